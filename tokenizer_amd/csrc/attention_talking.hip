// Attention whose heads' softmax weights are mixed with each other before they meet the values, over paged keys and
// values: w_h(i, j) = sum_g talk[h, g] p_g(i, j) with p_g head g's ordinary softmax over the keys j <= i, and head h's
// output is sum_j w_h(i, j) v(j) over the values of its own kv head.  Pages as everywhere: keys [n_pages, n_kv,
// page_size, d], values transposed inside a page, [n_pages, n_kv, dv, page_size].
#include "common.h"

#define TK_WAVES 4
#define TK_THREADS (TK_WAVES * WAVE)
#define TK_MAX_HEADS 128
#define TK_OUT 8               // outputs a thread keeps in the plain form

// ---------------------------------------------------------------------------------------------------------------
// The plain form, any storage type and any sizes, in float without matrix cores (the 32-bit path, and the yardstick of
// the kernels below): the softmax's maximum and sum of every head first, then the keys again with finished weights.

// stats[t, h] = (maximum, sum of exponentials under it) of the scaled scores; a workgroup a (token, head).
template <typename T>
__global__ void __launch_bounds__(TK_THREADS)
talking_stats_kernel(const T* __restrict__ q, int q_stride, const T* __restrict__ k_pages, const int* __restrict__ positions,
                     const int* __restrict__ entry_of_token, const int* __restrict__ block_table, int table_stride,
                     float* __restrict__ stats, int n_q, int n_kv, int d, int page_size, float scale) {
  __shared__ float q_s[512];
  __shared__ float m_s[TK_WAVES], l_s[TK_WAVES];
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
  const int entry = entry_of_token[t];
  if (entry < 0) return;
  const int n_keys = positions[t] + 1, kvh = h / (n_q / n_kv);
  const int* table = block_table + (size_t)entry * table_stride;
  for (int i = threadIdx.x; i < d; i += TK_THREADS) q_s[i] = ld(q + (size_t)t * q_stride + (size_t)h * d + i);
  __syncthreads();
  float m = -INFINITY, l = 0.f;
  for (int j = threadIdx.x; j < n_keys; j += TK_THREADS) {
    const T* kr = k_pages + (((size_t)table[j / page_size] * n_kv + kvh) * page_size + j % page_size) * d;
    float dot = 0.f;
    for (int i = 0; i < d; ++i) dot = fmaf(q_s[i], ld(kr + i), dot);
    const float s = dot * scale, top = fmaxf(m, s);
    l = l * expf(m - top) + expf(s - top);                   // (m = -inf at first: exp gives 0)
    m = top;
  }
  const float big = wave_max(m);
  l = wave_sum(m == -INFINITY ? 0.f : l * expf(m - big));
  if (lane == 0) { m_s[wave] = big; l_s[wave] = l; }
  __syncthreads();
  if (threadIdx.x == 0) {
    float top = -INFINITY, sum = 0.f;
    for (int w = 0; w < TK_WAVES; ++w) top = fmaxf(top, m_s[w]);
    for (int w = 0; w < TK_WAVES; ++w) sum += m_s[w] == -INFINITY ? 0.f : l_s[w] * expf(m_s[w] - top);
    stats[((size_t)t * n_q + h) * 2] = top;
    stats[((size_t)t * n_q + h) * 2 + 1] = sum;
  }
}

// A workgroup a (token, run of 2,048 outputs (head, value coordinate)): 64 keys at a time, all heads' weights into LDS,
// mixed there, then onto the values.  Dynamic LDS: two times n_q rows of 64 floats.
template <typename T>
__global__ void __launch_bounds__(TK_THREADS)
talking_apply_kernel(const T* __restrict__ q, int q_stride, T* __restrict__ out, const T* __restrict__ k_pages,
                     const T* __restrict__ v_pages, const int* __restrict__ positions, const int* __restrict__ entry_of_token,
                     const int* __restrict__ block_table, int table_stride, const float* __restrict__ stats,
                     const float* __restrict__ talk, int n_q, int n_kv, int d, int dv, int page_size, float scale) {
  extern __shared__ float tk_s[];
  float* p_s = tk_s;
  float* w_s = tk_s + n_q * WAVE;
  const int t = blockIdx.x, first = blockIdx.y * TK_THREADS * TK_OUT;
  const int entry = entry_of_token[t];
  if (entry < 0) return;
  const int n_keys = positions[t] + 1, group = n_q / n_kv, total = n_q * dv;
  const int* table = block_table + (size_t)entry * table_stride;
  float acc[TK_OUT] = {};
  for (int base = 0; base < n_keys; base += WAVE) {
    const int count = min(WAVE, n_keys - base);
    __syncthreads();                                         // the block before has been worked off
    for (int idx = threadIdx.x; idx < n_q * WAVE; idx += TK_THREADS) {
      const int h = idx / WAVE, jj = idx % WAVE, j = base + jj;
      float p = 0.f;
      if (jj < count) {
        const T* kr = k_pages + (((size_t)table[j / page_size] * n_kv + h / group) * page_size + j % page_size) * d;
        const T* qr = q + (size_t)t * q_stride + (size_t)h * d;
        float dot = 0.f;
        for (int i = 0; i < d; ++i) dot = fmaf(ld(qr + i), ld(kr + i), dot);
        const float* ml = stats + ((size_t)t * n_q + h) * 2;
        p = expf(dot * scale - ml[0]) / ml[1];
      }
      p_s[idx] = p;
    }
    __syncthreads();
    for (int idx = threadIdx.x; idx < n_q * WAVE; idx += TK_THREADS) {
      const int h = idx / WAVE, jj = idx % WAVE;
      float w = 0.f;
      for (int g = 0; g < n_q; ++g) w = fmaf(talk[(size_t)h * n_q + g], p_s[g * WAVE + jj], w);
      w_s[idx] = w;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < TK_OUT; ++r) {
      const int o = first + r * TK_THREADS + threadIdx.x;
      if (o >= total) continue;
      const int h = o / dv, i = o - h * dv, kvh = h / group;
      const float* w = w_s + h * WAVE;
      for (int jj = 0; jj < count;) {
        const int j = base + jj, off = j % page_size, run = min(count - jj, page_size - off);
        const T* v = v_pages + (((size_t)table[j / page_size] * n_kv + kvh) * dv + i) * page_size + off;
        for (int x = 0; x < run; ++x) acc[r] = fmaf(w[jj + x], ld(v + x), acc[r]);
        jj += run;
      }
    }
  }
#pragma unroll
  for (int r = 0; r < TK_OUT; ++r) {
    const int o = first + r * TK_THREADS + threadIdx.x;
    if (o < total) st(out + (size_t)t * total + o, acc[r]);
  }
}

// stats: float scratch [n_tokens, n_q, 2]; talk float [n_q, n_q]; out [n_tokens, n_q * dv].
extern "C" int ta_talking_attention_generic(const void* q, int q_stride, void* out, const void* k_pages, const void* v_pages,
                                            const void* positions, const void* entry_of_token, const void* block_table,
                                            int table_stride, void* stats, const void* talk, int n_tokens, int n_q, int n_kv,
                                            int d, int dv, int page_size, float scale, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (n_kv <= 0 || n_q <= 0 || n_q % n_kv || n_q > TK_MAX_HEADS || d <= 0 || d > 512 || dv <= 0 || page_size <= 0) return -1;
  const long slices = ((long)n_q * dv + TK_THREADS * TK_OUT - 1) / (TK_THREADS * TK_OUT);
  if (slices > 65535) return -1;
  dim3 g1(n_tokens, n_q), g2(n_tokens, (unsigned)slices);
  const size_t lds = sizeof(float) * 2 * n_q * WAVE;         // at most 64 KB
#define GO(TT)                                                                                                          \
  talking_stats_kernel<TT><<<g1, TK_THREADS, 0, stream>>>((const TT*)q, q_stride, (const TT*)k_pages, (const int*)positions, \
      (const int*)entry_of_token, (const int*)block_table, table_stride, (float*)stats, n_q, n_kv, d, page_size, scale);  \
  talking_apply_kernel<TT><<<g2, TK_THREADS, lds, stream>>>((const TT*)q, q_stride, (TT*)out, (const TT*)k_pages,          \
      (const TT*)v_pages, (const int*)positions, (const int*)entry_of_token, (const int*)block_table, table_stride,       \
      (const float*)stats, (const float*)talk, n_q, n_kv, d, dv, page_size, scale)
  if (dtype == DT_F32) { GO(float); } else { GO(bf16_t); }
#undef GO
  return LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------------------------------
// The matrix-core form for bfloat16.

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ bf16x8 tk_zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.0f;
  return z;
}

// Over the sixteen lanes of a row (lanes 16 i .. 16 i + 15), in every lane of the row: rotations within the row, which cost no
// trip through LDS.
#define TK_ROR(x, n) __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x120 | (n), 0xF, 0xF, false))
__device__ __forceinline__ float tk_row_sum16(float x) {
  x += TK_ROR(x, 8);
  x += TK_ROR(x, 4);
  x += TK_ROR(x, 2);
  x += TK_ROR(x, 1);
  return x;
}
__device__ __forceinline__ float tk_row_max16(float x) {
  x = fmaxf(x, TK_ROR(x, 8));
  x = fmaxf(x, TK_ROR(x, 4));
  x = fmaxf(x, TK_ROR(x, 2));
  x = fmaxf(x, TK_ROR(x, 1));
  return x;
}

// Where a key's page and slot lie; page sizes are powers of two as a rule, and a division costs thirty scalar instructions.
struct TalkPages {
  int size, shift;
  __device__ __forceinline__ explicit TalkPages(int page_size)
      : size(page_size), shift((page_size & (page_size - 1)) ? -1 : 31 - __builtin_clz(page_size)) {}
  __device__ __forceinline__ int page(int key) const { return shift >= 0 ? key >> shift : key / size; }
  __device__ __forceinline__ int slot(int key) const { return shift >= 0 ? key & (size - 1) : key % size; }
};

// Single tokens, in two passes over the keys' parts, since a part's weights can be mixed once every head's maximum and sum over
// all parts are known: the scores of every part from its keys, then the mixed weights of every part onto its values.
// d a multiple of 8 up to 256; split_keys a multiple of 32 up to 256.
#define TKD_BLOCKS 8

// A workgroup a (part of the keys, kv head and block of sixteen of its heads, token): scores, a wave a block of 32 keys at a
// time (the heads the N side of the instruction), through LDS to exponentials under the part's own maximum.
// e: float [items, splits, n_q, split_keys]; part_ml: float [items, splits, n_q, 2], maximum and sum (-inf and 0 for a part
// past the token).
__global__ void __launch_bounds__(4 * WAVE)
talking_scores_kernel(const bf16_t* __restrict__ q, int q_stride, const bf16_t* __restrict__ k_pages,
                      const int* __restrict__ rows, const int* __restrict__ positions, const int* __restrict__ entry_of_token,
                      const int* __restrict__ block_table, int table_stride, float* __restrict__ e, float* __restrict__ part_ml,
                      int n_q, int n_kv, int d, int page_size, float scale, int split_keys, int splits) {
  HELD(q, q_stride, k_pages, rows, positions, entry_of_token, block_table, table_stride, e, part_ml, n_q, n_kv, d, page_size,
       scale, split_keys, splits);
  __shared__ __attribute__((aligned(16))) float s_s[16][32 * TKD_BLOCKS + 4];
  const int split = blockIdx.x, item = blockIdx.z;
  const int t = rows ? scalar_int(rows + item) : item;
  if (t < 0) return;                                       // a row that only fills the list up
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, g = lane >> 4;
  const int* table = block_table + (size_t)(entry_of_token ? scalar_int(entry_of_token + t) : t) * table_stride;
  const int pos = scalar_int(positions + t), first = split * split_keys, last = min(pos, first + split_keys - 1);
  const int group = n_q / n_kv, head_blocks = (group + 15) / 16;
  const int kvh = blockIdx.y / head_blocks, hb = blockIdx.y - kvh * head_blocks;
  const int heads = min(16, group - hb * 16), head0 = kvh * group + hb * 16;
  const size_t part = (size_t)item * splits + split;
  if (first > pos) {
    if ((int)threadIdx.x < heads) {
      part_ml[(part * n_q + head0 + threadIdx.x) * 2] = -INFINITY;
      part_ml[(part * n_q + head0 + threadIdx.x) * 2 + 1] = 0.f;
    }
    return;
  }
  const TalkPages pages(page_size);
  const int blocks = (last - first) / 32 + 1;
  const bool has = col < heads;
  const bf16_t* qr = q + (size_t)t * q_stride + (size_t)(head0 + (has ? col : 0)) * d + 8 * g;
  for (int b = wave; b < blocks; b += 4) {
    const int kb = first + 32 * b;
    const bool there1 = kb + 16 <= last;                   // (a half without keys borrows the other's page; its scores are masked)
    const int kb1 = there1 ? kb + 16 : kb;
    const int page0 = scalar_int(table + pages.page(kb)), page1 = scalar_int(table + pages.page(kb1));
    const bf16_t* k0 = k_pages + (((size_t)page0 * n_kv + kvh) * page_size + pages.slot(kb) + col) * d + 8 * g;
    const bf16_t* k1 = k_pages + (((size_t)page1 * n_kv + kvh) * page_size + pages.slot(kb1) + col) * d + 8 * g;
    floatx4 st[2] = {(floatx4){0.f, 0.f, 0.f, 0.f}, (floatx4){0.f, 0.f, 0.f, 0.f}};
    for (int ks0 = 0; ks0 * 32 < d; ks0 += 4) {
      bf16x8 kf0[4], kf1[4], qf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int at = (ks0 + i) * 32;
        const bool in = at + 8 * g < d;
        kf0[i] = kf1[i] = qf[i] = tk_zero8();
        if (in) {
          kf0[i] = *reinterpret_cast<const bf16x8*>(k0 + at);
          kf1[i] = *reinterpret_cast<const bf16x8*>(k1 + at);
        }
        if (in && has) qf[i] = *reinterpret_cast<const bf16x8*>(qr + at);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        st[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf0[i], qf[i], st[0], 0, 0, 0);
        st[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf1[i], qf[i], st[1], 0, 0, 0);
      }
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int key = kb + 16 * u + 4 * g;
      float4 s;
      s.x = key <= last ? st[u][0] * scale : -INFINITY;
      s.y = key + 1 <= last ? st[u][1] * scale : -INFINITY;
      s.z = key + 2 <= last ? st[u][2] * scale : -INFINITY;
      s.w = key + 3 <= last ? st[u][3] * scale : -INFINITY;
      *reinterpret_cast<float4*>(&s_s[col][key - first]) = s;
    }
  }
  __syncthreads();
  // Maximum, exponentials and sum: sixteen lanes a head, four heads a wave.  (The part's first key is seen, so every maximum
  // is a number.)
  const int h = wave * 4 + g;
  float s[2 * TKD_BLOCKS], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int i = 0; i < 2 * TKD_BLOCKS; ++i) {
    s[i] = i < 2 * blocks ? s_s[h][col + 16 * i] : -INFINITY;
    m = fmaxf(m, s[i]);
  }
  m = tk_row_max16(m);
  float* to = e + (part * n_q + head0 + h) * split_keys + col;
#pragma unroll
  for (int i = 0; i < 2 * TKD_BLOCKS; ++i) {
    if (i >= 2 * blocks) continue;
    const float p = s[i] == -INFINITY ? 0.f : __expf(s[i] - m);
    l += p;
    if (h < heads) to[16 * i] = p;
  }
  l = tk_row_sum16(l);
  if (col == 0 && h < heads) {
    part_ml[(part * n_q + head0 + h) * 2] = m;
    part_ml[(part * n_q + head0 + h) * 2 + 1] = l;
  }
}

#define TK_MFMA32(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

// Every head's maximum over the parts and one over its sum under it, into m_s and inv_s: sixteen lanes a head, lane `col` parts
// col, col + 16, ....  ml: (maximum, sum) of part 0 of the item.
template <int NW>
__device__ __forceinline__ void talking_totals(const float2* __restrict__ ml, int n_q, int parts, float* m_s, float* inv_s,
                                               int wave, int col, int grp) {
  for (int g0 = wave * 4; g0 < n_q; g0 += NW * 4) {
    const int g = min(g0 + grp, n_q - 1);
    float m = -INFINITY, l = 0.f;
    for (int p0 = col; p0 < parts; p0 += 64) {
      float2 x[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] = p0 + 16 * i < parts ? ml[(size_t)(p0 + 16 * i) * n_q + g] : make_float2(-INFINITY, 0.f);
      float top = m;
#pragma unroll
      for (int i = 0; i < 4; ++i) top = fmaxf(top, x[i].x);
      if (top == -INFINITY) continue;
      l = m == -INFINITY ? 0.f : l * __expf(m - top);
#pragma unroll
      for (int i = 0; i < 4; ++i) l += x[i].x == -INFINITY ? 0.f : x[i].y * __expf(x[i].x - top);
      m = top;
    }
    const float big = tk_row_max16(m);
    l = tk_row_sum16(m == -INFINITY ? 0.f : l * __expf(m - big));
    if (col == 0 && g0 + grp < n_q) { m_s[g] = big; inv_s[g] = 1.0f / l; }
  }
}

// A workgroup a (part, kv head and block of sixteen of its heads, token): the part's weights of all heads g (exponentials times
// what brings them under the heads' totals), mixed by the rows of the talk table (float products on the matrix cores: heads
// the M side, sixteen keys the N side, g the contraction), rounded to bfloat16 once, onto the kv head's values.  part_o: float
// [items, splits, n_q, dv], plain sums (nothing where the part lies past the token).
template <int STEPS>
__global__ void __launch_bounds__(4 * WAVE)
talking_values_kernel(const float* __restrict__ e, const float* __restrict__ part_ml, const float* __restrict__ talk,
                      const bf16_t* __restrict__ vt_pages, const int* __restrict__ rows, const int* __restrict__ positions,
                      const int* __restrict__ entry_of_token, const int* __restrict__ block_table, int table_stride,
                      float* __restrict__ part_o, int n_q, int n_kv, int dv, int page_size, int split_keys, int splits) {
  HELD(e, part_ml, talk, vt_pages, rows, positions, entry_of_token, block_table, table_stride, part_o, n_q, n_kv, dv, page_size,
       split_keys, splits);
  __shared__ float m_s[4 * STEPS], inv_s[4 * STEPS];
  __shared__ __attribute__((aligned(16))) bf16_t w_s[16][32 * TKD_BLOCKS + 8];
  const int split = blockIdx.x, item = blockIdx.z;
  const int t = rows ? scalar_int(rows + item) : item;
  if (t < 0) return;
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, g = lane >> 4;
  const int* table = block_table + (size_t)(entry_of_token ? scalar_int(entry_of_token + t) : t) * table_stride;
  const int pos = scalar_int(positions + t), first = split * split_keys, last = min(pos, first + split_keys - 1);
  if (first > pos) return;
  const int group = n_q / n_kv, head_blocks = (group + 15) / 16;
  const int kvh = blockIdx.y / head_blocks, hb = blockIdx.y - kvh * head_blocks;
  const int heads = min(16, group - hb * 16), head0 = kvh * group + hb * 16;
  const TalkPages pages(page_size);
  const int blocks = (last - first) / 32 + 1;
  union VFrag { uint4 bits; bf16x8 v; };
  // Value rows rb * 16 .. + 15 over the part's keys: lane (col, g) has row col, keys 8 g .. 8 g + 7 of a block of 32.
  auto load_values = [&](VFrag (&vf)[TKD_BLOCKS], int rb) {
    const int row = min(rb * 16 + col, dv - 1);            // (a row past the last repeats it and is not written)
#pragma unroll
    for (int b = 0; b < TKD_BLOCKS; ++b) {
      vf[b].bits = make_uint4(0, 0, 0, 0);
      if (b >= blocks) continue;
      const int kb = first + 32 * b;
      const bool there1 = kb + 16 <= last;                 // (a half without keys borrows the other's page; its values are zeroed)
      const int page0 = scalar_int(table + pages.page(kb)), page1 = scalar_int(table + pages.page(there1 ? kb + 16 : kb));
      const int slot0 = pages.slot(kb), slot1 = pages.slot(kb + 16);
      const uint32_t at = (((uint32_t)((g >> 1) ? page1 : page0) * n_kv + kvh) * dv + row) * page_size +
                          ((g >> 1) ? slot1 : slot0) + 8 * (g & 1);
      vf[b].bits = *reinterpret_cast<const uint4*>(vt_pages + at);
    }
  };
  const int row_blocks = (dv + 15) / 16;
  VFrag vf[TKD_BLOCKS];
  if (wave < row_blocks) load_values(vf, wave);            // on their way while the weights are made
  const size_t part = (size_t)item * splits + split;
  const float* src = e + part * n_q * split_keys;
  float a[STEPS];                                          // the talk table's rows of this block of heads
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const int gg = 4 * s + g;
    a[s] = (col < heads && gg < n_q) ? talk[(size_t)(head0 + col) * n_q + gg] : 0.f;
  }
  // A wave's first block of sixteen keys is asked for beside the totals.
  const int key_blocks = 2 * blocks;
  float x[STEPS];
  auto load_weights = [&](int kb16) {
#pragma unroll
    for (int s = 0; s < STEPS; ++s) x[s] = 4 * s + g < n_q ? src[(size_t)(4 * s + g) * split_keys + 16 * kb16 + col] : 0.f;
  };
  if (wave < key_blocks) load_weights(wave);
  talking_totals<4>(reinterpret_cast<const float2*>(part_ml) + (size_t)item * splits * n_q, n_q, splits, m_s, inv_s, wave, col, g);
  float mine[STEPS];                                       // (maximum of this part, asked for with the totals)
#pragma unroll
  for (int s = 0; s < STEPS; ++s) mine[s] = part_ml[(part * n_q + min(4 * s + g, n_q - 1)) * 2];
  __syncthreads();
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const int gg = min(4 * s + g, n_q - 1);
    mine[s] = 4 * s + g < n_q ? __expf(mine[s] - m_s[gg]) * inv_s[gg] : 0.f;
  }
  for (int kb16 = wave; kb16 < key_blocks; kb16 += 4) {
    if (kb16 != wave) load_weights(kb16);
    floatx4 w = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < STEPS; ++s) w = TK_MFMA32(a[s], x[s] * mine[s], w);
#pragma unroll
    for (int r = 0; r < 4; ++r) st(&w_s[4 * g + r][16 * kb16 + col], w[r]);      // (rows past the last head hold zeros)
  }
  __syncthreads();
  for (int rb = wave; rb < row_blocks; rb += 4) {
    if (rb != wave) load_values(vf, rb);
    floatx4 acc = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < TKD_BLOCKS; ++b) {
      if (b >= blocks) continue;
      const int left = last - (first + 32 * b + 8 * g);    // the lane's keys that exist: 0 .. left; slots nobody wrote may hold anything
      if (left < 7) {
        uint4 v = vf[b].bits;
        if (left < 0) v.x = 0; else if (left < 1) v.x &= 0xffffu;
        if (left < 2) v.y = 0; else if (left < 3) v.y &= 0xffffu;
        if (left < 4) v.z = 0; else if (left < 5) v.z &= 0xffffu;
        if (left < 6) v.w = 0; else v.w &= 0xffffu;
        vf[b].bits = v;
      }
      const bf16x8 pf = *reinterpret_cast<const bf16x8*>(&w_s[col][32 * b + 8 * g]);
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[b].v, pf, acc, 0, 0, 0);
    }
    const int row = rb * 16 + 4 * g;
    if (col < heads) {
      float* dst = part_o + (part * n_q + head0 + col) * dv + row;
      if (dv % 4 == 0) {
        if (row < dv) *reinterpret_cast<float4*>(dst) = make_float4(acc[0], acc[1], acc[2], acc[3]);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (row + r < dv) dst[r] = acc[r];
      }
    }
  }
}

// out[t, i] = the sum of part_o[item, p, i] over the parts with keys of the token.  A workgroup an (item, 64 of its n_q dv
// outputs); its waves share the parts.
#define TKS_WAVES 4
__global__ void __launch_bounds__(TKS_WAVES * WAVE)
talking_sum_kernel(const float* __restrict__ part_o, const int* __restrict__ rows, const int* __restrict__ positions,
                   bf16_t* __restrict__ out, int outputs, int split_keys, int splits) {
  __shared__ float sum_s[TKS_WAVES][WAVE];
  const int item = blockIdx.y, lane = threadIdx.x & 63, wave = wave_index(), i = blockIdx.x * WAVE + lane;
  const int t = rows ? scalar_int(rows + item) : item;
  if (t < 0) return;
  const int parts = min(splits, scalar_int(positions + t) / split_keys + 1);
  const float* src = part_o + (size_t)item * splits * outputs + min(i, outputs - 1);
  float sum = 0.f;
  for (int p0 = wave; p0 < parts; p0 += TKS_WAVES * 8) {
    float v[8];
#pragma unroll
    for (int x = 0; x < 8; ++x) v[x] = p0 + TKS_WAVES * x < parts ? src[(size_t)(p0 + TKS_WAVES * x) * outputs] : 0.f;
#pragma unroll
    for (int x = 0; x < 8; ++x) sum += v[x];
  }
  sum_s[wave][lane] = sum;
  __syncthreads();
  if (wave > 0 || i >= outputs) return;
  sum = 0.f;
#pragma unroll
  for (int w = 0; w < TKS_WAVES; ++w) sum += sum_s[w][lane];
  st(out + (size_t)t * outputs + i, sum);
}

// Prompt portions, in one walk over the keys: the mix commutes with the product with the values.  With A_g = sum_j p_g(j) V(j)
// over the values of ALL kv heads side by side (W = n_kv dv numbers), head h's output is sum_g talk[h, g] times A_g's part at
// h's own kv head.  So every head is an ordinary softmax over its own keys against values W wide, and the mix is a small
// product at the end (`talking_mix_kernel`), in float.  The value pages hold exactly these wide values: a page's
// [n_kv, dv, page_size] read as [W, page_size].  The kernel leaves, per (token, part of its keys, head), the unnormalised sums
// [W] with the maximum and the sum of exponentials they stand under: part_o float [items, parts, n_q, W], part_ml float
// [items, parts, n_q, 2].
//
// A workgroup a (tile of sixteen tokens, kv head, block of 4 HG of its query heads, slab of 16 VB of the
// W value columns, part of the tile's keys); its four waves have HG heads each and walk the same blocks of KB keys, which
// come from the pages once for all of them straight into LDS, two buffers deep (the next block is on its way while the
// current one is worked on).  S^T = K Q^T and O^T = V^T P^T with 16x16x32 instructions, token index in `lane % 16`;
// softmax online in float; a row block of ones beside V^T gives the probabilities' sums.  A fragment of the values is
// read from LDS once for the wave's HG heads.
// Keys in LDS: rows of DP (d filled up to a power of two) elements; the sixteen bytes that hold elements 8 p .. 8 p + 7 of
// key k stand at place p ^ turn(k), so that rows read at once lie in different banks; a piece past d repeats the row's
// last one and meets a query of zeros.  Values: runs of sixteen keys, 16 VB rows of 32 bytes each.
template <int DP, int VB>
struct TalkBlock {
  static constexpr int KB = DP + 16 * VB > 256 ? 32 : 64;
  static constexpr int RUNS = KB / 16, SHARE = 4 / RUNS;     // runs of sixteen keys; waves that share a run's loads
  static constexpr int PIECES = DP / 8, KEYS_A_LOAD = 64 / PIECES, K_LOADS = 16 / KEYS_A_LOAD, V_LOADS = VB / 2;
  static constexpr int K_ROW = 2 * DP, K_BYTES = KB * K_ROW, V_RUN = 32 * 16 * VB, BYTES = K_BYTES + RUNS * V_RUN;
  __device__ static constexpr int turn(int key) { return ((key & 3) | ((key >> 1) & 4)) & (PIECES - 1); }
};

struct Whole { static constexpr bool value = true; };    // every key of the block is seen by every token of the tile
struct Edge { static constexpr bool value = false; };

template <int DP, int VB, int HG>
__global__ void __launch_bounds__(4 * WAVE, 2)
talking_prefill_kernel(const bf16_t* __restrict__ q, int q_stride, const bf16_t* __restrict__ k_pages,
                       const bf16_t* __restrict__ vt_pages, const int* __restrict__ tiles, int n_tiles,
                       const int* __restrict__ cu_q, const int* __restrict__ first_position,
                       const int* __restrict__ block_table, int table_stride, float* __restrict__ part_o,
                       float* __restrict__ part_ml, int n_q, int n_kv, int d, int wide, int page_size, float scale,
                       int slabs, int key_splits) {
  typedef TalkBlock<DP, VB> B;
  constexpr int KS = DP / 32, KB = B::KB, HALVES = KB / 32;
  HELD(q, q_stride, k_pages, vt_pages, tiles, n_tiles, cu_q, first_position, block_table, table_stride, part_o, part_ml,
       n_q, n_kv, d, wide, page_size, scale, slabs, key_splits);
  extern __shared__ __attribute__((aligned(16))) char tkp_lds[];
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, g = lane >> 4;
  const int group = n_q / n_kv, head_blocks = (group + 4 * HG - 1) / (4 * HG);
  // Late tiles first: they see the most keys.
  int which = blockIdx.x;
  const int split = which % key_splits; which /= key_splits;
  const int slab = which % slabs; which /= slabs;
  const int hb = which % head_blocks; which /= head_blocks;
  const int kvh = which % n_kv; which /= n_kv;
  const int tile_index = n_tiles - 1 - which;
  const int first_head = hb * 4 * HG + wave * HG, heads_here = max(0, min(HG, group - first_head));
  const int head0 = kvh * group + first_head;
  const int entry = scalar_int(tiles + 2 * tile_index), offset = scalar_int(tiles + 2 * tile_index + 1);
  const int entry_row = scalar_int(cu_q + entry), next_row = scalar_int(cu_q + entry + 1);
  const int entry_position = scalar_int(first_position + entry);
  HELD(entry_row, next_row, entry_position);
  const int row0 = entry_row + offset, n_valid = min(16, next_row - row0);
  if (n_valid <= 0) return;                                // a tile that only fills the list up
  const int p0 = entry_position + offset, hi = p0 + n_valid - 1;
  const int my_pos = p0 + min(col, n_valid - 1), my_row = row0 + min(col, n_valid - 1);
  const int* table = block_table + (size_t)entry * table_stride;
  // This workgroup's blocks: a run of whole turns of the walk.
  const int turns = hi / KB + 1, each = (turns + key_splits - 1) / key_splits;
  const int begin = split * each * KB, end = min(hi, begin + each * KB - 1);
  bf16x8 qf[HG][KS];
  floatx4 acc[HG][VB], l[HG];
  float m[HG];
#pragma unroll
  for (int h = 0; h < HG; ++h) {
    m[h] = -INFINITY;
    l[h] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int db = 0; db < VB; ++db) acc[h][db] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d0 = ks * 32 + 8 * g;
      qf[h][ks] = tk_zero8();
      if (h < heads_here && d0 < d)
        qf[h][ks] = *reinterpret_cast<const bf16x8*>(q + (size_t)my_row * q_stride + (size_t)(head0 + h) * d + d0);
    }
  }
  // What a lane brings of a run: offsets worked out once.
  const int run = wave % B::RUNS, share = wave / B::RUNS;
  uint32_t k_from[B::K_LOADS], v_from[B::V_LOADS];
#pragma unroll
  for (int j = 0; j < B::K_LOADS; ++j) {
    const int key = B::KEYS_A_LOAD * j + lane / B::PIECES, piece = (lane % B::PIECES) ^ B::turn(key);
    k_from[j] = (uint32_t)(key * d + min(piece * 8, d - 8)) * 2;
  }
#pragma unroll
  for (int j = 0; j < B::V_LOADS; ++j) {
    const int row = min(slab * 16 * VB + 32 * j + (lane >> 1), wide - 1);
    v_from[j] = (uint32_t)(row * page_size + (lane & 1) * 8) * 2;
  }
  const TalkPages pages(page_size);
  const auto page_of = [&](int kb) {                       // (a run past the last key borrows the last key's page: its keys are masked)
    return scalar_int(table + pages.page(min(kb + 16 * run, hi)));
  };
  const auto fetch = [&](int kb, int page, char* buf) {
    typedef const void __attribute__((address_space(1)))* from_t;
    typedef void __attribute__((address_space(3)))* to_t;
    const int slot = pages.slot(kb + 16 * run);
    const char* k_run = reinterpret_cast<const char*>(k_pages + (((uint32_t)page * n_kv + kvh) * page_size + slot) * d);
    const char* v_run = reinterpret_cast<const char*>(vt_pages + ((uint32_t)page * wide * page_size + slot));
    char* k_to = buf + run * 16 * B::K_ROW;
    char* v_to = buf + B::K_BYTES + run * B::V_RUN;
#pragma unroll
    for (int j = 0; j < B::K_LOADS; ++j)
      if (B::SHARE == 1 || j % B::SHARE == share)
        __builtin_amdgcn_global_load_lds((from_t)(k_run + k_from[j]), (to_t)(k_to + j * 1024), 16, 0, 0);
#pragma unroll
    for (int j = 0; j < B::V_LOADS; ++j)
      if (B::SHARE == 1 || j % B::SHARE == share)
        __builtin_amdgcn_global_load_lds((from_t)(v_run + v_from[j]), (to_t)(v_to + j * 1024), 16, 0, 0);
  };
  bf16x8 ones;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;
  const float c = scale * 1.4426950408889634f;
  const int turned = B::turn((col & 3) | ((col >> 2) & 1) << 3);     // of the lane's keys: the same in every instruction
  const auto block = [&](const char* buf, int kb, auto full) {
    constexpr bool FULL = decltype(full)::value;
    float s[HG][KB / 4];
#pragma unroll
    for (int t = 0; t < 2 * HALVES; ++t) {
      // Row r of the instruction is key 8 (r / 4) + 4 (t % 2) + r % 4 of its half of 32, whose score then lies in the lane
      // group that holds that key in the second product (lane group g: keys 8 g .. 8 g + 7).
      const int key = 32 * (t >> 1) + 8 * (col >> 2) + 4 * (t & 1) + (col & 3);
      bf16x8 kf[KS];
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        kf[ks] = *reinterpret_cast<const bf16x8*>(buf + key * B::K_ROW + ((ks * 4 + g) ^ turned) * 16);
#pragma unroll
      for (int h = 0; h < HG; ++h) {
        floatx4 st = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks], qf[h][ks], st, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int at = kb + 32 * (t >> 1) + 8 * g + 4 * (t & 1) + r;
          s[h][t * 4 + r] = FULL || at <= my_pos ? st[r] : -INFINITY;
        }
      }
    }
    bf16x8 pf[HG][HALVES];
#pragma unroll
    for (int h = 0; h < HG; ++h) {
      float mx = s[h][0];
#pragma unroll
      for (int i = 1; i < KB / 4; ++i) mx = __builtin_elementwise_maximum(mx, s[h][i]);
      mx = __builtin_elementwise_maximum(mx, __shfl_xor(mx, 16, WAVE));
      mx = __builtin_elementwise_maximum(mx, __shfl_xor(mx, 32, WAVE));
      const float m_new = __builtin_elementwise_maximum(m[h], mx);
      const float mc = (m_new == -INFINITY) ? 0.f : m_new * c;         // (no key seen yet: exp2 of inf - inf would be NaN)
      if (__any(m_new > m[h])) {                            // rescale only when some token's maximum moved
        const float corr = __builtin_amdgcn_exp2f(m[h] * c - mc);
#pragma unroll
        for (int r = 0; r < 4; ++r) l[h][r] *= corr;
#pragma unroll
        for (int db = 0; db < VB; ++db)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[h][db][r] *= corr;
        m[h] = m_new;
      }
#pragma unroll
      for (int i = 0; i < KB / 4; ++i)
        pf[h][i >> 3][i & 7] = (__bf16)__builtin_amdgcn_exp2f(fmaf(s[h][i], c, -mc));
    }
#pragma unroll
    for (int u = 0; u < HALVES; ++u) {
#pragma unroll
      for (int h = 0; h < HG; ++h) l[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[h][u], l[h], 0, 0, 0);
#pragma unroll
      for (int db = 0; db < VB; ++db) {
        bf16x8 vf = *reinterpret_cast<const bf16x8*>(buf + B::K_BYTES + (2 * u + (g >> 1)) * B::V_RUN +
                                                     (db * 16 + col) * 32 + (g & 1) * 16);
        if (!FULL) {                                        // slots nobody wrote may hold anything: 0 * NaN must stay 0
#pragma unroll
          for (int i = 0; i < 8; ++i)
            if (kb + 32 * u + 8 * g + i > hi) vf[i] = (__bf16)0.0f;
        }
#pragma unroll
        for (int h = 0; h < HG; ++h) acc[h][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[h][u], acc[h][db], 0, 0, 0);
      }
    }
  };
  // Turn by turn: ask for the next block into the buffer that the turn before read, work on the current one, wait for
  // what was asked for, meet.  The page of the block after the next is looked up meanwhile.
  int cur = 0, kb = begin;
  if (kb <= end) fetch(kb, page_of(kb), tkp_lds);
  int next_page = page_of(kb + KB);
  __builtin_amdgcn_s_waitcnt(0x0F70);                       // all that this wave fetched has arrived (vmcnt 0)
  __syncthreads();
#define TALK_TURN(KIND)                                                              \
  {                                                                                  \
    if (kb + KB <= end) fetch(kb + KB, next_page, tkp_lds + (cur ^ 1) * B::BYTES);   \
    next_page = page_of(kb + 2 * KB);                                                \
    if (heads_here > 0) block(tkp_lds + cur * B::BYTES, kb, KIND{});                 \
    __builtin_amdgcn_s_waitcnt(0x0F70);                                              \
    __syncthreads();                                                                 \
    cur ^= 1;                                                                        \
  }
  for (; kb <= end && kb + KB - 1 <= p0; kb += KB) TALK_TURN(Whole)
  for (; kb <= end; kb += KB) TALK_TURN(Edge)
#undef TALK_TURN
  if (col >= n_valid) return;
#pragma unroll
  for (int h = 0; h < HG; ++h) {
    if (h >= heads_here) break;
    const size_t at = (((size_t)tile_index * 16 + col) * key_splits + split) * n_q + head0 + h;
    if (slab == 0 && g == 0) {
      part_ml[at * 2] = m[h] * scale;                       // in units of the scaled scores
      part_ml[at * 2 + 1] = l[h][0];
    }
#pragma unroll
    for (int db = 0; db < VB; ++db) {
      const int row = slab * 16 * VB + db * 16 + 4 * g;
      float* dst = part_o + at * wide + row;
      if (wide % 4 == 0) {
        if (row < wide) *reinterpret_cast<float4*>(dst) = make_float4(acc[h][db][0], acc[h][db][1], acc[h][db][2], acc[h][db][3]);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (row + r < wide) dst[r] = acc[h][db][r];
      }
    }
  }
}

// The parts of every head brought together and the heads mixed: out of head h = sum_g talk[h, g] A_g at h's own kv head, float
// products on the matrix cores (16x16x4): the sixteen heads of a block are the M side, sixteen value columns the N side, the
// heads g the contraction; lane (col, grp) has row `col` of the talk table and column `col` of the A_g for g = 4 s + grp.
// STEPS: steps of four heads g.  A wave a token, for one (kv head, block of sixteen of its heads) and all its value columns;
// four workgroups a tile.
template <int STEPS>
__global__ void __launch_bounds__(4 * WAVE)
talking_mix_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, const float* __restrict__ talk,
                   const int* __restrict__ tiles, const int* __restrict__ cu_q, bf16_t* __restrict__ out, int n_q, int n_kv,
                   int dv, int parts) {
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, grp = lane >> 4;
  const int tile = blockIdx.x >> 2, token = 4 * (blockIdx.x & 3) + wave;
  const int group = n_q / n_kv, head_blocks = (group + 15) / 16, wide = n_kv * dv;
  const int kvh = blockIdx.y / head_blocks, first = (blockIdx.y - kvh * head_blocks) * 16, heads = min(16, group - first);
  const int head0 = kvh * group + first;
  const int entry = scalar_int(tiles + 2 * tile), row0 = scalar_int(cu_q + entry) + scalar_int(tiles + 2 * tile + 1);
  if (token >= scalar_int(cu_q + entry + 1) - row0) return;
  float t[STEPS];
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const int g = 4 * s + grp;
    t[s] = (col < heads && g < n_q) ? talk[(size_t)(head0 + col) * n_q + g] : 0.f;
  }
  const size_t base = ((size_t)tile * 16 + token) * parts * n_q;
  const float2* ml = reinterpret_cast<const float2*>(part_ml) + base;
  float m[STEPS], l[STEPS];
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const float2 x = ml[min(4 * s + grp, n_q - 1)];
    m[s] = x.x;                                          // (the first part always has keys)
    l[s] = x.y;
  }
  for (int p = 1; p < parts; ++p) {
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
      const float2 x = ml[(size_t)p * n_q + min(4 * s + grp, n_q - 1)];
      const float top = fmaxf(m[s], x.x);
      l[s] = l[s] * __expf(m[s] - top) + (x.x == -INFINITY ? 0.f : x.y * __expf(x.x - top));
      m[s] = top;
    }
  }
#pragma unroll
  for (int s = 0; s < STEPS; ++s) l[s] = 1.0f / l[s];
  const float* src = part_o + base * wide + (size_t)kvh * dv;
  for (int c0 = 0; c0 < dv; c0 += 64) {
    float a[4][STEPS];
#pragma unroll
    for (int cb = 0; cb < 4; ++cb)
#pragma unroll
      for (int s = 0; s < STEPS; ++s) a[cb][s] = 0.f;
    for (int p = 0; p < parts; ++p) {
      float f[STEPS];
#pragma unroll
      for (int s = 0; s < STEPS; ++s) {
        const float top = ml[(size_t)p * n_q + min(4 * s + grp, n_q - 1)].x;
        f[s] = 4 * s + grp >= n_q || top == -INFINITY ? 0.f : __expf(top - m[s]) * l[s];
      }
#pragma unroll
      for (int cb = 0; cb < 4; ++cb) {
        const float* from = src + (size_t)p * n_q * wide + min(c0 + 16 * cb + col, dv - 1);
        float v[STEPS];
#pragma unroll
        for (int s = 0; s < STEPS; ++s) v[s] = from[(size_t)min(4 * s + grp, n_q - 1) * wide];
#pragma unroll
        for (int s = 0; s < STEPS; ++s) a[cb][s] += f[s] == 0.f ? 0.f : f[s] * v[s];   // (unwritten sums of a part without keys: by selection)
      }
    }
#pragma unroll
    for (int cb = 0; cb < 4; ++cb) {
      floatx4 acc = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < STEPS; ++s) acc = TK_MFMA32(t[s], a[cb][s], acc);
      const int column = c0 + 16 * cb + col;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (4 * grp + r < heads && column < dv)
          st(out + (size_t)(row0 + token) * n_q * dv + (size_t)(head0 + 4 * grp + r) * dv + column, acc[r]);
    }
  }
}

// A launch that wants more dynamic LDS than every kernel may have says so first.
static int allow_lds(const void* kernel, int bytes) {
  if (bytes <= 48 * 1024) return 0;
  return (int)hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
}

// Whether the matrix-core kernels take these sizes.
static bool talking_fits(int n_q, int n_kv, int d, int dv, int page_size) {
  return n_kv > 0 && n_q > 0 && n_q % n_kv == 0 && n_q <= 64 && d >= 8 && d <= 256 && d % 8 == 0 && dv > 0 && page_size % 16 == 0 &&
         (long)n_kv * dv <= 65536;
}

// Single tokens: items are the rows of `rows` (or every row); entry_of_token null: row e is entry e.  e float
// [n_items, splits, n_q, split_keys], part_ml float [n_items, splits, n_q, 2], part_o float [n_items, splits, n_q, dv].
// Returns -2 for sizes without an instance.
extern "C" int ta_talking_decode_bf16(const void* q, int q_stride, void* out, const void* k_pages, const void* vt_pages,
                                      const void* rows, const void* positions, const void* entry_of_token,
                                      const void* block_table, int table_stride, void* e, void* part_ml, void* part_o,
                                      const void* talk, int n_items, int n_q, int n_kv, int d, int dv, int page_size, float scale,
                                      int split_keys, int splits, hipStream_t stream) {
  if (n_items <= 0) return 0;
  if (!talking_fits(n_q, n_kv, d, dv, page_size) || q_stride % 8) return -2;
  if (split_keys < 32 || split_keys % 32 || split_keys > 32 * TKD_BLOCKS || splits < 1 || splits > 0x7ffffff || n_items > 65535) return -1;
  dim3 grid(splits, n_kv * ((n_q / n_kv + 15) / 16), n_items);
  talking_scores_kernel<<<grid, 4 * WAVE, 0, stream>>>((const bf16_t*)q, q_stride, (const bf16_t*)k_pages, (const int*)rows,
      (const int*)positions, (const int*)entry_of_token, (const int*)block_table, table_stride, (float*)e, (float*)part_ml, n_q,
      n_kv, d, page_size, scale, split_keys, splits);
#define VALUES(SV) talking_values_kernel<SV><<<grid, 4 * WAVE, 0, stream>>>((const float*)e, (const float*)part_ml,          \
      (const float*)talk, (const bf16_t*)vt_pages, (const int*)rows, (const int*)positions, (const int*)entry_of_token,      \
      (const int*)block_table, table_stride, (float*)part_o, n_q, n_kv, dv, page_size, split_keys, splits)
  if (n_q <= 16) VALUES(4); else if (n_q <= 32) VALUES(8); else VALUES(16);
#undef VALUES
  const int outputs = n_q * dv;
  talking_sum_kernel<<<dim3((outputs + WAVE - 1) / WAVE, n_items), TKS_WAVES * WAVE, 0, stream>>>((const float*)part_o,
      (const int*)rows, (const int*)positions, (bf16_t*)out, outputs, split_keys, splits);
  return LAUNCH_STATUS();
}

// What a launch over `n_tiles` tiles that reach `reach` keys is cut into: slabs of the value columns (16 * *blocks columns
// each), and parts of the keys (a few tiles behind a long context would leave the device idle).
static void talking_plan(int n_tiles, int n_q, int n_kv, int d, int dv, int reach, int* blocks, int* slabs, int* heads, int* parts) {
  const int wide = n_kv * dv, group = n_q / n_kv;
  *blocks = wide <= 64 ? 4 : wide <= 128 ? 8 : 16;
  *slabs = (wide + 16 * *blocks - 1) / (16 * *blocks);
  *heads = (group > 4 && d <= 128) ? 2 : 1;
  const long groups = (long)n_tiles * n_kv * ((group + 4 * *heads - 1) / (4 * *heads)) * *slabs;
  int cut = 1;
  while (cut < 16 && groups * cut < 1024 && reach / (cut * 2) >= 256) cut *= 2;
  *parts = cut;
}

extern "C" int ta_talking_prefill_parts(int n_tiles, int n_q, int n_kv, int d, int dv, int reach) {
  if (n_tiles <= 0 || n_kv <= 0 || n_q % n_kv) return 1;
  int blocks, slabs, heads, parts;
  talking_plan(n_tiles, n_q, n_kv, d, dv, reach, &blocks, &slabs, &heads, &parts);
  return parts;
}

// Prompt portions: tiles [n_tiles, 2] = (entry, offset of the tile's first token inside the entry's tokens).  part_o float
// [n_tiles * 16, parts, n_q, n_kv dv], part_ml float [n_tiles * 16, parts, n_q, 2] with `parts` as
// ta_talking_prefill_parts says.  Returns -2 for sizes without an instance.
extern "C" int ta_talking_prefill_bf16(const void* q, int q_stride, void* out, const void* k_pages, const void* vt_pages,
                                       const void* tiles, int n_tiles, const void* cu_q, const void* first_position,
                                       const void* block_table, int table_stride, void* part_o, void* part_ml, const void* talk,
                                       int n_q, int n_kv, int d, int dv, int page_size, float scale, int reach, hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (!talking_fits(n_q, n_kv, d, dv, page_size) || q_stride % 8) return -2;
  int blocks, slabs, heads, parts;
  talking_plan(n_tiles, n_q, n_kv, d, dv, reach, &blocks, &slabs, &heads, &parts);
  const int wide = n_kv * dv, group = n_q / n_kv;
  const long total = (long)n_tiles * n_kv * ((group + 4 * heads - 1) / (4 * heads)) * slabs * parts;
  if (total > 0x7fffffffL || (long)n_tiles * 16 > 0x7fffffffL) return -1;
#define PREFILL(DPV, VBV, HGV)                                                                                            \
  {                                                                                                                       \
  if (const int bad = allow_lds(reinterpret_cast<const void*>(&talking_prefill_kernel<DPV, VBV, HGV>),                     \
                                2 * TalkBlock<DPV, VBV>::BYTES)) return bad;                                              \
  talking_prefill_kernel<DPV, VBV, HGV><<<(unsigned)total, 4 * WAVE, 2 * TalkBlock<DPV, VBV>::BYTES, stream>>>(             \
      (const bf16_t*)q, q_stride, (const bf16_t*)k_pages, (const bf16_t*)vt_pages, (const int*)tiles, n_tiles,             \
      (const int*)cu_q, (const int*)first_position, (const int*)block_table, table_stride, (float*)part_o,                 \
      (float*)part_ml, n_q, n_kv, d, wide, page_size, scale, slabs, parts);                                                \
  }
#define PREFILL_H(DPV, VBV) if (heads == 2) PREFILL(DPV, VBV, 2) else PREFILL(DPV, VBV, 1)
#define PREFILL_V(DPV) if (blocks == 4) { PREFILL_H(DPV, 4); } else if (blocks == 8) { PREFILL_H(DPV, 8); } else { PREFILL_H(DPV, 16); }
  if (d <= 32) { PREFILL_V(32); } else if (d <= 64) { PREFILL_V(64); } else if (d <= 128) { PREFILL_V(128); }
  else if (blocks == 4) PREFILL(256, 4, 1) else if (blocks == 8) PREFILL(256, 8, 1) else PREFILL(256, 16, 1)
#undef PREFILL_V
#undef PREFILL_H
#undef PREFILL
  const int status = LAUNCH_STATUS();
  if (status) return status;
  const dim3 grid(n_tiles * 4, n_kv * ((group + 15) / 16));
#define MIX(SV) talking_mix_kernel<SV><<<grid, 4 * WAVE, 0, stream>>>((const float*)part_o, (const float*)part_ml,             \
      (const float*)talk, (const int*)tiles, (const int*)cu_q, (bf16_t*)out, n_q, n_kv, dv, parts)
  if (n_q <= 16) MIX(4); else if (n_q <= 32) MIX(8); else MIX(16);
#undef MIX
  return LAUNCH_STATUS();
}
