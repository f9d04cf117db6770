// Retention: per head S <- c S + k v^T, o = S^T q with a fixed decay c, over a batch of portions, with the state of every
// request in its slot; the rotation of q and k in front of it, and behind it each head's norm and the silu gate.
// Everything here is float: rotation, state, decays, reads, norm.  A state row is [heads, dv, d] (S transposed).
#include "common.h"

// x summed over the sixteen lanes of a row (lanes 16 i .. 16 i + 15), in every lane of the row: four rotations within the
// row, which cost no trip through LDS.
__device__ __forceinline__ float rt_row_sum16(float x) {
#define RT_ROR(n) __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x120 | (n), 0xF, 0xF, false))
  x += RT_ROR(8);
  x += RT_ROR(4);
  x += RT_ROR(2);
  x += RT_ROR(1);
#undef RT_ROR
  return x;
}

__device__ __forceinline__ float ld_bf(const bf16_t* p) { return ld(p); }

#define RT_ROWS 4              // value rows of S^T a lane keeps (a part of)

// Token by token: a workgroup an (entry, head).  Sixteen lanes share a value row of S^T, lane p with columns p PER ..
// p PER + PER - 1 of it in registers; a lane works on up to RT_ROWS rows, THREADS / 16 apart.  Between two tokens only the
// next token's q, k, v and gate come from memory (asked for while the current one is worked on).
// qkvg: rows of `row_stride`, [heads d (q) | heads d (k) | heads dv (v) | heads dv (g)]; table: float [n_tokens, rot],
// [cosines | sines] of the rotation of the first `rot` coordinates of q and k; out [n_tokens, heads dv].
// Entries of more than `most` rows are left to the chunked form below.
template <typename T, int PER, int THREADS>
__global__ void __launch_bounds__(THREADS)
retention_scan_kernel(const T* __restrict__ qkvg, int row_stride, const float* __restrict__ table, int rot,
                      const float* __restrict__ decays, float* __restrict__ state, size_t state_stride,
                      const int* __restrict__ cu_q, const int* __restrict__ first_position, const int* __restrict__ state_slots,
                      T* __restrict__ out, int heads, int d, int dv, float eps, int most) {
  constexpr int DP = 16 * PER;
  __shared__ __attribute__((aligned(16))) float q_s[DP], k_s[DP];
  __shared__ float v_s[THREADS / 16 * RT_ROWS], o_s[THREADS / 16 * RT_ROWS], sq_s[THREADS / WAVE];
  const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lo = cu_q[e], hi = cu_q[e + 1];
  if (hi <= lo || hi - lo > most) return;
  const int part = tid & 15, row0 = tid >> 4;
  float* mem = state + (size_t)state_slots[e] * state_stride + (size_t)h * dv * d;
  const bool fresh = first_position[e] == 0;
  const float decay = decays[h], k_scale = 1.0f / sqrtf((float)d);
  const int half = rot / 2, units = d - half;                // a unit: a pair that turns, or a coordinate that passes
  // What a thread brings of a token: a unit of q or of k, a value, a gate.
  const bool brings = tid < 2 * units, of_k = tid >= units;
  const int unit = of_k ? tid - units : tid;
  const int c0 = unit < half ? unit : half + unit, c1 = unit < half ? unit + half : c0;
  float a = 0.f, b = 0.f, cs = 1.f, sn = 0.f, vv = 0.f, gg = 0.f;
  auto fetch = [&](int t) {
    const T* row = qkvg + (size_t)t * row_stride;
    if (brings) {
      const T* x = row + (size_t)(of_k ? heads + h : h) * d;
      a = ld(x + c0);
      if (unit < half) {
        b = ld(x + c1);
        cs = table[(size_t)t * rot + unit];
        sn = table[(size_t)t * rot + half + unit];
      }
    }
    if (tid < dv) {
      vv = ld(row + (size_t)2 * heads * d + (size_t)h * dv + tid);
      gg = ld(row + (size_t)2 * heads * d + (size_t)(heads + h) * dv + tid);
    }
  };
  fetch(lo);
  float S[RT_ROWS][PER];
#pragma unroll
  for (int i = 0; i < RT_ROWS; ++i) {
    const int r = row0 + i * (THREADS / 16);
#pragma unroll
    for (int j = 0; j < PER; ++j) S[i][j] = 0.f;
    if (!fresh && r < dv) {
      const float* src = mem + (size_t)r * d + part * PER;
      if (PER % 4 == 0 && d % 4 == 0) {
#pragma unroll
        for (int j = 0; j < PER; j += 4)
          if (part * PER + j < d) {
            const float4 x = *reinterpret_cast<const float4*>(src + j);
            S[i][j] = x.x; S[i][j + 1] = x.y; S[i][j + 2] = x.z; S[i][j + 3] = x.w;
          }
      } else {
#pragma unroll
        for (int j = 0; j < PER; ++j)
          if (part * PER + j < d) S[i][j] = src[j];
      }
    }
  }
  for (int j = d + tid; j < DP; j += THREADS) q_s[j] = k_s[j] = 0.f;
  for (int t = lo; t < hi; ++t) {
    __syncthreads();                                         // the token before has been worked off
    if (brings) {
      float* to = of_k ? k_s : q_s;
      const float f = of_k ? k_scale : 1.f;
      to[c0] = (unit < half ? a * cs - b * sn : a) * f;
      if (unit < half) to[c1] = (b * cs + a * sn) * f;
    }
    if (tid < dv) v_s[tid] = vv;
    const float gate = gg;
    if (t + 1 < hi) fetch(t + 1);
    __syncthreads();
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < RT_ROWS; ++i) {
      const int r = row0 + i * (THREADS / 16);
      const float v = r < dv ? v_s[r] : 0.f;
      float o = 0.f;
#pragma unroll
      for (int j = 0; j < PER; ++j) {
        S[i][j] = fmaf(decay, S[i][j], k_s[part * PER + j] * v);
        o = fmaf(S[i][j], q_s[part * PER + j], o);
      }
      o = rt_row_sum16(o);
      if (part == 0) {
        sq = fmaf(o, o, sq);
        if (r < dv) o_s[r] = o;
      }
    }
    sq = wave_sum(sq);
    if ((tid & (WAVE - 1)) == 0) sq_s[tid / WAVE] = sq;
    __syncthreads();
    if (tid < dv) {
      float total = 0.f;
#pragma unroll
      for (int w = 0; w < THREADS / WAVE; ++w) total += sq_s[w];
      const float inv = 1.0f / sqrtf(total / (float)dv + eps);
      st(out + (size_t)t * heads * dv + (size_t)h * dv + tid, o_s[tid] * inv * (gate / (1.0f + expf(-gate))));
    }
  }
#pragma unroll
  for (int i = 0; i < RT_ROWS; ++i) {
    const int r = row0 + i * (THREADS / 16);
    if (r >= dv) continue;
    float* dst = mem + (size_t)r * d + part * PER;
    if (PER % 4 == 0 && d % 4 == 0) {
#pragma unroll
      for (int j = 0; j < PER; j += 4)
        if (part * PER + j < d) *reinterpret_cast<float4*>(dst + j) = make_float4(S[i][j], S[i][j + 1], S[i][j + 2], S[i][j + 3]);
    } else {
#pragma unroll
      for (int j = 0; j < PER; ++j)
        if (part * PER + j < d) dst[j] = S[i][j];
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// Long portions of bfloat16 rows in chunks of 64 tokens: every chunk's own sum of decayed k v^T side by side, the state
// carried from chunk to chunk element by element, then every chunk's reads side by side,
//   o_t = c^(t+1) S_before^T q_t + sum_{s <= t} c^(t-s) (q_t . k_s) v_s   (t, s counted within the chunk),
// with the heads' norm and the gate behind them.  All products are float products on the matrix cores (16x16x4, true
// 32-bit); a lane's part of the contraction may take the indices in any order as long as both operands do.

#define RC_L 64
typedef float rc_floatx4 __attribute__((ext_vector_type(4)));
#define RC_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

struct rc_place { int lo, n, entry, index, base, count; };   // rows of the chunk; which of its entry's chunks

// Chunk g of the entries with more than `most` rows, in order; false past the last.
__device__ __forceinline__ bool rc_find(const int* cu_q, int n_entries, int g, int most, rc_place& p) {
  int seen = 0;
  for (int e = 0; e < n_entries; ++e) {
    const int lo = scalar_int(cu_q + e), len = scalar_int(cu_q + e + 1) - lo;
    if (len <= most) continue;
    const int count = (len + RC_L - 1) / RC_L;
    if (g < seen + count) {
      p.entry = e; p.index = g - seen; p.base = seen; p.count = count;
      p.lo = lo + p.index * RC_L;
      p.n = min(RC_L, len - p.index * RC_L);
      return true;
    }
    seen += count;
  }
  return false;
}

__device__ __forceinline__ void rc_unpack8(const uint4& raw, float (&v)[8]) {
  const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) { v[2 * i] = __uint_as_float(w[i] << 16); v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u); }
}

// The chunk's q or k of one head, rotated and multiplied by weight(row), as float rows of `ld` in LDS; rows from n on and
// columns d .. columns - 1 become zeros.  VEC: d, rot / 2 and the rows' addresses come in pieces of eight elements.
template <bool VEC, typename W>
__device__ __forceinline__ void rc_load_turned(float* dst, int ld, const bf16_t* rows, int row_stride, int n, int d, int columns,
                                               const float* table, int rot, W weight) {
  const int half = rot / 2;
  if (VEC) {
    const int pairs = half / 8, pieces = pairs + (d - rot) / 8;
    for (int idx = threadIdx.x; idx < RC_L * pieces; idx += 4 * WAVE) {
      const int t = idx / pieces, piece = idx - t * pieces;
      const int c0 = piece < pairs ? piece * 8 : rot + (piece - pairs) * 8;
      float a[8] = {}, b[8] = {};
      if (t < n) {
        const bf16_t* x = rows + (size_t)t * row_stride + c0;
        const float f = weight(t);
        rc_unpack8(*reinterpret_cast<const uint4*>(x), a);
        if (piece < pairs) {
          rc_unpack8(*reinterpret_cast<const uint4*>(x + half), b);
          const float* cs = table + (size_t)t * rot + c0;
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const float c = cs[i], sn = cs[half + i], u = a[i], v = b[i];
            a[i] = (u * c - v * sn) * f;
            b[i] = (v * c + u * sn) * f;
          }
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i) a[i] *= f;
        }
      }
      float* to = dst + t * ld + c0;
#pragma unroll
      for (int i = 0; i < 8; i += 4) *reinterpret_cast<float4*>(to + i) = make_float4(a[i], a[i + 1], a[i + 2], a[i + 3]);
      if (piece < pairs) {
#pragma unroll
        for (int i = 0; i < 8; i += 4) *reinterpret_cast<float4*>(to + half + i) = make_float4(b[i], b[i + 1], b[i + 2], b[i + 3]);
      }
    }
  } else {
    const int units = d - half;                              // pairs that turn, then coordinates that pass
    for (int idx = threadIdx.x; idx < RC_L * units; idx += 4 * WAVE) {
      const int t = idx / units, unit = idx - t * units;
      const int c0 = unit < half ? unit : half + unit;
      float a = 0.f, b = 0.f;
      if (t < n) {
        const bf16_t* x = rows + (size_t)t * row_stride + c0;
        const float f = weight(t);
        a = ld_bf(x);
        if (unit < half) {
          b = ld_bf(x + half);
          const float c = table[(size_t)t * rot + unit], sn = table[(size_t)t * rot + half + unit], u = a;
          a = (u * c - b * sn) * f;
          b = (b * c + u * sn) * f;
        } else {
          a *= f;
        }
      }
      dst[t * ld + c0] = a;
      if (unit < half) dst[t * ld + c0 + half] = b;
    }
  }
  if (d < columns)
    for (int idx = threadIdx.x; idx < RC_L * (columns - d); idx += 4 * WAVE)
      dst[idx / (columns - d) * ld + d + idx % (columns - d)] = 0.f;
}

// The chunk's values of one head as float rows of `ld`; rows from n on and columns from dv on become zeros.
template <bool VEC>
__device__ __forceinline__ void rc_load_values(float* dst, int ld, const bf16_t* rows, int row_stride, int n, int dv, int columns) {
  if (VEC) {
    const int pieces = dv / 8;
    for (int idx = threadIdx.x; idx < RC_L * pieces; idx += 4 * WAVE) {
      const int t = idx / pieces, c0 = (idx - t * pieces) * 8;
      float a[8] = {};
      if (t < n) rc_unpack8(*reinterpret_cast<const uint4*>(rows + (size_t)t * row_stride + c0), a);
#pragma unroll
      for (int i = 0; i < 8; i += 4) *reinterpret_cast<float4*>(dst + t * ld + c0 + i) = make_float4(a[i], a[i + 1], a[i + 2], a[i + 3]);
    }
  } else {
    for (int idx = threadIdx.x; idx < RC_L * dv; idx += 4 * WAVE) {
      const int t = idx / dv, c = idx - t * dv;
      dst[t * ld + c] = t < n ? ld_bf(rows + (size_t)t * row_stride + c) : 0.f;
    }
  }
  if (dv < columns)
    for (int idx = threadIdx.x; idx < RC_L * (columns - dv); idx += 4 * WAVE)
      dst[idx / (columns - dv) * ld + dv + idx % (columns - dv)] = 0.f;
}

// Rows in LDS, in floats: a row whose sixteen-byte pieces sixteen lanes read at once (one a row) lies 4 floats past a multiple
// of 32 from the next, a row of which sixteen lanes read neighbours 16 floats past one.
__host__ __device__ constexpr int rc_ld_rows(int columns) { return (columns + 31) / 32 * 32 + 4; }
__host__ __device__ constexpr int rc_ld_lines(int columns) { return (columns + 31) / 32 * 32 + 16; }

// local[g, h] [dv, d]: what chunk g adds to the state, sum_s c^(n-1-s) v_s k_s^T.  DB: blocks of sixteen columns of d.
// powers: float [heads, 65], c^0 .. c^64.  Dynamic LDS: 64 rows of k and 64 rows of v.
template <int DB, bool VEC>
__global__ void __launch_bounds__(4 * WAVE)
retention_chunk_local_kernel(const bf16_t* __restrict__ qkvg, int row_stride, const float* __restrict__ table, int rot,
                             const float* __restrict__ powers, const int* __restrict__ cu_q, int n_entries,
                             float* __restrict__ local, int heads, int d, int dv, int most) {
  extern __shared__ __attribute__((aligned(16))) float rc_lds[];
  constexpr int LDK = rc_ld_lines(16 * DB);
  const int g = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, grp = lane >> 4;
  rc_place p;
  if (!rc_find(cu_q, n_entries, g, most, p)) return;
  const int dvp = (dv + 15) / 16 * 16, ldv = rc_ld_lines(dvp);
  float* k_s = rc_lds;
  float* v_s = rc_lds + RC_L * LDK;
  const bf16_t* rows = qkvg + (size_t)p.lo * row_stride;
  const float* pw = powers + (size_t)h * (RC_L + 1);
  const float scale = 1.0f / sqrtf((float)d);
  const int last = p.n - 1;
  rc_load_turned<VEC>(k_s, LDK, rows + (size_t)(heads + h) * d, row_stride, p.n, d, 16 * DB, table + (size_t)p.lo * rot, rot,
                      [&](int t) { return scale * pw[last - t]; });
  rc_load_values<VEC>(v_s, ldv, rows + (size_t)2 * heads * d + (size_t)h * dv, row_stride, p.n, dv, dvp);
  __syncthreads();
  float* dst = local + ((size_t)g * heads + h) * dv * d;
  for (int vb = wave; vb * 16 < dv; vb += 4) {
    rc_floatx4 acc[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db) acc[db] = (rc_floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < RC_L; s += 4) {
      const float a = v_s[(s + grp) * ldv + vb * 16 + col];
#pragma unroll
      for (int db = 0; db < DB; ++db) acc[db] = RC_MFMA(a, k_s[(s + grp) * LDK + db * 16 + col], acc[db]);
    }
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int v = vb * 16 + 4 * grp + r, c = db * 16 + col;
        if (v < dv && c < d) dst[(size_t)v * d + c] = acc[db][r];
      }
  }
}

// From chunk to chunk, an element of the state a thread: local[g, h] becomes the state before chunk g, the state behind the
// entry's last chunk goes into its slot.
__global__ void __launch_bounds__(4 * WAVE)
retention_chunk_carry_kernel(float* __restrict__ state, size_t state_stride, const float* __restrict__ powers,
                             const int* __restrict__ cu_q, const int* __restrict__ first_position,
                             const int* __restrict__ state_slots, float* __restrict__ local, int heads, int plane, int most) {
  const int e = blockIdx.x, h = blockIdx.y, idx = blockIdx.z * (4 * WAVE) + threadIdx.x;
  const int len = cu_q[e + 1] - cu_q[e];
  if (len <= most || idx >= plane) return;
  int base = 0;
  for (int x = 0; x < e; ++x) {
    const int l = cu_q[x + 1] - cu_q[x];
    if (l > most) base += (l + RC_L - 1) / RC_L;
  }
  const int count = (len + RC_L - 1) / RC_L;
  float* mine = state + (size_t)state_slots[e] * state_stride + (size_t)h * plane + idx;
  const float whole = powers[(size_t)h * (RC_L + 1) + RC_L], rest = powers[(size_t)h * (RC_L + 1) + (len - (count - 1) * RC_L)];
  float x = first_position[e] == 0 ? 0.f : *mine;
  const size_t step = (size_t)heads * plane;
  float* src = local + ((size_t)base * heads + h) * plane + idx;
  for (int c0 = 0; c0 < count; c0 += 16) {
    float now[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) now[i] = c0 + i < count ? src[(size_t)(c0 + i) * step] : 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      if (c0 + i >= count) continue;
      src[(size_t)(c0 + i) * step] = x;
      x = fmaf(c0 + i == count - 1 ? rest : whole, x, now[i]);
    }
  }
  *mine = x;
}

// A chunk's reads.  Wave w has tokens 16 w .. 16 w + 15 and all values; `start` is what the carry left in `local`.  VB: blocks
// of sixteen values, DB: of sixteen coordinates.  Dynamic LDS: 64 rows of q (in whose place each wave then keeps its tokens'
// weights of the chunk's 64 keys), then 64 rows of k, later of v.
template <int DB, int VB, bool VEC>
__global__ void __launch_bounds__(4 * WAVE)
retention_chunk_read_kernel(const bf16_t* __restrict__ qkvg, int row_stride, const float* __restrict__ table, int rot,
                            const float* __restrict__ powers, const int* __restrict__ cu_q, int n_entries,
                            const int* __restrict__ first_position, const float* __restrict__ start,
                            bf16_t* __restrict__ out, int heads, int d,
                            int dv, float eps, int most) {
  extern __shared__ __attribute__((aligned(16))) float rc_lds[];
  constexpr int LDK = rc_ld_rows(16 * DB), LDQ = LDK > rc_ld_rows(RC_L) ? LDK : rc_ld_rows(RC_L), LDV = rc_ld_lines(16 * VB);
  const int g = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, grp = lane >> 4;
  rc_place p;
  if (!rc_find(cu_q, n_entries, g, most, p)) return;
  float* q_s = rc_lds;
  float* kv_s = rc_lds + RC_L * LDQ;
  const bf16_t* rows = qkvg + (size_t)p.lo * row_stride;
  const float* turn = table + (size_t)p.lo * rot;
  const float* pw = powers + (size_t)h * (RC_L + 1);
  const float scale = 1.0f / sqrtf((float)d);
  rc_load_turned<VEC>(q_s, LDQ, rows + (size_t)h * d, row_stride, p.n, d, 16 * DB, turn, rot, [](int) { return 1.f; });
  rc_load_turned<VEC>(kv_s, LDK, rows + (size_t)(heads + h) * d, row_stride, p.n, d, 16 * DB, turn, rot, [&](int) { return scale; });
  __syncthreads();
  const int t0 = 16 * wave;
  rc_floatx4 acc[VB], w[4];
#pragma unroll
  for (int vb = 0; vb < VB; ++vb) acc[vb] = (rc_floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kb = 0; kb < 4; ++kb) w[kb] = (rc_floatx4){0.f, 0.f, 0.f, 0.f};
  // The state before the chunk (none before a sequence's first), and q_t . k_s: both contract over d, a lane's four numbers
  // 16 step + 4 grp .. + 3 of a row of either operand serve four instructions.
  const bool carried = p.index > 0 || scalar_int(first_position + p.entry) != 0;
  const float* S = start + ((size_t)g * heads + h) * dv * d;
#pragma unroll
  for (int step = 0; step < DB; ++step) {
    const int c = 16 * step + 4 * grp;
    const float4 a = *reinterpret_cast<const float4*>(q_s + (t0 + col) * LDQ + c);
    if (carried) {
      float4 b[VB];
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) {
        const int v = vb * 16 + col;
        b[vb] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (VEC) {
          if (v < dv && c < d) b[vb] = *reinterpret_cast<const float4*>(S + (size_t)v * d + c);
        } else if (v < dv) {
          if (c < d) b[vb].x = S[(size_t)v * d + c];
          if (c + 1 < d) b[vb].y = S[(size_t)v * d + c + 1];
          if (c + 2 < d) b[vb].z = S[(size_t)v * d + c + 2];
          if (c + 3 < d) b[vb].w = S[(size_t)v * d + c + 3];
        }
      }
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) {
        acc[vb] = RC_MFMA(a.x, b[vb].x, acc[vb]);
        acc[vb] = RC_MFMA(a.y, b[vb].y, acc[vb]);
        acc[vb] = RC_MFMA(a.z, b[vb].z, acc[vb]);
        acc[vb] = RC_MFMA(a.w, b[vb].w, acc[vb]);
      }
    }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      if (kb > wave) continue;                               // keys behind all of the wave's tokens
      const float4 b = *reinterpret_cast<const float4*>(kv_s + (kb * 16 + col) * LDK + c);
      w[kb] = RC_MFMA(a.x, b.x, w[kb]);
      w[kb] = RC_MFMA(a.y, b.y, w[kb]);
      w[kb] = RC_MFMA(a.z, b.z, w[kb]);
      w[kb] = RC_MFMA(a.w, b.w, w[kb]);
    }
  }
  // Decays: token 4 grp + r of the wave in row r of a lane, key (or value) `col` in the lane.
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = t0 + 4 * grp + r;
    const float f = pw[t + 1];
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) acc[vb][r] *= f;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      const int s = kb * 16 + col;
      q_s[t * LDQ + s] = s <= t ? w[kb][r] * pw[s <= t ? t - s : 0] : 0.f;
    }
  }
  __syncthreads();                                           // the keys have been read by everybody
  rc_load_values<VEC>(kv_s, LDV, rows + (size_t)2 * heads * d + (size_t)h * dv, row_stride, p.n, dv, 16 * VB);
  __syncthreads();
#pragma unroll
  for (int step = 0; step < 4; ++step) {
    if (step > wave) continue;
    const float4 a = *reinterpret_cast<const float4*>(q_s + (t0 + col) * LDQ + 16 * step + 4 * grp);
    const float* v = kv_s + (16 * step + 4 * grp) * LDV + col;
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) {
      acc[vb] = RC_MFMA(a.x, v[vb * 16], acc[vb]);
      acc[vb] = RC_MFMA(a.y, v[LDV + vb * 16], acc[vb]);
      acc[vb] = RC_MFMA(a.z, v[2 * LDV + vb * 16], acc[vb]);
      acc[vb] = RC_MFMA(a.w, v[3 * LDV + vb * 16], acc[vb]);
    }
  }
  const bf16_t* gates = rows + (size_t)2 * heads * d + (size_t)(heads + h) * dv;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = t0 + 4 * grp + r;
    float sq = 0.f;
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) sq = fmaf(acc[vb][r], acc[vb][r], sq);
    const float inv = 1.0f / sqrtf(rt_row_sum16(sq) / (float)dv + eps);
    if (t >= p.n) continue;
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) {
      const int v = vb * 16 + col;
      if (v >= dv) continue;
      const float z = ld_bf(gates + (size_t)t * row_stride + v);
      st(out + (size_t)(p.lo + t) * heads * dv + (size_t)h * dv + v, acc[vb][r] * inv * (z / (1.0f + expf(-z))));
    }
  }
}

// The chunked form for entries of more than `most` rows (bfloat16 rows).  powers: float [heads, 65]; scratch: float
// [max_chunks, heads, dv, d], max_chunks at least the number of chunks of all entries (rows / 64 + entries is enough).
extern "C" int ta_retention_chunked(const void* qkvg, int row_stride, const void* table, int rot, const void* powers, void* state,
                                    long state_stride, const void* cu_q, const void* first_position, const void* state_slots,
                                    void* scratch, void* out, int n_entries, int max_chunks, int heads, int d, int dv, float eps,
                                    int most, hipStream_t stream) {
  if (n_entries <= 0 || max_chunks <= 0) return 0;
  if (d < 1 || d > 256 || dv < 1 || dv > 256 || heads < 1 || heads > 65535 || rot < 0 || rot % 2 || rot > d ||
      (rot > 0 && !table) || most < 0 || state_stride < (long)heads * d * dv)
    return -1;
  dim3 per_chunk(max_chunks, heads), per_entry(n_entries, heads, (unsigned)(((long)d * dv + 4 * WAVE - 1) / (4 * WAVE)));
  const bool vec = d % 8 == 0 && dv % 8 == 0 && (rot / 2) % 8 == 0 && row_stride % 8 == 0 && ((uintptr_t)qkvg & 15) == 0;
#define LOCAL(DBV, VV)                                                                                                    \
  {                                                                                                                       \
    const int lds = 4 * RC_L * (rc_ld_lines(16 * DBV) + rc_ld_lines((dv + 15) / 16 * 16));                                \
    if (lds > 48 * 1024) {                                                                                                \
      const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_chunk_local_kernel<DBV, VV>),   \
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, lds);                        \
      if (err != hipSuccess) return (int)err;                                                                             \
    }                                                                                                                     \
    retention_chunk_local_kernel<DBV, VV><<<per_chunk, 4 * WAVE, lds, stream>>>((const bf16_t*)qkvg, row_stride,           \
        (const float*)table, rot, (const float*)powers, (const int*)cu_q, n_entries, (float*)scratch, heads, d, dv, most); \
  }
#define READ(DBV, VBV, VV)                                                                                                \
  {                                                                                                                       \
    constexpr int ldk = rc_ld_rows(16 * DBV), ldq = ldk > rc_ld_rows(RC_L) ? ldk : rc_ld_rows(RC_L), ldv = rc_ld_lines(16 * VBV); \
    constexpr int lds = 4 * RC_L * (ldq + (ldk > ldv ? ldk : ldv));                                                        \
    static_assert(lds <= 160 * 1024, "a chunk's rows must fit a compute unit's LDS");                                     \
    if (lds > 48 * 1024) {                                                                                                \
      const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_chunk_read_kernel<DBV, VBV, VV>), \
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, lds);                        \
      if (err != hipSuccess) return (int)err;                                                                             \
    }                                                                                                                     \
    retention_chunk_read_kernel<DBV, VBV, VV><<<per_chunk, 4 * WAVE, lds, stream>>>((const bf16_t*)qkvg, row_stride,       \
        (const float*)table, rot, (const float*)powers, (const int*)cu_q, n_entries, (const int*)first_position,          \
        (const float*)scratch, (bf16_t*)out, heads, d, dv, eps, most);                                                     \
  }
  const int db = (d + 15) / 16, vb = (dv + 15) / 16;
#define BY_D(WHAT)                                                                                                        \
  if (db <= 1) WHAT(1) else if (db <= 2) WHAT(2) else if (db <= 4) WHAT(4) else if (db <= 8) WHAT(8) else WHAT(16)
#define LOCAL_D(DBV) { if (vec) LOCAL(DBV, true) else LOCAL(DBV, false) }
#define READ_V(DBV, VBV) { if (vec) READ(DBV, VBV, true) else READ(DBV, VBV, false) }
#define READ_D(DBV)                                                                                                       \
  { if (vb <= 1) READ_V(DBV, 1) else if (vb <= 2) READ_V(DBV, 2) else if (vb <= 4) READ_V(DBV, 4)                          \
    else if (vb <= 8) READ_V(DBV, 8) else READ_V(DBV, 16) }
  BY_D(LOCAL_D)
  retention_chunk_carry_kernel<<<per_entry, 4 * WAVE, 0, stream>>>((float*)state, (size_t)state_stride, (const float*)powers,
      (const int*)cu_q, (const int*)first_position, (const int*)state_slots, (float*)scratch, heads, d * dv, most);
  BY_D(READ_D)
#undef READ_D
#undef READ_V
#undef LOCAL_D
#undef BY_D
#undef READ
#undef LOCAL
  return LAUNCH_STATUS();
}

// Heads of up to 256 coordinates and 256 values.  `most`: the longest entry this form takes.
extern "C" int ta_retention_scan(const void* qkvg, int row_stride, const void* table, int rot, const void* decays, void* state,
                                 long state_stride, const void* cu_q, const void* first_position, const void* state_slots,
                                 void* out, int n_entries, int heads, int d, int dv, float eps, int most, int dtype,
                                 hipStream_t stream) {
  if (n_entries <= 0) return 0;
  if (d < 1 || d > 256 || dv < 1 || dv > 256 || heads < 1 || heads > 65535 || rot < 0 || rot % 2 || rot > d ||
      (rot > 0 && !table) || state_stride < (long)heads * d * dv)
    return -1;
  dim3 grid(n_entries, heads);
  // The threads have to cover 2 (d - rot / 2) units of q and k, the values, and dv rows of which a lane keeps four.
  const int need = 2 * d > 4 * dv ? 2 * d : 4 * dv, per = (d + 15) / 16;
#define SCAN(TT, PP, TH) retention_scan_kernel<TT, PP, TH><<<grid, TH, 0, stream>>>((const TT*)qkvg, row_stride,           \
      (const float*)table, rot, (const float*)decays, (float*)state, (size_t)state_stride, (const int*)cu_q,               \
      (const int*)first_position, (const int*)state_slots, (TT*)out, heads, d, dv, eps, most)
#define SCANS(TT, TH) if (per <= 1) SCAN(TT, 1, TH); else if (per <= 2) SCAN(TT, 2, TH); else if (per <= 4) SCAN(TT, 4, TH); \
                      else if (per <= 8) SCAN(TT, 8, TH); else SCAN(TT, 16, TH)
#define SIZES(TT) if (need <= 256) { SCANS(TT, 256); } else if (need <= 512) { SCANS(TT, 512); } else { SCANS(TT, 1024); }
  if (dtype == DT_F32) { SIZES(float); } else { SIZES(bf16_t); }
#undef SIZES
#undef SCANS
#undef SCAN
  return LAUNCH_STATUS();
}
