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
