// What stands between the joined q/k/v projection and the attention, for mixers whose rotation covers only the first
// coordinates of a head: bias, an RMS norm over all query rows at once and over all key rows at once, the rotation
// with angles formed in the kernel, and the write of keys and values into their pages.  A workgroup a token.
#include "common.h"

#define RP_THREADS 256
#define RP_MAX_HALF 128

// qkv: [n_tokens, row_stride]; a row holds n_q query heads and n_k key heads of d elements, then n_v value heads of dv
// elements (what lies behind them is not touched).  bias (float, or null) is added first.  q_norm / k_norm (float
// [n_q d] / [n_k d], or null): the query part (the key part) is divided by its root mean square over all its
// elements (eps inside the root) and multiplied by the weight.  rates (float [rot / 2]): coordinates i and
// i + rot / 2 of every query and key head turn by the angle position * rates[i], formed and taken sine and cosine of
// in float; coordinates from rot on pass.  slots (or null): page * page_size + offset of each token, negative =
// nothing is stored.  Key pages [n_pages, n_k, page_size, d]; value pages transposed inside a page,
// [n_pages, n_v, dv, page_size].
template <typename T>
__global__ void __launch_bounds__(RP_THREADS)
norm_rotate_store_kernel(T* __restrict__ qkv, int row_stride, const float* __restrict__ bias,
                         const int* __restrict__ positions, const float* __restrict__ rates, int rot,
                         const int* __restrict__ slots, T* __restrict__ k_pages, T* __restrict__ v_pages,
                         int n_q, int n_k, int n_v, int d, int dv, int page_size,
                         const float* __restrict__ q_norm, const float* __restrict__ k_norm, float eps) {
  __shared__ float scratch[16];
  __shared__ float cos_s[RP_MAX_HALF], sin_s[RP_MAX_HALF];
  const int t = blockIdx.x;
  T* row = qkv + (size_t)t * row_stride;
  const int q_size = n_q * d, k_size = n_k * d, half = rot / 2;
  const int slot = slots ? slots[t] : -1;
  const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  if (half > 0) {
    const float position = (float)positions[t];
    for (int i = threadIdx.x; i < half; i += RP_THREADS) {
      float s, c;
      sincosf(position * rates[i], &s, &c);
      cos_s[i] = c;
      sin_s[i] = s;
    }
  }
  float inv_q = 1.f, inv_k = 1.f;
  if (q_norm) {
    float sq = 0.f;
    for (int i = threadIdx.x; i < q_size; i += RP_THREADS) {
      const float v = ld(row + i) + (bias ? bias[i] : 0.f);
      sq += v * v;
    }
    inv_q = 1.0f / sqrtf(block_sum(sq, scratch) / (float)q_size + eps);
  }
  if (k_norm && k_size > 0) {
    float sq = 0.f;
    for (int i = threadIdx.x; i < k_size; i += RP_THREADS) {
      const float v = ld(row + q_size + i) + (bias ? bias[q_size + i] : 0.f);
      sq += v * v;
    }
    inv_k = 1.0f / sqrtf(block_sum(sq, scratch) / (float)k_size + eps);
  }
  __syncthreads();
  const bool changes = bias || q_norm || k_norm;
  // The pairs that turn.
  for (int idx = threadIdx.x; idx < (n_q + n_k) * half; idx += RP_THREADS) {
    const int head = idx / half, i = idx - head * half;
    const int at = head * d + i, with = at + half;
    float a = ld(row + at), b = ld(row + with);
    if (bias) { a += bias[at]; b += bias[with]; }
    const bool key = head >= n_q;
    if (!key && q_norm) { a *= inv_q * q_norm[at]; b *= inv_q * q_norm[with]; }
    if (key && k_norm) { a *= inv_k * k_norm[at - q_size]; b *= inv_k * k_norm[with - q_size]; }
    const float c = cos_s[i], s = sin_s[i];
    const float r1 = a * c - b * s, r2 = b * c + a * s;
    st(row + at, r1);
    st(row + with, r2);
    if (key && slot >= 0) {
      T* dst = k_pages + (((size_t)page * n_k + (head - n_q)) * page_size + off) * d;
      st(dst + i, r1);
      st(dst + half + i, r2);
    }
  }
  // The coordinates that pass.
  const int rest = d - rot;
  for (int idx = threadIdx.x; idx < (n_q + n_k) * rest; idx += RP_THREADS) {
    const int head = idx / rest, i = rot + (idx - head * rest);
    const int at = head * d + i;
    float a = ld(row + at);
    if (bias) a += bias[at];
    const bool key = head >= n_q;
    if (!key && q_norm) a *= inv_q * q_norm[at];
    if (key && k_norm) a *= inv_k * k_norm[at - q_size];
    if (changes) st(row + at, a);
    if (key && slot >= 0) {
      if (changes) a = ld(row + at);           // the page holds what the row holds, rounded the same way
      st(k_pages + (((size_t)page * n_k + (head - n_q)) * page_size + off) * d + i, a);
    }
  }
  // Values.
  const int v_at = q_size + k_size;
  for (int idx = threadIdx.x; idx < n_v * dv; idx += RP_THREADS) {
    float a = ld(row + v_at + idx);
    if (bias) { a += bias[v_at + idx]; st(row + v_at + idx, a); }
    if (slot >= 0) {
      const int head = idx / dv, i = idx - head * dv;
      st(v_pages + (((size_t)page * n_v + head) * dv + i) * page_size + off, a);
    }
  }
}

extern "C" int ta_norm_rotate_store(void* qkv, int row_stride, const void* bias, const void* positions, const void* rates,
                                    int rot, const void* slots, void* k_pages, void* v_pages, int n_tokens, int n_q,
                                    int n_k, int n_v, int d, int dv, int page_size, const void* q_norm,
                                    const void* k_norm, float eps, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (rot < 0 || rot % 2 || rot > d || rot / 2 > RP_MAX_HALF || d <= 0 || dv <= 0 || n_q < 0 || n_k < 0 || n_v < 0) return -1;
  if (rot > 0 && !rates) return -1;
  if (dtype == DT_F32)
    norm_rotate_store_kernel<float><<<n_tokens, RP_THREADS, 0, stream>>>(
        (float*)qkv, row_stride, (const float*)bias, (const int*)positions, (const float*)rates, rot, (const int*)slots,
        (float*)k_pages, (float*)v_pages, n_q, n_k, n_v, d, dv, page_size, (const float*)q_norm, (const float*)k_norm, eps);
  else
    norm_rotate_store_kernel<bf16_t><<<n_tokens, RP_THREADS, 0, stream>>>(
        (bf16_t*)qkv, row_stride, (const float*)bias, (const int*)positions, (const float*)rates, rot, (const int*)slots,
        (bf16_t*)k_pages, (bf16_t*)v_pages, n_q, n_k, n_v, d, dv, page_size, (const float*)q_norm, (const float*)k_norm, eps);
  return LAUNCH_STATUS();
}

// Rows of qkv as above without a bias: n_q query heads and n_k key heads of d elements, then n_k value heads of dv (tied: no
// value heads, the keys are the values too and dv = d; without v_pages only the keys are stored).  The query heads are multiplied by
// 1 + coef * ln(floor((position + 1) / every) + 1), formed in float, and go back into their rows; keys and values go into
// their pages as they are.  A workgroup a token.
template <typename T>
__global__ void __launch_bounds__(RP_THREADS)
temper_store_kernel(T* __restrict__ qkv, int row_stride, const int* __restrict__ positions, float coef, int every,
                    const int* __restrict__ slots, T* __restrict__ k_pages, T* __restrict__ v_pages, int n_q, int n_k, int d,
                    int dv, int page_size, int tied) {
  const int t = blockIdx.x;
  T* row = qkv + (size_t)t * row_stride;
  const int steps = (positions[t] + 1) / every;
  if (steps > 0 && coef != 0.f) {                            // (before the first step the factor is 1)
    const float factor = 1.f + coef * logf((float)steps + 1.f);
    for (int i = threadIdx.x; i < n_q * d; i += RP_THREADS) st(row + i, ld(row + i) * factor);
  }
  const int slot = slots ? slots[t] : -1;
  if (slot < 0) return;
  const int page = slot / page_size, off = slot % page_size;
  const T* keys = row + n_q * d;
  const T* values = tied ? keys : keys + n_k * d;
  for (int i = threadIdx.x; i < n_k * d; i += RP_THREADS)
    k_pages[(((size_t)page * n_k + i / d) * page_size + off) * d + i % d] = keys[i];
  if (!v_pages) return;
  for (int i = threadIdx.x; i < n_k * dv; i += RP_THREADS)    // head i / dv, coordinate i % dv: one line of a transposed page
    v_pages[((size_t)page * n_k * dv + i) * page_size + off] = values[i];
}

// The same for bfloat16 rows in whole pieces of eight elements (d and dv multiples of 8, everything 16-byte aligned): a
// thread a piece; the pieces of a token lie over grid.y workgroups.
__global__ void __launch_bounds__(RP_THREADS)
temper_store_vec_kernel(bf16_t* __restrict__ qkv, int row_stride, const int* __restrict__ positions, float coef, int every,
                        const int* __restrict__ slots, bf16_t* __restrict__ k_pages, bf16_t* __restrict__ v_pages, int n_q,
                        int n_k, int d, int dv, int page_size, int tied) {
  HELD(qkv, row_stride, positions, coef, every, slots, k_pages, v_pages, n_q, n_k, d, dv, page_size, tied);
  const int t = blockIdx.x, i = (blockIdx.y * RP_THREADS + threadIdx.x) * 8;
  const int q_size = n_q * d, k_size = n_k * d, used = q_size + k_size + (tied ? 0 : n_k * dv);
  if (i >= used) return;
  bf16_t* at = qkv + (size_t)t * row_stride + i;
  const uint4 raw = *reinterpret_cast<const uint4*>(at);
  const int position = scalar_int(positions + t), slot = slots ? scalar_int(slots + t) : -1;
  if (i < q_size) {
    const int steps = (position + 1) / every;
    if (steps == 0 || coef == 0.f) return;
    const float factor = 1.f + coef * logf((float)steps + 1.f);
    const uint32_t in[4] = {raw.x, raw.y, raw.z, raw.w};
    uint32_t out[4];
#pragma unroll
    for (int e = 0; e < 4; ++e)
      out[e] = (uint32_t)float_to_bf16_bits(bf16_bits_to_float(in[e] & 0xffffu) * factor) |
               ((uint32_t)float_to_bf16_bits(bf16_bits_to_float(in[e] >> 16) * factor) << 16);
    *reinterpret_cast<uint4*>(at) = make_uint4(out[0], out[1], out[2], out[3]);
    return;
  }
  if (slot < 0) return;
  const int page = slot / page_size, off = slot % page_size;
  const bool key = i < q_size + k_size;
  if (key) {
    const int j = i - q_size;
    *reinterpret_cast<uint4*>(k_pages + (((size_t)page * n_k + j / d) * page_size + off) * d + j % d) = raw;
  }
  if ((!key || tied) && v_pages) {
    const int j = i - q_size - (tied ? 0 : k_size);           // head j / dv, coordinate j % dv
    bf16_t* to = v_pages + ((size_t)page * n_k * dv + j) * page_size + off;
    const uint32_t in[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int e = 0; e < 8; ++e) to[(size_t)e * page_size].bits = (uint16_t)(in[e >> 1] >> (16 * (e & 1)));
  }
}

extern "C" int ta_temper_store(void* qkv, int row_stride, const void* positions, float coef, int every, const void* slots,
                               void* k_pages, void* v_pages, int n_tokens, int n_q, int n_k, int d, int dv, int page_size,
                               int tied, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (every < 1 || d <= 0 || dv <= 0 || n_q <= 0 || n_k < 0 || page_size <= 0 || (tied && dv != d) ||
      (slots && (!k_pages || (!v_pages && !tied))))
    return -1;
  const int used = (n_q + n_k) * d + (tied ? 0 : n_k * dv);
  if (used > row_stride) return -1;
  if (dtype == DT_BF16 && d % 8 == 0 && dv % 8 == 0 && row_stride % 8 == 0 &&
      (((uintptr_t)qkv | (uintptr_t)k_pages | (uintptr_t)v_pages) & 15) == 0) {
    temper_store_vec_kernel<<<dim3(n_tokens, (used / 8 + RP_THREADS - 1) / RP_THREADS), RP_THREADS, 0, stream>>>(
        (bf16_t*)qkv, row_stride, (const int*)positions, coef, every, (const int*)slots, (bf16_t*)k_pages, (bf16_t*)v_pages,
        n_q, n_k, d, dv, page_size, tied);
    return LAUNCH_STATUS();
  }
#define TEMPER(TT) temper_store_kernel<TT><<<n_tokens, RP_THREADS, 0, stream>>>((TT*)qkv, row_stride, (const int*)positions, \
      coef, every, (const int*)slots, (TT*)k_pages, (TT*)v_pages, n_q, n_k, d, dv, page_size, tied)
  if (dtype == DT_F32) TEMPER(float); else TEMPER(bf16_t);
#undef TEMPER
  return LAUNCH_STATUS();
}

// table[t] = [cosines | sines] (each rot / 2 floats) of positions[t] * rates[i], formed and taken in float, times magnitude.
__global__ void __launch_bounds__(RP_THREADS)
rotation_table_kernel(const int* __restrict__ positions, const float* __restrict__ rates, float magnitude, int half,
                      float* __restrict__ table, int total) {
  const int idx = blockIdx.x * RP_THREADS + threadIdx.x;
  if (idx >= total) return;
  const int t = idx / half, i = idx - t * half;
  float s, c;
  sincosf((float)positions[t] * rates[i], &s, &c);
  table[(size_t)t * 2 * half + i] = magnitude * c;
  table[(size_t)t * 2 * half + half + i] = magnitude * s;
}

// A wave a head of a token.  Rows of qkv as above: n_q query heads and n_k key heads of d elements, n_v value heads of dv.
// q_norm / k_norm (float [d], or null): the head is divided by its root mean square (eps inside the root) and multiplied
// by the weight; then the first `rot` coordinates turn by the token's row of `table` ([cosines | sines]).  norm_values:
// a value head is divided by its root mean square; share (float [1], or null): it becomes (1 - share) v + share * first,
// first[t * first_stride + ...] being the token's value heads of another layer.  Heads go back into their rows, keys and
// values also into their pages (slots as above), rounded once.
template <typename T, int PER>
__global__ void __launch_bounds__(RP_THREADS)
head_norm_rotate_store_kernel(T* __restrict__ qkv, int row_stride, const float* __restrict__ table, int rot,
                              const int* __restrict__ slots, T* __restrict__ k_pages, T* __restrict__ v_pages, int n_q,
                              int n_k, int n_v, int d, int dv, int page_size, const float* __restrict__ q_norm,
                              const float* __restrict__ k_norm, int norm_values, const T* __restrict__ first,
                              int first_stride, const float* __restrict__ share, float eps) {
  __shared__ float row_s[RP_THREADS / WAVE][PER * WAVE];
  const int t = blockIdx.x, lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
  const int head = blockIdx.y * (RP_THREADS / WAVE) + wave;
  if (head >= n_q + n_k + n_v) return;                       // (nobody waits for anybody in this kernel)
  const bool value = head >= n_q + n_k, key = !value && head >= n_q;
  const int h = value ? head - n_q - n_k : key ? head - n_q : head, n = value ? dv : d;
  T* row = qkv + (size_t)t * row_stride + (value ? (size_t)(n_q + n_k) * d + (size_t)h * dv : (size_t)head * d);
  const float* weight = value ? nullptr : key ? k_norm : q_norm;
  const T* other = (value && share) ? first + (size_t)t * first_stride + (size_t)h * dv : nullptr;
  const int slot = slots ? slots[t] : -1, half = rot / 2;
  float x[PER], w[PER], o[PER], c[PER], s[PER], sq = 0.f;
#pragma unroll
  for (int r = 0; r < PER; ++r) {
    const int i = lane + r * WAVE;
    x[r] = i < n ? ld(row + i) : 0.f;
    w[r] = (weight && i < n) ? weight[i] : 1.f;
    o[r] = (other && i < n) ? ld(other + i) : 0.f;
    const bool turns = !value && i < rot;
    c[r] = turns ? table[(size_t)t * rot + (i < half ? i : i - half)] : 1.f;
    s[r] = turns ? table[(size_t)t * rot + half + (i < half ? i : i - half)] : 0.f;
  }
  const float mix = other ? share[0] : 0.f;
  if (weight || (value && norm_values)) {
#pragma unroll
    for (int r = 0; r < PER; ++r) sq = fmaf(x[r], x[r], sq);
    const float inv = 1.0f / sqrtf(wave_sum(sq) / (float)n + eps);
#pragma unroll
    for (int r = 0; r < PER; ++r) x[r] *= inv * w[r];
  }
  if (other) {
#pragma unroll
    for (int r = 0; r < PER; ++r) x[r] = (1.0f - mix) * x[r] + mix * o[r];
  }
  if (!value && half > 0) {
    // A coordinate's partner lies with another lane: through the wave's own row in LDS.
#pragma unroll
    for (int r = 0; r < PER; ++r) row_s[wave][lane + r * WAVE] = x[r];
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int r = 0; r < PER; ++r) {
      const int i = lane + r * WAVE;
      if (i >= rot) continue;
      const float with = row_s[wave][i < half ? i + half : i - half];
      x[r] = i < half ? x[r] * c[r] - with * s[r] : x[r] * c[r] + with * s[r];
    }
  }
  const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
#pragma unroll
  for (int r = 0; r < PER; ++r) {
    const int i = lane + r * WAVE;
    if (i >= n) continue;
    st(row + i, x[r]);
    if (slot < 0) continue;
    if (key) st(k_pages + (((size_t)page * n_k + h) * page_size + off) * d + i, x[r]);
    if (value) st(v_pages + (((size_t)page * n_v + h) * dv + i) * page_size + off, x[r]);
  }
}

// The same for bfloat16 heads in whole pieces of eight elements (d, dv and rot / 2 multiples of 8, everything 16-byte aligned):
// LPH lanes a head, a piece a lane, so a wave has 64 / LPH heads of a token; a head's sum of squares goes over its LPH lanes,
// and the piece that turns together with a lane's lies with another of them.
template <int LPH>
__global__ void __launch_bounds__(RP_THREADS)
head_norm_rotate_store_vec_kernel(bf16_t* __restrict__ qkv, int row_stride, const float* __restrict__ table, int rot,
                                  const int* __restrict__ slots, bf16_t* __restrict__ k_pages, bf16_t* __restrict__ v_pages,
                                  int n_q, int n_k, int n_v, int d, int dv, int page_size, const float* __restrict__ q_norm,
                                  const float* __restrict__ k_norm, int norm_values, const bf16_t* __restrict__ first,
                                  int first_stride, const float* __restrict__ share, float eps) {
  const int t = blockIdx.x, lane = threadIdx.x & (WAVE - 1), piece = lane % LPH;
  const int head = (blockIdx.y * RP_THREADS + threadIdx.x) / LPH;
  const bool there = head < n_q + n_k + n_v;                 // (lanes without a head go along: they take part in the exchanges)
  const bool value = head >= n_q + n_k, key = !value && head >= n_q;
  const int h = value ? head - n_q - n_k : key ? head - n_q : head, n = value ? dv : d, i = piece * 8;
  const bool in = there && i < n;
  bf16_t* at = qkv + (size_t)t * row_stride + (value ? (size_t)(n_q + n_k) * d + (size_t)h * dv : (size_t)head * d) + i;
  const float* weight = value ? nullptr : key ? k_norm : q_norm;
  const int slot = slots ? slots[t] : -1, half = rot / 2;
  const bool turns = in && !value && i < rot, upper = i >= half;
  uint4 raw = make_uint4(0, 0, 0, 0), other = make_uint4(0, 0, 0, 0);
  float4 w0 = make_float4(1.f, 1.f, 1.f, 1.f), w1 = w0, c0 = w0, c1 = w0, s0 = make_float4(0.f, 0.f, 0.f, 0.f), s1 = s0;
  if (in) raw = *reinterpret_cast<const uint4*>(at);
  if (in && value && share) other = *reinterpret_cast<const uint4*>(first + (size_t)t * first_stride + (size_t)h * dv + i);
  if (in && weight) { w0 = *reinterpret_cast<const float4*>(weight + i); w1 = *reinterpret_cast<const float4*>(weight + i + 4); }
  if (turns) {
    const float4* cs = reinterpret_cast<const float4*>(table + (size_t)t * rot + (upper ? i - half : i));
    c0 = cs[0];
    c1 = cs[1];
    s0 = cs[half / 4];
    s1 = cs[half / 4 + 1];
  }
  float x[8] = {bf16_bits_to_float(raw.x & 0xffffu), bf16_bits_to_float(raw.x >> 16), bf16_bits_to_float(raw.y & 0xffffu),
                bf16_bits_to_float(raw.y >> 16), bf16_bits_to_float(raw.z & 0xffffu), bf16_bits_to_float(raw.z >> 16),
                bf16_bits_to_float(raw.w & 0xffffu), bf16_bits_to_float(raw.w >> 16)};
  float sq = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) sq = fmaf(x[e], x[e], sq);
#pragma unroll
  for (int off = LPH / 2; off > 0; off >>= 1) sq += __shfl_xor(sq, off, WAVE);
  if (weight || (value && norm_values)) {
    const float inv = 1.0f / sqrtf(sq / (float)n + eps);
    const float w[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] *= inv * w[e];
  }
  if (value && share) {
    const float mix = share[0];
    const float o[8] = {bf16_bits_to_float(other.x & 0xffffu), bf16_bits_to_float(other.x >> 16), bf16_bits_to_float(other.y & 0xffffu),
                        bf16_bits_to_float(other.y >> 16), bf16_bits_to_float(other.z & 0xffffu), bf16_bits_to_float(other.z >> 16),
                        bf16_bits_to_float(other.w & 0xffffu), bf16_bits_to_float(other.w >> 16)};
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = (1.0f - mix) * x[e] + mix * o[e];
  }
  if (half > 0) {
    const int partner = turns ? lane + (upper ? -half : half) / 8 : lane;
    const float c[8] = {c0.x, c0.y, c0.z, c0.w, c1.x, c1.y, c1.z, c1.w}, sn[8] = {s0.x, s0.y, s0.z, s0.w, s1.x, s1.y, s1.z, s1.w};
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float with = __shfl(x[e], partner, WAVE);
      x[e] = x[e] * c[e] + (upper ? with : -with) * sn[e];
    }
  }
  if (!in) return;
  uint32_t packed[4];
#pragma unroll
  for (int e = 0; e < 4; ++e)
    packed[e] = (uint32_t)float_to_bf16_bits(x[2 * e]) | ((uint32_t)float_to_bf16_bits(x[2 * e + 1]) << 16);
  const uint4 out = make_uint4(packed[0], packed[1], packed[2], packed[3]);
  *reinterpret_cast<uint4*>(at) = out;
  if (slot < 0) return;
  const int page = slot / page_size, off = slot % page_size;
  if (key) *reinterpret_cast<uint4*>(k_pages + (((size_t)page * n_k + h) * page_size + off) * d + i) = out;
  if (value) {
    bf16_t* to = v_pages + (((size_t)page * n_v + h) * dv + i) * page_size + off;
#pragma unroll
    for (int e = 0; e < 8; ++e) to[(size_t)e * page_size].bits = (uint16_t)(packed[e >> 1] >> (16 * (e & 1)));
  }
}

extern "C" int ta_rotation_table(const void* positions, const void* rates, float magnitude, int rot, void* table,
                                 int n_tokens, hipStream_t stream) {
  if (n_tokens <= 0 || rot <= 0) return 0;
  const long total = (long)n_tokens * (rot / 2);
  if (rot % 2 || total > 0x7fffffffL - RP_THREADS) return -1;
  rotation_table_kernel<<<(unsigned)((total + RP_THREADS - 1) / RP_THREADS), RP_THREADS, 0, stream>>>(
      (const int*)positions, (const float*)rates, magnitude, rot / 2, (float*)table, (int)total);
  return LAUNCH_STATUS();
}

extern "C" int ta_head_norm_rotate_store(void* qkv, int row_stride, const void* table, int rot, const void* slots, void* k_pages,
                                         void* v_pages, int n_tokens, int n_q, int n_k, int n_v, int d, int dv, int page_size,
                                         const void* q_norm, const void* k_norm, int norm_values, const void* first,
                                         int first_stride, const void* share, float eps, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (rot < 0 || rot % 2 || rot > d || d <= 0 || dv <= 0 || n_q < 0 || n_k < 0 || n_v < 0 || n_q + n_k + n_v <= 0) return -1;
  if ((rot > 0 && !table) || (share && !first) || d > 8 * WAVE || dv > 8 * WAVE) return -1;
  const int waves = RP_THREADS / WAVE, most = d > dv ? d : dv;
  dim3 grid(n_tokens, (n_q + n_k + n_v + waves - 1) / waves);
  const uintptr_t bases = (uintptr_t)qkv | (uintptr_t)table | (uintptr_t)k_pages | (uintptr_t)q_norm | (uintptr_t)k_norm |
                          (share ? (uintptr_t)first : 0);
  if (dtype == DT_BF16 && d % 8 == 0 && dv % 8 == 0 && rot % 16 == 0 && row_stride % 8 == 0 && most <= 256 && (bases & 15) == 0 &&
      (!share || first_stride % 8 == 0)) {
#define STORE_VEC(LL) head_norm_rotate_store_vec_kernel<LL><<<dim3(n_tokens, ((n_q + n_k + n_v) * LL + RP_THREADS - 1) / RP_THREADS), \
      RP_THREADS, 0, stream>>>((bf16_t*)qkv, row_stride, (const float*)table, rot, (const int*)slots, (bf16_t*)k_pages,       \
      (bf16_t*)v_pages, n_q, n_k, n_v, d, dv, page_size, (const float*)q_norm, (const float*)k_norm, norm_values,             \
      (const bf16_t*)first, first_stride, (const float*)share, eps)
    if (most <= 64) STORE_VEC(8); else if (most <= 128) STORE_VEC(16); else STORE_VEC(32);
#undef STORE_VEC
    return LAUNCH_STATUS();
  }
#define STORE(TT, PP) head_norm_rotate_store_kernel<TT, PP><<<grid, RP_THREADS, 0, stream>>>((TT*)qkv, row_stride,          \
      (const float*)table, rot, (const int*)slots, (TT*)k_pages, (TT*)v_pages, n_q, n_k, n_v, d, dv, page_size,              \
      (const float*)q_norm, (const float*)k_norm, norm_values, (const TT*)first, first_stride, (const float*)share, eps)
#define STORES(TT) if (most <= WAVE) STORE(TT, 1); else if (most <= 2 * WAVE) STORE(TT, 2);                                  \
                   else if (most <= 4 * WAVE) STORE(TT, 4); else STORE(TT, 8)
  if (dtype == DT_F32) { STORES(float); } else { STORES(bf16_t); }
#undef STORES
#undef STORE
  return LAUNCH_STATUS();
}
