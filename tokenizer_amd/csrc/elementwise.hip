// Embedding gather, residual-add + RMSNorm, gated activation.
#include "common.h"

// out[t, :] = table[ids[t], :] widened to float (the residual stream is float), times `scale`.
template <typename T>
__global__ void embedding_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                 float* __restrict__ out, int hidden, int vocab, float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  if (id < 0 || id >= vocab) id = 0;  // the host rejects such ids before the launch
  const T* row = table + (size_t)id * hidden;
  float* dst = out + (size_t)t * hidden;
  for (int h = threadIdx.x; h < hidden; h += blockDim.x) dst[h] = ld(row + h) * scale;
}

// The same for bfloat16 tables whose rows are a multiple of eight long: sixteen bytes a thread.
__global__ void __launch_bounds__(256)
embedding_vec_kernel(const int* __restrict__ ids, const bf16_t* __restrict__ table, float* __restrict__ out,
                     int hidden, int vocab, float scale) {
  HELD(ids, table, out, hidden, vocab, scale);
  const int t = blockIdx.x;
  int id = scalar_int(ids + t);
  if (id < 0 || id >= vocab) id = 0;  // the host rejects such ids before the launch
  const uint4* row = reinterpret_cast<const uint4*>(table + (size_t)id * hidden);
  float* dst = out + (size_t)t * hidden;
  for (int h8 = threadIdx.x; h8 * 8 < hidden; h8 += blockDim.x) {
    const uint4 raw = row[h8];
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
    float v[8];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16) * scale;
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u) * scale;
    }
    *reinterpret_cast<float4*>(dst + h8 * 8) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(dst + h8 * 8 + 4) = make_float4(v[4], v[5], v[6], v[7]);
  }
}

// For output row i: r = rows ? rows[i] : i;  x = residual[r] (+ delta[r]);
// if store_residual: residual[r] = x;  out[i] = x / sqrt(mean(x^2) + eps) * weight.
// Sum of squares, root and scaling are float.
template <typename T>
__global__ void add_rmsnorm_kernel(float* __restrict__ residual, const T* __restrict__ delta,
                                   const float* __restrict__ weight, T* __restrict__ out,
                                   const int* __restrict__ rows, int hidden, float eps, int store_residual) {
  __shared__ float scratch[16];
  const int i = blockIdx.x;
  const int r = rows ? rows[i] : i;
  float* res = residual + (size_t)r * hidden;
  const T* del = delta ? delta + (size_t)r * hidden : nullptr;
  float sq = 0.f;
  for (int h = threadIdx.x; h < hidden; h += blockDim.x) {
    float x = res[h];
    if (del) x += ld(del + h);
    sq += x * x;
  }
  const float total = block_sum(sq, scratch);
  const float inv = 1.0f / sqrtf(total / (float)hidden + eps);
  T* dst = out + (size_t)i * hidden;
  for (int h = threadIdx.x; h < hidden; h += blockDim.x) {
    float x = res[h];
    if (del) x += ld(del + h);
    if (store_residual) res[h] = x;
    st(dst + h, x * inv * weight[h]);
  }
}

// The same for rows of up to 4096 elements (a multiple of 4): every thread keeps its four-element pieces in
// registers, so the row is read once, 16 bytes at a time.
__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 ld4(const bf16_t* p) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  return make_float4(bf16_bits_to_float(raw.x & 0xffffu), bf16_bits_to_float(raw.x >> 16),
                     bf16_bits_to_float(raw.y & 0xffffu), bf16_bits_to_float(raw.y >> 16));
}
__device__ __forceinline__ void st4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void st4(bf16_t* p, float4 v) {
  uint2 raw;
  raw.x = (uint32_t)float_to_bf16_bits(v.x) | ((uint32_t)float_to_bf16_bits(v.y) << 16);
  raw.y = (uint32_t)float_to_bf16_bits(v.z) | ((uint32_t)float_to_bf16_bits(v.w) << 16);
  *reinterpret_cast<uint2*>(p) = raw;
}

// CHUNKS: runs of 1,024 floats that a row has (a thread takes four floats of each).  The old residual, the delta
// and the norm weight are all asked for at the start (a thread past the end of the row asks for the row's last
// floats and does not use them, so that no load stands behind a condition): one trip to memory where a chunk after
// the other, and the weight after the sum, were up to five.
template <typename T, int CHUNKS, bool DELTA>
__global__ void __launch_bounds__(256)
add_rmsnorm_vec_kernel(float* __restrict__ residual, const T* __restrict__ delta, const float* __restrict__ weight,
                       T* __restrict__ out, const int* __restrict__ rows, int hidden, float eps, int store_residual) {
  HELD(residual, delta, weight, out, rows, hidden, eps, store_residual);
  __shared__ float scratch[16];
  const int i = blockIdx.x;
  const int r = rows ? scalar_int(rows + i) : i;
  float* res = residual + (size_t)r * hidden;
  const T* del = delta + (size_t)r * hidden;
  float4 x[CHUNKS], d[CHUNKS], gain[CHUNKS];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = min((c * 256 + (int)threadIdx.x) * 4, hidden - 4);
    x[c] = ld4(res + h);
    if (DELTA) d[c] = ld4(del + h);
    gain[c] = ld4(weight + h);
  }
  float sq = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    if (DELTA) { x[c].x += d[c].x; x[c].y += d[c].y; x[c].z += d[c].z; x[c].w += d[c].w; }
    if (h >= hidden) x[c] = make_float4(0.f, 0.f, 0.f, 0.f);
    else if (DELTA && store_residual) st4(res + h, x[c]);
    sq += x[c].x * x[c].x + x[c].y * x[c].y + x[c].z * x[c].z + x[c].w * x[c].w;
  }
  const float total = block_sum(sq, scratch);
  const float inv = 1.0f / sqrtf(total / (float)hidden + eps);
  T* dst = out + (size_t)i * hidden;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    if (h >= hidden) continue;
    const float4 w = gain[c];
    st4(dst + h, make_float4(x[c].x * inv * w.x, x[c].y * inv * w.y, x[c].z * inv * w.z, x[c].w * inv * w.w));
  }
}

// The same with the delta still in parts: a product whose K was cut over workgroups left `splits` slabs of
// float sums [M, hidden]; they are added in their order, the bias joins, the sum goes into the residual stream
// (stored back) and the row is normalised.  One kernel instead of the addition and the norm after it.
// CHUNKS: runs of 1,024 floats that a row has (a thread takes four floats of each).  Everything a thread needs (the
// old residual, the bias, the norm weight and the first slabs) is asked for at once and nothing is used
// before all of it is under way: asked for one after the other as they are needed, these are five trips to memory
// in a kernel that is over after one.  A thread past the end of the row asks for the row's last floats and does
// not use them (no load stands behind a condition).
template <typename T, int CHUNKS>
__global__ void __launch_bounds__(256)
splitk_add_rmsnorm_kernel(float* __restrict__ residual, const float* __restrict__ partial, int splits,
                          const float* __restrict__ bias, const float* __restrict__ weight, T* __restrict__ out,
                          int n_rows, int hidden, float eps) {
  HELD(residual, partial, splits, bias, weight, out, n_rows, hidden, eps);
  __shared__ float scratch[16];
  const int i = blockIdx.x;
  float* res = residual + (size_t)i * hidden;
  const size_t slab_stride = (size_t)n_rows * hidden;
  const float* bias_or_any = bias ? bias : weight;           // (without a bias: loaded from a valid place, not used)
  constexpr int FIRST = CHUNKS == 1 ? 8 : 4;                 // slabs asked for at the start (registers: sixteen bytes each)
  float4 old[CHUNKS], gain[CHUNKS], extra[CHUNKS], first[CHUNKS][FIRST];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = min((c * 256 + (int)threadIdx.x) * 4, hidden - 4);
    old[c] = ld4(res + h);
    extra[c] = ld4(bias_or_any + h);
    gain[c] = ld4(weight + h);
    const float* slab = partial + (size_t)i * hidden + h;
#pragma unroll
    for (int j = 0; j < FIRST; ++j) first[c][j] = ld4(slab + (size_t)min(j, splits - 1) * slab_stride);
  }
  float4 x[CHUNKS];
  float sq = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    const int hc = min(h, hidden - 4);
    // The slabs are added in their order, eight asked for at a time after the first ones.
    float4 sum = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int j = 0; j < FIRST; ++j) {
      const float4 v = j < splits ? first[c][j] : make_float4(0.f, 0.f, 0.f, 0.f);
      sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
    }
    const float* slab = partial + (size_t)i * hidden + hc;
    for (int s0 = FIRST; s0 < splits; s0 += 8) {
      float4 v[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = ld4(slab + (size_t)min(s0 + j, splits - 1) * slab_stride);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float4 u = s0 + j < splits ? v[j] : make_float4(0.f, 0.f, 0.f, 0.f);
        sum.x += u.x; sum.y += u.y; sum.z += u.z; sum.w += u.w;
      }
    }
    if (bias) { sum.x += extra[c].x; sum.y += extra[c].y; sum.z += extra[c].z; sum.w += extra[c].w; }
    x[c] = make_float4(old[c].x + sum.x, old[c].y + sum.y, old[c].z + sum.z, old[c].w + sum.w);
    if (h < hidden) st4(res + h, x[c]);
    else x[c] = make_float4(0.f, 0.f, 0.f, 0.f);
    sq += x[c].x * x[c].x + x[c].y * x[c].y + x[c].z * x[c].z + x[c].w * x[c].w;
  }
  const float total = block_sum(sq, scratch);
  const float inv = 1.0f / sqrtf(total / (float)hidden + eps);
  T* dst = out + (size_t)i * hidden;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    if (h >= hidden) continue;
    const float4 w = gain[c];
    st4(dst + h, make_float4(x[c].x * inv * w.x, x[c].y * inv * w.y, x[c].z * inv * w.z, x[c].w * inv * w.w));
  }
}

// out[t, j] = silu(in[t, j]) * in[t, inner + j], silu(z) = z * sigmoid(z), in float.
template <typename T>
__global__ void silu_gate_kernel(const T* __restrict__ in, T* __restrict__ out, int inner, size_t total) {
  for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += (size_t)gridDim.x * blockDim.x) {
    const size_t t = idx / inner;
    const int j = (int)(idx - t * inner);
    const float g = ld(in + t * 2 * inner + j);
    const float u = ld(in + t * 2 * inner + inner + j);
    st(out + idx, g / (1.0f + expf(-g)) * u);
  }
}

// out[t, j] = g' * sigmoid(alpha g') * (u' + shift) with g' = min(in[t, j], limit), u' = clamp(in[t, inner + j], -limit, limit).
template <typename T>
__global__ void capped_gate_kernel(const T* __restrict__ in, T* __restrict__ out, int inner, size_t total, float alpha,
                                   float limit, float shift) {
  for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += (size_t)gridDim.x * blockDim.x) {
    const size_t t = idx / inner;
    const int j = (int)(idx - t * inner);
    const float g = fminf(ld(in + t * 2 * inner + j), limit);
    const float u = fminf(fmaxf(ld(in + t * 2 * inner + inner + j), -limit), limit);
    st(out + idx, g / (1.0f + expf(-alpha * g)) * (u + shift));
  }
}

// The same for bfloat16 rows whose length is a multiple of 8: sixteen bytes of gate and of up per thread.
__global__ void silu_gate_vec_kernel(const bf16_t* __restrict__ in, bf16_t* __restrict__ out, int inner8,
                                     unsigned total8) {
  for (unsigned idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total8; idx += gridDim.x * blockDim.x) {
    const unsigned t = idx / (unsigned)inner8, j = idx - t * (unsigned)inner8;
    const uint4* row = reinterpret_cast<const uint4*>(in) + (size_t)t * 2 * inner8;
    const uint4 gate = row[j], up = row[inner8 + j];
    const uint32_t gw[4] = {gate.x, gate.y, gate.z, gate.w}, uw[4] = {up.x, up.y, up.z, up.w};
    uint32_t packed[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float g0 = __uint_as_float(gw[i] << 16), g1 = __uint_as_float(gw[i] & 0xffff0000u);
      const float u0 = __uint_as_float(uw[i] << 16), u1 = __uint_as_float(uw[i] & 0xffff0000u);
      const float r0 = g0 / (1.0f + expf(-g0)) * u0, r1 = g1 / (1.0f + expf(-g1)) * u1;
      packed[i] = (uint32_t)float_to_bf16_bits(r0) | ((uint32_t)float_to_bf16_bits(r1) << 16);
    }
    reinterpret_cast<uint4*>(out)[idx] = make_uint4(packed[0], packed[1], packed[2], packed[3]);
  }
}

// The capped activation for bfloat16 rows whose length is a multiple of 8, in the same manner.
__global__ void capped_gate_vec_kernel(const bf16_t* __restrict__ in, bf16_t* __restrict__ out, int inner8,
                                       unsigned total8, float alpha, float limit, float shift) {
  for (unsigned idx = blockIdx.x * blockDim.x + threadIdx.x; idx < total8; idx += gridDim.x * blockDim.x) {
    const unsigned t = idx / (unsigned)inner8, j = idx - t * (unsigned)inner8;
    const uint4* row = reinterpret_cast<const uint4*>(in) + (size_t)t * 2 * inner8;
    const uint4 gate = row[j], up = row[inner8 + j];
    const uint32_t gw[4] = {gate.x, gate.y, gate.z, gate.w}, uw[4] = {up.x, up.y, up.z, up.w};
    uint32_t packed[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float g0 = fminf(__uint_as_float(gw[i] << 16), limit), g1 = fminf(__uint_as_float(gw[i] & 0xffff0000u), limit);
      const float u0 = fminf(fmaxf(__uint_as_float(uw[i] << 16), -limit), limit);
      const float u1 = fminf(fmaxf(__uint_as_float(uw[i] & 0xffff0000u), -limit), limit);
      const float r0 = g0 / (1.0f + expf(-alpha * g0)) * (u0 + shift), r1 = g1 / (1.0f + expf(-alpha * g1)) * (u1 + shift);
      packed[i] = (uint32_t)float_to_bf16_bits(r0) | ((uint32_t)float_to_bf16_bits(r1) << 16);
    }
    reinterpret_cast<uint4*>(out)[idx] = make_uint4(packed[0], packed[1], packed[2], packed[3]);
  }
}

extern "C" int ta_embedding(const void* ids, const void* table, void* out, int n_tokens, int hidden,
                            int vocab, int dtype, float scale, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (dtype == DT_F32)
    embedding_kernel<float><<<n_tokens, 256, 0, stream>>>((const int*)ids, (const float*)table, (float*)out, hidden, vocab, scale);
  else if (hidden % 8 == 0 && (((uintptr_t)table | (uintptr_t)out) & 15) == 0)
    embedding_vec_kernel<<<n_tokens, 256, 0, stream>>>((const int*)ids, (const bf16_t*)table, (float*)out, hidden, vocab, scale);
  else
    embedding_kernel<bf16_t><<<n_tokens, 256, 0, stream>>>((const int*)ids, (const bf16_t*)table, (float*)out, hidden, vocab, scale);
  return LAUNCH_STATUS();
}

// Two sub-layers' outputs that read the same normalised rows: for output row i, r = rows ? rows[i] : i;
// x = residual[r] + (first[r] + second[r]), all float; if store_residual: residual[r] = x;
// out[i] = weight ? x / sqrt(mean(x^2) + eps) * weight : x.  A row a workgroup; the row is read once and kept in
// registers (PER elements a thread, rows of up to 256 * PER).
template <typename T, int PER>
__global__ void __launch_bounds__(256)
add_pair_rmsnorm_kernel(float* __restrict__ residual, const T* __restrict__ first, const T* __restrict__ second,
                        const float* __restrict__ weight, T* __restrict__ out, const int* __restrict__ rows, int hidden,
                        float eps, int store_residual) {
  __shared__ float scratch[16];
  const int i = blockIdx.x;
  const int r = rows ? rows[i] : i;
  float* res = residual + (size_t)r * hidden;
  const T* a = first + (size_t)r * hidden;
  const T* b = second + (size_t)r * hidden;
  float x[PER];
  float sq = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int h = p * 256 + threadIdx.x;
    x[p] = 0.f;
    if (h < hidden) {
      x[p] = res[h] + (ld(a + h) + ld(b + h));
      if (store_residual) res[h] = x[p];
    }
    sq += x[p] * x[p];
  }
  float inv = 1.f;
  if (weight) inv = 1.0f / sqrtf(block_sum(sq, scratch) / (float)hidden + eps);
  T* dst = out + (size_t)i * hidden;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int h = p * 256 + threadIdx.x;
    if (h < hidden) st(dst + h, weight ? x[p] * inv * weight[h] : x[p]);
  }
}

// Sub-layers' outputs still to be weighted and added: up to four terms, term k = factor[k] * scale[k][h] * rows[k][r, h]
// (scale float [hidden] or null).  For output row i, r = rows ? rows[i] : i; x = residual[r] + (the terms' sum), all
// float; if store_residual: residual[r] = x; out[i] = weight ? x / sqrt(mean(x^2) + eps) * weight : x, in rows of
// `out_stride` elements; with out2, a second normalised copy under weight2 and eps2.  A row a workgroup; the row is
// read once and kept in registers.
#define TERMS_MAX 4
struct SumTerms {
  const void* rows[TERMS_MAX];
  const float* scale[TERMS_MAX];
  float factor[TERMS_MAX];
  int count;
};

template <typename T, int PER>
__global__ void __launch_bounds__(256)
add_terms_rmsnorm_kernel(float* __restrict__ residual, SumTerms terms, const float* __restrict__ weight, float eps,
                         T* __restrict__ out, int out_stride, const float* __restrict__ weight2, float eps2,
                         T* __restrict__ out2, const int* __restrict__ rows, int hidden, int store_residual) {
  __shared__ float scratch[16];
  const int i = blockIdx.x;
  const int r = rows ? rows[i] : i;
  float* res = residual + (size_t)r * hidden;
  float x[PER];
  float sq = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int h = p * 256 + threadIdx.x;
    x[p] = 0.f;
    if (h < hidden) {
      float sum = 0.f;
#pragma unroll
      for (int k = 0; k < TERMS_MAX; ++k)
        if (k < terms.count) {
          float v = terms.factor[k] * ld(reinterpret_cast<const T*>(terms.rows[k]) + (size_t)r * hidden + h);
          if (terms.scale[k]) v *= terms.scale[k][h];
          sum = k == 0 ? v : sum + v;
        }
      x[p] = terms.count > 0 ? res[h] + sum : res[h];
      if (store_residual) res[h] = x[p];
    }
    sq += x[p] * x[p];
  }
  float mean = 0.f;
  if (weight || out2) mean = block_sum(sq, scratch) / (float)hidden;
  const float inv = weight ? 1.0f / sqrtf(mean + eps) : 1.f;
  T* dst = out + (size_t)i * out_stride;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int h = p * 256 + threadIdx.x;
    if (h < hidden) st(dst + h, weight ? x[p] * inv * weight[h] : x[p]);
  }
  if (out2) {
    const float inv2 = 1.0f / sqrtf(mean + eps2);
    T* dst2 = out2 + (size_t)i * hidden;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int h = p * 256 + threadIdx.x;
      if (h < hidden) st(dst2 + h, x[p] * inv2 * weight2[h]);
    }
  }
}

// One more term that is a product still in parts: factor * scale[h] * the sum over `count` slabs [n_tokens, hidden] of floats,
// `stride` floats apart, added in their order.
struct SlabTerm {
  const float* slabs;
  const float* scale;
  float factor;
  int count;
  size_t stride;
};

// The same for rows of up to 4,096 elements (a multiple of 4) with a norm weight, in pieces of four elements: everything a
// thread needs (the old residual, the terms, their scales, the norm weights and the first slabs) is asked for at the start,
// as in add_rmsnorm_vec_kernel.  COUNT terms of rows, all of them with a scale (SCALED) or none; SLABS: and one term in
// parts behind them.
template <typename T, int CHUNKS, int COUNT, bool SCALED, bool SLABS>
__global__ void __launch_bounds__(256)
add_terms_rmsnorm_vec_kernel(float* __restrict__ residual, SumTerms terms, const float* __restrict__ weight, T* __restrict__ out,
                             const int* __restrict__ rows, int hidden, float eps, int store_residual, int out_stride,
                             const float* __restrict__ weight2, float eps2, T* __restrict__ out2, SlabTerm tail) {
  HELD(residual, weight, out, rows, hidden, eps, store_residual, out_stride, weight2, out2);
  __shared__ float scratch[16];
  constexpr int FIRST = CHUNKS == 1 ? 8 : 4;                 // slabs asked for at the start
  const int i = blockIdx.x;
  const int r = rows ? scalar_int(rows + i) : i;
  float* res = residual + (size_t)r * hidden;
  const float* gain2_at = out2 ? weight2 : weight;           // (without a second output: loaded from a valid place, not used)
  float4 x[CHUNKS], term[CHUNKS][COUNT], scale[CHUNKS][COUNT], gain[CHUNKS], gain2[CHUNKS];
  float4 slab[CHUNKS][SLABS ? FIRST : 1], tail_scale[CHUNKS];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = min((c * 256 + (int)threadIdx.x) * 4, hidden - 4);
    x[c] = ld4(res + h);
#pragma unroll
    for (int k = 0; k < COUNT; ++k) {
      term[c][k] = ld4(reinterpret_cast<const T*>(terms.rows[k]) + (size_t)r * hidden + h);
      if (SCALED) scale[c][k] = ld4(terms.scale[k] + h);
    }
    if (SLABS) {
      if (SCALED) tail_scale[c] = ld4(tail.scale + h);
#pragma unroll
      for (int j = 0; j < FIRST; ++j)                        // (past the last slab: the last one again, not used)
        slab[c][j] = ld4(tail.slabs + (size_t)min(j, tail.count - 1) * tail.stride + (size_t)r * hidden + h);
    }
    gain[c] = ld4(weight + h);
    gain2[c] = ld4(gain2_at + h);
  }
  float sq = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    float4 sum = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int k = 0; k < COUNT; ++k) {
      const float f = terms.factor[k];
      float4 v = make_float4(f * term[c][k].x, f * term[c][k].y, f * term[c][k].z, f * term[c][k].w);
      if (SCALED) { v.x *= scale[c][k].x; v.y *= scale[c][k].y; v.z *= scale[c][k].z; v.w *= scale[c][k].w; }
      if (k == 0) sum = v;
      else { sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w; }
    }
    if (SLABS) {
      float4 v = slab[c][0];
#pragma unroll
      for (int j = 1; j < FIRST; ++j)
        if (j < tail.count) { v.x += slab[c][j].x; v.y += slab[c][j].y; v.z += slab[c][j].z; v.w += slab[c][j].w; }
      for (int j = FIRST; j < tail.count; ++j) {
        const float4 more = ld4(tail.slabs + (size_t)j * tail.stride + (size_t)r * hidden + min(h, hidden - 4));
        v.x += more.x; v.y += more.y; v.z += more.z; v.w += more.w;
      }
      v.x *= tail.factor; v.y *= tail.factor; v.z *= tail.factor; v.w *= tail.factor;
      if (SCALED) { v.x *= tail_scale[c].x; v.y *= tail_scale[c].y; v.z *= tail_scale[c].z; v.w *= tail_scale[c].w; }
      sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
    }
    x[c].x += sum.x; x[c].y += sum.y; x[c].z += sum.z; x[c].w += sum.w;
    if (h >= hidden) x[c] = make_float4(0.f, 0.f, 0.f, 0.f);
    else if (store_residual) st4(res + h, x[c]);
    sq += x[c].x * x[c].x + x[c].y * x[c].y + x[c].z * x[c].z + x[c].w * x[c].w;
  }
  const float mean = block_sum(sq, scratch) / (float)hidden;
  const float inv = 1.0f / sqrtf(mean + eps);
  T* dst = out + (size_t)i * out_stride;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int h = (c * 256 + threadIdx.x) * 4;
    if (h >= hidden) continue;
    const float4 w = gain[c];
    st4(dst + h, make_float4(x[c].x * inv * w.x, x[c].y * inv * w.y, x[c].z * inv * w.z, x[c].w * inv * w.w));
    if (out2) {
      const float inv2 = 1.0f / sqrtf(mean + eps2);
      const float4 w2 = gain2[c];
      st4(out2 + (size_t)i * hidden + h,
          make_float4(x[c].x * inv2 * w2.x, x[c].y * inv2 * w2.y, x[c].z * inv2 * w2.z, x[c].w * inv2 * w2.w));
    }
  }
}

// The vector form, if these operands have it: 0 or an error of the launch; -2 if not.
static int launch_terms_vec(void* residual, const SumTerms& terms, const void* weight, float eps, void* out, int out_stride,
                            const void* weight2, float eps2, void* out2, const void* rows, int n_rows, int hidden,
                            int store_residual, const SlabTerm& tail, int dtype, hipStream_t stream) {
  const uintptr_t piece = dtype == DT_F32 ? 15 : 7;
  if (!weight || hidden % 4 || hidden > 4096 || out_stride % 4 || terms.count < 1 || terms.count > 3 ||
      (((uintptr_t)out | (uintptr_t)out2) & piece) ||
      (((uintptr_t)residual | (uintptr_t)weight | (uintptr_t)weight2 | (uintptr_t)tail.slabs | (uintptr_t)tail.scale) & 15))
    return -2;
  int scaled = tail.slabs && tail.scale ? 1 : 0;
  for (int k = 0; k < terms.count; ++k) {
    if (((uintptr_t)terms.rows[k] & piece) || ((uintptr_t)terms.scale[k] & 15)) return -2;
    scaled += terms.scale[k] ? 1 : 0;
  }
  if (scaled != 0 && scaled != terms.count + (tail.slabs ? 1 : 0)) return -2;
  if (tail.slabs && (dtype != DT_BF16 || terms.count != 1 || tail.count < 1)) return -2;
#define GO(TT, CC, NN, SS, LL) add_terms_rmsnorm_vec_kernel<TT, CC, NN, SS, LL><<<n_rows, 256, 0, stream>>>((float*)residual, terms, \
    (const float*)weight, (TT*)out, (const int*)rows, hidden, eps, store_residual, out_stride, (const float*)weight2, eps2,          \
    (TT*)out2, tail)
#define GO_CHUNKS(TT, NN, SS, LL) switch ((hidden + 1023) / 1024) { case 1: GO(TT, 1, NN, SS, LL); break; \
    case 2: GO(TT, 2, NN, SS, LL); break; case 3: GO(TT, 3, NN, SS, LL); break; default: GO(TT, 4, NN, SS, LL); break; }
#define GO_SCALED(TT, NN, LL) if (scaled) GO_CHUNKS(TT, NN, true, LL) else GO_CHUNKS(TT, NN, false, LL)
  if (tail.slabs) { GO_SCALED(bf16_t, 1, true) }
  else if (dtype == DT_F32) {
    if (terms.count == 1) { GO_SCALED(float, 1, false) } else if (terms.count == 2) { GO_SCALED(float, 2, false) } else return -2;
  } else {
    if (terms.count == 1) { GO_SCALED(bf16_t, 1, false) } else if (terms.count == 2) { GO_SCALED(bf16_t, 2, false) }
    else { GO_SCALED(bf16_t, 3, false) }
  }
#undef GO_SCALED
#undef GO_CHUNKS
#undef GO
  return LAUNCH_STATUS();
}

extern "C" int ta_add_terms_rmsnorm(void* residual, int count, const void* rows0, const void* rows1, const void* rows2,
                                    const void* rows3, const void* scale0, const void* scale1, const void* scale2,
                                    const void* scale3, float f0, float f1, float f2, float f3, const void* weight,
                                    float eps, void* out, int out_stride, const void* weight2, float eps2, void* out2,
                                    const void* rows, int n_rows, int hidden, int store_residual, int dtype,
                                    hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (hidden <= 0 || hidden > 256 * 32 || count < 0 || count > TERMS_MAX || out_stride < hidden || (out2 && !weight2)) return -1;
  SumTerms terms = {{rows0, rows1, rows2, rows3},
                    {(const float*)scale0, (const float*)scale1, (const float*)scale2, (const float*)scale3},
                    {f0, f1, f2, f3}, count};
  for (int k = 0; k < count; ++k)
    if (!terms.rows[k]) return -1;
  const int status = launch_terms_vec(residual, terms, weight, eps, out, out_stride, weight2, eps2, out2, rows, n_rows, hidden,
                                      store_residual, SlabTerm{nullptr, nullptr, 0.f, 0, 0}, dtype, stream);
  if (status != -2) return status;
#define TERMS(TT, PP) add_terms_rmsnorm_kernel<TT, PP><<<n_rows, 256, 0, stream>>>((float*)residual, terms,     (const float*)weight, eps, (TT*)out, out_stride, (const float*)weight2, eps2, (TT*)out2, (const int*)rows, hidden, store_residual)
#define TERMS_SIZES(TT) if (hidden <= 256) TERMS(TT, 1); else if (hidden <= 1024) TERMS(TT, 4); else if (hidden <= 2048) TERMS(TT, 8);                         else if (hidden <= 4096) TERMS(TT, 16); else TERMS(TT, 32)
  if (dtype == DT_F32) { TERMS_SIZES(float); } else { TERMS_SIZES(bf16_t); }
#undef TERMS_SIZES
#undef TERMS
  return LAUNCH_STATUS();
}

// One term of rows and one in parts (float slabs [n_slabs, n_tokens, hidden], `stride` floats apart) in bfloat16 mode.  Returns
// -2 for operands without the vector form (the caller then adds the parts first).
extern "C" int ta_add_slabs_rmsnorm(void* residual, const void* rows0, const void* scale0, float f0, const void* slabs,
                                    const void* slab_scale, float slab_factor, int n_slabs, size_t stride, const void* weight,
                                    float eps, void* out, const void* rows, int n_rows, int hidden, int store_residual,
                                    hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (hidden <= 0 || !rows0 || !slabs || n_slabs < 1 || !weight) return -1;
  const SumTerms terms = {{rows0, nullptr, nullptr, nullptr}, {(const float*)scale0, nullptr, nullptr, nullptr}, {f0, 0.f, 0.f, 0.f}, 1};
  return launch_terms_vec(residual, terms, weight, eps, out, hidden, nullptr, 0.f, nullptr, rows, n_rows, hidden, store_residual,
                          SlabTerm{(const float*)slabs, (const float*)slab_scale, slab_factor, n_slabs, stride}, DT_BF16, stream);
}

extern "C" int ta_add_pair_rmsnorm(void* residual, const void* first, const void* second, const void* weight, void* out,
                                   const void* rows, int n_rows, int hidden, float eps, int store_residual, int dtype,
                                   hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (hidden <= 0 || hidden > 256 * 32 || !first || !second) return -1;
  const SumTerms terms = {{first, second, nullptr, nullptr}, {nullptr, nullptr, nullptr, nullptr}, {1.f, 1.f, 0.f, 0.f}, 2};
  const int status = launch_terms_vec(residual, terms, weight, eps, out, hidden, nullptr, 0.f, nullptr, rows, n_rows, hidden,
                                      store_residual, SlabTerm{nullptr, nullptr, 0.f, 0, 0}, dtype, stream);
  if (status != -2) return status;
#define PAIR(TT, PP) add_pair_rmsnorm_kernel<TT, PP><<<n_rows, 256, 0, stream>>>((float*)residual, (const TT*)first, \
    (const TT*)second, (const float*)weight, (TT*)out, (const int*)rows, hidden, eps, store_residual)
#define PAIR_SIZES(TT) if (hidden <= 256) PAIR(TT, 1); else if (hidden <= 1024) PAIR(TT, 4); else if (hidden <= 2048) PAIR(TT, 8); \
                       else if (hidden <= 4096) PAIR(TT, 16); else PAIR(TT, 32)
  if (dtype == DT_F32) { PAIR_SIZES(float); } else { PAIR_SIZES(bf16_t); }
#undef PAIR_SIZES
#undef PAIR
  return LAUNCH_STATUS();
}

// x <- cap > 0 ? cap * tanh(scale * x / cap) : scale * x, in place, float.
__global__ void scale_cap_kernel(float* __restrict__ x, size_t total, float scale, float cap) {
  for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total; idx += (size_t)gridDim.x * blockDim.x) {
    const float v = x[idx] * scale;
    x[idx] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

extern "C" int ta_scale_cap(void* x, size_t total, float scale, float cap, hipStream_t stream) {
  if (total == 0) return 0;
  const int blocks = (int)((total + 255) / 256 < 65535 ? (total + 255) / 256 : 65535);
  scale_cap_kernel<<<blocks, 256, 0, stream>>>((float*)x, total, scale, cap);
  return LAUNCH_STATUS();
}

extern "C" int ta_add_rmsnorm(void* residual, const void* delta, const void* weight, void* out,
                              const void* rows, int n_rows, int hidden, float eps, int store_residual,
                              int dtype, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (hidden % 4 == 0 && hidden <= 4096) {
#define GO(TT, CC, DD) add_rmsnorm_vec_kernel<TT, CC, DD><<<n_rows, 256, 0, stream>>>( \
    (float*)residual, (const TT*)delta, (const float*)weight, (TT*)out, (const int*)rows, hidden, eps, store_residual)
#define GO_DELTA(TT, CC) if (delta) GO(TT, CC, true); else GO(TT, CC, false)
#define GO_CHUNKS(TT) switch ((hidden + 1023) / 1024) { case 1: GO_DELTA(TT, 1); break; case 2: GO_DELTA(TT, 2); break; \
                                                        case 3: GO_DELTA(TT, 3); break; default: GO_DELTA(TT, 4); break; }
    if (dtype == DT_F32) GO_CHUNKS(float) else GO_CHUNKS(bf16_t)
#undef GO_CHUNKS
#undef GO_DELTA
#undef GO
    return LAUNCH_STATUS();
  }
  if (dtype == DT_F32)
    add_rmsnorm_kernel<float><<<n_rows, 256, 0, stream>>>((float*)residual, (const float*)delta, (const float*)weight,
                                                          (float*)out, (const int*)rows, hidden, eps, store_residual);
  else
    add_rmsnorm_kernel<bf16_t><<<n_rows, 256, 0, stream>>>((float*)residual, (const bf16_t*)delta, (const float*)weight,
                                                           (bf16_t*)out, (const int*)rows, hidden, eps, store_residual);
  return LAUNCH_STATUS();
}

// residual [n_rows, hidden] += the slabs of `partial` ([splits, n_rows, hidden] floats, added in order) + bias;
// out = rmsnorm(residual) * weight.  hidden a multiple of 4 and at most 4096.
extern "C" int ta_splitk_add_rmsnorm(void* residual, const void* partial, int splits, const void* bias,
                                     const void* weight, void* out, int n_rows, int hidden, float eps, int dtype,
                                     hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (hidden % 4 || hidden > 4096 || splits < 1 || !partial) return -1;
#define GO(TT, CC) splitk_add_rmsnorm_kernel<TT, CC><<<n_rows, 256, 0, stream>>>( \
    (float*)residual, (const float*)partial, splits, (const float*)bias, (const float*)weight, (TT*)out, n_rows, hidden, eps)
#define GO_CHUNKS(TT) switch ((hidden + 1023) / 1024) { case 1: GO(TT, 1); break; case 2: GO(TT, 2); break; \
                                                        case 3: GO(TT, 3); break; default: GO(TT, 4); break; }
  if (dtype == DT_F32) GO_CHUNKS(float) else GO_CHUNKS(bf16_t)
#undef GO_CHUNKS
#undef GO
  return LAUNCH_STATUS();
}

extern "C" int ta_silu_gate(const void* in, void* out, int n_tokens, int inner, int dtype, hipStream_t stream) {
  const size_t total = (size_t)n_tokens * inner;
  if (total == 0) return 0;
  const int blocks = (int)((total + 255) / 256 < 65535 ? (total + 255) / 256 : 65535);
  if (dtype != DT_F32 && inner % 8 == 0 && total / 8 < 0xffffffffu && ((uintptr_t)in & 15) == 0 && ((uintptr_t)out & 15) == 0) {
    const size_t total8 = total / 8;
    const int blocks8 = (int)((total8 + 255) / 256 < 16384 ? (total8 + 255) / 256 : 16384);
    silu_gate_vec_kernel<<<blocks8, 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, inner / 8, (unsigned)total8);
    return LAUNCH_STATUS();
  }
  if (dtype == DT_F32)
    silu_gate_kernel<float><<<blocks, 256, 0, stream>>>((const float*)in, (float*)out, inner, total);
  else
    silu_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, inner, total);
  return LAUNCH_STATUS();
}

extern "C" int ta_capped_gate(const void* in, void* out, int n_tokens, int inner, float alpha, float limit, float shift,
                              int dtype, hipStream_t stream) {
  const size_t total = (size_t)n_tokens * inner;
  if (total == 0) return 0;
  const int blocks = (int)((total + 255) / 256 < 65535 ? (total + 255) / 256 : 65535);
  if (dtype != DT_F32 && inner % 8 == 0 && total / 8 < 0xffffffffu && ((uintptr_t)in & 15) == 0 && ((uintptr_t)out & 15) == 0) {
    const size_t total8 = total / 8;
    const int blocks8 = (int)((total8 + 255) / 256 < 16384 ? (total8 + 255) / 256 : 16384);
    capped_gate_vec_kernel<<<blocks8, 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, inner / 8, (unsigned)total8, alpha,
                                                        limit, shift);
    return LAUNCH_STATUS();
  }
  if (dtype == DT_F32)
    capped_gate_kernel<float><<<blocks, 256, 0, stream>>>((const float*)in, (float*)out, inner, total, alpha, limit, shift);
  else
    capped_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, inner, total, alpha, limit, shift);
  return LAUNCH_STATUS();
}

// The number of compute units that the launchers plan for (the current device's).
extern "C" int ta_compute_units() { return compute_units(); }

// A yardstick, not a model kernel: reads `n16` words of sixteen bytes once, in the access pattern of the
// weight-streaming kernels (a wave instruction reads 1 KB of one run, eight such loads of a lane in flight), and
// leaves the xor of everything it read per workgroup in `out` so that no load can be dropped.  What it reaches is
// what a kernel bound by HBM can reach on this device.
typedef uint32_t word4 __attribute__((ext_vector_type(4)));
__global__ void __launch_bounds__(256) read_stream_kernel(const word4* __restrict__ p, size_t n16, uint32_t* __restrict__ out) {
  const size_t stride = (size_t)gridDim.x * blockDim.x;
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  uint32_t acc = 0;
  for (; i + 7 * stride < n16; i += 8 * stride) {
    word4 v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = __builtin_nontemporal_load(p + i + u * stride);
#pragma unroll
    for (int u = 0; u < 8; ++u) acc ^= v[u].x ^ v[u].y ^ v[u].z ^ v[u].w;
  }
  for (; i < n16; i += stride) {
    const word4 v = __builtin_nontemporal_load(p + i);
    acc ^= v.x ^ v.y ^ v.z ^ v.w;
  }
#pragma unroll
  for (int off = WAVE / 2; off > 0; off >>= 1) acc ^= __shfl_xor(acc, off, WAVE);
  __shared__ uint32_t parts[4];
  if ((threadIdx.x & 63) == 0) parts[threadIdx.x >> 6] = acc;
  __syncthreads();
  if (threadIdx.x == 0) out[blockIdx.x] = parts[0] ^ parts[1] ^ parts[2] ^ parts[3];
}

// out: uint32 [workgroups]; bytes a multiple of 16; data 16-byte aligned.
extern "C" int ta_read_stream(const void* data, size_t bytes, void* out, int workgroups, hipStream_t stream) {
  if (bytes % 16 || workgroups <= 0 || ((uintptr_t)data & 15)) return -1;
  read_stream_kernel<<<workgroups, 256, 0, stream>>>((const word4*)data, bytes / 16, (uint32_t*)out);
  return LAUNCH_STATUS();
}
