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
