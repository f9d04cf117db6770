// Routed experts of few rows (decode steps): only the experts that some row chose are read.  Two kernels: the first
// product of every chosen expert with the rows that chose it, the activation and the rows' weights in its epilogue; and
// the second product, whose results lie pick by pick (slab k holds every row's k-th pick), for whoever adds them up.
// bfloat16 operands, float sums on the matrix cores (16x16x32), computed transposed, C^T = W x^T, as the weight-streaming
// product does: sixteen weight rows are the M side, up to sixteen (row, pick) pairs of the expert the N side, the waves of a
// workgroup take turns of 64 elements of K and add up through LDS.
#include "common.h"

typedef __bf16 ef_bf16x8 __attribute__((ext_vector_type(8)));
typedef float ef_floatx4 __attribute__((ext_vector_type(4)));

#define EF_MAX_PAIRS 256

__device__ __forceinline__ ef_bf16x8 ef_load8(const bf16_t* p, bool ok) {
  ef_bf16x8 z;
  if (ok) return *reinterpret_cast<const ef_bf16x8*>(p);
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.0f;
  return z;
}

// The pairs of this workgroup's expert, in rising order: every wave counts them for itself (the count is the same for all),
// the first wave lists them in LDS.
__device__ __forceinline__ int ef_pairs_of(const int* __restrict__ chosen, int n_pairs, int expert, int* list) {
  const int lane = threadIdx.x & (WAVE - 1);
  int count = 0;
#pragma unroll
  for (int base = 0; base < EF_MAX_PAIRS; base += WAVE) {
    if (base >= n_pairs) break;
    const int p = base + lane;
    const bool mine = p < n_pairs && chosen[p] == expert;
    const unsigned long long all = __ballot(mine);
    if (mine && threadIdx.x < WAVE) list[count + __popcll(all & ((1ull << lane) - 1))] = p;
    count += __popcll(all);
  }
  return __builtin_amdgcn_readfirstlane(count);
}

// acc[h] += sixteen rows of matrix h (row `wrow` + h * second of W, K elements `ldw` apart) times the lane's row of x, over this
// wave's turns of K.
template <int NW, int HALVES>
__device__ __forceinline__ void ef_walk(const bf16_t* const (&w_at)[HALVES], const bf16_t* x_at, bool x_ok, int K, int g, int wave,
                                        ef_floatx4 (&acc)[HALVES]) {
  constexpr int UN = HALVES == 2 ? 2 : 4;                    // turns asked for at once
  const int turns = (K + 63) / 64;
  for (int first = wave; first < turns; first += UN * NW) {
    ef_bf16x8 wf[UN][HALVES][2], xf[UN][2];
#pragma unroll
    for (int q = 0; q < UN; ++q) {
      const int turn = first + q * NW, at = min(turn, turns - 1) * 64;
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const bool in = turn < turns && at + 32 * s + 8 * g < K;
#pragma unroll
        for (int h = 0; h < HALVES; ++h) wf[q][h][s] = ef_load8(w_at[h] + at + 32 * s, in);
        xf[q][s] = ef_load8(x_at + at + 32 * s, in && x_ok);
      }
    }
#pragma unroll
    for (int q = 0; q < UN; ++q)
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int h = 0; h < HALVES; ++h)
          acc[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[q][h][s], xf[q][s], acc[h], 0, 0, 0);
  }
}

// x [n_rows, x_stride]; chosen int [n_rows * top], weights float [n_rows * top]; expert e's first matrix starts at
// W + e * HALVES * inner * hidden: [gate; up] of `inner` rows each (HALVES 2) or `up` alone (HALVES 1), rows of `hidden`.
// act [n_rows * top, inner]: pair p's row.  HALVES 2: weigh_input ? silu(w g) * (w u) : w * silu(g) * u; HALVES 1: w * max(u, 0)^2.
// Grid: (blocks of sixteen columns of inner, experts).
template <int NW, int HALVES>
__global__ void __launch_bounds__(NW * WAVE)
experts_few_up_kernel(const bf16_t* __restrict__ x, int x_stride, const int* __restrict__ chosen, const float* __restrict__ weights,
                      int n_pairs, int top, const bf16_t* __restrict__ W, int inner, int hidden, bf16_t* __restrict__ act,
                      int weigh_input) {
  HELD(x, x_stride, chosen, weights, n_pairs, top, W, inner, hidden, act, weigh_input);
  __shared__ int list[EF_MAX_PAIRS];
  __shared__ float red[NW][HALVES * 4][WAVE];
  const int expert = blockIdx.y, n0 = blockIdx.x * 16;
  const int count = ef_pairs_of(chosen, n_pairs, expert, list);
  if (count == 0) return;                                    // nobody's expert: the same for the whole workgroup
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, g = lane >> 4;
  const bf16_t* w_at[HALVES];
#pragma unroll
  for (int h = 0; h < HALVES; ++h)
    w_at[h] = W + ((size_t)expert * HALVES * inner + (size_t)h * inner + min(n0 + col, inner - 1)) * hidden + 8 * g;
  for (int p0 = 0; p0 < count; p0 += 16) {
    const bool ok = p0 + col < count;
    const bf16_t* x_at = x + (size_t)(list[min(p0 + col, count - 1)] / top) * x_stride + 8 * g;
    ef_floatx4 acc[HALVES];
#pragma unroll
    for (int h = 0; h < HALVES; ++h) acc[h] = (ef_floatx4){0.f, 0.f, 0.f, 0.f};
    ef_walk<NW, HALVES>(w_at, x_at, ok, hidden, g, wave, acc);
#pragma unroll
    for (int h = 0; h < HALVES; ++h)
#pragma unroll
      for (int r = 0; r < 4; ++r) red[wave][h * 4 + r][lane] = acc[h][r];
    __syncthreads();
    // Lane (col, g) held rows 4 g .. 4 g + 3 of column (pair) col: thread (pair, row) gathers its own.
    for (int idx = threadIdx.x; idx < 256; idx += NW * WAVE) {
      const int c = idx >> 4, r = idx & 15;
      if (p0 + c >= count || n0 + r >= inner) continue;
      float v[HALVES];
#pragma unroll
      for (int h = 0; h < HALVES; ++h) {
        v[h] = 0.f;
#pragma unroll
        for (int w = 0; w < NW; ++w) v[h] += red[w][h * 4 + (r & 3)][(r >> 2) * 16 + c];
        // (Rounded as the product over all experts leaves them, so that a row is the same in either form but for the
        // order of its sums.)
        v[h] = bf16_bits_to_float(float_to_bf16_bits(v[h]));
      }
      const int p = list[p0 + c];
      const float wgt = weights[p];
      float value;
      if constexpr (HALVES == 2) {
        const float before = weigh_input ? wgt : 1.f, z = before * v[0];
        value = (weigh_input ? 1.f : wgt) * (z / (1.0f + expf(-z)) * (before * v[1]));
      } else {
        const float z = fmaxf(v[0], 0.f);
        value = wgt * (z * z);
      }
      st(act + (size_t)p * inner + n0 + r, value);
    }
    __syncthreads();                                         // the sums are read before the next sixteen pairs' are written
  }
}

// out [top, n_rows, hidden] float: out[p % top, p / top] = act[p] times expert chosen[p]'s second matrix, which is columns
// e * inner .. of W [hidden, ldw].  Grid: (blocks of sixteen output columns, experts).
template <int NW>
__global__ void __launch_bounds__(NW * WAVE)
experts_few_down_kernel(const bf16_t* __restrict__ act, const int* __restrict__ chosen, int n_pairs, int top, int n_rows,
                        const bf16_t* __restrict__ W, int ldw, int inner, int hidden, float* __restrict__ out) {
  HELD(act, chosen, n_pairs, top, n_rows, W, ldw, inner, hidden, out);
  __shared__ int list[EF_MAX_PAIRS];
  __shared__ float red[NW][4][WAVE];
  const int expert = blockIdx.y, n0 = blockIdx.x * 16;
  const int count = ef_pairs_of(chosen, n_pairs, expert, list);
  if (count == 0) return;
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = wave_index(), col = lane & 15, g = lane >> 4;
  const bf16_t* const w_at[1] = {W + (size_t)min(n0 + col, hidden - 1) * ldw + (size_t)expert * inner + 8 * g};
  for (int p0 = 0; p0 < count; p0 += 16) {
    const bool ok = p0 + col < count;
    const bf16_t* x_at = act + (size_t)list[min(p0 + col, count - 1)] * inner + 8 * g;
    ef_floatx4 acc[1] = {(ef_floatx4){0.f, 0.f, 0.f, 0.f}};
    ef_walk<NW, 1>(w_at, x_at, ok, inner, g, wave, acc);
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wave][r][lane] = acc[0][r];
    __syncthreads();
    for (int idx = threadIdx.x; idx < 256; idx += NW * WAVE) {
      const int c = idx >> 4, r = idx & 15;
      if (p0 + c >= count || n0 + r >= hidden) continue;
      float v = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) v += red[w][r & 3][(r >> 2) * 16 + c];
      const int p = list[p0 + c];
      out[((size_t)(p % top) * n_rows + p / top) * hidden + n0 + r] = v;
    }
    __syncthreads();
  }
}

// Returns -2 for sizes the kernels do not take.  halves: 2 = gate and up rows (silu), 1 = up rows alone (squared ReLU).
extern "C" int ta_experts_few(const void* x, int x_stride, const void* chosen, const void* weights, int n_rows, int top,
                              int n_experts, const void* w_first, int halves, int inner, int hidden, int weigh_input, void* act,
                              const void* w_second, int ldw, void* out, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  const long pairs = (long)n_rows * top;
  if (top <= 0 || n_experts <= 0 || n_experts > 65535 || inner <= 0 || hidden <= 0 || (halves != 1 && halves != 2) ||
      ldw < n_experts * inner || x_stride < hidden)
    return -1;
  if (pairs > EF_MAX_PAIRS || inner % 8 || hidden % 8 || ldw % 8 || x_stride % 8 ||
      (((uintptr_t)x | (uintptr_t)w_first | (uintptr_t)w_second | (uintptr_t)act) & 15))
    return -2;
  const dim3 up((inner + 15) / 16, n_experts), down((hidden + 15) / 16, n_experts);
#define UP(NW, HH) experts_few_up_kernel<NW, HH><<<up, NW * WAVE, 0, stream>>>((const bf16_t*)x, x_stride, (const int*)chosen, \
    (const float*)weights, (int)pairs, top, (const bf16_t*)w_first, inner, hidden, (bf16_t*)act, weigh_input)
#define DOWN(NW) experts_few_down_kernel<NW><<<down, NW * WAVE, 0, stream>>>((const bf16_t*)act, (const int*)chosen, (int)pairs, top, \
    n_rows, (const bf16_t*)w_second, ldw, inner, hidden, (float*)out)
  if (halves == 2) { if (hidden <= 1024) UP(4, 2); else UP(8, 2); }
  else { if (hidden <= 1024) UP(4, 1); else UP(8, 1); }
  int status = LAUNCH_STATUS();
  if (status != 0) return status;
  if (inner <= 1024) DOWN(4); else DOWN(8);
#undef UP
#undef DOWN
  return LAUNCH_STATUS();
}
