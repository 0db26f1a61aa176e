// Projection of a few rows, out[n, m] = act(x[n, :] . W[m, :]), 2 <= n <= 32
// (gfx950).  The weights are the whole cost: they stream once, straight into
// MFMA operands, while the rows of x come from L2.
//
// A block owns 16 weight rows; its sixteen waves take every sixteenth 64-step
// stretch of K and their partial tiles are added in LDS.  (Fewer waves, or
// two row tiles per wave, leave too little of the stream in flight.)  A
// lane's 16 steps of a stretch are contiguous (the contraction order is free
// as long as both operands use it), so four lanes read one full 128-byte line
// of a row.

#include "hybrid_common.h"

namespace {

using f32x4 = __attribute__((__vector_size__(16))) float;
using bf16x8 = __attribute__((ext_vector_type(8))) __bf16;
using i32x4 = __attribute__((ext_vector_type(4))) int;

DEVINL bf16x8 load_stream(const bf16* p) {
  return __builtin_bit_cast(
      bf16x8, __builtin_nontemporal_load(reinterpret_cast<const i32x4*>(p)));
}

DEVINL bf16x8 load_row(const bf16* p) {
  return *reinterpret_cast<const bf16x8*>(p);
}

constexpr int NW = 16, STRIDE = NW * 64, UNR = 4;

// NT: tiles of 16 x rows
template <int NT, int ACT>
__global__ __launch_bounds__(NW * 64) void skinny_gemm_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ w,
    const bf16* __restrict__ x, int n, int m, int k, float act_p,
    float act_q) {
  __shared__ float red[NW][NT][16][17];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, quad = lane >> 4;
  const int m0 = blockIdx.x * 16;
  // rows past the end repeat the last one; they are never stored
  const bf16* wp = w + (size_t)min(m0 + c, m - 1) * k + quad * 16;
  const bf16* xp[NT];
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    xp[t] = x + (size_t)min(t * 16 + c, n - 1) * k + quad * 16;
    acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  auto step = [&](bf16x8 wa, bf16x8 wb, int at) {
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          wa, load_row(xp[t] + at), acc[t], 0, 0, 0);
      acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          wb, load_row(xp[t] + at + 8), acc[t], 0, 0, 0);
    }
  };
  int at = wave * 64;
  for (; at + (UNR - 1) * STRIDE < k; at += UNR * STRIDE) {
    bf16x8 wa[UNR], wb[UNR];
#pragma unroll
    for (int u = 0; u < UNR; ++u) {
      wa[u] = load_stream(wp + at + u * STRIDE);
      wb[u] = load_stream(wp + at + u * STRIDE + 8);
    }
#pragma unroll
    for (int u = 0; u < UNR; ++u) step(wa[u], wb[u], at + u * STRIDE);
  }
  for (; at < k; at += STRIDE)
    step(load_stream(wp + at), load_stream(wp + at + 8), at);

#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) red[wave][t][c][quad * 4 + i] = acc[t][i];
  __syncthreads();
  const int row = tid >> 4, j = tid & 15;
  if (row >= n || row >= NT * 16 || m0 + j >= m) return;
  float v = 0.f;
#pragma unroll
  for (int q = 0; q < NW; ++q) v += red[q][row >> 4][row & 15][j];
  if (ACT == 1) v = xielu(v, act_p, act_q);
  if (ACT == 2) v = gelu_erf(v);
  if (ACT == 3) v = relu2(v);
  out[(size_t)row * m + m0 + j] = from_f<bf16>(v);
}

}  // namespace

int launch_skinny_gemm(void* out, const void* w, const void* x, int n, int m,
                       int k, int act, float act_p, float act_q,
                       hipStream_t stream) {
  if (n < 1 || n > 32 || k % 64 != 0) return -1;
  const dim3 grid((m + 15) / 16);
#define SKINNY(NT, ACT)                                                  \
  skinny_gemm_kernel<NT, ACT><<<grid, NW * 64, 0, stream>>>(             \
      (bf16*)out, (const bf16*)w, (const bf16*)x, n, m, k, act_p, act_q)
  if (n <= 16) {
    if (act == 3) SKINNY(1, 3);
    else if (act == 2) SKINNY(1, 2);
    else if (act == 1) SKINNY(1, 1);
    else SKINNY(1, 0);
  } else {
    if (act == 3) SKINNY(2, 3);
    else if (act == 2) SKINNY(2, 2);
    else if (act == 1) SKINNY(2, 1);
    else SKINNY(2, 0);
  }
#undef SKINNY
  return 0;
}
