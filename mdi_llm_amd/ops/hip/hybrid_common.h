// Device helpers shared by the hybrid-stack kernels.
#pragma once

#include <hip/hip_bf16.h>
#include <hip/hip_runtime.h>

#include "hybrid_kernels.h"

#define DEVINL __device__ __forceinline__

using bf16 = __hip_bfloat16;

DEVINL float to_f(bf16 v) { return __bfloat162float(v); }
DEVINL float to_f(float v) { return v; }
template <typename T> DEVINL T from_f(float v);
template <> DEVINL bf16 from_f<bf16>(float v) { return __float2bfloat16(v); }
template <> DEVINL float from_f<float>(float v) { return v; }

template <typename T, int N>
struct alignas(sizeof(T) * N) Pack {
  T v[N];
};

DEVINL float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}

// sum over the 16 lanes of a DPP row, in every lane
DEVINL float row16_sum(float v) {
#define ROR_ADD(n)                                                         \
  v += __int_as_float(__builtin_amdgcn_update_dpp(                         \
      0, __float_as_int(v), 0x120 + n, 0xf, 0xf, false))
  ROR_ADD(8);
  ROR_ADD(4);
  ROR_ADD(2);
  ROR_ADD(1);
#undef ROR_ADD
  return v;
}

DEVINL float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
