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

// maximum over the wave, in every lane
DEVINL float wave_max(float v) {
#define ROR_MAX(n)                                                         \
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(                 \
                   0, __float_as_int(v), 0x120 + n, 0xf, 0xf, false)))
  ROR_MAX(8);
  ROR_MAX(4);
  ROR_MAX(2);
  ROR_MAX(1);
#undef ROR_MAX
  auto lane = [&](int l) {
    return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), l));
  };
  return fmaxf(fmaxf(lane(0), lane(16)), fmaxf(lane(32), lane(48)));
}

// Order of one kv head's 64 keys in a page.  A page is made of 16 x 32 blocks
// (K: keys x channels, V: columns x keys), each in the order in which a
// wave's lanes hold it as an MFMA operand: lane (quad, row) has steps
// quad*4 .. +3 of the first and of the second half of the 32.
struct PageLayout {
  static DEVINL int in_block(int row, int step) {
    return ((((step & 15) >> 2) * 16 + row) << 3) + ((step >> 4) << 2) +
           (step & 3);
  }
  static DEVINL int k_block(int key_tile, int chunk, int dpad) {
    return (key_tile * (dpad >> 5) + chunk) << 9;
  }
  static DEVINL int v_block(int col_tile, int key_half, int vpad) {
    return (key_half * (vpad >> 4) + col_tile) << 9;
  }
  static DEVINL int k(int key, int d, int dpad) {
    return k_block(key >> 4, d >> 5, dpad) + in_block(key & 15, d & 31);
  }
  static DEVINL int v(int key, int col, int vpad) {
    return v_block(col >> 4, key >> 5, vpad) + in_block(col & 15, key & 31);
  }
};

// z/2 plus p z^2 above zero, (1/2 + q)(e^z - 1 - z) below
DEVINL float xielu(float z, float p, float q) {
  return 0.5f * z + (z > 0.f ? p * z * z : (0.5f + q) * (expm1f(z) - z));
}

DEVINL float gelu_erf(float z) {
  return 0.5f * z * (1.f + erff(0.7071067811865476f * z));
}

DEVINL float relu2(float z) {
  const float p = fmaxf(z, 0.f);
  return p * p;
}

DEVINL float softplus(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

DEVINL float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }

DEVINL float gated(float gate, float up, int act) {
  if (act == 0) return gate * sigmoid(gate) * up;
  const float inner =
      0.7978845608028654f * (gate + 0.044715f * gate * gate * gate);
  return 0.5f * gate * (1.f + tanhf(inner)) * up;
}
