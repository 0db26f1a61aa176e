// MFMA operands of the hybrid-stack kernels, for bf16 and for float (gfx950).
// A Row holds 8 of the 32 contraction steps of one 16 x 16 x 32 product; which
// steps, the loader decides, the same way for both operands.
#pragma once

#include "hybrid_common.h"

using f32x4 = __attribute__((__vector_size__(16))) float;
using bf16x8 = __attribute__((ext_vector_type(8))) __bf16;
using bf16x4 = __attribute__((ext_vector_type(4))) __bf16;

template <typename T> struct Frag;

template <> struct Frag<bf16> {
  // 32 contraction steps of one row: steps quad*4 .. +3 of both halves
  using Row = bf16x8;
  static DEVINL Row load_row(const bf16* p, int quad) {
    const bf16x4 a = *reinterpret_cast<const bf16x4*>(p + quad * 4);
    const bf16x4 b = *reinterpret_cast<const bf16x4*>(p + 16 + quad * 4);
    return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
  }
  // 8 steps that lie together
  static DEVINL Row load_frag(const bf16* p) {
    return *reinterpret_cast<const bf16x8*>(p);
  }
  static DEVINL Row zero() { return Row{}; }
  static DEVINL void set(Row& r, int i, bf16 v) {
    r[i] = __builtin_bit_cast(__bf16, v);
  }
  static DEVINL f32x4 dot(Row a, Row b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
  }
  struct Weights {
    Row hi, lo;
  };
  static DEVINL Weights weights(const float* p0, const float* p1) {
    Weights w;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float v = i < 4 ? p0[i & 3] : p1[i & 3];
      w.hi[i] = (__bf16)v;
      w.lo[i] = (__bf16)(v - (float)w.hi[i]);
    }
    return w;
  }
  static DEVINL f32x4 weigh(Row v, const Weights& w, f32x4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w.lo, acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w.hi, acc, 0, 0, 0);
  }
};

template <> struct Frag<float> {
  struct Row {
    f32x4 a, b;
  };
  static DEVINL Row load_row(const float* p, int quad) {
    return {*reinterpret_cast<const f32x4*>(p + quad * 4),
            *reinterpret_cast<const f32x4*>(p + 16 + quad * 4)};
  }
  static DEVINL f32x4 dot(const Row& x, const Row& y, f32x4 acc) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a[i], y.a[i], acc, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.b[i], y.b[i], acc, 0, 0, 0);
    return acc;
  }
  static DEVINL Row load_frag(const float* p) {
    return {*reinterpret_cast<const f32x4*>(p),
            *reinterpret_cast<const f32x4*>(p + 4)};
  }
  static DEVINL Row zero() { return Row{}; }
  static DEVINL void set(Row& r, int i, float v) {
    if (i < 4) r.a[i] = v;
    else r.b[i - 4] = v;
  }
  using Weights = Row;
  static DEVINL Weights weights(const float* p0, const float* p1) {
    Row r;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      r.a[i] = p0[i];
      r.b[i] = p1[i];
    }
    return r;
  }
  static DEVINL f32x4 weigh(const Row& v, const Weights& w, f32x4 acc) {
    return dot(v, w, acc);
  }
};
