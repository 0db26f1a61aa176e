// 16 x 16 tiles of x w^T with the contraction split over a block's waves, for
// kernels with few rows and many small matrices (gfx950).
#pragma once

#include "mfma_frag.h"

// 8 contraction steps of a row of length k; vec: rows are 16-byte aligned
template <typename T>
DEVINL typename Frag<T>::Row load_steps(const T* row, int at, int k,
                                        bool vec) {
  using F = Frag<T>;
  if (vec && at + 8 <= k) return F::load_frag(row + at);
  typename F::Row r = F::zero();
#pragma unroll
  for (int j = 0; j < 8; ++j)
    if (at + j < k) F::set(r, j, row[at + j]);
  return r;
}

// out[row][m]: 16 x 16 tile of x w^T, the contraction split over NW waves in
// stretches of 64 (a lane's 16 steps of a stretch are contiguous), for NM sets
// of weight rows at once.  Every wave leaves its part in red[wave][set][row][m].
template <typename T, int NW, int NM>
DEVINL void tile_product(float (*red)[NM][16][17], const T* x,
                         const T* const (&w)[NM], int k, bool vec) {
  using F = Frag<T>;
  constexpr int STRIDE = NW * 64, UNR = NM == 1 ? 4 : 2;
  const int lane = threadIdx.x & 63, c = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  f32x4 acc[NM];
#pragma unroll
  for (int j = 0; j < NM; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  int at = wave * 64;
  // several stretches of the weight stream in flight
  for (; vec && at + (UNR - 1) * STRIDE + 64 <= k; at += UNR * STRIDE) {
    typename F::Row wa[UNR][NM], wb[UNR][NM];
#pragma unroll
    for (int u = 0; u < UNR; ++u)
#pragma unroll
      for (int j = 0; j < NM; ++j) {
        wa[u][j] = F::load_frag(w[j] + at + u * STRIDE + quad * 16);
        wb[u][j] = F::load_frag(w[j] + at + u * STRIDE + quad * 16 + 8);
      }
#pragma unroll
    for (int u = 0; u < UNR; ++u) {
      const auto xa = F::load_frag(x + at + u * STRIDE + quad * 16);
      const auto xb = F::load_frag(x + at + u * STRIDE + quad * 16 + 8);
#pragma unroll
      for (int j = 0; j < NM; ++j) {
        acc[j] = F::dot(wa[u][j], xa, acc[j]);
        acc[j] = F::dot(wb[u][j], xb, acc[j]);
      }
    }
  }
  for (; at < k; at += STRIDE) {
    const int s = at + quad * 16;
    const auto xa = load_steps<T>(x, s, k, vec);
    const auto xb = load_steps<T>(x, s + 8, k, vec);
#pragma unroll
    for (int j = 0; j < NM; ++j) {
      acc[j] = F::dot(load_steps<T>(w[j], s, k, vec), xa, acc[j]);
      acc[j] = F::dot(load_steps<T>(w[j], s + 8, k, vec), xb, acc[j]);
    }
  }
#pragma unroll
  for (int j = 0; j < NM; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) red[wave][j][c][quad * 4 + i] = acc[j][i];
  __syncthreads();
}

template <int NW, int NM>
DEVINL float tile_sum(const float (*red)[NM][16][17], int j, int row, int m) {
  float v = 0.f;
#pragma unroll
  for (int q = 0; q < NW; ++q) v += red[q][j][row][m];
  return v;
}
