// Recurrences over a [dim, vdim] state per head (gfx950): the one-token step
// and the walk over 16-token chunks, for any rule of the form
//     S <- diag(f) S + k v^T,   o = S^T q
// with decays f of at most 1.  What makes q, f and k of an input is a
// template argument of the step and a kernel of its own ahead of the walk.
#pragma once

#include "hybrid_common.h"

using f32x4 = __attribute__((__vector_size__(16))) float;

struct StepFactors {
  float q, f, k;
};

// ---------------------------------------------------------------------------
// One token per segment.  One block per (head, segment): the whole [dim, vdim]
// state of the head passes through registers once (16-byte accesses along
// vdim), so the block holds all of the head's output and can norm it before
// it leaves.  Rule has factors(row, h, d), value(row, h, c), put(row, h, c, v)
// and NORM: whether what put gets is the output of unit size.  A rule with
// NORMALISER has one more column whose values are 1; before the unit size the
// output is divided by size(what that column reads out), and enter and leave
// frame the step of a slot's head.
// ---------------------------------------------------------------------------
template <int NT, typename Rule>
__global__ __launch_bounds__(NT) void matrix_step_kernel(
    Rule rule, float* __restrict__ state, SegView seg, int heads, int dim,
    int vdim, int vstride, float eps) {
  extern __shared__ float sm[];
  __shared__ float red[NT / 64];
  const int tid = threadIdx.x, h = blockIdx.x, s = blockIdx.y;
  const int nq = vstride / 4;                 // float4 columns, at most NT
  const int groups = NT / nq;                 // row groups
  float* qs = sm;                             // [dim]
  float* fs = qs + dim;                       // [dim]
  float* ks = fs + dim;                       // [dim]
  float* part = ks + dim;                     // [groups][vstride]
  const size_t row = seg.start[s];
  float* S = state +
             ((size_t)seg.slot[s] * heads + h) * (size_t)dim * vstride;
  const bool fresh = seg.pos0[s] == 0;
  // a thread has one column of a row group; its first rows are on their way
  // while the factors are made
  constexpr int AHEAD = 8;
  const int g = tid / nq, c4 = tid % nq;
  float4 ahead[AHEAD];
  if (g < groups && !fresh) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (g + j * groups < dim)
        ahead[j] = *(reinterpret_cast<const float4*>(
                         S + (size_t)(g + j * groups) * vstride) + c4);
  }
  if constexpr (Rule::NORMALISER)
    rule.enter(row, h, seg.slot[s], seg.pos0[s] == 0);
  for (int d = tid; d < dim; d += NT) {
    const StepFactors x = rule.factors(row, h, d);
    qs[d] = x.q;
    fs[d] = x.f;
    ks[d] = x.k;
  }
  __syncthreads();
  if (g < groups) {
    float v[4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = c4 * 4 + j < vdim ? rule.value(row, h, c4 * 4 + j)
             : Rule::NORMALISER && c4 * 4 + j == vdim ? 1.f
                                                      : 0.f;
    auto update = [&](int d, float4 a) {
      if (fresh) a = make_float4(0.f, 0.f, 0.f, 0.f);
      const float f = fs[d], w = ks[d], q = qs[d];
      a.x = f * a.x + w * v[0];
      a.y = f * a.y + w * v[1];
      a.z = f * a.z + w * v[2];
      a.w = f * a.w + w * v[3];
      *(reinterpret_cast<float4*>(S + (size_t)d * vstride) + c4) = a;
      o[0] += q * a.x;
      o[1] += q * a.y;
      o[2] += q * a.z;
      o[3] += q * a.w;
    };
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (g + j * groups < dim) update(g + j * groups, ahead[j]);
#pragma unroll 8
    for (int d = g + AHEAD * groups; d < dim; d += groups)
      update(d, *(reinterpret_cast<const float4*>(S + (size_t)d * vstride) +
                  c4));
    *reinterpret_cast<float4*>(part + g * vstride + c4 * 4) =
        make_float4(o[0], o[1], o[2], o[3]);
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < vdim; c += NT) {
    float o = 0.f;
    for (int k = 0; k < groups; ++k) o += part[k * vstride + c];
    part[c] = o;  // only this thread reads column c
    ss += o * o;
  }
  float r = 1.f, inv = 1.f;
  if constexpr (Rule::NORMALISER) {
    float n = 0.f;
    for (int k = 0; k < groups; ++k) n += part[k * vstride + vdim];
    inv = 1.f / rule.size(n);
    if (tid == 0) rule.leave(h, seg.slot[s]);
  }
  if constexpr (Rule::NORM) {
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < NT / 64; ++k) ss += red[k];
    r = inv / sqrtf(ss * inv * inv / vdim + eps);
  }
  for (int c = tid; c < vdim; c += NT) rule.put(row, h, c, part[c] * r);
}

template <typename Rule>
void matrix_step(const Rule& rule, float* state, SegView seg, int heads,
                 int dim, int vdim, int vstride, float eps,
                 hipStream_t stream) {
  // few blocks with a large state each: more waves to keep loads in flight
  const int nt =
      dim * vstride >= 8192 && heads * seg.n <= 512 ? 1024 : 256;
  const size_t smem =
      (3 * (size_t)dim + (size_t)(nt / (vstride / 4)) * vstride) *
      sizeof(float);
  const dim3 grid(heads, seg.n);
  if (nt == 1024)
    matrix_step_kernel<1024, Rule><<<grid, 1024, smem, stream>>>(
        rule, state, seg, heads, dim, vdim, vstride, eps);
  else
    matrix_step_kernel<256, Rule><<<grid, 256, smem, stream>>>(
        rule, state, seg, heads, dim, vdim, vstride, eps);
}

// ---------------------------------------------------------------------------
// Longer segments, in chunks of 16 tokens.  With S the state at the chunk's
// start, per channel
//     R_t = f_first .. f_t          (decay from the start to t)
//     U_s = f_(s+1) .. f_last       (decay from s to the end)
// the chunk is three small matrix products,
//     o_t = (q_t R_t)^T S + sum_(s<=t) P[t][s] v_s
//     S  <- (f_first .. f_last) S + sum_s (U_s k_s) v_s^T
// with P[t][s] = sum_d q_t k_s f_(s+1) .. f_t.  Every factor is at most 1 and
// nothing is divided by; an underflow is a token that is forgotten.
// Everything is float and the products run on the float MFMA.
//
// A kernel per rule makes the factors of every (chunk, head) in parallel; the
// walk below takes a segment's chunks in order with a [dim, 16] slice of the
// state per block, held as MFMA accumulators split over the block's four
// waves by rows.  An accumulator tile is at the same time the right operand
// of (q R)^T S once the contraction index is permuted to its layout.
//
// Workspace of one (chunk, head), DP = dim padded to 64, 128 or 256:
//   qr [16][DP] | uk [DP][16] | decay [DP] | P [16][16]
// Segment s has its chunks from start[s] / 16 + s on, which cannot overlap
// as long as the segments are in the order of their rows.
//
// SUMS: one more column whose values are 1, which is a vector per head and
// needs no products: sums [chunk, heads, DP] has sum_s U_s k_s of each chunk,
// in whose place the head's last block leaves the column at the chunk's start.
// ---------------------------------------------------------------------------
template <int DP>
struct ChunkWork {
  static constexpr int QR = 0, UK = 16 * DP, DECAY = 32 * DP,
                       P = 33 * DP, SIZE = 33 * DP + 256;
};

template <int DP>
DEVINL void running_sums(float* __restrict__ sums, const float* __restrict__ w,
                         float* __restrict__ column, bool fresh, int chunks,
                         int heads, int dim, int vstride) {
  constexpr int AHEAD = 8;
  const int d = threadIdx.x;
  if (d >= DP) return;
  const size_t step = (size_t)heads * DP;
  const size_t wstep = (size_t)heads * ChunkWork<DP>::SIZE;
  sums += d;
  w += ChunkWork<DP>::DECAY + d;
  float n = !fresh && d < dim ? column[(size_t)d * vstride] : 0.f;
  float u[2][AHEAD], f[2][AHEAD];
  auto load = [&](int b, int c0) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const int c = min(c0 + j, chunks - 1);
      u[b][j] = sums[c * step];
      f[b][j] = w[c * wstep];
    }
  };
  auto run = [&](int b, int c0) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (c0 + j < chunks) {
        sums[(c0 + j) * step] = n;
        n = f[b][j] * n + u[b][j];
      }
  };
  // (a chunk is loaded before its place is written: loads run ahead, and what
  // they repeat past the end is not used)
  load(0, 0);
  for (int c0 = 0; c0 < chunks; c0 += 2 * AHEAD) {
    load(1, c0 + AHEAD);
    run(0, c0);
    load(0, c0 + 2 * AHEAD);
    run(1, c0 + AHEAD);
  }
  if (d < dim) column[(size_t)d * vstride] = n;
}

template <typename T, int TPW, bool SUMS = false>
__global__ __launch_bounds__(256) void matrix_chunks_kernel(
    float* __restrict__ o, const float* __restrict__ work,
    const T* __restrict__ values, long long ld, float* __restrict__ state,
    SegView seg, int heads, int dim, int vdim, int vstride,
    float* __restrict__ sums = nullptr) {
  constexpr int DP = 64 * TPW;
  using W = ChunkWork<DP>;
  __shared__ float red[2][4][16][17];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, quad = lane >> 4;
  // heads vary fastest: the column blocks of a head share an XCD's L2
  const int s = blockIdx.z, h = blockIdx.x, c0 = blockIdx.y * 16;
  const int col = c0 + c, d0 = wave * TPW * 16;
  const int len = seg.len[s], n = (len + 15) / 16;
  const size_t row0 = seg.start[s];
  const float* w = work + ((row0 / 16 + s) * heads + h) * W::SIZE;
  const size_t wstep = (size_t)heads * W::SIZE;
  if constexpr (SUMS) {
    if (blockIdx.y + 1 == gridDim.y) {
      running_sums<DP>(
          sums + ((row0 / 16 + s) * heads + h) * DP, w,
          state + ((size_t)seg.slot[s] * heads + h) * (size_t)dim * vstride +
              vdim,
          seg.pos0[s] == 0, n, heads, dim, vstride);
      return;
    }
  }
  // values: head h of row r at r * ld + h * vdim
  const T* vp = values + row0 * ld + h * vdim + min(col, vdim - 1);
  float* S = state +
             ((size_t)seg.slot[s] * heads + h) * (size_t)dim * vstride + col;
  const bool keep = col < vdim && seg.pos0[s] != 0;

  f32x4 st[TPW];
#pragma unroll
  for (int k = 0; k < TPW; ++k)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = d0 + k * 16 + quad * 4 + i;
      st[k][i] = keep && d < dim ? S[(size_t)d * vstride] : 0.f;
    }

  // operands of the next chunks on their way (values stay unconverted, so
  // that nothing waits for them early)
  constexpr int AHEAD = TPW <= 2 ? 4 : 2;
  struct Operands {
    f32x4 qr[TPW], uk[TPW], decay[TPW];
    float p;
    T v[4], vw;
  } ring[AHEAD];
  auto load = [&](Operands& a, int ch) {
    const float* wc = w + ch * wstep;
#pragma unroll
    for (int k = 0; k < TPW; ++k) {
      a.qr[k] = *reinterpret_cast<const f32x4*>(
          wc + W::QR + c * DP + d0 + k * 16 + quad * 4);
      a.uk[k] = *reinterpret_cast<const f32x4*>(
          wc + W::UK + (d0 + k * 16 + c) * 16 + quad * 4);
      a.decay[k] = *reinterpret_cast<const f32x4*>(
          wc + W::DECAY + d0 + k * 16 + quad * 4);
    }
    a.p = wc[W::P + c * 16 + quad * 4 + wave];
    // rows and columns past the end repeat the last: they meet zero factors
    // or are not stored
    auto value = [&](int t) { return vp[(size_t)min(t, len - 1) * ld]; };
#pragma unroll
    for (int i = 0; i < 4; ++i) a.v[i] = value(ch * 16 + quad * 4 + i);
    a.vw = value(ch * 16 + quad * 4 + wave);
  };
  auto chunk = [&](const Operands& a, int ch) {
    // two accumulators: half the dependent chain
    f32x4 a0{0.f, 0.f, 0.f, 0.f}, a1 = a0;
    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.p, to_f(a.vw), a0, 0, 0, 0);
#pragma unroll
    for (int k = 0; k < TPW; ++k) {
      a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.qr[k][0], st[k][0], a1, 0, 0, 0);
      a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.qr[k][1], st[k][1], a0, 0, 0, 0);
      a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.qr[k][2], st[k][2], a1, 0, 0, 0);
      a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.qr[k][3], st[k][3], a0, 0, 0, 0);
    }
#pragma unroll
    for (int k = 0; k < TPW; ++k) st[k] *= a.decay[k];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int k = 0; k < TPW; ++k)
        st[k] = __builtin_amdgcn_mfma_f32_16x16x4f32(a.uk[k][i], to_f(a.v[i]),
                                                     st[k], 0, 0, 0);
    a0 += a1;
#pragma unroll
    for (int i = 0; i < 4; ++i) red[ch & 1][wave][quad * 4 + i][c] = a0[i];
  };
  auto emit = [&](int ch) {
    __syncthreads();  // one per chunk: the other half is written next
    const int t = tid >> 4, e = tid & 15, tt = ch * 16 + t;
    if (tt < len && c0 + e < vdim) {
      float v = 0.f;
#pragma unroll
      for (int k = 0; k < 4; ++k) v += red[ch & 1][k][t][e];
      o[(row0 + tt) * (size_t)(heads * vdim) + h * vdim + c0 + e] = v;
    }
  };
#pragma unroll
  for (int r = 0; r < AHEAD; ++r) load(ring[r], min(r, n - 1));
  int base = 0;
  for (; base + AHEAD <= n; base += AHEAD) {
#pragma unroll
    for (int r = 0; r < AHEAD; ++r) {
      chunk(ring[r], base + r);
      load(ring[r], min(base + r + AHEAD, n - 1));
      emit(base + r);
    }
  }
#pragma unroll
  for (int r = 0; r < AHEAD - 1; ++r)
    if (base + r < n) {
      chunk(ring[r], base + r);
      emit(base + r);
    }
  if (col < vdim) {
#pragma unroll
    for (int k = 0; k < TPW; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = d0 + k * 16 + quad * 4 + i;
        if (d < dim) S[(size_t)d * vstride] = st[k][i];
      }
  }
}

inline int chunk_dpad(int dim) {
  return dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 0;
}

inline long long chunk_work_floats(int rows, int segments, int heads,
                                   int dim) {
  const long long chunks = rows / 16 + segments + 1;
  return chunks * heads * (33 * chunk_dpad(dim) + 256);
}

inline long long chunk_sums_floats(int rows, int segments, int heads,
                                   int dim) {
  return (long long)(rows / 16 + segments + 1) * heads * chunk_dpad(dim);
}
