// Mixture of experts over a ragged batch (gfx950): float router, top
// experts and their weights, the pairs (row, choice) ordered by expert, and
// the experts' products over tiles of pairs of one expert.  Nothing comes
// back to the host, so decode steps can be captured.

#include "mfma_tile.h"

namespace {

constexpr int MAX_EXPERTS = 256;
constexpr int FUSED_ROWS = 64;  // up to here one block chooses and orders

// ---------------------------------------------------------------------------
template <typename T, int NW>
__global__ __launch_bounds__(NW * 64) void router_kernel(
    float* __restrict__ z, const T* __restrict__ x, const T* __restrict__ w,
    int n, int experts, int k, bool vec) {
  __shared__ float red[NW][1][16][17];
  const int c = threadIdx.x & 15, r0 = blockIdx.y * 16, e0 = blockIdx.x * 16;
  const T* const wp[1] = {w + (size_t)min(e0 + c, experts - 1) * k};
  tile_product<T, NW, 1>(red, x + (size_t)min(r0 + c, n - 1) * k, wp, k, vec);
  for (int i = threadIdx.x; i < 256; i += NW * 64) {
    const int row = i >> 4, e = i & 15;
    if (r0 + row < n && e0 + e < experts)
      z[(size_t)(r0 + row) * experts + e0 + e] =
          tile_sum<NW, 1>(red, 0, row, e);
  }
}

// One wave: the choice of a row (lower index first among equals) and its
// weights.  Without correction the top logits and their softmax; with it the
// softmax over all outputs plus the correction chooses, and the weights are
// the chosen scores over their sum, times scale.
DEVINL void choose(float* weight, int* chosen, const float* z,
                   const MoePlan& p, int lane) {
  constexpr int NV = MAX_EXPERTS / 64;
  const int outputs = p.outputs, top = p.top;
  float v[NV], score[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int e = j * 64 + lane;
    v[j] = e < outputs ? z[e] : -__builtin_huge_valf();
  }
  if (p.correction != nullptr) {
    float m = v[0], total = 0.f;
#pragma unroll
    for (int j = 1; j < NV; ++j) m = fmaxf(m, v[j]);
    m = wave_max(m);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      score[j] = expf(v[j] - m);
      total += score[j];
    }
    total = wave_sum(total);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int e = j * 64 + lane;
      score[j] /= total;
      if (e < outputs) v[j] = score[j] + p.correction[e];
    }
  }
  float zmax = 0.f, sum = 0.f, mine = 0.f;
  for (int t = 0; t < top; ++t) {
    float best = v[0];
#pragma unroll
    for (int j = 1; j < NV; ++j) best = fmaxf(best, v[j]);
    best = wave_max(best);
    int at = outputs - 1;  // kept only if a logit is not a number
#pragma unroll
    for (int j = NV - 1; j >= 0; --j) {
      const unsigned long long hit = __ballot(v[j] == best);
      if (hit != 0) at = min(j * 64 + __ffsll(hit) - 1, outputs - 1);
    }
    if (t == 0) zmax = best;
    float e;
    if (p.correction != nullptr) {
      float s = score[0];
#pragma unroll
      for (int j = 1; j < NV; ++j)
        if (at >> 6 == j) s = score[j];
      e = __shfl(s, at & 63, 64);
    } else {
      e = expf(best - zmax);
    }
    sum += e;
    // a wave holds up to 64 choices, one per lane
    if (lane == t) {
      mine = e;
      chosen[t] = at;
    }
#pragma unroll
    for (int j = 0; j < NV; ++j)
      if (at == j * 64 + lane) v[j] = -__builtin_huge_valf();
  }
  if (p.correction != nullptr) sum = (sum + 1e-20f) / p.scale;
  if (lane < top) weight[lane] = mine / sum;
  if (p.gated && lane == 0) weight[top] = sigmoid(z[outputs]);
}

__global__ __launch_bounds__(256) void choose_kernel(
    float* __restrict__ weight, const float* __restrict__ z, MoePlan p,
    int n) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= n) return;
  choose(weight + (size_t)row * (p.top + p.gated),
         p.chosen + (size_t)row * p.top,
         z + (size_t)row * (p.outputs + p.gated), p, threadIdx.x & 63);
}

// One block: the pairs ordered by expert, and the tiles.  Pairs of outputs
// that are not experts are left out.
__global__ __launch_bounds__(1024) void order_kernel(
    float* __restrict__ weight, const float* __restrict__ z, MoePlan p,
    int n, bool choose_here) {
  __shared__ int count[MAX_EXPERTS], next[MAX_EXPERTS];
  const int tid = threadIdx.x;
  if (choose_here)
    for (int row = tid >> 6; row < n; row += 16)
      choose(weight + row * (p.top + p.gated), p.chosen + row * p.top,
             z + row * (p.outputs + p.gated), p, tid & 63);
  if (tid < p.experts) count[tid] = 0;
  __syncthreads();
  // (the block's own global writes are visible to it after the barrier)
  for (int i = tid; i < p.pairs; i += 1024)
    if (p.chosen[i] < p.experts) atomicAdd(&count[p.chosen[i]], 1);
  __syncthreads();
  if (tid < p.experts) {
    const int shift = 31 - __clz(p.tile_rows);  // a power of two
    int first = 0, tile = 0;
    for (int e = 0; e < tid; ++e) {
      first += count[e];
      tile += (count[e] + p.tile_rows - 1) >> shift;
    }
    next[tid] = first;
    const int tile0 = tile, n_tiles = (count[tid] + p.tile_rows - 1) >> shift;
    for (int at = 0; at < count[tid]; at += p.tile_rows, ++tile)
      p.tiles[tile] = MoeTile{tid, first + at,
                              min(p.tile_rows, count[tid] - at), tile0,
                              n_tiles};
    if (tid == p.experts - 1) *p.n_tiles = tile;
  }
  __syncthreads();
  for (int i = tid; i < p.pairs; i += 1024)
    if (p.chosen[i] < p.experts)
      p.order[atomicAdd(&next[p.chosen[i]], 1)] = i;
}

// ---------------------------------------------------------------------------
// Products of up to 16 pairs of one expert; the weights stream once.
// ---------------------------------------------------------------------------
template <typename T, int NW, bool UP>
__global__ __launch_bounds__(NW * 64) void expert_rows_kernel(
    T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    MoePlan p, int m, int k, int act, bool vec) {
  constexpr int NM = UP ? 2 : 1;
  __shared__ float red[NW][NM][16][17];
  const int tile = blockIdx.y;
  if (tile >= *p.n_tiles) return;
  const int e = p.tiles[tile].expert, first = p.tiles[tile].first;
  const int rows = p.tiles[tile].rows;
  const int c = threadIdx.x & 15, m0 = blockIdx.x * 16;
  const int pair = p.order[first + min(c, rows - 1)];
  const T* xp = x + (size_t)(UP ? pair / p.top : pair) * k;
  const T* we = w + ((size_t)e * NM * m + min(m0 + c, m - 1)) * k;
  const T* wp[NM];
#pragma unroll
  for (int j = 0; j < NM; ++j) wp[j] = we + (size_t)j * m * k;
  tile_product<T, NW, NM>(red, xp, wp, k, vec);
  for (int i = threadIdx.x; i < 256; i += NW * 64) {
    const int row = i >> 4, j = i & 15;
    if (row >= rows || m0 + j >= m) continue;
    float v = tile_sum<NW, NM>(red, 0, row, j);
    if (UP) v = gated(v, tile_sum<NW, NM>(red, NM - 1, row, j), act);
    out[(size_t)p.order[first + row] * m + m0 + j] = from_f<T>(v);
  }
}

template <typename T, bool UP>
void expert_rows_t(void* out, const void* x, const void* w, MoePlan p, int m,
                   int k, int act, hipStream_t stream) {
  const dim3 grid((m + 15) / 16, p.max_tiles);
  const bool vec = k % (16 / sizeof(T)) == 0;
#define EXPERT(NW)                                                      \
  expert_rows_kernel<T, NW, UP><<<grid, NW * 64, 0, stream>>>(          \
      (T*)out, (const T*)x, (const T*)w, p, m, k, act, vec)
  if (k >= 2048) EXPERT(8);
  else EXPERT(4);
#undef EXPERT
}

// ---------------------------------------------------------------------------
// Products of up to 128 pairs of one expert with 256 weight rows, bf16, k a
// multiple of 64.  Four waves hold 64 pairs x 128 outputs each; two blocks
// fit a CU, and one computes while the other stores its next tile.  That tile
// travels through registers during the MFMAs.  16-byte chunks of an LDS row
// are permuted by the row so that both the stores and the operand loads
// spread over the banks.  UP: half of the weight rows are an expert's gate
// rows, half the up rows of the same outputs.
// ---------------------------------------------------------------------------
constexpr int BIG_ROWS = 128, BIG_COLS = 256, BIG_K = 64;

template <bool UP, int ACT>
__global__ __launch_bounds__(256, 2) void expert_tiles_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x,
    const bf16* __restrict__ w, MoePlan p, int m, int k, int m_tiles) {
  constexpr int MT = UP ? BIG_COLS / 2 : BIG_COLS;  // outputs of a block
  constexpr int XI = BIG_ROWS / 32, WI = BIG_COLS / 32;
  extern __shared__ __attribute__((aligned(16))) bf16 sm[];
  // an XCD's blocks are neighbours in the list of (weight tile, pair tile)
  const int total = *p.n_tiles * m_tiles, per = (total + 7) / 8;
  const int at = blockIdx.x / 8, unit = (blockIdx.x % 8) * per + at;
  if (at >= per || unit >= total) return;
  const MoeTile head = p.tiles[unit / m_tiles];
  const int u = unit - head.tile0 * m_tiles;
  const MoeTile tile = p.tiles[head.tile0 + u % head.n_tiles];
  // the last tile of outputs may overlap the one before
  const int m0 = min(u / head.n_tiles * MT, m - MT);

  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, quad = lane >> 4;
  const int wr = wave >> 1, wc = wave & 1;
  // rows of a thread's chunks: r0, r0 + 32, ..
  const int r0 = tid >> 3, ch = tid & 7;
  // byte offsets in 32 bits; the weight rows of a thread are 32 apart
  const char* xb = reinterpret_cast<const char*>(x);
  unsigned xo[XI];
#pragma unroll
  for (int i = 0; i < XI; ++i) {
    // rows past the end repeat the last one; they are never stored
    const int pair =
        p.order[tile.first + min(i * 32 + r0, tile.rows - 1)];
    xo[i] = ((unsigned)(UP ? pair / p.top : pair) * k + ch * 8) * 2;
  }
  const char* wb = reinterpret_cast<const char*>(
      w + ((size_t)tile.expert * (UP ? 2 : 1) * m + m0) * k);
  const unsigned wo = ((unsigned)r0 * k + ch * 8) * 2;
  // up rows lie m after the gate rows of the same outputs
  auto wskip = [&](int i) {
    return (size_t)(UP && i * 32 >= MT ? m + i * 32 - MT : i * 32) * k * 2;
  };
  const int put = r0 * BIG_K + ((ch ^ (r0 & 7)) << 3);
  bf16x8 xr[XI], wreg[WI];
  auto load = [&](int k0) {
#pragma unroll
    for (int i = 0; i < XI; ++i)
      xr[i] = *reinterpret_cast<const bf16x8*>(xb + (xo[i] + k0 * 2));
#pragma unroll
    for (int i = 0; i < WI; ++i)
      wreg[i] = *reinterpret_cast<const bf16x8*>(wb + wskip(i) + (wo + k0 * 2));
  };
  auto store = [&](bf16* b) {
#pragma unroll
    for (int i = 0; i < XI; ++i)
      *reinterpret_cast<bf16x8*>(b + i * 32 * BIG_K + put) = xr[i];
#pragma unroll
    for (int i = 0; i < WI; ++i)
      *reinterpret_cast<bf16x8*>(b + (BIG_ROWS + i * 32) * BIG_K + put) =
          wreg[i];
  };
  // first LDS row of this wave's j-th 16 weight rows
  auto wrow = [&](int j) {
    return BIG_ROWS + (UP ? (j / 4) * MT + wc * 64 + (j % 4) * 16
                          : wc * 128 + j * 16);
  };
  f32x4 acc[4][8];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int steps = k / BIG_K;
  load(0);
  for (int s = 0; s < steps; ++s) {
    if (s) __syncthreads();
    store(sm);
    if (s + 1 < steps) load((s + 1) * BIG_K);
    __syncthreads();
    // operand loads run a few products ahead of the MFMAs
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const int chunk = ((kk * 4 + quad) ^ (c & 7)) << 3;
      bf16x8 xf[4], wf[8];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        xf[i] = *reinterpret_cast<const bf16x8*>(
            sm + (wr * 64 + i * 16 + c) * BIG_K + chunk);
#pragma unroll
      for (int j = 0; j < 8; ++j)
        wf[j] = *reinterpret_cast<const bf16x8*>(
            sm + (wrow(j) + c) * BIG_K + chunk);
#pragma unroll
      for (int j = 0; j < 8; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[j], xf[i], acc[i][j], 0, 0, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x100, 6, 0);
#pragma unroll
    for (int g = 0; g < 18; ++g) {
      __builtin_amdgcn_sched_group_barrier(0x008, 3, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x008, 10, 0);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = wr * 64 + i * 16 + c;
    if (row >= tile.rows) continue;
    bf16* o = out + (size_t)p.order[tile.first + row] * m;
#pragma unroll
    for (int j = 0; j < (UP ? 4 : 8); ++j) {
      const int col = m0 + (UP ? wc * 64 : wc * 128) + j * 16 + quad * 4;
      Pack<bf16, 4> v;
#pragma unroll
      for (int q = 0; q < 4; ++q)
        v.v[q] = from_f<bf16>(UP ? gated(acc[i][j][q], acc[i][(j + 4) % 8][q], ACT)
                                 : acc[i][j][q]);
      // m is a multiple of 4
      if (col < m) *reinterpret_cast<Pack<bf16, 4>*>(o + col) = v;
    }
  }
}

template <bool UP, int ACT>
void expert_tiles(void* out, const void* x, const void* w, MoePlan p, int m,
                  int k, hipStream_t stream) {
  constexpr size_t smem = (BIG_ROWS + BIG_COLS) * BIG_K * sizeof(bf16);
  const int m_tiles = (m + (UP ? BIG_COLS / 2 : BIG_COLS) - 1) /
                      (UP ? BIG_COLS / 2 : BIG_COLS);
  const long long units = (long long)p.max_tiles * m_tiles;
  auto kernel = expert_tiles_kernel<UP, ACT>;
  (void)hipFuncSetAttribute((const void*)kernel,
                            hipFuncAttributeMaxDynamicSharedMemorySize,
                            (int)smem);
  kernel<<<(unsigned)((units + 7) / 8 * 8), 256, smem, stream>>>(
      (bf16*)out, (const bf16*)x, (const bf16*)w, p, m, k, m_tiles);
}

}  // namespace

MoePlan moe_plan(int* buffer, int n, int top, int experts, int tile_rows) {
  MoePlan p{};
  p.outputs = experts;
  p.pairs = n * top;
  p.top = top;
  p.experts = experts;
  p.tile_rows = tile_rows;
  // every expert's last tile may be short
  const long long tiles = p.pairs / p.tile_rows + experts;
  p.max_tiles = (int)(tiles < p.pairs ? tiles : p.pairs);
  p.chosen = buffer;
  p.order = p.chosen + p.pairs;
  p.n_tiles = p.order + p.pairs;
  p.tiles = reinterpret_cast<MoeTile*>(p.n_tiles + 1);
  return p;
}

long long moe_plan_ints(int n, int top, int experts, int tile_rows) {
  const long long pairs = (long long)n * top;
  return 2 * pairs + 1 +
         (pairs / tile_rows + experts) * (sizeof(MoeTile) / sizeof(int));
}

void launch_moe_route(float* weight, float* z, const void* x,
                      const void* router, MoePlan p, int n, int k, int f32,
                      hipStream_t stream) {
  const int cols = p.outputs + p.gated;
  const dim3 grid((cols + 15) / 16, (n + 15) / 16);
  if (f32)
    router_kernel<float, 16><<<grid, 1024, 0, stream>>>(
        z, (const float*)x, (const float*)router, n, cols, k, k % 4 == 0);
  else
    router_kernel<bf16, 16><<<grid, 1024, 0, stream>>>(
        z, (const bf16*)x, (const bf16*)router, n, cols, k, k % 8 == 0);
  const bool fused = n <= FUSED_ROWS;
  if (!fused) choose_kernel<<<(n + 3) / 4, 256, 0, stream>>>(weight, z, p, n);
  order_kernel<<<1, 1024, 0, stream>>>(weight, z, p, n, fused);
}

void launch_moe_up(void* mid, const void* x, const void* w, MoePlan p,
                   int ff, int k, int act, int f32, hipStream_t stream) {
  if (p.tile_rows == BIG_ROWS && act == 0)
    expert_tiles<true, 0>(mid, x, w, p, ff, k, stream);
  else if (p.tile_rows == BIG_ROWS)
    expert_tiles<true, 1>(mid, x, w, p, ff, k, stream);
  else if (f32) expert_rows_t<float, true>(mid, x, w, p, ff, k, act, stream);
  else expert_rows_t<bf16, true>(mid, x, w, p, ff, k, act, stream);
}

void launch_moe_down(void* out, const void* mid, const void* w, MoePlan p,
                     int m, int ff, int f32, hipStream_t stream) {
  if (p.tile_rows == BIG_ROWS)
    expert_tiles<false, 0>(out, mid, w, p, m, ff, stream);
  else if (f32) expert_rows_t<float, false>(out, mid, w, p, m, ff, 0, stream);
  else expert_rows_t<bf16, false>(out, mid, w, p, m, ff, 0, stream);
}
