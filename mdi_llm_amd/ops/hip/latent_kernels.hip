// Row kernels of latent attention and gated feed-forwards, and the per-head
// products between a head's own sizes and the latent (gfx950).

#include "mfma_frag.h"

namespace {

// ---------------------------------------------------------------------------
// What follows the first product of a parallel block, in one launch: norms of
// a row's query and key/value latents (the latter goes to its place in the
// cache), one wave per (row, latent), and the gated activation.
// ---------------------------------------------------------------------------
template <typename T, int V>
DEVINL void wave_norm(T* dst, const T* src, const float* w, int n, float eps,
                      int lane) {
  using P = Pack<T, V>;
  float r = 1.f;
  if (w != nullptr) {
    float ss = 0.f;
    for (int i = lane * V; i < n; i += 64 * V) {
      const P a = *reinterpret_cast<const P*>(src + i);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += to_f(a.v[j]) * to_f(a.v[j]);
    }
    r = 1.f / sqrtf(wave_sum(ss) / n + eps);
  }
  for (int i = lane * V; i < n; i += 64 * V) {
    P a = *reinterpret_cast<const P*>(src + i);
    if (w != nullptr) {
#pragma unroll
      for (int j = 0; j < V; ++j) a.v[j] = from_f<T>(to_f(a.v[j]) * r * w[i + j]);
    }
    *reinterpret_cast<P*>(dst + i) = a;
  }
}

template <typename T, int V>
DEVINL void act_row(const BranchArgs& a, size_t row, int i) {
  using P = Pack<T, V>;
  if (i >= a.cols) return;
  const P g = *reinterpret_cast<const P*>((const T*)a.gate + row * a.in_ld + i);
  const P u = *reinterpret_cast<const P*>((const T*)a.up + row * a.in_ld + i);
  P o;
#pragma unroll
  for (int j = 0; j < V; ++j)
    o.v[j] = from_f<T>(gated(to_f(g.v[j]), to_f(u.v[j]), a.act));
  *reinterpret_cast<P*>((T*)a.out + row * a.out_ld + i) = o;
}

// blockIdx.y: 0 query latents, 1 key/value latents (four rows a block), then
// the gated activation in blocks of 256 * AV columns of four rows
template <typename T, int V, int AV>
__global__ __launch_bounds__(256) void branch_kernel(BranchArgs a) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const size_t row = (size_t)blockIdx.x * 4 + wave;
  if (blockIdx.y == 0) {
    if (row >= a.n || a.q == nullptr) return;
    wave_norm<T, V>((T*)a.q_out + row * a.q_rank,
                    (const T*)a.q + row * a.q_ld, a.q_w, a.q_rank, a.eps,
                    lane);
  } else if (blockIdx.y == 1) {
    if (row >= a.n || a.kv == nullptr) return;
    const int pos = a.row_pos[row];
    const size_t page =
        a.table[(size_t)a.row_slot[row] * a.table_stride + (pos >> 6)];
    wave_norm<T, V>((T*)a.pages + (page * 64 + (pos & 63)) * a.rpad,
                    (const T*)a.kv + row * a.kv_ld, a.kv_w, a.rank, a.eps,
                    lane);
  } else {
    const int i = ((blockIdx.y - 2) * 256 + threadIdx.x) * AV;
    for (int r = 0; r < 4; ++r)
      if ((size_t)blockIdx.x * 4 + r < a.n)
        act_row<T, AV>(a, (size_t)blockIdx.x * 4 + r, i);
  }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void latent_gather_kernel(
    T* __restrict__ out, const T* __restrict__ pages,
    const int* __restrict__ table, int table_stride, SegView seg, int rank,
    int rpad) {
  const int s = blockIdx.y, lane = threadIdx.x & 63;
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= seg.len[s]) return;
  const int pos = seg.pos0[s] + t;
  const size_t page =
      table[(size_t)seg.slot[s] * table_stride + (pos >> 6)];
  const T* src = pages + (page * 64 + (pos & 63)) * rpad;
  T* dst = out + ((size_t)seg.start[s] + t) * rank;
  for (int i = lane * V; i < rank; i += 64 * V)
    *reinterpret_cast<Pack<T, V>*>(dst + i) =
        *reinterpret_cast<const Pack<T, V>*>(src + i);
}

// ---------------------------------------------------------------------------
// Per-head products of a few rows.  A block has 16 rows of one head in LDS
// (merged from the attention's partial results, if it has those) and its four
// waves take 16 outputs each; the weights are the MFMA's A operand, straight
// from memory.
// ---------------------------------------------------------------------------
constexpr int HEAD_COLS = 64;

template <typename T, bool PARTS>
__global__ __launch_bounds__(256) void head_proj_kernel(HeadProjArgs a) {
  using F = Frag<T>;
  constexpr int N = 16 / sizeof(T);
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, quad = lane >> 4;
  const int h = blockIdx.y, r0 = blockIdx.z * 16;
  const int ld = a.k + N;
  T* xs = reinterpret_cast<T*>(smem);
  // the weights set out first: they need nothing of what follows
  constexpr int PRE = sizeof(T) == 2 ? 16 : 8;
  const int m0 = blockIdx.x * HEAD_COLS + wave * 16;
  const T* wp = (const T*)a.w +
                ((size_t)h * a.m + min(m0 + c, a.m - 1)) * a.k + quad * 8;
  typename F::Row pre[PRE];
#pragma unroll
  for (int i = 0; i < PRE; ++i)
    if (i * 32 < a.k) pre[i] = F::load_frag(wp + i * 32);
  if (PARTS) {
    float* we = reinterpret_cast<float*>(xs + 16 * ld);  // [16][splits]
    // parts that saw keys come first; the others have no values
    __shared__ int live[16];
    // 16 lanes per row
    const int row = tid >> 4, k = tid & 15;
    if (r0 + row < a.n) {
      const size_t cell = ((size_t)(r0 + row) * a.heads + h) * a.splits;
      const float* ml = a.part_ml + cell * 2;
      float mm = -__builtin_huge_valf();
      int used = 0;
      for (int s = k; s < a.splits; s += 16) {
        const float ms = ml[s * 2];
        mm = fmaxf(mm, ms);
        if (ms != -__builtin_huge_valf()) used = s + 1;
      }
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) {
        mm = fmaxf(mm, __shfl_xor(mm, off, 64));
        used = max(used, __shfl_xor(used, off, 64));
      }
      if (k == 0) live[row] = used;
      float sum = 0.f;
      for (int s = k; s < a.splits; s += 16)
        sum += __builtin_amdgcn_exp2f(ml[s * 2] - mm) * ml[s * 2 + 1];
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
      for (int s = k; s < a.splits; s += 16)
        we[row * a.splits + s] =
            __builtin_amdgcn_exp2f(ml[s * 2] - mm) / sum;
    }
    __syncthreads();
    for (int i = tid * 4; i < 16 * a.k; i += 1024) {
      const int row = i / a.k, k = i % a.k;
      float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
      if (r0 + row < a.n) {
        const float* po =
            a.part_o +
            ((size_t)(r0 + row) * a.heads + h) * a.splits * a.k + k;
        const int used = live[row];
#pragma unroll 8
        for (int s = 0; s < used; ++s) {
          const float e = we[row * a.splits + s];
          const float4 v = *reinterpret_cast<const float4*>(
              po + (size_t)s * a.k);
          acc.x += e * v.x;
          acc.y += e * v.y;
          acc.z += e * v.z;
          acc.w += e * v.w;
        }
      }
      Pack<T, 4> o;
      o.v[0] = from_f<T>(acc.x);
      o.v[1] = from_f<T>(acc.y);
      o.v[2] = from_f<T>(acc.z);
      o.v[3] = from_f<T>(acc.w);
      *reinterpret_cast<Pack<T, 4>*>(xs + row * ld + k) = o;
    }
  } else {
    const bool vec = a.xk % N == 0 && a.x_ld % N == 0;
    for (int i = tid * N; i < 16 * a.k; i += 256 * N) {
      const int row = i / a.k, k = i % a.k;
      Pack<T, N> v{};
      if (r0 + row < a.n) {
        const size_t r = a.x_rows ? a.x_rows[r0 + row] : r0 + row;
        const T* p = (const T*)a.x + r * (size_t)a.x_ld + (size_t)h * a.xk;
        if (vec) {
          if (k < a.xk) v = *reinterpret_cast<const Pack<T, N>*>(p + k);
        } else {
#pragma unroll
          for (int j = 0; j < N; ++j)
            if (k + j < a.xk) v.v[j] = p[k + j];
        }
      }
      *reinterpret_cast<Pack<T, N>*>(xs + row * ld + k) = v;
    }
  }
  __syncthreads();
  if (m0 >= a.m) return;
  const T* xp = xs + c * ld + quad * 8;
  f32x4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < PRE; ++i)
    if (i * 32 < a.k)
      acc = F::dot(pre[i], F::load_frag(xp + i * 32), acc);
  for (int k = PRE * 32; k < a.k; k += 32)
    acc = F::dot(F::load_frag(wp + k), F::load_frag(xp + k), acc);
  if (r0 + c >= a.n) return;
  const size_t r = a.out_rows ? a.out_rows[r0 + c] : r0 + c;
  float f = 1.f;
  if (a.gate != nullptr)
    f = sigmoid(to_f(((const T*)a.gate)[r * (size_t)a.gate_ld + h]));
  T* op = (T*)a.out + r * (size_t)a.out_ld + (size_t)h * a.m;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + quad * 4 + i;
    if (m < a.m) op[m] = from_f<T>(acc[i] * f);
  }
}

template <typename T>
void head_proj_t(const HeadProjArgs& a, hipStream_t stream) {
  const dim3 grid((a.m + HEAD_COLS - 1) / HEAD_COLS, a.heads, (a.n + 15) / 16);
  size_t smem = 16 * (a.k + 16 / sizeof(T)) * sizeof(T);
  if (a.part_o != nullptr) {
    smem += (size_t)16 * a.splits * sizeof(float);
    head_proj_kernel<T, true><<<grid, 256, smem, stream>>>(a);
  } else {
    head_proj_kernel<T, false><<<grid, 256, smem, stream>>>(a);
  }
}

}  // namespace

void launch_head_proj(const HeadProjArgs& a, int f32, hipStream_t stream) {
  if (f32) head_proj_t<float>(a, stream);
  else head_proj_t<bf16>(a, stream);
}

void launch_branch(const BranchArgs& a, int f32, hipStream_t stream) {
  auto norms = [&](int v) {
    return a.q_rank % v == 0 && a.q_ld % v == 0 && a.rank % v == 0 &&
           a.kv_ld % v == 0 && ((size_t)a.q | (size_t)a.kv) % 16 == 0;
  };
  auto acts = [&](int v) {
    return a.cols % v == 0 && a.out_ld % v == 0 && a.in_ld % v == 0 &&
           ((size_t)a.out | (size_t)a.gate | (size_t)a.up) % 16 == 0;
  };
#define BRANCH(T, V, AV)                                                   \
  branch_kernel<T, V, AV>                                                  \
      <<<dim3((a.n + 3) / 4, 2 + (a.cols + 256 * AV - 1) / (256 * AV)),    \
         256, 0, stream>>>(a)
#define BY_ALIGNMENT(T, V)                   \
  if (norms(V) && acts(V)) BRANCH(T, V, V);  \
  else if (norms(V)) BRANCH(T, V, 1);        \
  else if (acts(V)) BRANCH(T, 1, V);         \
  else BRANCH(T, 1, 1)
  if (f32) {
    BY_ALIGNMENT(float, 4);
  } else {
    BY_ALIGNMENT(bf16, 8);
  }
#undef BY_ALIGNMENT
#undef BRANCH
}

void launch_latent_gather(void* out, const void* pages, const int* table,
                          int table_stride, SegView seg, int max_len,
                          int rank, int rpad, int f32, hipStream_t stream) {
  const dim3 grid((max_len + 3) / 4, seg.n);
#define GATHER(T, V)                                                    \
  latent_gather_kernel<T, V><<<grid, 256, 0, stream>>>(                 \
      (T*)out, (const T*)pages, table, table_stride, seg, rank, rpad)
  if (f32) {
    if (rank % 4 == 0) GATHER(float, 4);
    else GATHER(float, 1);
  } else {
    if (rank % 8 == 0) GATHER(bf16, 8);
    else GATHER(bf16, 1);
  }
#undef GATHER
}
