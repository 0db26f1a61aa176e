// Row kernels of latent attention and gated feed-forwards, and the per-head
// products between a head's own sizes and the latent (gfx950).

#include "mfma_frag.h"

namespace {

// ---------------------------------------------------------------------------
// Norms of a row's query and key/value latents; the latter goes to its place
// in the cache.  One wave per (row, latent).
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
__global__ __launch_bounds__(256) void latent_norm_append_kernel(
    T* __restrict__ q_out, const T* __restrict__ q,
    const float* __restrict__ q_w, T* __restrict__ pages,
    const T* __restrict__ kv, const float* __restrict__ kv_w,
    const int* __restrict__ row_slot, const int* __restrict__ row_pos,
    const int* __restrict__ table, int table_stride, int n, int q_rank,
    long long q_ld, int rank, long long kv_ld, int rpad, float eps) {
  const int lane = threadIdx.x & 63;
  const size_t row = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= n) return;
  if (blockIdx.y == 0) {
    if (q == nullptr) return;
    wave_norm<T, V>(q_out + row * q_rank, q + row * q_ld, q_w, q_rank, eps,
                    lane);
  } else {
    const int pos = row_pos[row];
    const size_t page =
        table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
    wave_norm<T, V>(pages + (page * 64 + (pos & 63)) * rpad, kv + row * kv_ld,
                    kv_w, rank, eps, lane);
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
template <typename T, int V>
__global__ __launch_bounds__(256) void gated_act_kernel(
    T* __restrict__ out, long long out_ld, const T* __restrict__ gate,
    const T* __restrict__ up, long long in_ld, int cols, int act) {
  using P = Pack<T, V>;
  const size_t row = blockIdx.y;
  const int i = (blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= cols) return;
  const P a = *reinterpret_cast<const P*>(gate + row * in_ld + i);
  const P b = *reinterpret_cast<const P*>(up + row * in_ld + i);
  P o;
#pragma unroll
  for (int j = 0; j < V; ++j)
    o.v[j] = from_f<T>(gated(to_f(a.v[j]), to_f(b.v[j]), act));
  *reinterpret_cast<P*>(out + row * out_ld + i) = o;
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
  if (PARTS) {
    float* we = reinterpret_cast<float*>(xs + 16 * ld);  // [16][splits]
    // 16 lanes per row
    const int row = tid >> 4, k = tid & 15;
    if (r0 + row < a.n) {
      const size_t cell = ((size_t)(r0 + row) * a.heads + h) * a.splits;
      const float* ml = a.part_ml + cell * 2;
      float mm = -__builtin_huge_valf();
      for (int s = k; s < a.splits; s += 16) mm = fmaxf(mm, ml[s * 2]);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1)
        mm = fmaxf(mm, __shfl_xor(mm, off, 64));
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
        for (int s = 0; s < a.splits; ++s) {
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
  const int m0 = blockIdx.x * HEAD_COLS + wave * 16;
  if (m0 >= a.m) return;
  const T* wp = (const T*)a.w +
                ((size_t)h * a.m + min(m0 + c, a.m - 1)) * a.k + quad * 8;
  const T* xp = xs + c * ld + quad * 8;
  f32x4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < a.k; k += 32)
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

void launch_latent_norm_append(void* q_out, const void* q, const float* q_w,
                               void* pages, const void* kv,
                               const float* kv_w, const int* row_slot,
                               const int* row_pos, const int* table,
                               int table_stride, int n, int q_rank,
                               long long q_ld, int rank, long long kv_ld,
                               int rpad, float eps, int f32,
                               hipStream_t stream) {
  const dim3 grid((n + 3) / 4, kv != nullptr ? 2 : 1);
#define APPEND(T, V)                                                       \
  latent_norm_append_kernel<T, V><<<grid, 256, 0, stream>>>(               \
      (T*)q_out, (const T*)q, q_w, (T*)pages, (const T*)kv, kv_w,          \
      row_slot, row_pos, table, table_stride, n, q_rank, q_ld, rank,       \
      kv_ld, rpad, eps)
  auto fits = [&](int v, size_t bytes) {
    return q_rank % v == 0 && q_ld % v == 0 && rank % v == 0 &&
           kv_ld % v == 0 && (size_t)q % bytes == 0 && (size_t)kv % bytes == 0;
  };
  if (f32) {
    if (fits(4, 16)) APPEND(float, 4);
    else APPEND(float, 1);
  } else {
    if (fits(8, 16)) APPEND(bf16, 8);
    else APPEND(bf16, 1);
  }
#undef APPEND
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

void launch_gated_act(void* out, long long out_ld, const void* gate,
                      const void* up, long long in_ld, int n, int cols,
                      int act, int f32, hipStream_t stream) {
  auto fits = [&](int v) {
    return cols % v == 0 && out_ld % v == 0 && in_ld % v == 0 &&
           ((size_t)out | (size_t)gate | (size_t)up) % 16 == 0;
  };
#define ACT(T, V)                                                          \
  gated_act_kernel<T, V>                                                   \
      <<<dim3((cols + 256 * V - 1) / (256 * V), n), 256, 0, stream>>>(     \
          (T*)out, out_ld, (const T*)gate, (const T*)up, in_ld, cols, act)
  if (f32) {
    if (fits(4)) ACT(float, 4);
    else ACT(float, 1);
  } else {
    if (fits(8)) ACT(bf16, 8);
    else ACT(bf16, 1);
  }
#undef ACT
}
