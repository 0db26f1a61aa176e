// Row kernels of blocks that norm their sublayers' outputs (gfx950): residual
// step with grouped norms, routed rows, the average over depth and the token
// shift; and the gated group norm behind a state-space read-out.

#include <algorithm>

#include "hybrid_common.h"

namespace {

// 1 / sqrt(mean + eps) of each of `groups` equal parts of a row, from the
// sums of squares of its chunks of V elements (chunk k * NT + tid in ss[k]);
// part holds e / V floats, inv the result.
template <int V, int NT, int KEEP>
DEVINL void group_scales(const float (&ss)[KEEP], float* part, float* inv,
                         int e, int groups, float eps) {
  const int chunks = e / V, per = chunks / groups;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = k * NT + threadIdx.x;
    if (c < chunks) part[c] = ss[k];
  }
  __syncthreads();
  const int lane = threadIdx.x & 63;
  for (int g = threadIdx.x >> 6; g < groups; g += NT / 64) {
    float s = 0.f;
    for (int c = lane; c < per; c += 64) s += part[g * per + c];
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.f / sqrtf(s / (per * V) + eps);
  }
  __syncthreads();
}

constexpr int PAST_COLS = 128;  // vectors of a block below

// The weighted sum of earlier results by blocks of their own, beside the
// blocks of the rows: NT / PAST_COLS threads share a column.
template <int V, int NT>
DEVINL void past_sum(const StreamArgs& p, float* part, int block) {
  using PF = Pack<float, V>;
  constexpr int SPLIT = NT / PAST_COLS;
  const int col = threadIdx.x % PAST_COLS, first = threadIdx.x / PAST_COLS;
  const size_t total = (size_t)p.n * p.e;
  const size_t at = ((size_t)block * PAST_COLS + col) * V;
  PF sum{};
  if (at < total) {
#pragma unroll 8
    for (int d = first; d < p.depth; d += SPLIT) {
      const float f = p.coef[d];
      const PF v = *reinterpret_cast<const PF*>(p.hist + d * total + at);
#pragma unroll
      for (int j = 0; j < V; ++j) sum.v[j] += f * v.v[j];
    }
  }
#pragma unroll
  for (int j = 0; j < V; ++j)
    part[(first * V + j) * PAST_COLS + col] = sum.v[j];
  __syncthreads();
  if (first == 0 && at < total) {
#pragma unroll
    for (int j = 0; j < V; ++j)
#pragma unroll
      for (int k = 1; k < SPLIT; ++k)
        sum.v[j] += part[(k * V + j) * PAST_COLS + col];
    *reinterpret_cast<PF*>(p.past + at) = sum;
  }
}

template <typename T, int V, int NT, int KEEP>
__global__ __launch_bounds__(NT) void stream_step_kernel(StreamArgs p) {
  extern __shared__ float part[];
  if ((int)blockIdx.x >= p.n) {
    past_sum<V, NT>(p, part, blockIdx.x - p.n);
    return;
  }
  const int e = p.e, per = e / V / p.groups;
  float* inv = part + e / V;
  const size_t row = blockIdx.x;
  float* __restrict__ x = p.x + row * e;
  using PT = Pack<T, V>;
  using PF = Pack<float, V>;
  PF a[KEEP];
#define EACH(i)                                                 \
  _Pragma("unroll") for (int k = 0; k < KEEP; ++k)              \
    if (const int i = (k * NT + threadIdx.x) * V; i < e)
#define LOAD(type, ptr) *reinterpret_cast<const type*>(ptr)
  if (p.tokens != nullptr) {
    const T* t = (const T*)p.table + (size_t)p.tokens[row] * e;
    EACH(i) {
      const PT b = LOAD(PT, t + i);
#pragma unroll
      for (int j = 0; j < V; ++j) a[k].v[j] = to_f(b.v[j]) * p.scale;
    }
  } else {
    EACH(i) a[k] = LOAD(PF, x + i);
    if (p.y != nullptr || p.routed != nullptr) {
      PF b[KEEP];
      const int cols = p.top + (p.y != nullptr);
      const float* rw = p.routed_w + row * cols;
      if (p.y != nullptr) {
        const T* y = (const T*)p.y + row * e;
        const float f = p.routed != nullptr ? rw[p.top] : 1.f;
        EACH(i) {
          const PT v = LOAD(PT, y + i);
#pragma unroll
          for (int j = 0; j < V; ++j) b[k].v[j] = f * to_f(v.v[j]);
        }
      } else {
        EACH(i) b[k] = PF{};
      }
      for (int r = 0; r < p.top; ++r) {
        const float f = rw[r];
        if (p.chosen[row * p.top + r] >= p.experts) {
          EACH(i) {
#pragma unroll
            for (int j = 0; j < V; ++j) b[k].v[j] += f * a[k].v[j];
          }
        } else {
          const T* z = (const T*)p.routed + (row * p.top + r) * e;
          EACH(i) {
            const PT v = LOAD(PT, z + i);
#pragma unroll
            for (int j = 0; j < V; ++j) b[k].v[j] += f * to_f(v.v[j]);
          }
        }
      }
      if (p.post_w != nullptr) {
        float ss[KEEP] = {};
        EACH(i) {
#pragma unroll
          for (int j = 0; j < V; ++j) ss[k] += b[k].v[j] * b[k].v[j];
        }
        group_scales<V, NT, KEEP>(ss, part, inv, e, p.groups, p.eps);
        EACH(i) {
          const PF w = LOAD(PF, p.post_w + i);
          const float r = inv[i / V / per];
#pragma unroll
          for (int j = 0; j < V; ++j) b[k].v[j] *= r * w.v[j];
        }
      }
      EACH(i) {
#pragma unroll
        for (int j = 0; j < V; ++j) a[k].v[j] += b[k].v[j];
      }
    }
  }
  if (p.keep != nullptr) {
    EACH(i) *reinterpret_cast<PF*>(p.keep + row * e + i) = a[k];
  }
  if (p.coef != nullptr && p.past == nullptr) {
    const float own = p.coef[p.depth];
    EACH(i) {
#pragma unroll
      for (int j = 0; j < V; ++j) a[k].v[j] *= own;
    }
    const size_t step = (size_t)p.n * e;
    const float* hist = p.hist + row * e;
#pragma unroll 4
    for (int d = 0; d < p.depth; ++d) {
      const float f = p.coef[d];
      EACH(i) {
        const PF v = LOAD(PF, hist + d * step + i);
#pragma unroll
        for (int j = 0; j < V; ++j) a[k].v[j] += f * v.v[j];
      }
    }
  }
  EACH(i) *reinterpret_cast<PF*>(x + i) = a[k];
  if (p.xn == nullptr) return;
  T* xn = (T*)p.xn + row * e;
  if (p.next_w != nullptr) {
    float ss[KEEP] = {};
    EACH(i) {
#pragma unroll
      for (int j = 0; j < V; ++j) ss[k] += a[k].v[j] * a[k].v[j];
    }
    group_scales<V, NT, KEEP>(ss, part, inv, e, p.groups, p.eps);
    EACH(i) {
      const PF w = LOAD(PF, p.next_w + i);
      const float r = inv[i / V / per];
#pragma unroll
      for (int j = 0; j < V; ++j) a[k].v[j] *= r * w.v[j];
    }
  } else if (p.shift != nullptr) {
    float* prev = p.prev + (size_t)p.row_slot[row] * e;
    const bool fresh = p.row_pos[row] == 0;
    EACH(i) {
      const PF w = LOAD(PF, p.shift + i);
      PF h{};
      if (!fresh) h = LOAD(PF, prev + i);
      *reinterpret_cast<PF*>(prev + i) = a[k];
#pragma unroll
      for (int j = 0; j < V; ++j)
        a[k].v[j] += (h.v[j] - a[k].v[j]) * w.v[j];
    }
  }
  EACH(i) {
    PT o;
#pragma unroll
    for (int j = 0; j < V; ++j) o.v[j] = from_f<T>(a[k].v[j]);
    *reinterpret_cast<PT*>(xn + i) = o;
  }
}

// picks a block shape for rows of e elements; 0 if one fits
#define ROW_SHAPES(V, few)                                   \
  if constexpr (V == 1) {                                    \
    if (e <= 1024) RUN(V, 256, 4);                           \
    else if (e <= 12288) RUN(V, 1024, 12);                   \
    else return -1;                                          \
  } else if (few && e >= 2048 && e <= 16384) {               \
    if (e <= 4096) RUN(V, 1024, 1);                          \
    else RUN(V, 1024, 4);                                    \
  } else if (e <= 1024) {                                    \
    RUN(V, 256, 1);                                          \
  } else if (e <= 4096) {                                    \
    RUN(V, 256, 4);                                          \
  } else if (e <= 8192) {                                    \
    RUN(V, 512, 4);                                          \
  } else if (e <= 32768) {                                   \
    RUN(V, 1024, 8);                                         \
  } else {                                                   \
    return -1;                                               \
  }                                                          \
  return 0;

template <typename T, int V>
int stream_step_t(const StreamArgs& a, hipStream_t stream) {
  const int e = a.e;
  size_t smem = (e / V + a.groups) * sizeof(float);
  int blocks = a.n;
  if (a.past != nullptr) {
    const size_t vectors = (size_t)a.n * e / V;
    blocks += (int)((vectors + PAST_COLS - 1) / PAST_COLS);
    smem = std::max(smem, 1024 * V * sizeof(float));
  }
#define RUN(V, NT, KEEP) \
  stream_step_kernel<T, V, NT, KEEP><<<blocks, NT, smem, stream>>>(a)
  ROW_SHAPES(V, a.n <= 256)
#undef RUN
}

// one block per (token, segment)
template <typename T, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(
    T* __restrict__ xn, const float* __restrict__ x,
    const float* __restrict__ shift, float* __restrict__ prev, SegView seg,
    int e) {
  const int t = blockIdx.x, s = blockIdx.y, len = seg.len[s];
  if (t >= len) return;
  const size_t row = (size_t)seg.start[s] + t;
  float* slot = prev + (size_t)seg.slot[s] * e;
  const bool fresh = seg.pos0[s] == 0;
  using PF = Pack<float, V>;
  for (int i = threadIdx.x * V; i < e; i += 256 * V) {
    const PF a = LOAD(PF, x + row * e + i), w = LOAD(PF, shift + i);
    PF h{};
    if (t > 0) {
      h = LOAD(PF, x + (row - 1) * e + i);
    } else {
      if (!fresh) h = LOAD(PF, slot + i);
      // only this block looks at the slot
      *reinterpret_cast<PF*>(slot + i) =
          LOAD(PF, x + (row + len - 1) * e + i);
    }
    Pack<T, V> o;
#pragma unroll
    for (int j = 0; j < V; ++j)
      o.v[j] = from_f<T>(a.v[j] + (h.v[j] - a.v[j]) * w.v[j]);
    *reinterpret_cast<Pack<T, V>*>(xn + row * e + i) = o;
  }
}

template <typename T, int V, int NT, int KEEP>
__global__ __launch_bounds__(NT) void gated_norm_kernel(GatedNormArgs p) {
  extern __shared__ float part[];
  const int e = p.inner, per = e / V / p.groups;
  float* inv = part + e / V;
  const size_t row = blockIdx.x;
  using PT = Pack<T, V>;
  using PF = Pack<float, V>;
  const T* x = (const T*)p.x + row * p.xld;
  const T* z = (const T*)p.z + row * p.zld;
  PF a[KEEP];
  float ss[KEEP] = {};
  EACH(i) {
    a[k] = LOAD(PF, p.o + row * e + i);
    const PT b = LOAD(PT, x + i), g = LOAD(PT, z + i);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float zz = to_f(g.v[j]);
      a[k].v[j] = (a[k].v[j] + p.skip[(i + j) / p.vdim] * to_f(b.v[j])) * zz *
                  sigmoid(zz);
      ss[k] += a[k].v[j] * a[k].v[j];
    }
  }
  group_scales<V, NT, KEEP>(ss, part, inv, e, p.groups, p.eps);
  T* out = (T*)p.out + row * e;
  EACH(i) {
    const PF w = LOAD(PF, p.w + i);
    const float r = inv[i / V / per];
    PT o;
#pragma unroll
    for (int j = 0; j < V; ++j) o.v[j] = from_f<T>(a[k].v[j] * r * w.v[j]);
    *reinterpret_cast<PT*>(out + i) = o;
  }
}
#undef LOAD
#undef EACH

template <typename T, int V>
int gated_norm_t(const GatedNormArgs& a, hipStream_t stream) {
  const int e = a.inner;
  const size_t smem = (e / V + a.groups) * sizeof(float);
#define RUN(V, NT, KEEP) \
  gated_norm_kernel<T, V, NT, KEEP><<<a.n, NT, smem, stream>>>(a)
  ROW_SHAPES(V, a.n <= 256)
#undef RUN
}

}  // namespace

int launch_stream_step(const StreamArgs& a, int f32, hipStream_t stream) {
  const bool vec = a.e % (4 * a.groups) == 0;
  if (f32)
    return vec ? stream_step_t<float, 4>(a, stream)
               : stream_step_t<float, 1>(a, stream);
  return vec ? stream_step_t<bf16, 4>(a, stream)
             : stream_step_t<bf16, 1>(a, stream);
}

void launch_token_shift(void* xn, const float* x, const float* shift,
                        float* prev, SegView seg, int max_len, int e, int f32,
                        hipStream_t stream) {
  const dim3 grid(max_len, seg.n);
#define SHIFT(T, V)                                                    \
  token_shift_kernel<T, V><<<grid, 256, 0, stream>>>((T*)xn, x, shift, \
                                                     prev, seg, e)
  if (f32) {
    if (e % 4 == 0) SHIFT(float, 4);
    else SHIFT(float, 1);
  } else {
    if (e % 4 == 0) SHIFT(bf16, 4);
    else SHIFT(bf16, 1);
  }
#undef SHIFT
}

int launch_gated_norm(const GatedNormArgs& a, int f32, hipStream_t stream) {
  const bool vec = a.vec && a.inner % (4 * a.groups) == 0;
  if (f32)
    return vec ? gated_norm_t<float, 4>(a, stream)
               : gated_norm_t<float, 1>(a, stream);
  return vec ? gated_norm_t<bf16, 4>(a, stream)
             : gated_norm_t<bf16, 1>(a, stream);
}
