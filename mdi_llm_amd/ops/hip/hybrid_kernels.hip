// Row, gate, recurrence and cache-append kernels of the hybrid stacks
// (gfx950).  All of them take a flat batch of token rows; nothing here knows
// whether a row belongs to a prompt or to a decode step.

#include "matrix_state.h"

// ---------------------------------------------------------------------------
// Residual + norms, one block of NT threads per row.  Every thread keeps its
// KEEP accesses of V elements in registers, so a row is read once and all of
// it is in flight before the first reduction.
// ---------------------------------------------------------------------------
template <int NT>
DEVINL float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  v = 0.f;
#pragma unroll
  for (int k = 0; k < NT / 64; ++k) v += red[k];
  __syncthreads();
  return v;
}

template <typename T, int V, int NT, int KEEP>
__global__ __launch_bounds__(NT) void residual_norm_kernel(ResidualArgs p) {
  __shared__ float red[NT / 64];
  const size_t row = blockIdx.x;
  const int e = p.e;
  const float offset = p.offset, eps = p.eps;
  float* __restrict__ x = p.x + row * e;
  const T* __restrict__ y = (const T*)p.y;
  using PT = Pack<T, V>;
  using PF = Pack<float, V>;
  PF a[KEEP];
  float ss = 0.f;
#define EACH(i)                                                 \
  _Pragma("unroll") for (int k = 0; k < KEEP; ++k)              \
    if (const int i = (k * NT + threadIdx.x) * V; i < e)
  if (p.tokens != nullptr) {
    const T* t = (const T*)p.table + (size_t)p.tokens[row] * e;
    EACH(i) {
      const PT b = *reinterpret_cast<const PT*>(t + i);
#pragma unroll
      for (int j = 0; j < V; ++j) a[k].v[j] = to_f(b.v[j]) * p.scale;
    }
    if (p.pos_table != nullptr) {
      const T* t = (const T*)p.pos_table + (size_t)p.row_pos[row] * e;
      EACH(i) {
        const PT b = *reinterpret_cast<const PT*>(t + i);
#pragma unroll
        for (int j = 0; j < V; ++j) a[k].v[j] += to_f(b.v[j]);
      }
    }
    EACH(i) *reinterpret_cast<PF*>(x + i) = a[k];
  } else {
    EACH(i) a[k] = *reinterpret_cast<const PF*>(x + i);
    if (y != nullptr) {
      y += row * e;
      PT b[KEEP];
      EACH(i) b[k] = *reinterpret_cast<const PT*>(y + i);
      if (p.y2 != nullptr) {
        const T* y2 = (const T*)p.y2 + row * e;
        PT b2[KEEP];
        EACH(i) b2[k] = *reinterpret_cast<const PT*>(y2 + i);
        float s = 0.f, s2 = 0.f;
        EACH(i) {
#pragma unroll
          for (int j = 0; j < V; ++j) {
            s += to_f(b[k].v[j]) * to_f(b[k].v[j]);
            s2 += to_f(b2[k].v[j]) * to_f(b2[k].v[j]);
          }
        }
        const float r = p.mult / sqrtf(block_sum<NT>(s, red) / e + eps);
        const float r2 = p.mult / sqrtf(block_sum<NT>(s2, red) / e + eps);
        EACH(i) {
          const PF w = *reinterpret_cast<const PF*>(p.post_w + i);
          const PF w2 = *reinterpret_cast<const PF*>(p.post_w2 + i);
#pragma unroll
          for (int j = 0; j < V; ++j)
            a[k].v[j] += to_f(b[k].v[j]) * r * (offset + w.v[j]) +
                         to_f(b2[k].v[j]) * r2 * (offset + w2.v[j]);
        }
      } else if (p.post_w != nullptr) {
        PF w[KEEP];
        EACH(i) w[k] = *reinterpret_cast<const PF*>(p.post_w + i);
        float s = 0.f;
        EACH(i) {
#pragma unroll
          for (int j = 0; j < V; ++j) s += to_f(b[k].v[j]) * to_f(b[k].v[j]);
        }
        const float r = 1.f / sqrtf(block_sum<NT>(s, red) / e + eps);
        EACH(i) {
#pragma unroll
          for (int j = 0; j < V; ++j)
            a[k].v[j] +=
                to_f(b[k].v[j]) * r * (offset + w[k].v[j]) * p.mult;
        }
      } else if (p.gain != nullptr) {
        EACH(i) {
          const PF w = *reinterpret_cast<const PF*>(p.gain + i);
#pragma unroll
          for (int j = 0; j < V; ++j)
            a[k].v[j] += to_f(b[k].v[j]) * w.v[j] * p.mult;
        }
      } else {
        EACH(i) {
#pragma unroll
          for (int j = 0; j < V; ++j) a[k].v[j] += to_f(b[k].v[j]) * p.mult;
        }
      }
      for (int r = 0; r < p.top; ++r) {
        const float f = p.routed_w[row * p.top + r] * p.mult;
        const T* z = (const T*)p.routed + (row * p.top + r) * e;
        EACH(i) {
          const PT v = *reinterpret_cast<const PT*>(z + i);
#pragma unroll
          for (int j = 0; j < V; ++j) a[k].v[j] += f * to_f(v.v[j]);
        }
      }
      EACH(i) *reinterpret_cast<PF*>(x + i) = a[k];
    }
  }
  if (p.next_w == nullptr) return;
  PF w[KEEP];
  EACH(i) {
    w[k] = *reinterpret_cast<const PF*>(p.next_w + i);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += a[k].v[j] * a[k].v[j];
  }
  const float r = 1.f / sqrtf(block_sum<NT>(ss, red) / e + eps);
  T* __restrict__ xn = (T*)p.xn + row * e;
  EACH(i) {
    PT o;
#pragma unroll
    for (int j = 0; j < V; ++j)
      o.v[j] = from_f<T>(a[k].v[j] * r * (offset + w[k].v[j]));
    *reinterpret_cast<PT*>(xn + i) = o;
  }
#undef EACH
}

template <typename T>
static int residual_norm_t(const ResidualArgs& a, hipStream_t stream) {
  const int n = a.n, e = a.e;
#define ROWS(V, NT, KEEP) \
  residual_norm_kernel<T, V, NT, KEEP><<<n, NT, 0, stream>>>(a)
  if (e % 4 != 0) {
    if (e > 1024 * 16) return -1;
    if (e <= 1024) ROWS(1, 256, 4);
    else ROWS(1, 1024, 16);
  } else if (n <= 256 && e >= 2048 && e <= 16384) {
    if (e <= 4096) ROWS(4, 1024, 1);  // few rows: latency counts
    else ROWS(4, 1024, 4);
  } else if (e <= 1024) {
    ROWS(4, 256, 1);
  } else if (e <= 4096) {
    ROWS(4, 256, 4);
  } else if (e <= 8192) {
    ROWS(4, 512, 4);
  } else if (e <= 32768) {
    ROWS(4, 1024, 8);
  } else {
    return -1;
  }
#undef ROWS
  return 0;
}

int launch_residual_norm(const ResidualArgs& a, int f32, hipStream_t stream) {
  return f32 ? residual_norm_t<float>(a, stream)
             : residual_norm_t<bf16>(a, stream);
}

// ---------------------------------------------------------------------------
// xIELU (1), exact GELU (2) or squared ReLU (3) on a whole GEMM output (single
// rows have it in the GEMV epilogue)
// ---------------------------------------------------------------------------
template <typename T, int V, int ACT>
__global__ __launch_bounds__(256) void act_kernel(T* __restrict__ z,
                                                  long long n, float p,
                                                  float q) {
  const long long stride = (long long)gridDim.x * 256 * V;
  for (long long i = ((long long)blockIdx.x * 256 + threadIdx.x) * V; i < n;
       i += stride) {
    Pack<T, V> a = *reinterpret_cast<Pack<T, V>*>(z + i);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float f = to_f(a.v[j]);
      a.v[j] = from_f<T>(ACT == 3   ? relu2(f)
                         : ACT == 2 ? gelu_erf(f)
                                    : xielu(f, p, q));
    }
    *reinterpret_cast<Pack<T, V>*>(z + i) = a;
  }
}

template <typename T, int V, int ACT>
static void act_t(void* z, long long n, float p, float q,
                  hipStream_t stream) {
  const long long blocks = (n + 256 * V - 1) / (256 * V);
  act_kernel<T, V, ACT>
      <<<(int)(blocks < 8192 ? blocks : 8192), 256, 0, stream>>>((T*)z, n, p,
                                                                 q);
}

template <int ACT>
static void act_any(void* z, long long n, float p, float q, int f32,
                    hipStream_t stream) {
  if (f32) {
    if (n % 4 == 0) act_t<float, 4, ACT>(z, n, p, q, stream);
    else act_t<float, 1, ACT>(z, n, p, q, stream);
  } else {
    if (n % 8 == 0) act_t<bf16, 8, ACT>(z, n, p, q, stream);
    else act_t<bf16, 1, ACT>(z, n, p, q, stream);
  }
}

void launch_xielu(void* z, long long n, float p, float q, int f32,
                  hipStream_t stream) {
  act_any<1>(z, n, p, q, f32, stream);
}

void launch_gelu(void* z, long long n, int f32, hipStream_t stream) {
  act_any<2>(z, n, 0.f, 0.f, f32, stream);
}

void launch_relu2(void* z, long long n, int f32, hipStream_t stream) {
  act_any<3>(z, n, 0.f, 0.f, f32, stream);
}

// ---------------------------------------------------------------------------
// HGRN2: f is a gate with a lower bound, k = 1 - f (see matrix_state.h).
// ---------------------------------------------------------------------------
template <typename T>
struct Hgrn2Rule {
  static constexpr bool NORM = true, NORMALISER = false;
  T* out;
  const T* proj;
  const float* f_bias;
  const float* lower;
  const float* norm_w;
  int heads, dim, vdim;
  DEVINL const T* at(size_t row) const {
    return proj + row * (size_t)(heads * (2 * dim + vdim));
  }
  DEVINL StepFactors factors(size_t row, int h, int d) const {
    const int c = h * dim + d;
    const float q = to_f(at(row)[c]), l = lower[c];
    const float f = l + (1.f - l) * sigmoid(to_f(at(row)[heads * dim + c]) +
                                            f_bias[c]);
    return {q * sigmoid(q), f, 1.f - f};
  }
  DEVINL float value(size_t row, int h, int c) const {
    return to_f(at(row)[2 * heads * dim + h * vdim + c]);
  }
  DEVINL void put(size_t row, int h, int c, float v) const {
    out[row * (size_t)(heads * vdim) + h * vdim + c] =
        from_f<T>(v * norm_w[c]);
  }
};

void launch_hgrn2_step(void* out, const void* proj, float* state,
                       const float* f_bias, const float* lower,
                       const float* norm_w, SegView seg, int heads, int dim,
                       int vdim, int vstride, float eps, int f32,
                       hipStream_t stream) {
#define STEP(T)                                                              \
  matrix_step(Hgrn2Rule<T>{(T*)out, (const T*)proj, f_bias, lower, norm_w,   \
                           heads, dim, vdim},                                \
              state, seg, heads, dim, vdim, vstride, eps, stream)
  if (f32) STEP(float);
  else STEP(bf16);
#undef STEP
}

// Factors of a 16-token chunk: all decays are plain products of gates.
template <typename T, int DP>
__global__ __launch_bounds__(256) void hgrn2_factors_kernel(
    float* __restrict__ work, const T* __restrict__ proj,
    const float* __restrict__ f_bias, const float* __restrict__ lower,
    SegView seg, int heads, int dim, int vdim) {
  using W = ChunkWork<DP>;
  constexpr int CH = DP / 16;
  const int s = blockIdx.z, h = blockIdx.y, t0 = blockIdx.x * 16;
  const int tn = min(16, seg.len[s] - t0);
  if (tn <= 0) return;
  __shared__ __attribute__((aligned(16))) float fs[16][DP];
  __shared__ __attribute__((aligned(16))) float qs[16][DP];
  const int tid = threadIdx.x;
  const size_t row0 = (size_t)seg.start[s] + t0;
  const size_t ld = (size_t)heads * (2 * dim + vdim);
  float* w = work + (((size_t)seg.start[s] / 16 + s + blockIdx.x) * heads +
                     h) * W::SIZE;
  for (int i = tid; i < 16 * DP; i += 256) {
    const int t = i / DP, d = i % DP;
    float f = 1.f, q = 0.f;  // past the end: nothing decays or is written
    if (d >= dim) {
      f = 0.f;
    } else if (t < tn) {
      const T* pr = proj + (row0 + t) * ld + h * dim + d;
      const int c = h * dim + d;
      const float qv = to_f(pr[0]), l = lower[c];
      q = qv * sigmoid(qv);
      f = l + (1.f - l) * sigmoid(to_f(pr[heads * dim]) + f_bias[c]);
    }
    fs[t][d] = f;
    qs[t][d] = q;
  }
  __syncthreads();
  for (int i = tid; i < 2 * DP; i += 256) {
    const int d = i % DP;
    if (i < DP) {
      float r = 1.f;
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        r *= fs[t][d];
        w[W::QR + t * DP + d] = qs[t][d] * r;
      }
    } else {
      float u = 1.f;
      Pack<float, 4> k[4];
#pragma unroll
      for (int t = 15; t >= 0; --t) {
        const float f = fs[t][d];
        k[t / 4].v[t % 4] = d < dim ? u * (1.f - f) : 0.f;
        u *= f;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        *reinterpret_cast<Pack<float, 4>*>(w + W::UK + d * 16 + j * 4) = k[j];
      w[W::DECAY + d] = u;
    }
  }
  // P: thread (s', channels CH*dc ..) carries (1 - f_s') f .. f along t
  const int sp = tid >> 4, dc = tid & 15;
  float k[CH];
#pragma unroll
  for (int c = 0; c < CH; ++c) k[c] = 0.f;
#pragma unroll 4
  for (int t = 0; t < 16; ++t) {
    float acc = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const float f = fs[t][dc * CH + c];
      k[c] = t == sp ? 1.f - f : k[c] * f;
      acc += qs[t][dc * CH + c] * k[c];  // q is 0 in padding channels
    }
    acc = row16_sum(acc);
    if (dc == 0) w[W::P + t * 16 + sp] = acc;
  }
}

long long hgrn2_work_floats(int rows, int segments, int heads, int dim) {
  return chunk_work_floats(rows, segments, heads, dim);
}

template <typename T, int TPW>
static void hgrn2_scan_sized(float* o, float* work, const void* proj,
                             float* state, const float* f_bias,
                             const float* lower, SegView seg, int max_len,
                             int heads, int dim, int vdim, int vstride,
                             hipStream_t stream) {
  hgrn2_factors_kernel<T, 64 * TPW>
      <<<dim3((max_len + 15) / 16, heads, seg.n), 256, 0, stream>>>(
          work, (const T*)proj, f_bias, lower, seg, heads, dim, vdim);
  matrix_chunks_kernel<T, TPW>
      <<<dim3(heads, (vdim + 15) / 16, seg.n), 256, 0, stream>>>(
          o, work, (const T*)proj + 2 * heads * dim,
          (long long)heads * (2 * dim + vdim), state, seg, heads, dim, vdim,
          vstride);
}

template <typename T>
static int hgrn2_scan_t(float* o, float* work, const void* proj,
                        float* state, const float* f_bias,
                        const float* lower, SegView seg, int max_len,
                        int heads, int dim, int vdim, int vstride,
                        hipStream_t stream) {
#define SCAN(TPW)                                                          \
  hgrn2_scan_sized<T, TPW>(o, work, proj, state, f_bias, lower, seg,       \
                           max_len, heads, dim, vdim, vstride, stream)
  switch (chunk_dpad(dim)) {
    case 64: SCAN(1); return 0;
    case 128: SCAN(2); return 0;
    case 256: SCAN(4); return 0;
  }
#undef SCAN
  return -1;
}

int launch_hgrn2_scan(float* o, float* work, const void* proj, float* state,
                      const float* f_bias, const float* lower, SegView seg,
                      int max_len, int heads, int dim, int vdim, int vstride,
                      int f32, hipStream_t stream) {
  return f32 ? hgrn2_scan_t<float>(o, work, proj, state, f_bias, lower, seg,
                                   max_len, heads, dim, vdim, vstride, stream)
             : hgrn2_scan_t<bf16>(o, work, proj, state, f_bias, lower, seg,
                                  max_len, heads, dim, vdim, vstride, stream);
}

// one wave per (row, head); V columns per access, up to 4 accesses kept
template <typename T, int V>
__global__ __launch_bounds__(256) void head_norm_kernel(
    T* __restrict__ out, const float* __restrict__ o,
    const float* __restrict__ w, SegView seg, int heads, int vdim,
    float eps) {
  constexpr int KEEP = 16 / V;
  const int s = blockIdx.z, lane = threadIdx.x & 63;
  const long long i =
      ((long long)blockIdx.x * 256 + threadIdx.x) >> 6;  // (row, head)
  if (i >= (long long)seg.len[s] * heads) return;
  const size_t base = ((size_t)seg.start[s] * heads + i) * vdim;
  Pack<float, V> a[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (k * 64 + lane) * V;
    if (c >= vdim) break;
    a[k] = *reinterpret_cast<const Pack<float, V>*>(o + base + c);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += a[k].v[j] * a[k].v[j];
  }
  const float r = 1.f / sqrtf(wave_sum(ss) / vdim + eps);
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (k * 64 + lane) * V;
    if (c >= vdim) break;
    Pack<T, V> b;
#pragma unroll
    for (int j = 0; j < V; ++j) b.v[j] = from_f<T>(a[k].v[j] * r * w[c + j]);
    *reinterpret_cast<Pack<T, V>*>(out + base + c) = b;
  }
}

template <typename T>
static void head_norm_t(void* out, const float* o, const float* w,
                        SegView seg, int max_len, int heads, int vdim,
                        float eps, hipStream_t stream) {
  dim3 grid((unsigned)(((long long)max_len * heads + 3) / 4), 1, seg.n);
  if (vdim % 2 == 0)
    head_norm_kernel<T, 2><<<grid, 256, 0, stream>>>((T*)out, o, w, seg,
                                                     heads, vdim, eps);
  else
    head_norm_kernel<T, 1><<<grid, 256, 0, stream>>>((T*)out, o, w, seg,
                                                     heads, vdim, eps);
}

void launch_head_norm(void* out, const float* o, const float* w, SegView seg,
                      int max_len, int heads, int vdim, float eps, int f32,
                      hipStream_t stream) {
  if (f32)
    head_norm_t<float>(out, o, w, seg, max_len, heads, vdim, eps, stream);
  else
    head_norm_t<bf16>(out, o, w, seg, max_len, heads, vdim, eps, stream);
}

// ---------------------------------------------------------------------------
// q/k head norms + cache append.  q and k: a group of L lanes per (row,
// head), V channels per lane.  v: pages run along the keys, so a wave takes
// 64 consecutive rows by V columns.  rope [positions, rot / 2, 2], if given,
// rotates neighbouring channels (2i, 2i + 1) below rot after the norm.
// ---------------------------------------------------------------------------
template <typename T, int V, int L>
__global__ __launch_bounds__(256) void qk_norm_append_kernel(
    T* __restrict__ q_out, T* __restrict__ kpages,
    const T* __restrict__ proj, const float* __restrict__ q_w,
    const float* __restrict__ k_w, const int* __restrict__ row_slot,
    const int* __restrict__ row_pos, const int* __restrict__ table,
    int table_stride, int n, int heads, int kv_heads, int dim, long long ld,
    int dpad, float eps, const float* __restrict__ rope, int rot) {
  constexpr int PER = 256 / L;  // (row, head) pairs per block
  using P = Pack<T, V>;
  const int hk = heads + kv_heads;
  const long long i = (long long)blockIdx.x * PER + threadIdx.x / L;
  if (i >= (long long)n * hk) return;
  const int lane = threadIdx.x % L;
  // (fewer pairs than 2^31: the host checks)
  const unsigned r32 = (unsigned)i / (unsigned)hk;
  const size_t row = r32;
  const int hd = (int)((unsigned)i - r32 * hk);
  const bool is_q = hd < heads;
  const T* src = proj + row * (size_t)ld + (size_t)hd * dim;
  const float* w = is_q ? q_w : k_w;
  T* dst;
  int key = 0;
  if (is_q) {
    dst = q_out + (row * heads + hd) * (size_t)dpad;
  } else {
    const int pos = row_pos[row];
    const size_t page =
        table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
    key = pos & 63;
    dst = kpages + (page * kv_heads + (hd - heads)) * (size_t)(64 * dpad);
  }
  // dpad <= 256: at most 256 / (V * L) accesses per lane
  constexpr int KEEP = 256 / (V * L);
  P a[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int d = (k * L + lane) * V;
    if (d >= dim) break;
    a[k] = *reinterpret_cast<const P*>(src + d);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += to_f(a[k].v[j]) * to_f(a[k].v[j]);
  }
#pragma unroll
  for (int off = L / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
  const float r = 1.f / sqrtf(ss / dim + eps);
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int d = (k * L + lane) * V;
    if (d >= dpad) break;
    float f[V];
#pragma unroll
    for (int j = 0; j < V; ++j)
      f[j] = d < dim ? to_f(a[k].v[j]) * r * w[d + j] : 0.f;
    if (rope != nullptr) {
      const float* cs = rope + (size_t)row_pos[row] * rot;
      if constexpr (V == 1) {
        // the partner is the neighbouring lane (rot is even, and so is L)
        const float other = __shfl_xor(f[0], 1, 64);
        if (d < rot) {
          const float c = cs[d & ~1], si = cs[d | 1];
          f[0] = d & 1 ? f[0] * c + other * si : f[0] * c - other * si;
        }
      } else {
#pragma unroll
        for (int j = 0; j < V; j += 2)
          if (d + j < rot) {
            const float c = cs[d + j], si = cs[d + j + 1];
            const float u = f[j], v = f[j + 1];
            f[j] = u * c - v * si;
            f[j + 1] = v * c + u * si;
          }
      }
    }
    P b;
#pragma unroll
    for (int j = 0; j < V; ++j) b.v[j] = from_f<T>(f[j]);
    if (is_q) {
      *reinterpret_cast<P*>(dst + d) = b;
    } else {
      // runs of four channels stay together in a page
      constexpr int RUN = V < 4 ? V : 4;
#pragma unroll
      for (int j = 0; j < V; j += RUN)
        *reinterpret_cast<Pack<T, RUN>*>(
            dst + PageLayout::k(key, d + j, dpad)) =
            *reinterpret_cast<const Pack<T, RUN>*>(b.v + j);
    }
  }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void v_append_kernel(
    T* __restrict__ vpages, const T* __restrict__ values, long long ld,
    const int* __restrict__ row_slot, const int* __restrict__ row_pos,
    const int* __restrict__ table, int table_stride, int n, int heads,
    int vdim, int vpad) {
  const int chunks = heads * (vdim / V);
  const int ch = blockIdx.y * 4 + (threadIdx.x >> 6);
  const size_t row = (size_t)blockIdx.x * 64 + (threadIdx.x & 63);
  if (ch >= chunks || row >= n) return;
  const int g = ch / (vdim / V), c = (ch % (vdim / V)) * V;
  const Pack<T, V> a = *reinterpret_cast<const Pack<T, V>*>(
      values + row * (size_t)ld + (size_t)g * vdim + c);
  const int pos = row_pos[row];
  const size_t page =
      table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
  T* dst = vpages + (page * heads + g) * (size_t)(64 * vpad);
#pragma unroll
  for (int j = 0; j < V; ++j)
    dst[PageLayout::v(pos & 63, c + j, vpad)] = a.v[j];
}

template <typename T, int V, int L>
static void append_t(const QkAppendArgs& a, hipStream_t stream) {
  const int k_heads = a.kpages != nullptr ? a.k_heads : 0;
  const long long pairs = (long long)a.n * (a.heads + k_heads);
  const long long qk = (long long)(a.heads + k_heads) * a.dim;
  const long long ld = qk + (k_heads > 0 ? a.v_heads * a.vdim : 0);
  qk_norm_append_kernel<T, V, L>
      <<<(unsigned)((pairs + 256 / L - 1) / (256 / L)), 256, 0, stream>>>(
          (T*)a.q_out, (T*)a.kpages, (const T*)a.proj, a.q_w, a.k_w,
          a.row_slot, a.row_pos, a.table, a.table_stride, a.n, a.heads,
          k_heads, a.dim, ld, a.dpad, a.eps, a.rope, a.rot);
  if (k_heads == 0) return;
  const int chunks = a.v_heads * (a.vdim / V);
  v_append_kernel<T, V>
      <<<dim3((a.n + 63) / 64, (chunks + 3) / 4), 256, 0, stream>>>(
          (T*)a.vpages, (const T*)a.proj + qk, ld, a.row_slot, a.row_pos,
          a.table, a.table_stride, a.n, a.v_heads, a.vdim, a.vpad);
}

void launch_qk_norm_append(const QkAppendArgs& a, int f32,
                           hipStream_t stream) {
  if (f32) {
    if (a.dim % 4 == 0 && a.vdim % 4 == 0) append_t<float, 4, 16>(a, stream);
    else append_t<float, 1, 64>(a, stream);
  } else {
    if (a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dpad <= 64)
      append_t<bf16, 8, 8>(a, stream);
    else if (a.dim % 8 == 0 && a.vdim % 8 == 0)
      append_t<bf16, 8, 16>(a, stream);
    else append_t<bf16, 1, 64>(a, stream);
  }
}

// ---------------------------------------------------------------------------
// Norms over all query and all key channels of a row + cache append: one block
// per row.  VALUES: the row's values as well, a wave per head; for prompts the
// kernel below takes 64 rows of a head, so that it writes runs of keys.
// ---------------------------------------------------------------------------
template <typename T, int V, int NT, bool VALUES>
__global__ __launch_bounds__(NT) void row_norm_append_kernel(RowAppendArgs p) {
  __shared__ float red[NT / 64];
  using P = Pack<T, V>;
  const QkAppendArgs& a = p.qk;
  const size_t row = blockIdx.x;
  const int tid = threadIdx.x, nq = a.heads * a.dim, nk = a.k_heads * a.dim;
  const T* src = (const T*)a.proj + row * (size_t)p.ld;
  const int pos = a.row_pos[row];
  const size_t page =
      a.table[(size_t)a.row_slot[row] * a.table_stride + (pos >> 6)];
  float sq = 0.f, sk = 0.f;
  for (int i = tid * V; i < nq + nk; i += NT * V) {
    const P b = *reinterpret_cast<const P*>(src + i);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) s += to_f(b.v[j]) * to_f(b.v[j]);
    if (i < nq) sq += s;
    else sk += s;
  }
  const float heat = p.q_scale != nullptr ? p.q_scale[pos] : 1.f;
  const float rq = heat / sqrtf(block_sum<NT>(sq, red) / nq + a.eps);
  const float rk = 1.f / sqrtf(block_sum<NT>(sk, red) / nk + a.eps);
  const int per = a.dpad / V, total = (a.heads + a.k_heads) * per;
  for (int i = tid; i < total; i += NT) {
    const int h = i / per, d = (i - h * per) * V;
    const bool is_q = h < a.heads;
    const int c = h * a.dim + d;    // channel of the row, and of its weights
    P b{};
    if (d < a.dim) {
      b = *reinterpret_cast<const P*>(src + c);
      const float* w = is_q ? a.q_w + c : a.k_w + (c - nq);
      const float r = is_q ? rq : rk;
#pragma unroll
      for (int j = 0; j < V; ++j)
        b.v[j] = from_f<T>(to_f(b.v[j]) * r * w[j]);
    }
    if (is_q) {
      *reinterpret_cast<P*>((T*)a.q_out + (row * a.heads + h) * a.dpad + d) =
          b;
    } else {
      T* dst = (T*)a.kpages +
               (page * a.k_heads + (h - a.heads)) * (size_t)(64 * a.dpad);
      constexpr int RUN = V < 4 ? V : 4;
#pragma unroll
      for (int j = 0; j < V; j += RUN)
        *reinterpret_cast<Pack<T, RUN>*>(
            dst + PageLayout::k(pos & 63, d + j, a.dpad)) =
            *reinterpret_cast<const Pack<T, RUN>*>(b.v + j);
    }
  }
  if constexpr (VALUES) {
    const int lane = tid & 63;
    for (int g = tid >> 6; g < a.v_heads; g += NT / 64) {
      const T* v = src + nq + nk + g * a.vdim;
      T* dst = (T*)a.vpages + (page * a.v_heads + g) * (size_t)(64 * a.vpad);
      float f[4], s = 0.f;  // (vdim is at most 256)
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int c = k * 64 + lane;
        f[k] = c < a.vdim ? to_f(v[c]) : 0.f;
        s += f[k] * f[k];
      }
      float r = 1.f;
      if (p.unit_values) r = 1.f / sqrtf(wave_sum(s) / a.vdim + a.eps);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int c = k * 64 + lane;
        if (c < a.vdim)
          dst[PageLayout::v(pos & 63, c, a.vpad)] = from_f<T>(f[k] * r);
      }
    }
  }
}

// 64 rows of one value head per block, through LDS
template <typename T, int V>
__global__ __launch_bounds__(256) void unit_v_append_kernel(RowAppendArgs p) {
  extern __shared__ __attribute__((aligned(16))) char sm_raw[];
  const QkAppendArgs& a = p.qk;
  T* sm = reinterpret_cast<T*>(sm_raw);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int g = blockIdx.y, ld = a.vdim + 2;  // (an odd number of banks)
  const size_t row0 = (size_t)blockIdx.x * 64;
  const int rows = min(64, a.n - (int)row0);
  const T* src = (const T*)a.proj + (a.heads + a.k_heads) * a.dim + g * a.vdim;
  using P = Pack<T, V>;
  // four lanes a row
  const int r = tid >> 2, part = tid & 3;
  float s = 0.f;
  if (r < rows)
    for (int c = part * V; c < a.vdim; c += 4 * V) {
      const P b = *reinterpret_cast<const P*>(src + (row0 + r) * p.ld + c);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        s += to_f(b.v[j]) * to_f(b.v[j]);
        sm[r * ld + c + j] = b.v[j];
      }
    }
  s += __shfl_xor(s, 1, 64);
  s += __shfl_xor(s, 2, 64);
  __shared__ float inv[64];
  if (part == 0)
    inv[r] = p.unit_values ? 1.f / sqrtf(s / a.vdim + a.eps) : 1.f;
  __syncthreads();
  if (lane >= rows) return;
  const size_t row = row0 + lane;
  const int pos = a.row_pos[row];
  const size_t page =
      a.table[(size_t)a.row_slot[row] * a.table_stride + (pos >> 6)];
  T* dst = (T*)a.vpages + (page * a.v_heads + g) * (size_t)(64 * a.vpad);
  for (int c = wave; c < a.vdim; c += 4)
    dst[PageLayout::v(pos & 63, c, a.vpad)] =
        from_f<T>(to_f(sm[lane * ld + c]) * inv[lane]);
}

template <typename T, int V>
static int row_append_t(const RowAppendArgs& a, hipStream_t stream) {
  const QkAppendArgs& q = a.qk;
  if (q.n <= 64) {
    if ((q.heads + q.k_heads) * q.dim > 512 * V)
      row_norm_append_kernel<T, V, 1024, true><<<q.n, 1024, 0, stream>>>(a);
    else
      row_norm_append_kernel<T, V, 256, true><<<q.n, 256, 0, stream>>>(a);
    return 0;
  }
  row_norm_append_kernel<T, V, 256, false><<<q.n, 256, 0, stream>>>(a);
  const size_t smem = 64 * (q.vdim + 2) * sizeof(T);
  auto kernel = unit_v_append_kernel<T, V>;
  if (smem > 60000 &&
      hipFuncSetAttribute((const void*)kernel,
                          hipFuncAttributeMaxDynamicSharedMemorySize,
                          (int)smem) != hipSuccess)
    return -1;
  kernel<<<dim3((q.n + 63) / 64, q.v_heads), 256, smem, stream>>>(a);
  return 0;
}

int launch_row_norm_append(const RowAppendArgs& a, int f32,
                           hipStream_t stream) {
  if (f32)
    return a.vec ? row_append_t<float, 4>(a, stream)
                 : row_append_t<float, 1>(a, stream);
  return a.vec ? row_append_t<bf16, 8>(a, stream)
               : row_append_t<bf16, 1>(a, stream);
}

// Keys and values of some tokens as flat rows [k heads * dim | v heads *
// vdim], into the pages or out of them.
template <typename T, bool STORE>
__global__ __launch_bounds__(256) void kv_rows_kernel(
    T* __restrict__ rows, T* __restrict__ kpages, T* __restrict__ vpages,
    const int* __restrict__ row_slot, const int* __restrict__ row_pos,
    const int* __restrict__ table, int table_stride, int k_heads, int v_heads,
    int dim, int vdim, int dpad, int vpad) {
  const size_t row = blockIdx.x;
  const int cols = k_heads * dim + v_heads * vdim, pos = row_pos[row];
  const size_t page =
      table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
  for (int i = threadIdx.x; i < cols; i += 256) {
    T* at;
    if (i < k_heads * dim) {
      at = kpages + (page * k_heads + i / dim) * (size_t)(64 * dpad) +
           PageLayout::k(pos & 63, i % dim, dpad);
    } else {
      const int c = i - k_heads * dim;
      at = vpages + (page * v_heads + c / vdim) * (size_t)(64 * vpad) +
           PageLayout::v(pos & 63, c % vdim, vpad);
    }
    if (STORE) *at = rows[row * cols + i];
    else rows[row * cols + i] = *at;
  }
}

void launch_kv_rows(const QkAppendArgs& a, void* rows, int store, int f32,
                    hipStream_t stream) {
#define ROWS(T, ST)                                                         \
  kv_rows_kernel<T, ST><<<a.n, 256, 0, stream>>>(                           \
      (T*)rows, (T*)a.kpages, (T*)a.vpages, a.row_slot, a.row_pos, a.table, \
      a.table_stride, a.k_heads, a.v_heads, a.dim, a.vdim, a.dpad, a.vpad)
  if (f32) {
    if (store) ROWS(float, true);
    else ROWS(float, false);
  } else {
    if (store) ROWS(bf16, true);
    else ROWS(bf16, false);
  }
#undef ROWS
}

// ---------------------------------------------------------------------------
// decode bookkeeping (graph-replayable)
// ---------------------------------------------------------------------------
__global__ void advance_batch_kernel(const int* slots, const int* sampled,
                                     int* pos, int* tokens, int spare,
                                     int n) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n || slots[i] == spare) return;
  tokens[i] = sampled[i];
  pos[i] += 1;
}

void launch_advance_batch(const int* slots, const int* sampled, int* pos,
                          int* tokens, int spare, int n,
                          hipStream_t stream) {
  advance_batch_kernel<<<(n + 255) / 256, 256, 0, stream>>>(
      slots, sampled, pos, tokens, spare, n);
}
