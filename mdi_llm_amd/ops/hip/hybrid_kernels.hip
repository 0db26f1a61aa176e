// Row, gate, recurrence and cache-append kernels of the hybrid stacks
// (gfx950).  All of them take a flat batch of token rows; nothing here knows
// whether a row belongs to a prompt or to a decode step.

#include "hybrid_common.h"

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
      if (p.post_w != nullptr) {
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
// xIELU on a whole GEMM output (single rows have it in the GEMV epilogue)
// ---------------------------------------------------------------------------
template <typename T, int V>
__global__ __launch_bounds__(256) void xielu_kernel(T* __restrict__ z,
                                                    long long n, float p,
                                                    float q) {
  const long long stride = (long long)gridDim.x * 256 * V;
  for (long long i = ((long long)blockIdx.x * 256 + threadIdx.x) * V; i < n;
       i += stride) {
    Pack<T, V> a = *reinterpret_cast<Pack<T, V>*>(z + i);
#pragma unroll
    for (int j = 0; j < V; ++j) a.v[j] = from_f<T>(xielu(to_f(a.v[j]), p, q));
    *reinterpret_cast<Pack<T, V>*>(z + i) = a;
  }
}

template <typename T, int V>
static void xielu_t(void* z, long long n, float p, float q,
                    hipStream_t stream) {
  const long long blocks = (n + 256 * V - 1) / (256 * V);
  xielu_kernel<T, V><<<(int)(blocks < 8192 ? blocks : 8192), 256, 0, stream>>>(
      (T*)z, n, p, q);
}

void launch_xielu(void* z, long long n, float p, float q, int f32,
                  hipStream_t stream) {
  if (f32) {
    if (n % 4 == 0) xielu_t<float, 4>(z, n, p, q, stream);
    else xielu_t<float, 1>(z, n, p, q, stream);
  } else {
    if (n % 8 == 0) xielu_t<bf16, 8>(z, n, p, q, stream);
    else xielu_t<bf16, 1>(z, n, p, q, stream);
  }
}

// ---------------------------------------------------------------------------
// HGRN2, one token per segment.  One block per (head, segment): the whole
// [dim, vdim] state of the head passes through registers once (16-byte
// accesses along vdim), so the block holds all of the head's output and can
// norm it before it leaves.
// ---------------------------------------------------------------------------
template <typename T, int NT>
__global__ __launch_bounds__(NT) void hgrn2_step_kernel(
    T* __restrict__ out, const T* __restrict__ proj,
    float* __restrict__ state, const float* __restrict__ f_bias,
    const float* __restrict__ lower, const float* __restrict__ norm_w,
    SegView seg, int heads, int dim, int vdim, int vstride, float eps) {
  extern __shared__ float sm[];
  __shared__ float red[NT / 64];
  const int tid = threadIdx.x, h = blockIdx.x, s = blockIdx.y;
  const int nq = vstride / 4;                 // float4 columns
  const int lanes = nq < NT ? nq : NT;      // threads along the columns
  const int groups = NT / lanes;             // row groups
  float* qs = sm;                             // [dim]
  float* fs = qs + dim;                       // [dim]
  float* part = fs + dim;                     // [groups][vstride]
  const size_t row = seg.start[s];
  const T* pr = proj + row * (size_t)(heads * (2 * dim + vdim));
  for (int d = tid; d < dim; d += NT) {
    const int c = h * dim + d;
    const float qv = to_f(pr[c]);
    qs[d] = qv * sigmoid(qv);
    const float l = lower[c];
    fs[d] = l + (1.f - l) * sigmoid(to_f(pr[heads * dim + c]) + f_bias[c]);
  }
  __syncthreads();
  const T* vr = pr + 2 * heads * dim + h * vdim;
  float* S = state +
             ((size_t)seg.slot[s] * heads + h) * (size_t)dim * vstride;
  const bool fresh = seg.pos0[s] == 0;
  const int g = tid / lanes;
  if (g < groups) {
    for (int c4 = tid % lanes; c4 < nq; c4 += lanes) {
      float v[4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j)
        v[j] = c4 * 4 + j < vdim ? to_f(vr[c4 * 4 + j]) : 0.f;
#pragma unroll 8
      for (int d = g; d < dim; d += groups) {
        float4* p = reinterpret_cast<float4*>(S + (size_t)d * vstride) + c4;
        float4 a = fresh ? make_float4(0.f, 0.f, 0.f, 0.f) : *p;
        const float f = fs[d], w = 1.f - f, q = qs[d];
        a.x = f * a.x + w * v[0];
        a.y = f * a.y + w * v[1];
        a.z = f * a.z + w * v[2];
        a.w = f * a.w + w * v[3];
        *p = a;
        o[0] += q * a.x;
        o[1] += q * a.y;
        o[2] += q * a.z;
        o[3] += q * a.w;
      }
      *reinterpret_cast<float4*>(part + g * vstride + c4 * 4) =
          make_float4(o[0], o[1], o[2], o[3]);
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < vdim; c += NT) {
    float o = 0.f;
    for (int k = 0; k < groups; ++k) o += part[k * vstride + c];
    part[c] = o;  // only this thread reads column c
    ss += o * o;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int k = 0; k < NT / 64; ++k) ss += red[k];
  const float r = 1.f / sqrtf(ss / vdim + eps);
  T* o_row = out + row * (size_t)(heads * vdim) + h * vdim;
  for (int c = tid; c < vdim; c += NT)
    o_row[c] = from_f<T>(part[c] * r * norm_w[c]);
}

template <typename T, int NT>
static void hgrn2_step_t(void* out, const void* proj, float* state,
                         const float* f_bias, const float* lower,
                         const float* norm_w, SegView seg, int heads, int dim,
                         int vdim, int vstride, float eps,
                         hipStream_t stream) {
  const int nq = vstride / 4;
  const int lanes = nq < NT ? nq : NT;
  const size_t smem =
      (2 * (size_t)dim + (size_t)(NT / lanes) * vstride) * sizeof(float);
  hgrn2_step_kernel<T, NT><<<dim3(heads, seg.n), NT, smem, stream>>>(
      (T*)out, (const T*)proj, state, f_bias, lower, norm_w, seg, heads, dim,
      vdim, vstride, eps);
}

void launch_hgrn2_step(void* out, const void* proj, float* state,
                       const float* f_bias, const float* lower,
                       const float* norm_w, SegView seg, int heads, int dim,
                       int vdim, int vstride, float eps, int f32,
                       hipStream_t stream) {
  // few blocks with a large state each: more waves to keep loads in flight
  const bool wide = dim * vstride >= 8192 && heads * seg.n <= 512;
#define STEP(T, NT)                                                       \
  hgrn2_step_t<T, NT>(out, proj, state, f_bias, lower, norm_w, seg,       \
                      heads, dim, vdim, vstride, eps, stream)
  if (f32) {
    if (wide) STEP(float, 1024);
    else STEP(float, 256);
  } else {
    if (wide) STEP(bf16, 1024);
    else STEP(bf16, 256);
  }
#undef STEP
}

// ---------------------------------------------------------------------------
// HGRN2 over longer segments, in chunks of 16 tokens.  With S the state at
// the chunk's start, per channel
//     R_t = f_first .. f_t          (decay from the start to t)
//     U_s = f_(s+1) .. f_last       (decay from s to the end)
// the chunk is three small matrix products,
//     o_t = (q_t R_t)^T S + sum_(s<=t) P[t][s] v_s
//     S  <- (f_first .. f_last) S + sum_s (U_s (1 - f_s)) v_s^T
// with P[t][s] = sum_d q_t (1 - f_s) f_(s+1) .. f_t.  All decays are plain
// products of gates, so every factor is at most 1 and nothing is divided
// by; an underflow is a token that is forgotten.  Everything is float and
// the products run on the float MFMA.
//
// The first kernel makes the factors of every (chunk, head) in parallel;
// the second walks a segment's chunks with a [dim, 16] slice of the state
// per block, held as MFMA accumulators split over the block's four waves by
// rows.  An accumulator tile is at the same time the right operand of
// (q R)^T S once the contraction index is permuted to its layout.
//
// Workspace of one (chunk, head), DP = dim padded to 64, 128 or 256:
//   qr [16][DP] | uk [DP][16] | decay [DP] | P [16][16]
// Segment s has its chunks from start[s] / 16 + s on, which cannot overlap
// as long as the segments are in the order of their rows.
// ---------------------------------------------------------------------------
using f32x4 = __attribute__((__vector_size__(16))) float;

template <int DP>
struct ChunkWork {
  static constexpr int QR = 0, UK = 16 * DP, DECAY = 32 * DP,
                       P = 33 * DP, SIZE = 33 * DP + 256;
};

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

template <typename T, int TPW>
__global__ __launch_bounds__(256) void hgrn2_chunks_kernel(
    float* __restrict__ o, const float* __restrict__ work,
    const T* __restrict__ proj, float* __restrict__ state, SegView seg,
    int heads, int dim, int vdim, int vstride) {
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
  const size_t ld = (size_t)heads * (2 * dim + vdim);
  const float* w = work + ((row0 / 16 + s) * heads + h) * W::SIZE;
  const size_t wstep = (size_t)heads * W::SIZE;
  const T* vp = proj + row0 * ld + 2 * heads * dim + h * vdim +
                min(col, vdim - 1);
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

static int chunk_dpad(int dim) {
  return dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 0;
}

long long hgrn2_work_floats(int rows, int segments, int heads, int dim) {
  const long long chunks = rows / 16 + segments + 1;
  return chunks * heads * (33 * chunk_dpad(dim) + 256);
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
  hgrn2_chunks_kernel<T, TPW>
      <<<dim3(heads, (vdim + 15) / 16, seg.n), 256, 0, stream>>>(
          o, work, (const T*)proj, state, seg, heads, dim, vdim, vstride);
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
// 64 consecutive rows by V columns.
// ---------------------------------------------------------------------------
template <typename T, int V, int L>
__global__ __launch_bounds__(256) void qk_norm_append_kernel(
    T* __restrict__ q_out, T* __restrict__ kpages,
    const T* __restrict__ proj, const float* __restrict__ q_w,
    const float* __restrict__ k_w, const int* __restrict__ row_slot,
    const int* __restrict__ row_pos, const int* __restrict__ table,
    int table_stride, int n, int heads, int kv_heads, int dim, int vdim,
    int dpad, float eps) {
  constexpr int PER = 256 / L;  // (row, head) pairs per block
  using P = Pack<T, V>;
  const int hk = heads + kv_heads;
  const long long i = (long long)blockIdx.x * PER + threadIdx.x / L;
  if (i >= (long long)n * hk) return;
  const int lane = threadIdx.x % L;
  const size_t row = i / hk;
  const int hd = (int)(i - row * hk);
  const bool is_q = hd < heads;
  const T* src = proj + row * (size_t)(hk * dim + kv_heads * vdim) +
                 (size_t)hd * dim;
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
    P b;
#pragma unroll
    for (int j = 0; j < V; ++j)
      b.v[j] = from_f<T>(d < dim ? to_f(a[k].v[j]) * r * w[d + j] : 0.f);
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
    T* __restrict__ vpages, const T* __restrict__ proj,
    const int* __restrict__ row_slot, const int* __restrict__ row_pos,
    const int* __restrict__ table, int table_stride, int n, int heads,
    int kv_heads, int dim, int vdim, int vpad) {
  const int chunks = kv_heads * (vdim / V);
  const int ch = blockIdx.y * 4 + (threadIdx.x >> 6);
  const size_t row = (size_t)blockIdx.x * 64 + (threadIdx.x & 63);
  if (ch >= chunks || row >= n) return;
  const int g = ch / (vdim / V), c = (ch % (vdim / V)) * V;
  const size_t qk = (size_t)(heads + kv_heads) * dim;
  const Pack<T, V> a = *reinterpret_cast<const Pack<T, V>*>(
      proj + row * (qk + kv_heads * vdim) + qk + (size_t)g * vdim + c);
  const int pos = row_pos[row];
  const size_t page =
      table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
  T* dst = vpages + (page * kv_heads + g) * (size_t)(64 * vpad);
#pragma unroll
  for (int j = 0; j < V; ++j)
    dst[PageLayout::v(pos & 63, c + j, vpad)] = a.v[j];
}

template <typename T, int V, int L>
static void append_t(void* q_out, void* kpages, void* vpages,
                     const void* proj, const float* q_w, const float* k_w,
                     const int* row_slot, const int* row_pos,
                     const int* table, int table_stride, int n, int heads,
                     int kv_heads, int dim, int vdim, int dpad, int vpad,
                     float eps, hipStream_t stream) {
  const long long pairs = (long long)n * (heads + kv_heads);
  qk_norm_append_kernel<T, V, L>
      <<<(unsigned)((pairs + 256 / L - 1) / (256 / L)), 256, 0, stream>>>(
          (T*)q_out, (T*)kpages, (const T*)proj, q_w, k_w, row_slot, row_pos,
          table, table_stride, n, heads, kv_heads, dim, vdim, dpad, eps);
  const int chunks = kv_heads * (vdim / V);
  v_append_kernel<T, V>
      <<<dim3((n + 63) / 64, (chunks + 3) / 4), 256, 0, stream>>>(
          (T*)vpages, (const T*)proj, row_slot, row_pos, table, table_stride,
          n, heads, kv_heads, dim, vdim, vpad);
}

void launch_qk_norm_append(void* q_out, void* kpages, void* vpages,
                           const void* proj, const float* q_w,
                           const float* k_w, const int* row_slot,
                           const int* row_pos, const int* table,
                           int table_stride, int n, int heads, int kv_heads,
                           int dim, int vdim, int dpad, int vpad, float eps,
                           int f32, hipStream_t stream) {
#define APPEND(T, V, L)                                                     \
  append_t<T, V, L>(q_out, kpages, vpages, proj, q_w, k_w, row_slot,        \
                    row_pos, table, table_stride, n, heads, kv_heads, dim,  \
                    vdim, dpad, vpad, eps, stream)
  if (f32) {
    if (dim % 4 == 0 && vdim % 4 == 0) APPEND(float, 4, 16);
    else APPEND(float, 1, 64);
  } else {
    if (dim % 8 == 0 && vdim % 8 == 0) APPEND(bf16, 8, 16);
    else APPEND(bf16, 1, 64);
  }
#undef APPEND
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
