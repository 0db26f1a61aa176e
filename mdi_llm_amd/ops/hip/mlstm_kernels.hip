// mLSTM over ragged batches (gfx950): the rule of the matrix-state step, and
// for prompts the gates with their running maximum, the factors of the chunk
// walk, and the normalised, gated read-out.
//
// State and normaliser are kept relative to exp(m).  m is a scan of maps m ->
// max(F + m, I), which compose, so all gates of a prompt are known before its
// chunks; what a chunk multiplies by are then exponentials of numbers that
// are never above 0.

#include "matrix_state.h"
#include "mfma_tile.h"

namespace {

constexpr float NEG_INF = -__builtin_huge_valf();

struct Gates {
  float i, f;  // logarithms
};

DEVINL Gates log_gates(float zi, float zf, float cap) {
  const float f = cap * tanhf(zf / cap);
  return {cap * tanhf(zi / cap), fminf(f, 0.f) - log1pf(expf(-fabsf(f)))};
}

template <typename T>
struct MLstmRule {
  static constexpr bool NORM = true, NORMALISER = true;
  T* out;
  const T* proj;
  float* peak;
  const float* gate_bias;
  const float* norm_w;
  int heads, dim, vdim;
  float cap, q_scale;
  float keep, write, m;
  DEVINL const T* at(size_t row) const {
    return proj + row * (size_t)(2 * heads * (dim + vdim + 1));
  }
  DEVINL void enter(size_t row, int h, int slot, bool fresh) {
    const T* z = at(row) + 2 * heads * (dim + vdim);
    const Gates g = log_gates(to_f(z[h]) + gate_bias[h],
                              to_f(z[heads + h]) + gate_bias[heads + h], cap);
    const float before = fresh ? 0.f : peak[(size_t)slot * heads + h];
    m = fmaxf(g.f + before, g.i);
    keep = expf(g.f + before - m);
    write = expf(g.i - m);
  }
  DEVINL void leave(int h, int slot) const {
    peak[(size_t)slot * heads + h] = m;
  }
  DEVINL float size(float n) const {
    return fmaxf(fabsf(n), expf(-m)) + 1e-6f;
  }
  DEVINL StepFactors factors(size_t row, int h, int d) const {
    const T* p = at(row) + h * dim + d;
    return {to_f(p[0]) * q_scale, keep, to_f(p[heads * dim]) * write};
  }
  DEVINL float value(size_t row, int h, int c) const {
    return to_f(at(row)[2 * heads * dim + h * vdim + c]);
  }
  DEVINL void put(size_t row, int h, int c, float v) const {
    const float g = to_f(at(row)[heads * (2 * dim + vdim) + h * vdim + c]);
    out[row * (size_t)(heads * vdim) + h * vdim + c] =
        from_f<T>(v * norm_w[h * vdim + c] * sigmoid(g));
  }
};

template <typename T>
void step_t(const MLstmArgs& a, hipStream_t stream) {
  matrix_step(MLstmRule<T>{(T*)a.out, (const T*)a.proj, a.peak, a.gate_bias,
                           a.norm_w, a.heads, a.dim, a.vdim, a.cap, a.q_scale,
                           0.f, 0.f, 0.f},
              a.state, a.seg, a.heads, a.dim, a.vdim, a.vstride, a.eps,
              stream);
}

// Workspace of a scan: chunk factors and sums, the raw read-out; by head and
// row the log gates, m after each token, and the normaliser's read-out as
// n . q = from * (n at the chunk's start . q) + own; m before each segment.
struct ScanWork {
  float *chunks, *sums, *o, *i, *f, *m, *from, *own, *start;
};

ScanWork scan_work(const MLstmArgs& a) {
  const size_t cells = (size_t)a.n * a.heads;
  ScanWork w;
  w.chunks = a.work;
  w.sums = w.chunks + chunk_work_floats(a.n, a.seg.n, a.heads, a.dim);
  w.o = w.sums + chunk_sums_floats(a.n, a.seg.n, a.heads, a.dim);
  w.i = w.o + cells * a.vdim;
  w.f = w.i + cells;
  w.m = w.f + cells;
  w.from = w.m + cells;
  w.own = w.from + cells;
  w.start = w.own + cells;
  return w;
}

// One block per (head, segment), TC tokens a thread
template <typename T>
__global__ __launch_bounds__(256) void mlstm_gates_kernel(MLstmArgs p,
                                                          ScanWork w) {
  constexpr int TC = 4, TILE = 256 * TC;
  __shared__ float sf[2][4], si[2][4];
  const int h = blockIdx.x, s = blockIdx.y, len = p.seg.len[s];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t row0 = p.seg.start[s], at = (size_t)h * p.n + row0;
  const long long ld = 2LL * p.heads * (p.dim + p.vdim + 1);
  const T* z = (const T*)p.proj + row0 * ld + 2 * p.heads * (p.dim + p.vdim);
  const float bi = p.gate_bias[h], bf = p.gate_bias[p.heads + h];
  float* peak = p.peak + (size_t)p.seg.slot[s] * p.heads + h;
  float m0 = p.seg.pos0[s] == 0 ? 0.f : *peak;
  if (tid == 0) w.start[s * p.heads + h] = m0;
  for (int t0 = 0, buf = 0; t0 < len; t0 += TILE, buf ^= 1) {
    Gates g[TC];
    float F = 0.f, I = NEG_INF;
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      const int t = t0 + tid * TC + j;
      const T* r = z + min(t, len - 1) * ld;
      g[j] = log_gates(to_f(r[h]) + bi, to_f(r[p.heads + h]) + bf, p.cap);
      if (t >= len) g[j] = {NEG_INF, 0.f};  // m stays as it is
      F += g[j].f;
      I = fmaxf(g[j].f + I, g[j].i);
    }
    // the maps of all threads up to this one
#pragma unroll
    for (int off = 1; off < 64; off *= 2) {
      const float f = __shfl_up(F, off, 64), i = __shfl_up(I, off, 64);
      if (lane >= off) {
        I = fmaxf(F + i, I);
        F += f;
      }
    }
    if (lane == 63) {
      sf[buf][wave] = F;
      si[buf][wave] = I;
    }
    __syncthreads();  // one per tile: the other half is written next
    float m = m0;
    for (int k = 0; k < wave; ++k) m = fmaxf(sf[buf][k] + m, si[buf][k]);
    const float f = __shfl_up(F, 1, 64), i = __shfl_up(I, 1, 64);
    if (lane > 0) m = fmaxf(f + m, i);
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      m = fmaxf(g[j].f + m, g[j].i);
      const int t = t0 + tid * TC + j;
      if (t < len) {
        w.i[at + t] = g[j].i;
        w.f[at + t] = g[j].f;
        w.m[at + t] = m;
      }
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) m0 = fmaxf(sf[buf][k] + m0, si[buf][k]);
  }
  if (tid == 0) *peak = m0;
}

// Factors of a 16-token chunk (matrix_state.h); q . k on MFMA
template <typename T, int DP>
__global__ __launch_bounds__(256) void mlstm_factors_kernel(MLstmArgs p,
                                                            ScanWork sw,
                                                            bool vec) {
  using W = ChunkWork<DP>;
  using F = Frag<T>;
  __shared__ T ks[16][DP + 2];
  __shared__ float red[4][16][17];
  __shared__ float cum[16], li[16], lm[16], from[16], to[16];
  const int s = blockIdx.z, h = blockIdx.y, t0 = blockIdx.x * 16;
  const int tn = min(16, p.seg.len[s] - t0);
  if (tn <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t row0 = (size_t)p.seg.start[s] + t0, at = (size_t)h * p.n + row0;
  const size_t chunk =
      ((size_t)p.seg.start[s] / 16 + s + blockIdx.x) * p.heads + h;
  float* w = sw.chunks + chunk * W::SIZE;
  const long long ld = 2LL * p.heads * (p.dim + p.vdim + 1);
  const T* q = (const T*)p.proj + row0 * ld + h * p.dim;
  const T* k = q + p.heads * p.dim;
  const float m0 = t0 == 0 ? sw.start[s * p.heads + h] : sw.m[at - 1];
  {
    // every wave a part of the channels; rows past the end repeat the last
    const int c = lane & 15, quad = lane >> 4;
    const T* qr = q + min(c, tn - 1) * ld;
    const T* kr = k + min(c, tn - 1) * ld;
    f32x4 acc{0.f, 0.f, 0.f, 0.f};
    for (int d = wave * 32; d < p.dim; d += 128)
      acc = F::dot(load_steps<T>(kr, d + quad * 8, p.dim, vec),
                   load_steps<T>(qr, d + quad * 8, p.dim, vec), acc);
#pragma unroll
    for (int i = 0; i < 4; ++i) red[wave][c][quad * 4 + i] = acc[i];
  }
  if (tid < 16) {
    const int t = tid;
    float sum = t < tn ? sw.f[at + t] : 0.f;
    const float i = t < tn ? sw.i[at + t] : NEG_INF;
    const float m = sw.m[at + min(t, tn - 1)];
#pragma unroll
    for (int off = 1; off < 16; off *= 2) {
      const float v = __shfl_up(sum, off, 16);
      if (t >= off) sum += v;
    }
    cum[t] = sum;
    li[t] = i;
    lm[t] = m;
    const float total = __shfl(sum, 15, 16), end = __shfl(m, 15, 16);
    from[t] = t < tn ? expf(sum + m0 - m) * p.q_scale : 0.f;
    if (t < tn) sw.from[at + t] = from[t];
    to[t] = expf(i + (total - sum) - end);
  }
  for (int i = tid; i < 16 * DP; i += 256) {
    const int t = i / DP, d = i % DP;
    ks[t][d] = t < tn && d < p.dim ? k[t * ld + d] : from_f<T>(0.f);
  }
  __syncthreads();
  const float decay = expf(cum[15] + m0 - lm[15]);
  for (int i = tid; i < 16 * DP; i += 256) {
    const int t = i / DP, d = i % DP;
    w[W::QR + i] =
        t < tn && d < p.dim ? to_f(q[t * ld + d]) * from[t] : 0.f;
    w[W::UK + i] = to_f(ks[i & 15][i >> 4]) * to[i & 15];
  }
  for (int d = tid; d < DP; d += 256) {
    w[W::DECAY + d] = decay;
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) sum += to_f(ks[t][d]) * to[t];
    sw.sums[chunk * DP + d] = sum;
  }
  const int t = tid >> 4, sp = tid & 15;
  float dot = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) dot += red[j][t][sp];
  const float weight =
      sp <= t && t < tn ? dot * p.q_scale *
                              expf(li[sp] + (cum[t] - cum[sp]) - lm[t])
                        : 0.f;
  w[W::P + tid] = weight;
  const float own = row16_sum(weight);
  if (sp == 0 && t < tn) sw.own[at + t] = own;
}

// Normalised, of unit size, gated: a wave has ROWS neighbouring rows of a head
// (all of one chunk), V columns per access.
template <typename T, int TPW, int V, int KEEP, int ROWS>
__global__ __launch_bounds__(256) void mlstm_out_kernel(MLstmArgs p,
                                                        ScanWork w) {
  const int s = blockIdx.y, lane = threadIdx.x & 63, len = p.seg.len[s];
  const unsigned unit = blockIdx.x * 4u + (threadIdx.x >> 6);
  const int h = unit % p.heads, t0 = unit / p.heads * ROWS;
  if (t0 >= len) return;
  const size_t row0 = p.seg.start[s];
  const int col0 = h * p.vdim, inner = p.heads * p.vdim;
  const size_t ld = 2 * p.heads * (size_t)(p.dim + p.vdim + 1);
  const float* sum =
      w.sums + ((row0 / 16 + s + t0 / 16) * p.heads + h) * (64 * TPW);
  // all loads ahead of the first use
  Pack<float, V> a[ROWS][KEEP];
  Pack<T, V> b[ROWS][KEEP];
  T q[ROWS][TPW];
  float u[TPW], from[ROWS], own[ROWS], m[ROWS];
#pragma unroll
  for (int k = 0; k < TPW; ++k) u[k] = sum[k * 64 + lane];  // 0 past dim
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    // rows past the end repeat the last one; they are not stored
    const size_t row = row0 + min(t0 + r, len - 1);
    const size_t at = (size_t)h * p.n + row;
    const T* proj = (const T*)p.proj + row * ld;
    const float* o = w.o + row * inner + col0;
    const T* g = proj + 2 * p.heads * p.dim + inner + col0;
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = (k * 64 + lane) * V;
      if (c >= p.vdim) break;
      a[r][k] = *reinterpret_cast<const Pack<float, V>*>(o + c);
      b[r][k] = *reinterpret_cast<const Pack<T, V>*>(g + c);
    }
#pragma unroll
    for (int k = 0; k < TPW; ++k)
      q[r][k] = proj[h * p.dim + min(k * 64 + lane, p.dim - 1)];
    from[r] = w.from[at];
    own[r] = w.own[at];
    m[r] = w.m[at];
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    float ss = 0.f, dot = 0.f;
#pragma unroll
    for (int k = 0; k < TPW; ++k) dot += to_f(q[r][k]) * u[k];
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      if ((k * 64 + lane) * V >= p.vdim) break;
#pragma unroll
      for (int j = 0; j < V; ++j) ss += a[r][k].v[j] * a[r][k].v[j];
    }
    const float n = from[r] * wave_sum(dot) + own[r];
    const float inv = 1.f / (fmaxf(fabsf(n), expf(-m[r])) + 1e-6f);
    const float f = inv / sqrtf(wave_sum(ss) * inv * inv / p.vdim + p.eps);
    if (t0 + r >= len) break;
    T* out = (T*)p.out + (row0 + t0 + r) * inner + col0;
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = (k * 64 + lane) * V;
      if (c >= p.vdim) break;
      Pack<T, V> y;
#pragma unroll
      for (int j = 0; j < V; ++j)
        y.v[j] = from_f<T>(a[r][k].v[j] * f * p.norm_w[col0 + c + j] *
                           sigmoid(to_f(b[r][k].v[j])));
      *reinterpret_cast<Pack<T, V>*>(out + c) = y;
    }
  }
}

template <typename T, int TPW, int V, int KEEP, int ROWS>
void out_sized(const MLstmArgs& a, const ScanWork& w, hipStream_t stream) {
  const long long units =
      (long long)((a.max_len + ROWS - 1) / ROWS) * a.heads;
  mlstm_out_kernel<T, TPW, V, KEEP, ROWS>
      <<<dim3((unsigned)((units + 3) / 4), a.seg.n), 256, 0, stream>>>(a, w);
}

template <typename T, int TPW>
void scan_sized(const MLstmArgs& a, hipStream_t stream) {
  const ScanWork w = scan_work(a);
  const long long ld = 2LL * a.heads * (a.dim + a.vdim + 1);
  const int n = 16 / sizeof(T);
  mlstm_gates_kernel<T>
      <<<dim3(a.heads, a.seg.n), 256, 0, stream>>>(a, w);
  mlstm_factors_kernel<T, 64 * TPW>
      <<<dim3((a.max_len + 15) / 16, a.heads, a.seg.n), 256, 0, stream>>>(
          a, w, a.dim % n == 0 && ld % n == 0);
  matrix_chunks_kernel<T, TPW, true>
      <<<dim3(a.heads, (a.vdim + 15) / 16 + 1, a.seg.n), 256, 0, stream>>>(
          w.o, w.chunks, (const T*)a.proj + 2 * a.heads * a.dim, ld, a.state,
          a.seg, a.heads, a.dim, a.vdim, a.vstride, w.sums);
  if (a.vdim % 2 != 0) {
    if (a.vdim <= 64) out_sized<T, TPW, 1, 1, 4>(a, w, stream);
    else out_sized<T, TPW, 1, 16, 1>(a, w, stream);
  } else {
    if (a.vdim <= 128) out_sized<T, TPW, 2, 1, 4>(a, w, stream);
    else if (a.vdim <= 256) out_sized<T, TPW, 2, 2, 4>(a, w, stream);
    else out_sized<T, TPW, 2, 8, 1>(a, w, stream);
  }
}

template <typename T>
int scan_t(const MLstmArgs& a, hipStream_t stream) {
  switch (chunk_dpad(a.dim)) {
    case 64: scan_sized<T, 1>(a, stream); return 0;
    case 128: scan_sized<T, 2>(a, stream); return 0;
    case 256: scan_sized<T, 4>(a, stream); return 0;
  }
  return -1;
}

}  // namespace

void launch_mlstm_step(const MLstmArgs& a, int f32, hipStream_t stream) {
  if (f32) step_t<float>(a, stream);
  else step_t<bf16>(a, stream);
}

long long mlstm_work_floats(int rows, int segments, int heads, int dim,
                            int vdim) {
  return chunk_work_floats(rows, segments, heads, dim) +
         chunk_sums_floats(rows, segments, heads, dim) +
         (long long)rows * heads * (vdim + 5) + (long long)segments * heads;
}

int launch_mlstm_scan(const MLstmArgs& a, int f32, hipStream_t stream) {
  return f32 ? scan_t<float>(a, stream) : scan_t<bf16>(a, stream);
}
