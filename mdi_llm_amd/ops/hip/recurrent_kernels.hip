// Recurrent mixers over ragged batches (gfx950): the short convolution, the
// scan per channel with RG-LRU (block-diagonal gates) and minGRU, and the
// Mamba-2 rule of the matrix-state kernels.

#include "matrix_state.h"
#include "mfma_tile.h"

namespace {

constexpr int CONV_TILE = 16;  // tokens of a block, and the most taps

// ---------------------------------------------------------------------------
// Causal convolution: a thread has V channels of a tile of tokens and keeps
// the last K - 1 inputs in registers.  K = 0: any number of taps, inputs are
// read again.  The first tile's block alone reads the slot's inputs, and
// writes the new ones after that.
// ---------------------------------------------------------------------------
template <typename T, int V, int K>
__global__ __launch_bounds__(256) void causal_conv_kernel(ConvArgs p) {
  const int s = blockIdx.z, t0 = blockIdx.y * CONV_TILE;
  const int len = p.seg.len[s];
  const int c = (blockIdx.x * 256 + threadIdx.x) * V;
  if (t0 >= len || c >= p.c) return;
  const int taps = K ? K : p.taps, back = taps - 1;
  const int keep = max(1, back);  // rows of a slot
  const int pos0 = p.seg.pos0[s];
  const size_t row0 = p.seg.start[s];
  const T* x = (const T*)p.x + row0 * p.ld + c;
  T* state = (T*)p.state + (size_t)p.seg.slot[s] * keep * p.c + c;
  using PT = Pack<T, V>;
  using PF = Pack<float, V>;
  PF in_bias{};
  if (p.in_bias != nullptr)
    in_bias = *reinterpret_cast<const PF*>(p.in_bias + c);
  const PF bias = *reinterpret_cast<const PF*>(p.bias + c);
  // raw input of token t of the segment, -back <= t < len
  auto raw = [&](int t) {
    return *reinterpret_cast<const PT*>(
        t >= 0 ? x + (size_t)t * p.ld : state + (size_t)(back + t) * p.c);
  };
  auto input = [&](int t) {
    PF f{};
    if (pos0 + t >= 0) {  // zeros before the sequence's start
      const PT r = raw(t);
#pragma unroll
      for (int j = 0; j < V; ++j) f.v[j] = to_f(r.v[j]) + in_bias.v[j];
    }
    return f;
  };
  const int tn = min(CONV_TILE, len - t0);
  T* out = (T*)p.out + (row0 + t0) * p.c + c;
  auto put = [&](int t, PF y) {
    PT o;
#pragma unroll
    for (int j = 0; j < V; ++j)
      o.v[j] = from_f<T>(p.act ? y.v[j] * sigmoid(y.v[j]) : y.v[j]);
    *reinterpret_cast<PT*>(out + (size_t)t * p.c) = o;
  };
  if constexpr (K > 0) {
    PF w[K], win[K];
#pragma unroll
    for (int k = 0; k < K; ++k) {
      w[k] = *reinterpret_cast<const PF*>(p.w + (size_t)k * p.c + c);
      if (k < K - 1) win[k] = input(t0 - (K - 1) + k);
    }
    for (int t = 0; t < tn; ++t) {
      win[K - 1] = input(t0 + t);
      PF y = bias;
#pragma unroll
      for (int k = 0; k < K; ++k)
#pragma unroll
        for (int j = 0; j < V; ++j) y.v[j] += w[k].v[j] * win[k].v[j];
      put(t, y);
#pragma unroll
      for (int k = 0; k + 1 < K; ++k) win[k] = win[k + 1];
    }
  } else {
    for (int t = 0; t < tn; ++t) {
      PF y = bias;
      for (int k = 0; k < taps; ++k) {
        const PF f = input(t0 + t - back + k);
        const PF w = *reinterpret_cast<const PF*>(p.w + (size_t)k * p.c + c);
#pragma unroll
        for (int j = 0; j < V; ++j) y.v[j] += w.v[j] * f.v[j];
      }
      put(t, y);
    }
  }
  // the last inputs; rows move towards the front, so none is lost early
  if (t0 == 0)
    for (int k = 0; k < back; ++k)
      *reinterpret_cast<PT*>(state + (size_t)k * p.c) = raw(len - back + k);
}

template <typename T, int V>
void causal_conv_t(const ConvArgs& a, hipStream_t stream) {
  const dim3 grid((a.c + 256 * V - 1) / (256 * V),
                  (a.max_len + CONV_TILE - 1) / CONV_TILE, a.seg.n);
  switch (a.taps) {
    case 2: causal_conv_kernel<T, V, 2><<<grid, 256, 0, stream>>>(a); break;
    case 3: causal_conv_kernel<T, V, 3><<<grid, 256, 0, stream>>>(a); break;
    case 4: causal_conv_kernel<T, V, 4><<<grid, 256, 0, stream>>>(a); break;
    default: causal_conv_kernel<T, V, 0><<<grid, 256, 0, stream>>>(a);
  }
}

// ---------------------------------------------------------------------------
// RG-LRU
// ---------------------------------------------------------------------------
struct Decay {
  float a, x;  // S <- a S + x
};

// float stages take the library's functions; a bf16 stage the hardware's,
// which are good to about one unit in the last place of a float
template <typename T> struct Math {
  static DEVINL float exp(float x) {
    return __builtin_amdgcn_exp2f(1.4426950408889634f * x);
  }
  static DEVINL float inv(float x) { return __builtin_amdgcn_rcpf(x); }
  static DEVINL float sqrt(float x) { return __builtin_amdgcn_sqrtf(x); }
};
template <> struct Math<float> {
  static DEVINL float exp(float x) { return expf(x); }
  static DEVINL float inv(float x) { return 1.f / x; }
  static DEVINL float sqrt(float x) { return sqrtf(x); }
};

// a = exp(rate r), and u times the input gate and sqrt(1 - a^2), which is
// taken from the Taylor series of exp where a is close to 1
template <typename T>
DEVINL Decay rglru_decay(float zr, float zi, float rate, float u) {
  using M = Math<T>;
  const float log_a = rate * M::inv(1.f + M::exp(-zr));
  const float a = M::exp(log_a), y = 2.f * log_a;
  float e = fmaf(y, 1.f / 720, 1.f / 120);
  e = fmaf(y, e, 1.f / 24);
  e = fmaf(y, e, 1.f / 6);
  e = fmaf(y, e, 0.5f);
  e = fmaf(y, e, 1.f) * -y;
  const float rest = y > -0.3f ? e : 1.f - a * a;
  return {a, M::sqrt(rest) * M::inv(1.f + M::exp(-zi)) * u};
}

// z (1 + tanh(p(z))) / 2 is z / (1 + exp(-2 p(z)))
template <typename T>
DEVINL float gelu_tanh(float z) {
  using M = Math<T>;
  return z * M::inv(1.f + M::exp(-1.5957691216057308f *
                                 (z + 0.044715f * z * z * z)));
}

// Both gates of 64 rows x 32 channels per wave; a and x to work [2, n, width].
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void rglru_gates_kernel(RgLruArgs p) {
  using F = Frag<T>;
  constexpr int RT = 4, CT = 2;
  const int part = p.width / p.blocks, tiles = (part + CT * 16 - 1) / (CT * 16);
  const int lane = threadIdx.x & 63, c = lane & 15, quad = lane >> 4;
  const int unit =
      blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (unit >= tiles * p.blocks) return;
  const int b = unit / tiles, m0 = unit % tiles * CT * 16;
  const int r0 = blockIdx.y * RT * 16;
  const T* w[2][CT];
#pragma unroll
  for (int j = 0; j < CT; ++j) {
    w[0][j] = (const T*)p.gates +
              ((size_t)b * part + min(m0 + j * 16 + c, part - 1)) * part;
    w[1][j] = w[0][j] + (size_t)p.width * part;
  }
  const T* u[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t)
    u[t] = (const T*)p.u + (size_t)min(r0 + t * 16 + c, p.n - 1) * p.width +
           (size_t)b * part;
  f32x4 acc[2][CT][RT];
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int j = 0; j < CT; ++j)
#pragma unroll
      for (int t = 0; t < RT; ++t) acc[g][j][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  struct Operands {
    typename F::Row x[RT], w[2][CT];
  };
  auto load = [&](Operands& o, int at) {
#pragma unroll
    for (int t = 0; t < RT; ++t) o.x[t] = load_steps<T>(u[t], at, part, VEC);
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int j = 0; j < CT; ++j)
        o.w[g][j] = load_steps<T>(w[g][j], at, part, VEC);
  };
  auto dot = [&](const Operands& o) {
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int j = 0; j < CT; ++j)
#pragma unroll
        for (int t = 0; t < RT; ++t)
          acc[g][j][t] = F::dot(o.w[g][j], o.x[t], acc[g][j][t]);
  };
  const int steps = (part + 31) / 32;
  Operands o[2];
  load(o[0], quad * 8);
  for (int k = 0; k < steps; k += 2) {
    if (k + 1 < steps) load(o[1], (k + 1) * 32 + quad * 8);
    dot(o[0]);
    if (k + 2 < steps) load(o[0], (k + 2) * 32 + quad * 8);
    if (k + 1 < steps) dot(o[1]);
  }
#pragma unroll
  for (int j = 0; j < CT; ++j) {
    const int m = m0 + j * 16 + quad * 4;
    if (m >= part) continue;
    float br[4], bi[4], rate[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int ch = b * part + min(m + i, part - 1);
      br[i] = p.gate_bias[ch];
      bi[i] = p.gate_bias[p.width + ch];
      rate[i] = p.rate[ch];
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      const int row = r0 + t * 16 + c;
      if (row >= p.n) continue;
      const size_t base = (size_t)row * p.width + (size_t)b * part;
      f32x4 da, dx;
      const T* up = (const T*)p.u + base;
      Pack<T, 4> uu;
      if (VEC) {
        uu = *reinterpret_cast<const Pack<T, 4>*>(up + m);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) uu.v[i] = up[min(m + i, part - 1)];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const Decay d = rglru_decay<T>(acc[0][j][t][i] + br[i],
                                       acc[1][j][t][i] + bi[i], rate[i],
                                       to_f(uu.v[i]));
        da[i] = d.a;
        dx[i] = d.x;
      }
      float* oa = p.work + base + m;
      float* ox = oa + (size_t)p.n * p.width;
      if (VEC) {
        *reinterpret_cast<f32x4*>(oa) = da;
        *reinterpret_cast<f32x4*>(ox) = dx;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (m + i < part) {
            oa[i] = da[i];
            ox[i] = dx[i];
          }
      }
    }
  }
}

// A recurrence S <- a S + x over a segment, 16 channels per block: SUB threads
// share a channel and take TC tokens each of a tile, whose maps S -> A S + B are
// composed through LDS.  The next tile's operands are in flight meanwhile.
// Rule has TC, SUB, In (a token's operands), enter(c), load(row, c), map(in) and
// put(row, c, S, in).
template <typename Rule>
__global__ __launch_bounds__(Rule::SUB * 16) void channel_scan_kernel(
    Rule rule, float* __restrict__ states, SegView seg, int width) {
  constexpr int TC = Rule::TC, SUB = Rule::SUB, TILE = TC * SUB;
  __shared__ float ma[2][SUB][17], mx[2][SUB][17];
  const int s = blockIdx.y, len = seg.len[s];
  const int cl = threadIdx.x & 15, sub = threadIdx.x >> 4;
  // blocks of one XCD are neighbours: they share lines in its L2
  const int c = ((int)(blockIdx.x & 7) * (gridDim.x >> 3) +
                 (int)(blockIdx.x >> 3)) * 16 + cl;
  const bool live = c < width;
  const int cc = min(c, width - 1);
  const size_t row0 = seg.start[s];
  float* state = states + (size_t)seg.slot[s] * width + cc;
  rule.enter(cc);
  float S = seg.pos0[s] != 0 ? *state : 0.f;
  struct Tile {
    typename Rule::In in[TC];
  };
  auto load = [&](Tile& t, int t0) {
#pragma unroll
    for (int j = 0; j < TC; ++j)
      // tokens past the end repeat the last: their map is replaced below
      t.in[j] = rule.load(row0 + min(t0 + sub * TC + j, len - 1), cc);
  };
  auto run = [&](Tile& t, int t0, int buf) {
    float A = 1.f, B = 0.f;
    Decay d[TC];
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      d[j] = t0 + sub * TC + j < len ? rule.map(t.in[j]) : Decay{1.f, 0.f};
      A *= d[j].a;
      B = d[j].a * B + d[j].x;
    }
    ma[buf][sub][cl] = A;
    mx[buf][sub][cl] = B;
    __syncthreads();  // one per tile: the other half is written next
    float in = S;
#pragma unroll
    for (int k = 0; k < SUB; ++k) {
      if (k == sub) in = S;
      S = ma[buf][k][cl] * S + mx[buf][k][cl];
    }
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      in = d[j].a * in + d[j].x;
      const int tt = t0 + sub * TC + j;
      if (live && tt < len) rule.put(row0 + tt, cc, in, t.in[j]);
    }
  };
  Tile t[2];
  load(t[0], 0);
  for (int t0 = 0; t0 < len; t0 += 2 * TILE) {
    load(t[1], t0 + TILE);
    run(t[0], t0, 0);
    if (t0 + TILE >= len) break;
    load(t[0], t0 + 2 * TILE);
    run(t[1], t0 + TILE, 1);
  }
  if (live && sub == 0) *state = S;
}

template <typename Rule>
void channel_scan(const Rule& rule, float* state, SegView seg, int width,
                  hipStream_t stream) {
  channel_scan_kernel<Rule>
      <<<dim3((width + 127) / 128 * 8, seg.n), Rule::SUB * 16, 0, stream>>>(
          rule, state, seg, width);
}

template <typename T>
struct RgLruScan {
  static constexpr int TC = 8, SUB = 16;
  struct In {
    float a, x;
    T y;
  };
  T* out;
  const float* a;
  const float* x;
  const T* y;
  const float* bias;
  long long y_ld;
  int width;
  float y_bias;
  DEVINL void enter(int c) { y_bias = bias[c]; }
  DEVINL In load(size_t row, int c) const {
    const size_t at = row * width + c;
    return {a[at], x[at], y[row * y_ld + c]};
  }
  DEVINL Decay map(const In& i) const { return {i.a, i.x}; }
  DEVINL void put(size_t row, int c, float S, const In& i) const {
    out[row * width + c] = from_f<T>(S * gelu_tanh<T>(to_f(i.y) + y_bias));
  }
};

// One token per segment: gates, recurrence and the second branch in one
// launch; a block has 16 channels of up to 16 segments.
template <typename T, int NW>
__global__ __launch_bounds__(NW * 64) void rglru_step_kernel(RgLruArgs p,
                                                             bool vec) {
  __shared__ float red[NW][2][16][17];
  const int part = p.width / p.blocks, tiles = (part + 15) / 16;
  const int b = blockIdx.x / tiles, m0 = blockIdx.x % tiles * 16;
  const int s0 = blockIdx.y * 16, c = threadIdx.x & 15;
  const T* w0 = (const T*)p.gates +
                ((size_t)b * part + min(m0 + c, part - 1)) * part;
  const T* const w[2] = {w0, w0 + (size_t)p.width * part};
  const size_t mine = p.seg.start[min(s0 + c, p.seg.n - 1)];
  tile_product<T, NW, 2>(red, (const T*)p.u + mine * p.width +
                                  (size_t)b * part, w, part, vec);
  for (int i = threadIdx.x; i < 256; i += NW * 64) {
    const int r = i >> 4, m = m0 + (i & 15), s = s0 + r;
    if (s >= p.seg.n || m >= part) continue;
    const int ch = b * part + m;
    const size_t row = p.seg.start[s];
    const Decay d = rglru_decay<T>(
        tile_sum<NW, 2>(red, 0, r, i & 15) + p.gate_bias[ch],
        tile_sum<NW, 2>(red, 1, r, i & 15) + p.gate_bias[p.width + ch],
        p.rate[ch], to_f(((const T*)p.u)[row * p.width + ch]));
    float* state = p.state + (size_t)p.seg.slot[s] * p.width + ch;
    float S = p.seg.pos0[s] != 0 ? *state : 0.f;
    S = d.a * S + d.x;
    *state = S;
    ((T*)p.out)[row * p.width + ch] = from_f<T>(
        S * gelu_tanh<T>(to_f(((const T*)p.y)[row * p.y_ld + ch]) +
                      p.y_bias[ch]));
  }
}

template <typename T>
void rglru_step_t(const RgLruArgs& a, hipStream_t stream) {
  const int part = a.width / a.blocks;
  rglru_step_kernel<T, 4>
      <<<dim3((part + 15) / 16 * a.blocks, (a.seg.n + 15) / 16), 256, 0,
         stream>>>(a, part % (16 / sizeof(T)) == 0);
}

template <typename T>
void rglru_scan_t(const RgLruArgs& a, hipStream_t stream) {
  const int part = a.width / a.blocks;
  const int units = (part + 31) / 32 * a.blocks;
  const dim3 grid((units + 3) / 4, (a.n + 63) / 64);
  if (part % (16 / sizeof(T)) == 0)
    rglru_gates_kernel<T, true><<<grid, 256, 0, stream>>>(a);
  else
    rglru_gates_kernel<T, false><<<grid, 256, 0, stream>>>(a);
  channel_scan(RgLruScan<T>{(T*)a.out, a.work,
                            a.work + (size_t)a.n * a.width, (const T*)a.y,
                            a.y_bias, a.y_ld, a.width, 0.f},
               a.state, a.seg, a.width, stream);
}

// ---------------------------------------------------------------------------
// minGRU: the maps come from the projections alone
// ---------------------------------------------------------------------------
template <typename T>
struct MinGruScan {
  static constexpr int TC = 8, SUB = 32;
  using M = Math<T>;
  struct In {
    T z, u, g;
  };
  T* out;
  const T* proj;
  const float* bias;
  long long ld;
  int width;
  float bz, bu;
  static DEVINL float gate(float v) { return M::inv(1.f + M::exp(-v)); }
  DEVINL void enter(int c) {
    bz = bias[c];
    bu = bias[width + c];
  }
  DEVINL In load(size_t row, int c) const {
    const T* p = proj + row * ld + c;
    return {p[0], p[width], p[2 * width]};
  }
  DEVINL Decay map(const In& i) const {
    // z = 1 / (1 + e) and 1 - z = e / (1 + e), for any z
    const float e = M::exp(fminf(-(to_f(i.z) + bz), 80.f));
    const float z = M::inv(1.f + e), u = to_f(i.u) + bu;
    const float c = u >= 0.f ? u + 0.5f : gate(u);
    return {e * z, z * c};
  }
  DEVINL void put(size_t row, int c, float S, const In& i) const {
    const float g = to_f(i.g);
    out[row * width + c] = from_f<T>(S * g * gate(g));
  }
};

template <typename T>
MinGruScan<T> mingru_rule(const MinGruArgs& a) {
  return {(T*)a.out, (const T*)a.proj, a.bias, a.ld, a.width, 0.f, 0.f};
}

template <typename T>
__global__ __launch_bounds__(256) void mingru_step_kernel(MinGruScan<T> rule,
                                                          float* states,
                                                          SegView seg) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.y;
  if (c >= rule.width) return;
  const size_t row = seg.start[s];
  float* state = states + (size_t)seg.slot[s] * rule.width + c;
  rule.enter(c);
  const typename MinGruScan<T>::In in = rule.load(row, c);
  const float S = seg.pos0[s] != 0 ? *state : 0.f;
  const Decay d = rule.map(in);
  const float next = d.a * S + d.x;
  *state = next;
  rule.put(row, c, next, in);
}

template <typename T>
void mingru_step_t(const MinGruArgs& a, hipStream_t stream) {
  mingru_step_kernel<T><<<dim3((a.width + 255) / 256, a.seg.n), 256, 0,
                          stream>>>(mingru_rule<T>(a), a.state, a.seg);
}

// ---------------------------------------------------------------------------
// Mamba-2: one decay per head, keys dt * B, queries C.
// ---------------------------------------------------------------------------
template <typename T>
struct Mamba2Rule {
  static constexpr bool NORM = false, NORMALISER = false;
  float* o;
  const T* xbc;
  const T* dt;
  const float* dt_bias;
  const float* rate;
  long long dt_ld;
  int heads, groups, dim, vdim;
  DEVINL const T* at(size_t row) const {
    return xbc + row * (size_t)(heads * vdim + 2 * groups * dim);
  }
  DEVINL StepFactors factors(size_t row, int h, int d) const {
    const float t = softplus(to_f(dt[row * dt_ld + h]) + dt_bias[h]);
    const T* b = at(row) + heads * vdim + h / (heads / groups) * dim;
    return {to_f(b[groups * dim + d]), expf(rate[h] * t), t * to_f(b[d])};
  }
  DEVINL float value(size_t row, int h, int c) const {
    return to_f(at(row)[h * vdim + c]);
  }
  DEVINL void put(size_t row, int h, int c, float v) const {
    o[row * (size_t)(heads * vdim) + h * vdim + c] = v;
  }
};

// Factors of a 16-token chunk (matrix_state.h); decays are exponentials of
// differences of the running sum of log decays, none above 0.
template <typename T, int DP>
__global__ __launch_bounds__(256) void mamba2_factors_kernel(Mamba2Args p) {
  using W = ChunkWork<DP>;
  __shared__ float bs[16][DP + 1], cs[16][DP + 1], dts[16], cum[16];
  const int s = blockIdx.z, h = blockIdx.y, t0 = blockIdx.x * 16;
  const int tn = min(16, p.seg.len[s] - t0);
  if (tn <= 0) return;
  const int tid = threadIdx.x;
  const size_t row0 = (size_t)p.seg.start[s] + t0;
  float* w = p.work + (((size_t)p.seg.start[s] / 16 + s + blockIdx.x) *
                           p.heads + h) * W::SIZE;
  if (tid < 64) {
    const int t = tid & 15;
    float dt = 0.f;  // past the end: nothing decays or is written
    if (t < tn)
      dt = softplus(to_f(((const T*)p.dt)[(row0 + t) * p.dt_ld + h]) +
                    p.dt_bias[h]);
    float sum = p.rate[h] * dt;
#pragma unroll
    for (int off = 1; off < 16; off *= 2) {
      const float v = __shfl_up(sum, off, 16);
      if (t >= off) sum += v;
    }
    if (tid < 16) {
      dts[t] = dt;
      cum[t] = sum;
    }
  }
  const size_t ld = (size_t)p.heads * p.vdim + 2 * p.groups * p.dim;
  const T* bc = (const T*)p.xbc + row0 * ld + p.heads * p.vdim +
                h / (p.heads / p.groups) * p.dim;
  for (int i = tid; i < 16 * DP; i += 256) {
    const int t = i / DP, d = i % DP;
    const bool in = t < tn && d < p.dim;
    bs[t][d] = in ? to_f(bc[t * ld + d]) : 0.f;
    cs[t][d] = in ? to_f(bc[t * ld + p.groups * p.dim + d]) : 0.f;
  }
  __syncthreads();
  const float total = cum[15];
  for (int i = tid; i < 16 * DP; i += 256) {
    const int t = i / DP, d = i % DP;
    w[W::QR + i] = cs[t][d] * expf(cum[t]);
    const int ku = i >> 4, tu = i & 15;
    w[W::UK + i] = bs[tu][ku] * (dts[tu] * expf(total - cum[tu]));
  }
  for (int d = tid; d < DP; d += 256) w[W::DECAY + d] = expf(total);
  const int t = tid >> 4, sp = tid & 15;
  float acc = 0.f;
  if (sp <= t) {
#pragma unroll 8
    for (int d = 0; d < DP; ++d) acc += cs[t][d] * bs[sp][d];
    acc *= dts[sp] * expf(cum[t] - cum[sp]);
  }
  w[W::P + tid] = acc;
}

template <typename T, int TPW>
void mamba2_scan_sized(const Mamba2Args& a, hipStream_t stream) {
  mamba2_factors_kernel<T, 64 * TPW>
      <<<dim3((a.max_len + 15) / 16, a.heads, a.seg.n), 256, 0, stream>>>(a);
  matrix_chunks_kernel<T, TPW>
      <<<dim3(a.heads, (a.vdim + 15) / 16, a.seg.n), 256, 0, stream>>>(
          a.o, a.work, (const T*)a.xbc,
          (long long)a.heads * a.vdim + 2 * a.groups * a.dim, a.state, a.seg,
          a.heads, a.dim, a.vdim, a.vstride);
}

template <typename T>
int mamba2_scan_t(const Mamba2Args& a, hipStream_t stream) {
  switch (chunk_dpad(a.dim)) {
    case 64: mamba2_scan_sized<T, 1>(a, stream); return 0;
    case 128: mamba2_scan_sized<T, 2>(a, stream); return 0;
    case 256: mamba2_scan_sized<T, 4>(a, stream); return 0;
  }
  return -1;
}

template <typename T>
void mamba2_step_t(const Mamba2Args& a, hipStream_t stream) {
  matrix_step(Mamba2Rule<T>{a.o, (const T*)a.xbc, (const T*)a.dt, a.dt_bias,
                            a.rate, a.dt_ld, a.heads, a.groups, a.dim,
                            a.vdim},
              a.state, a.seg, a.heads, a.dim, a.vdim, a.vstride, 0.f, stream);
}

}  // namespace

void launch_causal_conv(const ConvArgs& a, int f32, hipStream_t stream) {
  if (f32) {
    if (a.vec) causal_conv_t<float, 4>(a, stream);
    else causal_conv_t<float, 1>(a, stream);
  } else {
    if (a.vec) causal_conv_t<bf16, 8>(a, stream);
    else causal_conv_t<bf16, 1>(a, stream);
  }
}

void launch_rglru_step(const RgLruArgs& a, int f32, hipStream_t stream) {
  if (f32) rglru_step_t<float>(a, stream);
  else rglru_step_t<bf16>(a, stream);
}

void launch_rglru_scan(const RgLruArgs& a, int f32, hipStream_t stream) {
  if (f32) rglru_scan_t<float>(a, stream);
  else rglru_scan_t<bf16>(a, stream);
}

void launch_mingru_step(const MinGruArgs& a, int f32, hipStream_t stream) {
  if (f32) mingru_step_t<float>(a, stream);
  else mingru_step_t<bf16>(a, stream);
}

void launch_mingru_scan(const MinGruArgs& a, int f32, hipStream_t stream) {
  if (f32)
    channel_scan(mingru_rule<float>(a), a.state, a.seg, a.width, stream);
  else
    channel_scan(mingru_rule<bf16>(a), a.state, a.seg, a.width, stream);
}

void launch_mamba2_step(const Mamba2Args& a, int f32, hipStream_t stream) {
  if (f32) mamba2_step_t<float>(a, stream);
  else mamba2_step_t<bf16>(a, stream);
}

int launch_mamba2_scan(const Mamba2Args& a, int f32, hipStream_t stream) {
  return f32 ? mamba2_scan_t<float>(a, stream) : mamba2_scan_t<bf16>(a, stream);
}
