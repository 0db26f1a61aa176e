// Row, gate, recurrence and cache-append kernels of the hybrid stacks
// (gfx950).  All of them take a flat batch of token rows; nothing here knows
// whether a row belongs to a prompt or to a decode step.

#include "hybrid_common.h"

// ---------------------------------------------------------------------------
// Residual + norms.  One 256-thread block per row; every thread only ever
// touches its own elements of the row, so x can be re-read from cache
// between the two reductions without a fence.
// ---------------------------------------------------------------------------
DEVINL float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  v = red[0] + red[1] + red[2] + red[3];
  __syncthreads();
  return v;
}

template <typename T, int V>
__global__ __launch_bounds__(256) void residual_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const float* __restrict__ post_w, T* __restrict__ xn,
    const float* __restrict__ next_w, const int* __restrict__ tokens,
    const T* __restrict__ table, float scale, float offset, float eps,
    int e) {
  __shared__ float red[4];
  const size_t row = blockIdx.x;
  x += row * e;
  float ss = 0.f;
  using PT = Pack<T, V>;
  using PF = Pack<float, V>;
  if (tokens != nullptr) {
    const T* t = table + (size_t)tokens[row] * e;
    for (int i = threadIdx.x * V; i < e; i += 256 * V) {
      PT a = *reinterpret_cast<const PT*>(t + i);
      PF o;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        o.v[j] = to_f(a.v[j]) * scale;
        ss += o.v[j] * o.v[j];
      }
      *reinterpret_cast<PF*>(x + i) = o;
    }
  } else if (y != nullptr) {
    y += row * e;
    float r = 1.f;
    if (post_w != nullptr) {
      float s = 0.f;
      for (int i = threadIdx.x * V; i < e; i += 256 * V) {
        PT a = *reinterpret_cast<const PT*>(y + i);
#pragma unroll
        for (int j = 0; j < V; ++j) s += to_f(a.v[j]) * to_f(a.v[j]);
      }
      r = 1.f / sqrtf(block_sum(s, red) / e + eps);
    }
    for (int i = threadIdx.x * V; i < e; i += 256 * V) {
      PT a = *reinterpret_cast<const PT*>(y + i);
      PF o = *reinterpret_cast<const PF*>(x + i);
      if (post_w != nullptr) {
        PF w = *reinterpret_cast<const PF*>(post_w + i);
#pragma unroll
        for (int j = 0; j < V; ++j)
          o.v[j] += to_f(a.v[j]) * r * (offset + w.v[j]);
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) o.v[j] += to_f(a.v[j]);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) ss += o.v[j] * o.v[j];
      *reinterpret_cast<PF*>(x + i) = o;
    }
  } else {
    for (int i = threadIdx.x * V; i < e; i += 256 * V) {
      PF o = *reinterpret_cast<const PF*>(x + i);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += o.v[j] * o.v[j];
    }
  }
  if (next_w == nullptr) return;
  const float r = 1.f / sqrtf(block_sum(ss, red) / e + eps);
  xn += row * e;
  for (int i = threadIdx.x * V; i < e; i += 256 * V) {
    PF a = *reinterpret_cast<const PF*>(x + i);
    PF w = *reinterpret_cast<const PF*>(next_w + i);
    PT o;
#pragma unroll
    for (int j = 0; j < V; ++j)
      o.v[j] = from_f<T>(a.v[j] * r * (offset + w.v[j]));
    *reinterpret_cast<PT*>(xn + i) = o;
  }
}

template <typename T>
static void residual_norm_t(float* x, const void* y, const float* post_w,
                            void* xn, const float* next_w, const int* tokens,
                            const void* table, float scale, float offset,
                            float eps, int n, int e, hipStream_t stream) {
  if (e % 4 == 0)
    residual_norm_kernel<T, 4><<<n, 256, 0, stream>>>(
        x, (const T*)y, post_w, (T*)xn, next_w, tokens, (const T*)table,
        scale, offset, eps, e);
  else
    residual_norm_kernel<T, 1><<<n, 256, 0, stream>>>(
        x, (const T*)y, post_w, (T*)xn, next_w, tokens, (const T*)table,
        scale, offset, eps, e);
}

void launch_residual_norm(float* x, const void* y, const float* post_w,
                          void* xn, const float* next_w, const int* tokens,
                          const void* table, float scale, float offset,
                          float eps, int n, int e, int f32,
                          hipStream_t stream) {
  if (f32)
    residual_norm_t<float>(x, y, post_w, xn, next_w, tokens, table, scale,
                           offset, eps, n, e, stream);
  else
    residual_norm_t<bf16>(x, y, post_w, xn, next_w, tokens, table, scale,
                          offset, eps, n, e, stream);
}

// ---------------------------------------------------------------------------
// xIELU on a whole GEMM output (single rows have it in the GEMV epilogue)
// ---------------------------------------------------------------------------
DEVINL float xielu(float z, float p, float q) {
  return 0.5f * z + (z > 0.f ? p * z * z : (0.5f + q) * (expm1f(z) - z));
}

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
template <typename T>
__global__ __launch_bounds__(256) void hgrn2_step_kernel(
    T* __restrict__ out, const T* __restrict__ proj,
    float* __restrict__ state, const float* __restrict__ f_bias,
    const float* __restrict__ lower, const float* __restrict__ norm_w,
    SegView seg, int heads, int dim, int vdim, int vstride, float eps) {
  extern __shared__ float sm[];
  __shared__ float red[4];
  const int tid = threadIdx.x, h = blockIdx.x, s = blockIdx.y;
  const int nq = vstride / 4;                 // float4 columns
  const int lanes = nq < 256 ? nq : 256;      // threads along the columns
  const int groups = 256 / lanes;             // row groups
  float* qs = sm;                             // [dim]
  float* fs = qs + dim;                       // [dim]
  float* part = fs + dim;                     // [groups][vstride]
  const size_t row = seg.start[s];
  const T* pr = proj + row * (size_t)(heads * (2 * dim + vdim));
  for (int d = tid; d < dim; d += 256) {
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
  for (int c = tid; c < vdim; c += 256) {
    float o = 0.f;
    for (int k = 0; k < groups; ++k) o += part[k * vstride + c];
    part[c] = o;  // only this thread reads column c
    ss += o * o;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float r =
      1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / vdim + eps);
  T* o_row = out + row * (size_t)(heads * vdim) + h * vdim;
  for (int c = tid; c < vdim; c += 256)
    o_row[c] = from_f<T>(part[c] * r * norm_w[c]);
}

void launch_hgrn2_step(void* out, const void* proj, float* state,
                       const float* f_bias, const float* lower,
                       const float* norm_w, SegView seg, int heads, int dim,
                       int vdim, int vstride, float eps, int f32,
                       hipStream_t stream) {
  const int nq = vstride / 4;
  const int lanes = nq < 256 ? nq : 256;
  const size_t smem =
      (2 * (size_t)dim + (size_t)(256 / lanes) * vstride) * sizeof(float);
  dim3 grid(heads, seg.n);
  if (f32)
    hgrn2_step_kernel<float><<<grid, 256, smem, stream>>>(
        (float*)out, (const float*)proj, state, f_bias, lower, norm_w, seg,
        heads, dim, vdim, vstride, eps);
  else
    hgrn2_step_kernel<bf16><<<grid, 256, smem, stream>>>(
        (bf16*)out, (const bf16*)proj, state, f_bias, lower, norm_w, seg,
        heads, dim, vdim, vstride, eps);
}

// ---------------------------------------------------------------------------
// HGRN2 over longer segments.  The columns of the state never mix, so a
// block keeps a [dim, 16] slice of one head in registers for the whole
// segment: 16 lanes of a DPP row share a column, R rows each.  Tokens are
// staged in LDS (gates computed once per block) TB at a time.
// ---------------------------------------------------------------------------
template <typename T, int R>
__global__ __launch_bounds__(256) void hgrn2_scan_kernel(
    float* __restrict__ o, const T* __restrict__ proj,
    float* __restrict__ state, const float* __restrict__ f_bias,
    const float* __restrict__ lower, SegView seg, int heads, int dim,
    int vdim, int vstride) {
  constexpr int DP = 16 * R, TB = 16;
  __shared__ __attribute__((aligned(16))) float fs[TB][DP];
  __shared__ __attribute__((aligned(16))) float qs[TB][DP];
  __shared__ float vs[TB][16], os[TB][17];
  const int tid = threadIdx.x, h = blockIdx.y, s = blockIdx.z;
  const int c0 = blockIdx.x * 16;
  const int rl = tid & 15, cl = tid >> 4, col = c0 + cl;
  const int len = seg.len[s];
  const size_t row0 = seg.start[s];
  const int ld = heads * (2 * dim + vdim);
  float* S = state +
             ((size_t)seg.slot[s] * heads + h) * (size_t)dim * vstride;
  const bool live = col < vstride;
  float st[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = rl * R + r;
    st[r] = (live && d < dim && seg.pos0[s] != 0)
                ? S[(size_t)d * vstride + col] : 0.f;
  }
  for (int t0 = 0; t0 < len; t0 += TB) {
    const int tn = min(TB, len - t0);
    for (int i = tid; i < TB * DP; i += 256) {
      const int t = i / DP, d = i % DP;
      float f = 0.f, q = 0.f;
      if (t < tn && d < dim) {
        const T* pr = proj + (row0 + t0 + t) * (size_t)ld;
        const int c = h * dim + d;
        const float qv = to_f(pr[c]), l = lower[c];
        q = qv * sigmoid(qv);
        f = l + (1.f - l) *
                    sigmoid(to_f(pr[heads * dim + c]) + f_bias[c]);
      }
      fs[t][d] = f;
      qs[t][d] = q;
    }
    {
      const int t = tid >> 4, c = c0 + (tid & 15);
      float v = 0.f;
      if (t < tn && c < vdim)
        v = to_f(proj[(row0 + t0 + t) * (size_t)ld + 2 * heads * dim +
                      h * vdim + c]);
      vs[t][tid & 15] = v;
    }
    __syncthreads();
    for (int t = 0; t < tn; ++t) {
      const float v = vs[t][cl];
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float f = fs[t][rl * R + r];
        // rows past dim hold f = q = 0: their state stays out of the sum
        st[r] = f * st[r] + (1.f - f) * v;
        acc += qs[t][rl * R + r] * st[r];
      }
      acc = row16_sum(acc);
      if (rl == 0) os[t][cl] = acc;
    }
    __syncthreads();
    {
      const int t = tid >> 4, c = c0 + (tid & 15);
      if (t < tn && c < vdim)
        o[(row0 + t0 + t) * (size_t)(heads * vdim) + h * vdim + c] =
            os[t][tid & 15];
    }
  }
  if (live) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int d = rl * R + r;
      if (d < dim) S[(size_t)d * vstride + col] = st[r];
    }
  }
}

template <typename T>
static int hgrn2_scan_t(float* o, const void* proj, float* state,
                        const float* f_bias, const float* lower, SegView seg,
                        int heads, int dim, int vdim, int vstride,
                        hipStream_t stream) {
  dim3 grid((vdim + 15) / 16, heads, seg.n);
#define SCAN(R)                                                          \
  hgrn2_scan_kernel<T, R><<<grid, 256, 0, stream>>>(                     \
      o, (const T*)proj, state, f_bias, lower, seg, heads, dim, vdim,    \
      vstride)
  if (dim <= 16) SCAN(1);
  else if (dim <= 32) SCAN(2);
  else if (dim <= 64) SCAN(4);
  else if (dim <= 128) SCAN(8);
  else if (dim <= 256) SCAN(16);
  else return -1;
#undef SCAN
  return 0;
}

int launch_hgrn2_scan(float* o, const void* proj, float* state,
                      const float* f_bias, const float* lower, SegView seg,
                      int heads, int dim, int vdim, int vstride, int f32,
                      hipStream_t stream) {
  return f32 ? hgrn2_scan_t<float>(o, proj, state, f_bias, lower, seg, heads,
                                   dim, vdim, vstride, stream)
             : hgrn2_scan_t<bf16>(o, proj, state, f_bias, lower, seg, heads,
                                  dim, vdim, vstride, stream);
}

template <typename T>
__global__ __launch_bounds__(256) void head_norm_kernel(
    T* __restrict__ out, const float* __restrict__ o,
    const float* __restrict__ w, SegView seg, int heads, int vdim,
    float eps) {
  const int s = blockIdx.z, t = blockIdx.x;
  if (t >= seg.len[s]) return;
  const int lane = threadIdx.x & 63;
  for (int h = blockIdx.y * 4 + (threadIdx.x >> 6); h < heads;
       h += gridDim.y * 4) {
    const size_t base =
        ((size_t)seg.start[s] + t) * heads * vdim + (size_t)h * vdim;
    float ss = 0.f;
    for (int c = lane; c < vdim; c += 64) ss += o[base + c] * o[base + c];
    const float r = 1.f / sqrtf(wave_sum(ss) / vdim + eps);
    for (int c = lane; c < vdim; c += 64)
      out[base + c] = from_f<T>(o[base + c] * r * w[c]);
  }
}

void launch_head_norm(void* out, const float* o, const float* w, SegView seg,
                      int max_len, int heads, int vdim, float eps, int f32,
                      hipStream_t stream) {
  dim3 grid(max_len, (heads + 3) / 4, seg.n);
  if (f32)
    head_norm_kernel<float><<<grid, 256, 0, stream>>>((float*)out, o, w, seg,
                                                      heads, vdim, eps);
  else
    head_norm_kernel<bf16><<<grid, 256, 0, stream>>>((bf16*)out, o, w, seg,
                                                     heads, vdim, eps);
}

// ---------------------------------------------------------------------------
// q/k head norms + cache append: one wave per (row, head of q, k or v)
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void qk_norm_append_kernel(
    T* __restrict__ q_out, T* __restrict__ kpages, T* __restrict__ vpages,
    const T* __restrict__ proj, const float* __restrict__ q_w,
    const float* __restrict__ k_w, const int* __restrict__ row_slot,
    const int* __restrict__ row_pos, const int* __restrict__ table,
    int table_stride, int heads, int kv_heads, int dim, int vdim, int dpad,
    int vpad, float eps) {
  const int hd = blockIdx.y * 4 + (threadIdx.x >> 6);
  if (hd >= heads + 2 * kv_heads) return;
  const int lane = threadIdx.x & 63;
  const size_t row = blockIdx.x;
  const T* pr = proj + row * (size_t)((heads + kv_heads) * dim +
                                      kv_heads * vdim);
  const int pos = row_pos[row];
  const size_t page =
      table[(size_t)row_slot[row] * table_stride + (pos >> 6)];
  if (hd >= heads + kv_heads) {
    const int g = hd - heads - kv_heads;
    const T* v = pr + (size_t)(heads + kv_heads) * dim + g * vdim;
    T* dst = vpages + (page * kv_heads + g) * (size_t)vpad * 64 + (pos & 63);
    for (int c = lane; c < vdim; c += 64) dst[(size_t)c * 64] = v[c];
    return;
  }
  const T* src = pr + (size_t)hd * dim;
  float ss = 0.f;
  for (int d = lane; d < dim; d += 64) ss += to_f(src[d]) * to_f(src[d]);
  const float r = 1.f / sqrtf(wave_sum(ss) / dim + eps);
  const bool is_q = hd < heads;
  const float* w = is_q ? q_w : k_w;
  T* dst = is_q ? q_out + (row * heads + hd) * (size_t)dpad
                : kpages + ((page * kv_heads + (hd - heads)) * 64 +
                            (pos & 63)) * (size_t)dpad;
  for (int d = lane; d < dpad; d += 64)
    dst[d] = from_f<T>(d < dim ? to_f(src[d]) * r * w[d] : 0.f);
}

void launch_qk_norm_append(void* q_out, void* kpages, void* vpages,
                           const void* proj, const float* q_w,
                           const float* k_w, const int* row_slot,
                           const int* row_pos, const int* table,
                           int table_stride, int n, int heads, int kv_heads,
                           int dim, int vdim, int dpad, int vpad, float eps,
                           int f32, hipStream_t stream) {
  dim3 grid(n, (heads + 2 * kv_heads + 3) / 4);
  if (f32)
    qk_norm_append_kernel<float><<<grid, 256, 0, stream>>>(
        (float*)q_out, (float*)kpages, (float*)vpages, (const float*)proj,
        q_w, k_w, row_slot, row_pos, table, table_stride, heads, kv_heads,
        dim, vdim, dpad, vpad, eps);
  else
    qk_norm_append_kernel<bf16><<<grid, 256, 0, stream>>>(
        (bf16*)q_out, (bf16*)kpages, (bf16*)vpages, (const bf16*)proj, q_w,
        k_w, row_slot, row_pos, table, table_stride, heads, kv_heads, dim,
        vdim, dpad, vpad, eps);
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
