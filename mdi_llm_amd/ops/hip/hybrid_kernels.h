// Launchers of the kernels for stacks that mix recurrent and windowed-
// attention layers over ragged batches (hybrid_kernels.hip, paged_attn.inc).
//
// `f32` picks the activation type: 0 bf16, 1 float.  The residual stream,
// norm weights, gates, recurrent state and bias tables are always float.
#pragma once

#include <hip/hip_runtime.h>

// One ragged batch: segment s is `len[s]` tokens of slot `slot[s]`, at rows
// start[s].. of the flat activations and positions pos0[s].. of its sequence.
struct SegView {
  const int* start;
  const int* len;
  const int* slot;
  const int* pos0;
  int n;
};

// Residual + norm step, one row per block.  x [n, e] float:
//   tokens != null : x = scale * table[token]
//   y != null      : x += post_w ? rms(y) * (offset + post_w) : y
// then, if next_w, xn = rms(x) * (offset + next_w).  -1: e is too large.
int launch_residual_norm(float* x, const void* y, const float* post_w,
                         void* xn, const float* next_w, const int* tokens,
                         const void* table, float scale, float offset,
                         float eps, int n, int e, int f32,
                         hipStream_t stream);

// z <- xIELU(z), p and q already through softplus
void launch_xielu(void* z, long long n, float p, float q, int f32,
                  hipStream_t stream);

// HGRN2 over segments of one token each: gates, state update, read-out and
// the per-head norm in one launch.  proj [rows, 2*H*D + H*E] = q|f|v.
void launch_hgrn2_step(void* out, const void* proj, float* state,
                       const float* f_bias, const float* lower,
                       const float* norm_w, SegView seg, int heads, int dim,
                       int vdim, int vstride, float eps, int f32,
                       hipStream_t stream);

// HGRN2 over longer segments, which must be in the order of their rows; o is
// the raw read-out [rows, H*E] float, work holds hgrn2_work_floats(...).
// Returns -1 when dim has no instantiation.
long long hgrn2_work_floats(int rows, int segments, int heads, int dim);
int launch_hgrn2_scan(float* o, float* work, const void* proj, float* state,
                      const float* f_bias, const float* lower, SegView seg,
                      int max_len, int heads, int dim, int vdim, int vstride,
                      int f32, hipStream_t stream);

// out[row] = rms(o[row]) * w per head, for the rows of the segments
void launch_head_norm(void* out, const float* o, const float* w, SegView seg,
                      int max_len, int heads, int vdim, float eps, int f32,
                      hipStream_t stream);

// Per-head q/k norms, q to a padded buffer, k and v into the paged cache.
// proj [n, (H+G)*D + G*E] = q|k|v; k pages [P, G, 64 * dpad] and v pages
// [P, G, 64 * vpad] in the order of PageLayout.
void launch_qk_norm_append(void* q_out, void* kpages, void* vpages,
                           const void* proj, const float* q_w,
                           const float* k_w, const int* row_slot,
                           const int* row_pos, const int* table,
                           int table_stride, int n, int heads, int kv_heads,
                           int dim, int vdim, int dpad, int vpad, float eps,
                           int f32, hipStream_t stream);

struct PagedAttnArgs {
  void* out;            // [rows, H*vdim]
  const void* q;        // [rows, H, dpad]
  const void* kpages;
  const void* vpages;
  const float* bias;    // [H, bias_len] in log2 units, by distance
  const int* table;
  float* part_o;        // split mode: [n, H, splits, vpad]
  float* part_ml;       // split mode: [n, H, splits, 2]
  SegView seg;
  int bias_len, table_stride;
  int heads, kv_heads, vdim, dpad, vpad;
  int window, keep_first;
  float scale_log2;
  int splits;           // 0: whole rows per wave; >=1: split the keys
  int max_len;          // longest segment
};

// Returns -1 when (dpad, vpad) has no instantiation.
int launch_paged_attn_bf16(const PagedAttnArgs& a, hipStream_t stream);
int launch_paged_attn_f32(const PagedAttnArgs& a, hipStream_t stream);

// Between the steps of an unchanged decode batch: tokens = sampled,
// pos += 1; entries of the spare slot stay where they are.
void launch_advance_batch(const int* slots, const int* sampled, int* pos,
                          int* tokens, int spare, int n, hipStream_t stream);

// out[n, m] = x[n, :] . w[m, :] in bf16 for up to 32 rows of x, with xIELU
// if act.  Returns -1 when n or k (a multiple of 64) does not fit.
int launch_skinny_gemm(void* out, const void* w, const void* x, int n, int m,
                       int k, int act, float act_p, float act_q,
                       hipStream_t stream);
