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
//                    (+ pos_table[row_pos] if there is one)
//   y != null      : x += mult * (post_w ? rms(y) * (offset + post_w) : y
//                    (times gain, if there is one), plus a second output
//                    rms(y2) * (offset + post_w2) and the weighted routed
//                    rows [n, top, e] if any); post_w if y2
// then, if next_w, xn = rms(x) * (offset + next_w).
struct ResidualArgs {
  float* x;
  const void* y;
  const float* post_w;
  const float* gain;
  const void* y2;
  const float* post_w2;
  void* xn;
  const float* next_w;
  const int* tokens;
  const void* table;
  const void* pos_table;
  const int* row_pos;
  const void* routed;
  const float* routed_w;
  int top;
  float scale, offset, eps, mult;
  int n, e;
};

// -1: e is too large
int launch_residual_norm(const ResidualArgs& a, int f32, hipStream_t stream);

// z <- xIELU(z), p and q already through softplus
void launch_xielu(void* z, long long n, float p, float q, int f32,
                  hipStream_t stream);

// z <- exact GELU
void launch_gelu(void* z, long long n, int f32, hipStream_t stream);

// z <- max(z, 0)^2
void launch_relu2(void* z, long long n, int f32, hipStream_t stream);

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

// Per-head q/k norms (and rotation), q to a padded buffer [n, heads, dpad], k
// and v into the paged cache.  proj = q|k|v rows; k pages [P, k_heads, 64 *
// dpad] and v pages [P, v_heads, 64 * vpad] in the order of PageLayout.  No
// pages: proj = q rows, nothing is stored.
struct QkAppendArgs {
  void* q_out;
  void* kpages;
  void* vpages;
  const void* proj;
  const float* q_w;
  const float* k_w;
  const int* row_slot;
  const int* row_pos;
  const int* table;
  const float* rope;  // [positions, rot / 2, 2] or null
  int table_stride, n, heads, k_heads, v_heads, dim, vdim, dpad, vpad, rot;
  float eps;
};

void launch_qk_norm_append(const QkAppendArgs& a, int f32,
                           hipStream_t stream);

// rows [n, k_heads * dim + v_heads * vdim] <-> pages
void launch_kv_rows(const QkAppendArgs& a, void* rows, int store, int f32,
                    hipStream_t stream);

// The same for norms over a whole row of queries and of keys (q_w [heads *
// dim], k_w [k_heads * dim]), queries times q_scale[position] if it is there,
// values divided by their head's root mean square if unit_values.  rope is
// not used; proj rows are ld apart; vec: 8 (bf16) or 4 (float) channels per
// access are aligned and stay within a head.
struct RowAppendArgs {
  QkAppendArgs qk;
  const float* q_scale;
  long long ld;
  int unit_values, vec;
};

// -1: no room for the values' tile
int launch_row_norm_append(const RowAppendArgs& a, int f32,
                           hipStream_t stream);

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
  // score <- cap * tanh(score / cap): scale / cap and cap in log2 units
  float cap_in, cap_log2;  // cap_log2 0: no cap
  // maps 2: q [rows, H, 2, dpad] and k pages [P, kv_heads * 2, ..], part_o
  // [n, H, 2, splits, vpad]; out = unit-size (o1 - map_weight * o2) *
  // out_scale.  Split mode always leaves parts.
  int maps;
  float map_weight, out_scale, eps;
  // one map only:
  const float* slopes;  // [H] in log2 units, taken off per distance; no bias
  const float* sink;    // [H] score of one more term of the softmax
  const void* gate;     // out *= sigmoid(gate[row * gate_ld + h * vdim + ..])
  long long gate_ld;
};

// Returns -1 when (dpad, vpad) has no instantiation.
int launch_paged_attn_bf16(const PagedAttnArgs& a, hipStream_t stream);
int launch_paged_attn_f32(const PagedAttnArgs& a, hipStream_t stream);
int launch_diff_attn_bf16(const PagedAttnArgs& a, hipStream_t stream);  // maps 2
int launch_diff_attn_f32(const PagedAttnArgs& a, hipStream_t stream);
int launch_slope_attn_bf16(const PagedAttnArgs& a, hipStream_t stream);  // slopes
int launch_slope_attn_f32(const PagedAttnArgs& a, hipStream_t stream);

struct RowAttnArgs {
  void* out;              // head h of row r at r * out_row + h * vdim
  const void* q;          // head h of row r at r * q_row + h * dim
  const void* k;          // latent: pages [P, 64, dim]; head: flat rows
  const void* v;          // head: flat rows (kv_row apart, as k)
  const int* table;       // latent: pages of a slot
  const int* ctx_start;   // head: flat row of position ctx_first, by segment
  const int* ctx_first;
  const void* gate;       // head: sigmoid(gate[r * gate_row + h]) or null
  float* part_o;          // latent, splits > 1: [rows, H, splits, dim]
  float* part_ml;         // and [rows, H, splits, 2]
  long long out_row, q_row, kv_row, gate_row;
  SegView seg;
  int table_stride;
  int heads, groups;      // groups: 1 (latent) or heads
  int dim, vdim;          // latent: the padded row, both
  int window;
  float scale_log2;
  int splits, max_len;
  int vec, out_vec;       // 16-byte loads and 4-element stores are aligned
};

// Return -1 when the sizes have no instantiation.
int launch_latent_attn_bf16(const RowAttnArgs& a, hipStream_t stream);
int launch_latent_attn_f32(const RowAttnArgs& a, hipStream_t stream);
int launch_head_attn_bf16(const RowAttnArgs& a, hipStream_t stream);
int launch_head_attn_f32(const RowAttnArgs& a, hipStream_t stream);

// What follows the first product of a parallel block; any part may be absent
// (null, with its sizes 0).  Norms of a row's two latents: q [n, q_rank] to
// q_out, kv [n, rank] to its place in the pages [P, 64, rpad] (kv_w null: as
// it is).  out = act(gate) * up over [n, cols]; act 0 silu, 1 tanh-gelu.
struct BranchArgs {
  void* q_out;
  const void* q;
  const float* q_w;
  void* pages;
  const void* kv;
  const float* kv_w;
  const int* row_slot;
  const int* row_pos;
  const int* table;
  void* out;
  const void* gate;
  const void* up;
  long long q_ld, kv_ld, in_ld, out_ld;
  int n, table_stride, q_rank, rank, rpad, cols, act;
  float eps;
};

void launch_branch(const BranchArgs& a, int f32, hipStream_t stream);

// out[start[s] + t, :rank] = the cached row of position pos0[s] + t
void launch_latent_gather(void* out, const void* pages, const int* table,
                          int table_stride, SegView seg, int max_len,
                          int rank, int rpad, int f32, hipStream_t stream);

// Per-head product out[r, h*m ..] = w[h] x[r, h*xk ..] with w [H, m, k], k a
// multiple of 32 and xk <= k.  x_rows / out_rows map the n rows (null: as
// they are); gate is by output row.  part_o [n, H, splits, k] and part_ml, if
// given, are merged to make x.
struct HeadProjArgs {
  void* out;
  const void* x;
  const void* w;
  const int* x_rows;
  const int* out_rows;
  const void* gate;
  const float* part_o;
  const float* part_ml;
  long long out_ld, x_ld, gate_ld;
  int n, heads, m, k, xk, splits;
};

void launch_head_proj(const HeadProjArgs& a, int f32, hipStream_t stream);

// Routing.  plan is one int buffer:
//   chosen experts [n*top] | pairs ordered by expert [n*top] | number of
//   tiles | tiles
// where pair p is choice p % top of row p / top and a tile is up to
// tile_rows pairs of one expert.
struct MoeTile {
  int expert, first, rows;  // pairs order[first] .. order[first + rows - 1]
  int tile0, n_tiles;       // the expert's tiles
};

struct MoePlan {
  int* chosen;
  int* order;
  int* n_tiles;
  MoeTile* tiles;
  int pairs, top, experts, tile_rows, max_tiles;
  // the router: outputs >= experts, those past the experts stand for the row
  // itself; correction [outputs] or null; gated: one more column of z is a
  // gate, whose sigmoid is one more weight of each row
  int outputs, gated;
  const float* correction;
  float scale;
};

// tile_rows: 16, or 128 (bf16, contractions multiples of 64, at least 128
// expert and 256 model channels)
MoePlan moe_plan(int* buffer, int n, int top, int experts, int tile_rows);
long long moe_plan_ints(int n, int top, int experts, int tile_rows);

// z [n, outputs + gated] = x router^T in float; chosen outputs and weight [n,
// top + gated].
void launch_moe_route(float* weight, float* z, const void* x,
                      const void* router, MoePlan p, int n, int k, int f32,
                      hipStream_t stream);

// mid[pair] = act(gate x) * (up x), w [experts, 2 * ff, k]
void launch_moe_up(void* mid, const void* x, const void* w, MoePlan p,
                   int ff, int k, int act, int f32, hipStream_t stream);

// out[pair] = w x, w [experts, m, ff], x [pairs, ff]
void launch_moe_down(void* out, const void* mid, const void* w, MoePlan p,
                     int m, int ff, int f32, hipStream_t stream);

// Between the steps of an unchanged decode batch: tokens = sampled,
// pos += 1; entries of the spare slot stay where they are.
void launch_advance_batch(const int* slots, const int* sampled, int* pos,
                          int* tokens, int spare, int n, hipStream_t stream);

// Residual step of blocks with norms on the sublayers' outputs, one row per
// block.  x [n, e] float:
//   tokens != null : x = scale * table[token]
//   y or routed    : a = y (times the last weight, if there are routed rows)
//                        + weighted routed rows [n, top, e], where a chosen
//                        output >= experts stands for x itself;
//                    x += post_w ? groups of rms(a) * post_w : a
// keep = x; if coef, x = sum_j coef[j] hist[j] + coef[depth] x; then xn is
//   next_w : groups of rms(x) * next_w
//   shift  : x + (prev[slot] - x) * shift, and prev[slot] = x
//   else   : x
struct StreamArgs {
  float* x;
  const void* y;
  const float* post_w;
  void* xn;
  const float* next_w;
  const int* tokens;
  const void* table;
  const void* routed;
  const float* routed_w;
  const int* chosen;
  const float* hist;   // [depth, n, e]
  const float* coef;   // [depth + 1]
  float* past;         // [n, e]: only the sum over hist, the stream is as it was
  float* keep;
  const float* shift;
  float* prev;         // [slots, e]
  const int* row_slot;
  const int* row_pos;
  int top, experts, depth, groups, n, e;
  float scale, eps;
};

// -1: e is too large
int launch_stream_step(const StreamArgs& a, int f32, hipStream_t stream);

// xn = x + (the row before - x) * shift over segments; prev [slots, e] is the
// row before a segment and takes its last one
void launch_token_shift(void* xn, const float* x, const float* shift,
                        float* prev, SegView seg, int max_len, int e, int f32,
                        hipStream_t stream);

// out = act(bias + sum_k w[k] * (x[t - taps + 1 + k] + in_bias)) per channel
// over segments, zeros before position 0; w [taps, c], x rows ld apart, state
// [slots, max(1, taps - 1), c] the last rows of x; act: silu.  At most 16
// taps.
struct ConvArgs {
  void* out;
  const void* x;
  const float* w;
  const float* bias;
  const float* in_bias;  // or null
  void* state;
  SegView seg;
  long long ld;
  int max_len, c, taps, act;
  int vec;  // 8 (bf16) or 4 (float) channels per access are aligned
};

void launch_causal_conv(const ConvArgs& a, int f32, hipStream_t stream);

// RG-LRU: r, i = sigmoid(block-diagonal products of u + gate_bias), a =
// exp(rate * r), S = a S + sqrt(1 - a^2) i u, out = S * gelu_tanh(y + y_bias).
// gates [2, blocks, part, part], state [slots, width].
struct RgLruArgs {
  void* out;
  const void* u;      // [rows, width]
  const void* y;      // rows y_ld apart
  const float* y_bias;
  const void* gates;
  const float* gate_bias;
  const float* rate;
  float* state;
  float* work;        // scan: [2, n, width]
  SegView seg;
  long long y_ld;
  int n, width, blocks, max_len;
};

void launch_rglru_step(const RgLruArgs& a, int f32, hipStream_t stream);
void launch_rglru_scan(const RgLruArgs& a, int f32, hipStream_t stream);

// Mamba-2: dt = softplus(dt + dt_bias), S = exp(rate dt) S + dt B x^T, o =
// S^T C.  xbc [rows, inner + 2 * groups * dim] = x|B|C, dt rows dt_ld apart,
// state [slots, heads, dim, vstride], o [rows, inner] float.
struct Mamba2Args {
  float* o;
  const void* xbc;
  const void* dt;
  float* state;
  const float* dt_bias;
  const float* rate;
  float* work;        // scan: hgrn2_work_floats(...)
  SegView seg;
  long long dt_ld;
  int heads, groups, dim, vdim, vstride, max_len;
};

void launch_mamba2_step(const Mamba2Args& a, int f32, hipStream_t stream);
// -1: dim has no instantiation
int launch_mamba2_scan(const Mamba2Args& a, int f32, hipStream_t stream);

// mLSTM: per head, with log gates i = cap tanh(z_i / cap) and f =
// logsigmoid(cap tanh(z_f / cap)), m' = max(f + m, i), S = exp(f + m - m') S +
// exp(i - m') k v^T and the same for the normaliser n with v = 1; o = S^T q /
// (max(|n . q|, exp(-m')) + 1e-6), brought to unit size, times norm_w and
// sigmoid(g).  proj rows = q|k|v|g|z_i|z_f, gate_bias [2 H], state [slots, H,
// dim, vstride] with n in column vdim, peak [slots, H] = m, norm_w [H * vdim].
struct MLstmArgs {
  void* out;            // [rows, H * vdim]
  const void* proj;
  float* state;
  float* peak;
  const float* gate_bias;
  const float* norm_w;
  float* work;          // scan: mlstm_work_floats(...)
  SegView seg;
  int n, heads, dim, vdim, vstride, max_len;
  float cap, q_scale, eps;
};

void launch_mlstm_step(const MLstmArgs& a, int f32, hipStream_t stream);
long long mlstm_work_floats(int rows, int segments, int heads, int dim,
                            int vdim);
// segments in the order of their rows; -1: dim has no instantiation
int launch_mlstm_scan(const MLstmArgs& a, int f32, hipStream_t stream);

// minGRU: z = sigmoid(. + bias), c = u + 1/2 or sigmoid(u) below 0 with u = .
// + bias, S = (1 - z) S + z c, out = S silu(g).  proj rows = z|u|g, ld apart,
// bias [2 * width], state [slots, width].
struct MinGruArgs {
  void* out;
  const void* proj;
  const float* bias;
  float* state;
  SegView seg;
  long long ld;
  int width, max_len;
};

void launch_mingru_step(const MinGruArgs& a, int f32, hipStream_t stream);
void launch_mingru_scan(const MinGruArgs& a, int f32, hipStream_t stream);

// out = groups of rms((o + skip x) silu(z)) * w; x rows are xld, z rows zld
// apart, skip [heads].  -1: rows are too long
struct GatedNormArgs {
  void* out;
  const float* o;
  const void* x;
  const void* z;
  const float* skip;
  const float* w;
  long long xld, zld;
  int n, inner, vdim, groups;
  float eps;
  int vec;
};

int launch_gated_norm(const GatedNormArgs& a, int f32, hipStream_t stream);

// out[n, m] = x[n, :] . w[m, :] in bf16 for up to 32 rows of x, with act 1
// xIELU, 2 exact GELU, 3 squared ReLU.  Returns -1 when n or k (a multiple of 64) does not fit.
int launch_skinny_gemm(void* out, const void* w, const void* x, int n, int m,
                       int k, int act, float act_p, float act_q,
                       hipStream_t stream);
