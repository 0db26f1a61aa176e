// Torch bindings of the hybrid-stack kernels: every size that a kernel
// trusts is checked against the tensors here.

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>

#include "hybrid_kernels.h"

namespace {

using Opt = c10::optional<torch::Tensor>;

hipStream_t cur_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

const float* f32_ptr(const torch::Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 &&
                  t.is_contiguous() && t.numel() == n,
              name, ": expected ", n, " contiguous floats on the GPU");
  return t.data_ptr<float>();
}

const int* i32_ptr(const torch::Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 &&
                  t.is_contiguous() && t.numel() >= n,
              name, ": expected at least ", n, " contiguous int32 on the GPU");
  return t.data_ptr<int>();
}

// activations: bf16 or float, one type per call
int act_type(const torch::Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() &&
                  (t.scalar_type() == torch::kBFloat16 ||
                   t.scalar_type() == torch::kFloat32),
              name, ": expected contiguous bf16 or float on the GPU");
  return t.scalar_type() == torch::kFloat32 ? 1 : 0;
}

void check_like(const torch::Tensor& t, int f32, const char* name) {
  TORCH_CHECK(act_type(t, name) == f32, name, ": activation type mismatch");
}

// seg: int32 [4, n] = start, len, slot, pos0
SegView seg_view(const torch::Tensor& seg) {
  TORCH_CHECK(seg.is_cuda() && seg.scalar_type() == torch::kInt32 &&
                  seg.dim() == 2 && seg.size(0) == 4 && seg.size(1) > 0 &&
                  seg.stride(1) == 1,
              "seg: expected int32 [4, n] on the GPU");
  const int* p = seg.data_ptr<int>();
  const int64_t st = seg.stride(0);
  return SegView{p, p + st, p + 2 * st, p + 3 * st, (int)seg.size(1)};
}

// rows of a wider matrix: contiguous columns, any row stride
struct Rows {
  void* p;
  int n, cols;
  long long ld;
};

Rows rows_of(const torch::Tensor& t, int f32, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) > 0 && t.size(1) > 0 &&
                  t.stride(1) == 1 && t.stride(0) >= t.size(1) &&
                  t.scalar_type() ==
                      (f32 ? torch::kFloat32 : torch::kBFloat16),
              name, ": expected rows of the activation type on the GPU");
  return Rows{t.data_ptr(), (int)t.size(0), (int)t.size(1), t.stride(0)};
}

int row_type(const torch::Tensor& t, const char* name) {
  TORCH_CHECK(t.scalar_type() == torch::kBFloat16 ||
                  t.scalar_type() == torch::kFloat32,
              name, ": expected bf16 or float");
  return t.scalar_type() == torch::kFloat32 ? 1 : 0;
}

void residual_norm(torch::Tensor x, Opt y, Opt post_w, Opt xn, Opt next_w,
                   Opt tokens, Opt table, double scale, double offset,
                   double eps, double mult, Opt pos_table, Opt row_pos,
                   Opt routed, Opt routed_w, Opt gain, Opt y2, Opt post_w2) {
  TORCH_CHECK(x.dim() == 2 && x.size(0) > 0, "x must be [n, e]");
  const int n = (int)x.size(0), e = (int)x.size(1);
  float* xp = const_cast<float*>(f32_ptr(x, (int64_t)n * e, "x"));
  TORCH_CHECK(!(y && tokens) && !!tokens == !!table && !!xn == !!next_w,
              "residual_norm: bad combination of operands");
  int f32 = 0;
  const torch::Tensor* act = y ? &*y : xn ? &*xn : table ? &*table : nullptr;
  if (act) f32 = act_type(*act, "activation");
  if (y) {
    check_like(*y, f32, "y");
    TORCH_CHECK(y->numel() == x.numel(), "y size");
  }
  if (xn) {
    check_like(*xn, f32, "xn");
    TORCH_CHECK(xn->numel() == x.numel(), "xn size");
  }
  if (table) {
    check_like(*table, f32, "table");
    TORCH_CHECK(table->dim() == 2 && table->size(1) == e, "table size");
  }
  TORCH_CHECK(!!pos_table == !!row_pos && (!pos_table || tokens) &&
                  !!routed == !!routed_w && (!routed || y),
              "residual_norm: bad combination of operands");
  TORCH_CHECK(!(gain && (post_w || !y)) && !!y2 == !!post_w2 &&
                  (!y2 || (y && post_w)),
              "residual_norm: bad combination of operands");
  ResidualArgs a{};
  if (gain) a.gain = f32_ptr(*gain, e, "gain");
  if (y2) {
    check_like(*y2, f32, "y2");
    TORCH_CHECK(y2->numel() == x.numel(), "y2 size");
    a.y2 = y2->data_ptr();
    a.post_w2 = f32_ptr(*post_w2, e, "post_w2");
  }
  if (pos_table) {
    check_like(*pos_table, f32, "pos_table");
    TORCH_CHECK(pos_table->dim() == 2 && pos_table->size(1) == e,
                "pos_table size");
    a.pos_table = pos_table->data_ptr();
    a.row_pos = i32_ptr(*row_pos, n, "row_pos");
  }
  if (routed) {
    check_like(*routed, f32, "routed");
    TORCH_CHECK(routed->dim() == 3 && routed->size(0) == n &&
                    routed->size(2) == e,
                "routed must be [n, top, e]");
    a.top = (int)routed->size(1);
    a.routed = routed->data_ptr();
    a.routed_w = f32_ptr(*routed_w, (int64_t)n * a.top, "routed_w");
  }
  a.x = xp;
  a.y = y ? y->data_ptr() : nullptr;
  a.post_w = post_w ? f32_ptr(*post_w, e, "post_w") : nullptr;
  a.xn = xn ? xn->data_ptr() : nullptr;
  a.next_w = next_w ? f32_ptr(*next_w, e, "next_w") : nullptr;
  a.tokens = tokens ? i32_ptr(*tokens, n, "tokens") : nullptr;
  a.table = table ? table->data_ptr() : nullptr;
  a.scale = (float)scale;
  a.offset = (float)offset;
  a.eps = (float)eps;
  a.mult = (float)mult;
  a.n = n;
  a.e = e;
  const int rc = launch_residual_norm(a, f32, cur_stream());
  TORCH_CHECK(rc == 0, "residual_norm: row of ", e, " elements");
}

void xielu(torch::Tensor z, double p, double q) {
  const int f32 = act_type(z, "z");
  launch_xielu(z.data_ptr(), (long long)z.numel(), (float)p, (float)q, f32,
               cur_stream());
}

void gelu(torch::Tensor z) {
  launch_gelu(z.data_ptr(), (long long)z.numel(), act_type(z, "z"),
              cur_stream());
}

void relu2(torch::Tensor z) {
  launch_relu2(z.data_ptr(), (long long)z.numel(), act_type(z, "z"),
               cur_stream());
}

struct Recurrent {
  int heads, dim, vdim, vstride, f32;
  float* state;
  const float* f_bias;
  const float* lower;
};

Recurrent recurrent(const torch::Tensor& proj, const torch::Tensor& state,
                    const torch::Tensor& f_bias, const torch::Tensor& lower,
                    int64_t vdim) {
  TORCH_CHECK(state.dim() == 4, "state must be [slots, H, D, vstride]");
  Recurrent r;
  r.heads = (int)state.size(1);
  r.dim = (int)state.size(2);
  r.vstride = (int)state.size(3);
  r.vdim = (int)vdim;
  r.f32 = act_type(proj, "proj");
  TORCH_CHECK(r.vstride % 4 == 0 && r.vdim <= r.vstride && r.vdim > 0,
              "state columns");
  TORCH_CHECK(proj.dim() == 2 &&
                  proj.size(1) == r.heads * (2 * r.dim + r.vdim),
              "proj columns");
  r.state = const_cast<float*>(f32_ptr(state, state.numel(), "state"));
  r.f_bias = f32_ptr(f_bias, r.heads * r.dim, "f_bias");
  r.lower = f32_ptr(lower, r.heads * r.dim, "lower");
  return r;
}

void hgrn2_step(torch::Tensor out, torch::Tensor proj, torch::Tensor state,
                torch::Tensor f_bias, torch::Tensor lower,
                torch::Tensor norm_w, torch::Tensor seg, double eps) {
  const Recurrent r =
      recurrent(proj, state, f_bias, lower, norm_w.numel());
  check_like(out, r.f32, "out");
  TORCH_CHECK(out.numel() == proj.size(0) * r.heads * r.vdim, "out size");
  TORCH_CHECK(r.dim <= 1024 && r.vstride <= 1024, "hgrn2_step: sizes");
  launch_hgrn2_step(out.data_ptr(), proj.data_ptr(), r.state, r.f_bias,
                    r.lower, f32_ptr(norm_w, r.vdim, "norm_w"),
                    seg_view(seg), r.heads, r.dim, r.vdim, r.vstride,
                    (float)eps, r.f32, cur_stream());
}

void hgrn2_scan(torch::Tensor out, torch::Tensor proj, torch::Tensor state,
                torch::Tensor f_bias, torch::Tensor lower,
                torch::Tensor norm_w, torch::Tensor seg, int64_t max_len,
                double eps) {
  const Recurrent r =
      recurrent(proj, state, f_bias, lower, norm_w.numel());
  check_like(out, r.f32, "out");
  TORCH_CHECK(out.numel() == proj.size(0) * r.heads * r.vdim, "out size");
  TORCH_CHECK(r.dim <= 256 && r.vdim <= 1024, "hgrn2_scan: sizes");
  TORCH_CHECK(max_len > 0 && max_len <= proj.size(0), "max_len");
  const SegView sv = seg_view(seg);
  const auto fp = proj.options().dtype(torch::kFloat32);
  torch::Tensor o = torch::empty({out.numel()}, fp);
  torch::Tensor work = torch::empty(
      {hgrn2_work_floats((int)proj.size(0), sv.n, r.heads, r.dim)}, fp);
  float* op = o.data_ptr<float>();
  const int rc = launch_hgrn2_scan(
      op, work.data_ptr<float>(), proj.data_ptr(), r.state, r.f_bias,
      r.lower, sv, (int)max_len, r.heads, r.dim, r.vdim, r.vstride, r.f32,
      cur_stream());
  TORCH_CHECK(rc == 0, "hgrn2_scan: unsupported dim ", r.dim);
  launch_head_norm(out.data_ptr(), op, f32_ptr(norm_w, r.vdim, "norm_w"), sv,
                   (int)max_len, r.heads, r.vdim, (float)eps, r.f32,
                   cur_stream());
}

struct Pages {
  int kv_heads, maps, dpad, vpad;
};

// one K page per value head, or two (two maps)
Pages pages(const torch::Tensor& k, const torch::Tensor& v, int f32) {
  check_like(k, f32, "kpages");
  check_like(v, f32, "vpages");
  TORCH_CHECK(k.dim() == 3 && v.dim() == 3 && k.size(0) == v.size(0) &&
                  (k.size(1) == v.size(1) || k.size(1) == 2 * v.size(1)) &&
                  k.size(2) % (64 * 32) == 0 && v.size(2) % (64 * 32) == 0,
              "pages: expected k [P, G * maps, 64 * dpad] and v [P, G, 64 * "
              "vpad]");
  return Pages{(int)v.size(1), (int)(k.size(1) / v.size(1)),
               (int)k.size(2) / 64, (int)v.size(2) / 64};
}

void set_places(QkAppendArgs& a, const torch::Tensor& row_slot,
                const torch::Tensor& row_pos, const torch::Tensor& table) {
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  a.row_slot = i32_ptr(row_slot, a.n, "row_slot");
  a.row_pos = i32_ptr(row_pos, a.n, "row_pos");
  a.table = i32_ptr(table, table.numel(), "table");
  a.table_stride = (int)table.size(1);
}

void set_pages(QkAppendArgs& a, const torch::Tensor& kpages,
               const torch::Tensor& vpages, int64_t dim, int64_t vdim,
               int f32) {
  const Pages pg = pages(kpages, vpages, f32);
  a.kpages = kpages.data_ptr();
  a.vpages = vpages.data_ptr();
  a.k_heads = pg.kv_heads * pg.maps;
  a.v_heads = pg.kv_heads;
  a.dim = (int)dim;
  a.vdim = (int)vdim;
  a.dpad = pg.dpad;
  a.vpad = pg.vpad;
  TORCH_CHECK(dim > 0 && dim <= pg.dpad && vdim > 0 && vdim <= pg.vpad,
              "head sizes of the pages");
}

void qk_norm_append(torch::Tensor q_out, Opt kpages, Opt vpages,
                    torch::Tensor proj, torch::Tensor q_w, Opt k_w,
                    torch::Tensor row_slot, torch::Tensor row_pos,
                    torch::Tensor table, int64_t vdim, double eps, Opt rope) {
  const int f32 = act_type(proj, "proj");
  check_like(q_out, f32, "q_out");
  QkAppendArgs a{};
  TORCH_CHECK(proj.dim() == 2 && q_out.dim() == 3 &&
                  q_out.size(0) == proj.size(0) && q_out.size(2) % 32 == 0 &&
                  q_out.size(2) <= 256,
              "q_out must be [n, H, dpad]");
  TORCH_CHECK(!!kpages == !!vpages && !!kpages == !!k_w,
              "qk_norm_append: bad combination of operands");
  a.n = (int)proj.size(0);
  a.heads = (int)q_out.size(1);
  a.dim = (int)q_w.numel();
  a.vdim = (int)vdim;
  a.dpad = (int)q_out.size(2);
  TORCH_CHECK(a.n > 0 && a.dim > 0 && a.dim <= a.dpad, "q_out columns");
  if (kpages) {
    set_pages(a, *kpages, *vpages, a.dim, vdim, f32);
    TORCH_CHECK(a.dpad == q_out.size(2), "q_out must be [n, H, dpad]");
    a.k_w = f32_ptr(*k_w, a.dim, "k_w");
  }
  TORCH_CHECK(proj.size(1) == (a.heads + a.k_heads) * a.dim + a.v_heads * vdim,
              "proj columns");
  if (rope) {
    // (positions beyond the table are the caller's limit on sequences)
    TORCH_CHECK(rope->dim() == 3 && rope->size(2) == 2 &&
                    2 * rope->size(1) <= a.dim,
                "rope must be [positions, pairs, 2]");
    TORCH_CHECK(rope->size(0) > 0, "rope positions");
    a.rope = f32_ptr(*rope, rope->numel(), "rope");
    a.rot = 2 * (int)rope->size(1);
  }
  TORCH_CHECK((int64_t)a.n * (a.heads + a.k_heads) < (int64_t)1 << 31,
              "qk_norm_append: rows");
  a.q_out = q_out.data_ptr();
  a.proj = proj.data_ptr();
  a.q_w = f32_ptr(q_w, a.dim, "q_w");
  a.eps = (float)eps;
  set_places(a, row_slot, row_pos, table);
  launch_qk_norm_append(a, f32, cur_stream());
}

void row_norm_append(torch::Tensor q_out, torch::Tensor kpages,
                     torch::Tensor vpages, torch::Tensor proj,
                     torch::Tensor q_w, torch::Tensor k_w,
                     torch::Tensor row_slot, torch::Tensor row_pos,
                     torch::Tensor table, int64_t vdim, double eps,
                     Opt q_scale, bool unit_values) {
  const int f32 = act_type(q_out, "q_out");
  const Rows r = rows_of(proj, f32, "proj");
  RowAppendArgs a{};
  TORCH_CHECK(q_out.dim() == 3 && q_out.size(0) == r.n && q_out.size(1) > 0 &&
                  q_out.size(2) <= 256 && q_w.numel() % q_out.size(1) == 0,
              "q_out must be [n, H, dpad]");
  a.qk.n = r.n;
  a.qk.heads = (int)q_out.size(1);
  const int64_t dim = q_w.numel() / a.qk.heads;
  set_pages(a.qk, kpages, vpages, dim, vdim, f32);
  TORCH_CHECK(a.qk.dpad == q_out.size(2) && a.qk.k_heads == a.qk.v_heads &&
                  a.qk.vpad <= 256,
              "row_norm_append: pages");
  TORCH_CHECK(r.cols == (a.qk.heads + a.qk.k_heads) * dim +
                            a.qk.v_heads * vdim,
              "proj columns");
  a.qk.q_out = q_out.data_ptr();
  a.qk.proj = r.p;
  a.qk.q_w = f32_ptr(q_w, a.qk.heads * dim, "q_w");
  a.qk.k_w = f32_ptr(k_w, a.qk.k_heads * dim, "k_w");
  a.qk.eps = (float)eps;
  set_places(a.qk, row_slot, row_pos, table);
  // (positions beyond the table are the caller's limit on sequences)
  if (q_scale) a.q_scale = f32_ptr(*q_scale, q_scale->numel(), "q_scale");
  a.ld = r.ld;
  a.unit_values = unit_values ? 1 : 0;
  const int v = f32 ? 4 : 8;
  a.vec = dim % v == 0 && vdim % v == 0 && r.ld % v == 0 &&
          (size_t)r.p % 16 == 0;
  TORCH_CHECK(launch_row_norm_append(a, f32, cur_stream()) == 0,
              "row_norm_append: values of ", vdim);
}

void kv_rows(torch::Tensor rows, torch::Tensor kpages, torch::Tensor vpages,
             torch::Tensor row_slot, torch::Tensor row_pos,
             torch::Tensor table, int64_t dim, int64_t vdim, bool store) {
  const int f32 = act_type(rows, "rows");
  QkAppendArgs a{};
  set_pages(a, kpages, vpages, dim, vdim, f32);
  TORCH_CHECK(rows.dim() == 2 && rows.size(0) > 0 &&
                  rows.size(1) == a.k_heads * dim + a.v_heads * vdim,
              "kv_rows: columns");
  a.n = (int)rows.size(0);
  set_places(a, row_slot, row_pos, table);
  launch_kv_rows(a, rows.data_ptr(), store ? 1 : 0, f32, cur_stream());
}

void paged_attn(torch::Tensor out, torch::Tensor q, torch::Tensor kpages,
                torch::Tensor vpages, Opt bias, torch::Tensor table,
                torch::Tensor seg, int64_t max_len, int64_t window,
                int64_t keep_first, double scale, int64_t splits, Opt part_o,
                Opt part_ml, double softcap, double map_weight,
                double out_scale, double eps, Opt slopes, Opt sink,
                Opt gate) {
  const int f32 = act_type(q, "q");
  const Pages pg = pages(kpages, vpages, f32);
  check_like(out, f32, "out");
  TORCH_CHECK(q.dim() == 3 && q.size(2) == pg.dpad &&
                  q.size(1) % pg.maps == 0,
              "q must be [n, H * maps, dpad]");
  PagedAttnArgs a{};
  a.maps = pg.maps;
  a.heads = (int)q.size(1) / pg.maps;
  TORCH_CHECK(softcap >= 0.0, "softcap");
  if (softcap > 0.0) {
    a.cap_in = (float)(scale / softcap);
    a.cap_log2 = (float)(softcap * 1.4426950408889634);
  }
  a.map_weight = (float)map_weight;
  a.out_scale = (float)out_scale;
  a.eps = (float)eps;
  a.kv_heads = pg.kv_heads;
  TORCH_CHECK(a.heads % a.kv_heads == 0, "heads per kv head");
  TORCH_CHECK(out.dim() == 2 && out.size(0) == q.size(0) &&
                  out.size(1) % a.heads == 0,
              "out must be [n, H*vdim]");
  a.vdim = (int)out.size(1) / a.heads;
  a.dpad = pg.dpad;
  a.vpad = pg.vpad;
  TORCH_CHECK(a.vdim <= a.vpad, "vdim");
  TORCH_CHECK(!!bias != !!slopes, "paged_attn: a bias table or slopes");
  TORCH_CHECK(a.maps == 1 || !(slopes || sink || gate),
              "paged_attn: slopes, sink and gate go with one map");
  if (bias) {
    TORCH_CHECK(bias->dim() == 2 && bias->size(0) == a.heads &&
                    bias->size(1) > 0,
                "bias must be [H, n]");
    a.bias = f32_ptr(*bias, bias->numel(), "bias");
    a.bias_len = (int)bias->size(1);
  } else {
    a.slopes = f32_ptr(*slopes, a.heads, "slopes");
  }
  if (sink) a.sink = f32_ptr(*sink, a.heads, "sink");
  if (gate) {
    const Rows g = rows_of(*gate, f32, "gate");
    TORCH_CHECK(g.n == out.size(0) && g.cols == out.size(1),
                "gate must be [n, H*vdim]");
    a.gate = g.p;
    a.gate_ld = g.ld;
  }
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  a.table = i32_ptr(table, table.numel(), "table");
  a.table_stride = (int)table.size(1);
  a.seg = seg_view(seg);
  a.out = out.data_ptr();
  a.q = q.data_ptr();
  a.kpages = kpages.data_ptr();
  a.vpages = vpages.data_ptr();
  TORCH_CHECK(window > 0 && keep_first >= 0, "mask");
  a.window = (int)std::min<int64_t>(window, INT32_MAX / 2);
  a.keep_first = (int)std::min<int64_t>(keep_first, INT32_MAX / 2);
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.splits = (int)splits;
  a.max_len = (int)max_len;
  TORCH_CHECK(splits >= 0 && max_len > 0, "splits and max_len");
  TORCH_CHECK(splits <= 1 || max_len == 1,
              "split keys: one token per segment");
  if (splits > 1 || (splits == 1 && a.maps > 1)) {
    TORCH_CHECK(max_len == 1, "two maps: parts hold one token per segment");
    TORCH_CHECK(part_o && part_ml, "split keys need scratch");
    const int64_t cells = (int64_t)a.seg.n * a.heads * a.maps * splits;
    TORCH_CHECK(part_o->numel() >= cells * a.vpad &&
                    part_ml->numel() >= cells * 2,
                "split scratch too small");
    a.part_o = const_cast<float*>(
        f32_ptr(*part_o, part_o->numel(), "part_o"));
    a.part_ml = const_cast<float*>(
        f32_ptr(*part_ml, part_ml->numel(), "part_ml"));
  }
  const auto launch =
      a.maps == 2 ? (f32 ? launch_diff_attn_f32 : launch_diff_attn_bf16)
      : slopes ? (f32 ? launch_slope_attn_f32 : launch_slope_attn_bf16)
               : (f32 ? launch_paged_attn_f32 : launch_paged_attn_bf16);
  const int rc = launch(a, cur_stream());
  TORCH_CHECK(rc == 0, "paged_attn: unsupported padded sizes ", a.dpad, ", ",
              a.vpad);
}

// latent pages [P, 64, rpad]
int latent_pages(const torch::Tensor& pages, int f32) {
  check_like(pages, f32, "pages");
  TORCH_CHECK(pages.dim() == 3 && pages.size(1) == 64 &&
                  pages.size(2) % 64 == 0,
              "pages: expected [P, 64, rpad]");
  return (int)pages.size(2);
}

void set_act(BranchArgs& a, const torch::Tensor& out,
             const torch::Tensor& gate, const torch::Tensor& up, int64_t act,
             int f32) {
  const Rows o = rows_of(out, f32, "act_out"), g = rows_of(gate, f32, "gate"),
             u = rows_of(up, f32, "up");
  TORCH_CHECK(o.n == g.n && o.n == u.n && o.cols == g.cols &&
                  o.cols == u.cols && g.ld == u.ld,
              "gated activation: sizes");
  TORCH_CHECK(act == 0 || act == 1, "gated activation: act");
  a.out = o.p;
  a.out_ld = o.ld;
  a.gate = g.p;
  a.up = u.p;
  a.in_ld = g.ld;
  a.cols = o.cols;
  a.act = (int)act;
  a.n = o.n;
}

void latent_norm_append(torch::Tensor pages, Opt kv, Opt kv_w,
                        torch::Tensor row_slot, torch::Tensor row_pos,
                        torch::Tensor table, double eps, Opt q_out, Opt q,
                        Opt q_w, Opt act_out, Opt gate, Opt up,
                        int64_t act) {
  const int f32 = act_type(pages, "pages");
  BranchArgs a{};
  a.pages = pages.data_ptr();
  a.rpad = latent_pages(pages, f32);
  a.eps = (float)eps;
  TORCH_CHECK((kv || q) && !!q == !!q_out && !!q == !!q_w && (kv || !kv_w) &&
                  !!act_out == !!gate && !!act_out == !!up,
              "latent_norm_append: bad combination of operands");
  if (act_out) set_act(a, *act_out, *gate, *up, act, f32);
  auto same_rows = [&](const Rows& r) {
    TORCH_CHECK(a.n == 0 || a.n == r.n, "latent_norm_append: rows");
    a.n = r.n;
  };
  if (kv) {
    const Rows r = rows_of(*kv, f32, "kv");
    same_rows(r);
    TORCH_CHECK(r.cols <= a.rpad, "kv columns");
    a.kv = r.p;
    a.kv_ld = r.ld;
    a.rank = r.cols;
    if (kv_w) a.kv_w = f32_ptr(*kv_w, r.cols, "kv_w");
  }
  if (q) {
    const Rows r = rows_of(*q, f32, "q");
    same_rows(r);
    check_like(*q_out, f32, "q_out");
    TORCH_CHECK(q_out->numel() == (int64_t)r.n * r.cols, "q_out size");
    a.q = r.p;
    a.q_ld = r.ld;
    a.q_rank = r.cols;
    a.q_out = q_out->data_ptr();
    a.q_w = f32_ptr(*q_w, r.cols, "q_w");
  }
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  a.row_slot = i32_ptr(row_slot, a.n, "row_slot");
  a.row_pos = i32_ptr(row_pos, a.n, "row_pos");
  a.table = i32_ptr(table, table.numel(), "table");
  a.table_stride = (int)table.size(1);
  launch_branch(a, f32, cur_stream());
}

void gated_act(torch::Tensor out, torch::Tensor gate, torch::Tensor up,
               int64_t act) {
  const int f32 = row_type(out, "out");
  BranchArgs a{};
  set_act(a, out, gate, up, act, f32);
  launch_branch(a, f32, cur_stream());
}

void latent_gather(torch::Tensor out, torch::Tensor pages,
                   torch::Tensor table, torch::Tensor seg, int64_t max_len) {
  const int f32 = act_type(pages, "pages");
  const int rpad = latent_pages(pages, f32);
  check_like(out, f32, "out");
  TORCH_CHECK(out.dim() == 2 && out.size(1) <= rpad && max_len > 0 &&
                  max_len <= out.size(0),
              "latent_gather: out must be [rows, rank]");
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  launch_latent_gather(out.data_ptr(), pages.data_ptr(),
                       i32_ptr(table, table.numel(), "table"),
                       (int)table.size(1), seg_view(seg), (int)max_len,
                       (int)out.size(1), rpad, f32, cur_stream());
}

struct Parts {
  float *o = nullptr, *ml = nullptr;
};

Parts parts(const Opt& part_o, const Opt& part_ml, int64_t cells, int k) {
  TORCH_CHECK(part_o && part_ml, "split keys need scratch");
  return Parts{
      const_cast<float*>(f32_ptr(*part_o, cells * k, "part_o")),
      const_cast<float*>(f32_ptr(*part_ml, cells * 2, "part_ml"))};
}

void head_proj(torch::Tensor out, Opt x, torch::Tensor w, Opt x_rows,
               Opt out_rows, Opt gate, Opt part_o, Opt part_ml) {
  const int f32 = act_type(w, "w");
  const Rows o = rows_of(out, f32, "out");
  HeadProjArgs a{};
  TORCH_CHECK(w.dim() == 3 && w.size(2) % 32 == 0, "w must be [H, m, k]");
  a.heads = (int)w.size(0);
  a.m = (int)w.size(1);
  a.k = (int)w.size(2);
  TORCH_CHECK(o.cols == a.heads * a.m, "head_proj: out columns");
  TORCH_CHECK(!!x != !!part_o, "head_proj: x or partial results");
  if (x) {
    const Rows r = rows_of(*x, f32, "x");
    TORCH_CHECK(r.cols % a.heads == 0, "head_proj: x columns");
    a.x = r.p;
    a.x_ld = r.ld;
    a.xk = r.cols / a.heads;
    a.n = x_rows ? (int)x_rows->numel() : r.n;
    TORCH_CHECK(a.xk <= a.k, "head_proj: x columns");
    if (x_rows) a.x_rows = i32_ptr(*x_rows, a.n, "x_rows");
  } else {
    TORCH_CHECK(part_o->dim() == 4 && part_o->size(1) == a.heads &&
                    part_o->size(3) == a.k && !x_rows,
                "part_o must be [n, H, splits, k]");
    a.n = (int)part_o->size(0);
    a.splits = (int)part_o->size(2);
    a.xk = a.k;
    const Parts p = parts(part_o, part_ml,
                          (int64_t)a.n * a.heads * a.splits, a.k);
    a.part_o = p.o;
    a.part_ml = p.ml;
  }
  if (out_rows) {
    a.out_rows = i32_ptr(*out_rows, a.n, "out_rows");
  } else {
    TORCH_CHECK(o.n >= a.n, "head_proj: out rows");
  }
  if (gate) {
    const Rows g = rows_of(*gate, f32, "gate");
    TORCH_CHECK(g.n == o.n && g.cols == a.heads, "gate must be [n, H]");
    a.gate = g.p;
    a.gate_ld = g.ld;
  }
  a.out = o.p;
  a.out_ld = o.ld;
  a.w = w.data_ptr();
  TORCH_CHECK(a.n > 0 && 16 * (a.k + 8) * (f32 ? 4 : 2) +
                      16 * a.splits * 4 <= 65536,
              "head_proj: sizes");
  launch_head_proj(a, f32, cur_stream());
}

void latent_attn(Opt out, torch::Tensor q, torch::Tensor pages,
                 torch::Tensor table, torch::Tensor seg, int64_t max_len,
                 int64_t window, double scale, int64_t splits, Opt part_o,
                 Opt part_ml) {
  const int f32 = act_type(q, "q");
  RowAttnArgs a{};
  a.dim = a.vdim = latent_pages(pages, f32);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == a.dim, "q must be [n, H, rpad]");
  a.heads = (int)q.size(1);
  a.groups = 1;
  a.q = q.data_ptr();
  a.q_row = (int64_t)a.heads * a.dim;
  a.k = a.v = pages.data_ptr();
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  a.table = i32_ptr(table, table.numel(), "table");
  a.table_stride = (int)table.size(1);
  a.seg = seg_view(seg);
  a.max_len = (int)max_len;
  a.splits = (int)splits;
  a.window = (int)std::min<int64_t>(window, INT32_MAX / 2);
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.vec = a.out_vec = 1;
  TORCH_CHECK(window > 0 && max_len > 0 && max_len <= q.size(0) &&
                  splits > 0 && splits <= 256,
              "latent_attn: sizes");
  if (splits > 1) {
    TORCH_CHECK(part_o && part_o->dim() == 4 &&
                    part_o->size(0) == q.size(0) &&
                    part_o->size(2) == splits,
                "part_o must be [n, H, splits, rpad]");
    const Parts p = parts(part_o, part_ml, q.size(0) * a.heads * splits,
                          a.dim);
    a.part_o = p.o;
    a.part_ml = p.ml;
  } else {
    TORCH_CHECK(out, "latent_attn: out");
    check_like(*out, f32, "out");
    TORCH_CHECK(out->numel() == q.numel(), "latent_attn: out size");
    a.out = out->data_ptr();
    a.out_row = a.q_row;
  }
  const int rc = f32 ? launch_latent_attn_f32(a, cur_stream())
                     : launch_latent_attn_bf16(a, cur_stream());
  TORCH_CHECK(rc == 0, "latent_attn: unsupported row size ", a.dim);
}

void head_attn(torch::Tensor out, torch::Tensor q, torch::Tensor kv,
               torch::Tensor seg, torch::Tensor ctx_seg, int64_t max_len,
               int64_t heads, int64_t dim, int64_t vdim, int64_t window,
               double scale, Opt gate) {
  const int f32 = row_type(q, "q");
  const Rows o = rows_of(out, f32, "out"), r = rows_of(q, f32, "q"),
             k = rows_of(kv, f32, "kv");
  TORCH_CHECK(heads > 0 && r.cols == heads * dim && o.cols == heads * vdim &&
                  k.cols == heads * (dim + vdim) && o.n == r.n,
              "head_attn: columns");
  RowAttnArgs a{};
  a.heads = a.groups = (int)heads;
  a.dim = (int)dim;
  a.vdim = (int)vdim;
  a.out = o.p;
  a.out_row = o.ld;
  a.q = r.p;
  a.q_row = r.ld;
  const int size = f32 ? 4 : 2, n = 16 / size;
  a.k = k.p;
  a.v = (char*)k.p + heads * dim * size;
  a.kv_row = k.ld;
  a.seg = seg_view(seg);
  const SegView c = seg_view(ctx_seg);
  TORCH_CHECK(c.n == a.seg.n, "head_attn: segments");
  a.ctx_start = c.start;
  a.ctx_first = c.pos0;
  if (gate) {
    const Rows g = rows_of(*gate, f32, "gate");
    TORCH_CHECK(g.n == o.n && g.cols == heads, "gate must be [n, H]");
    a.gate = g.p;
    a.gate_row = g.ld;
  }
  TORCH_CHECK(window > 0 && max_len > 0 && max_len <= r.n, "head_attn: sizes");
  a.window = (int)std::min<int64_t>(window, INT32_MAX / 2);
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.splits = 1;
  a.max_len = (int)max_len;
  a.vec = dim % n == 0 && vdim % n == 0 && r.ld % n == 0 && k.ld % n == 0 &&
          (size_t)r.p % 16 == 0 && (size_t)k.p % 16 == 0;
  a.out_vec = vdim % 4 == 0 && o.ld % 4 == 0 && (size_t)o.p % (4 * size) == 0;
  const int rc = f32 ? launch_head_attn_f32(a, cur_stream())
                     : launch_head_attn_bf16(a, cur_stream());
  TORCH_CHECK(rc == 0, "head_attn: unsupported sizes ", dim, ", ", vdim);
}

void check_tile_rows(int64_t tile_rows, int f32, int64_t k) {
  TORCH_CHECK(tile_rows == 16 || (tile_rows == 128 && !f32 && k % 64 == 0),
              "expert tiles: 16 rows, or 128 in bf16 with k a multiple of 64");
}

// the plan that moe_route made for n rows
MoePlan plan_of(const torch::Tensor& w, const torch::Tensor& plan,
                int64_t pairs, int64_t top, int64_t tile_rows, int f32) {
  TORCH_CHECK(top > 0 && pairs % top == 0 && pairs > 0, "expert rows");
  check_tile_rows(tile_rows, f32, w.size(2));
  const int n = (int)(pairs / top), e = (int)w.size(0), t = (int)tile_rows;
  const int64_t ints = moe_plan_ints(n, (int)top, e, t);
  TORCH_CHECK(plan.numel() == ints, "plan of another shape");
  return moe_plan(const_cast<int*>(i32_ptr(plan, ints, "plan")), n, (int)top,
                  e, t);
}

torch::Tensor moe_route(torch::Tensor weight, torch::Tensor x,
                        torch::Tensor router, int64_t top,
                        int64_t tile_rows, Opt correction, double scale,
                        int64_t identity, bool gated) {
  const int f32 = act_type(x, "x");
  check_like(router, f32, "router");
  TORCH_CHECK(x.dim() == 2 && router.dim() == 2 &&
                  router.size(1) == x.size(1),
              "moe_route: sizes");
  const int n = (int)x.size(0), cols = (int)router.size(0);
  const int outputs = cols - (gated ? 1 : 0);
  TORCH_CHECK(n > 0 && outputs <= 256 && top >= 1 && top <= outputs &&
                  top <= 64,
              "moe_route: at most 256 outputs, 64 of them for a token");
  TORCH_CHECK(identity >= 0 && identity < outputs, "moe_route: identity");
  float* wp = const_cast<float*>(
      f32_ptr(weight, n * (top + (gated ? 1 : 0)), "weight"));
  check_tile_rows(tile_rows, f32, x.size(1));
  const int e = outputs - (int)identity;
  torch::Tensor plan =
      torch::empty({moe_plan_ints(n, (int)top, e, (int)tile_rows)},
                   x.options().dtype(torch::kInt32));
  torch::Tensor z =
      torch::empty({n, cols}, x.options().dtype(torch::kFloat32));
  MoePlan p = moe_plan(plan.data_ptr<int>(), n, (int)top, e, (int)tile_rows);
  p.outputs = outputs;
  p.gated = gated ? 1 : 0;
  p.scale = (float)scale;
  if (correction) p.correction = f32_ptr(*correction, outputs, "correction");
  launch_moe_route(wp, z.data_ptr<float>(), x.data_ptr(), router.data_ptr(),
                   p, n, (int)x.size(1), f32, cur_stream());
  return plan;
}

void moe_up(torch::Tensor mid, torch::Tensor x, torch::Tensor w,
            torch::Tensor plan, int64_t act, int64_t tile_rows) {
  const int f32 = act_type(x, "x");
  check_like(mid, f32, "mid");
  check_like(w, f32, "w");
  TORCH_CHECK(x.dim() == 2 && mid.dim() == 2 && w.dim() == 3 &&
                  w.size(1) == 2 * mid.size(1) && w.size(2) == x.size(1) &&
                  mid.size(0) % x.size(0) == 0,
              "moe_up: sizes");
  TORCH_CHECK(act == 0 || act == 1, "moe_up: act");
  // (the large tiles have 32-bit byte offsets)
  TORCH_CHECK(tile_rows == 16 || (mid.size(1) % 4 == 0 &&
                                  mid.size(1) >= 128 &&
                                  x.numel() < (1LL << 30) &&
                                  128 * x.size(1) < (1LL << 30)),
              "moe_up: columns");
  const MoePlan p = plan_of(w, plan, mid.size(0), mid.size(0) / x.size(0),
                            tile_rows, f32);
  launch_moe_up(mid.data_ptr(), x.data_ptr(), w.data_ptr(), p,
                (int)mid.size(1), (int)x.size(1), (int)act, f32,
                cur_stream());
}

void moe_down(torch::Tensor out, torch::Tensor mid, torch::Tensor w,
              torch::Tensor plan, int64_t tile_rows) {
  const int f32 = act_type(mid, "mid");
  check_like(out, f32, "out");
  check_like(w, f32, "w");
  TORCH_CHECK(out.dim() == 3 && mid.dim() == 2 && w.dim() == 3 &&
                  w.size(1) == out.size(2) && w.size(2) == mid.size(1) &&
                  mid.size(0) == out.size(0) * out.size(1),
              "moe_down: sizes");
  TORCH_CHECK(tile_rows == 16 || (out.size(2) % 4 == 0 &&
                                  out.size(2) >= 256 &&
                                  mid.numel() < (1LL << 30)),
              "moe_down: columns");
  const MoePlan p =
      plan_of(w, plan, mid.size(0), out.size(1), tile_rows, f32);
  launch_moe_down(out.data_ptr(), mid.data_ptr(), w.data_ptr(), p,
                  (int)out.size(2), (int)mid.size(1), f32, cur_stream());
}

void skinny_gemm(torch::Tensor out, torch::Tensor w, torch::Tensor x,
                 int64_t act, double act_p, double act_q) {
  TORCH_CHECK(act >= 0 && act <= 3, "skinny_gemm: act");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && out.dim() == 2, "2-D operands");
  const int n = (int)x.size(0), m = (int)w.size(0), k = (int)x.size(1);
  for (const auto* t : {&out, &w, &x})
    TORCH_CHECK(act_type(*t, "operand") == 0, "skinny_gemm: bf16 operands");
  TORCH_CHECK(w.size(1) == k && out.size(0) == n && out.size(1) == m,
              "skinny_gemm: sizes");
  const int rc = launch_skinny_gemm(out.data_ptr(), w.data_ptr(),
                                    x.data_ptr(), n, m, k, (int)act,
                                    (float)act_p, (float)act_q, cur_stream());
  TORCH_CHECK(rc == 0, "skinny_gemm: unsupported n ", n, " or k ", k);
}

void stream_step(torch::Tensor x, Opt y, Opt post_w, Opt xn, Opt next_w,
                 int64_t groups, double eps, Opt tokens, Opt table,
                 double scale, Opt routed, Opt routed_w, Opt chosen,
                 int64_t experts, Opt hist, Opt coef, Opt keep, Opt past,
                 Opt shift, Opt prev, Opt row_slot, Opt row_pos) {
  TORCH_CHECK(x.dim() == 2 && x.size(0) > 0, "x must be [n, e]");
  const int64_t n = x.size(0), e = x.size(1);
  StreamArgs a{};
  a.x = const_cast<float*>(f32_ptr(x, n * e, "x"));
  TORCH_CHECK(groups > 0 && e % groups == 0, "stream_step: groups");
  TORCH_CHECK(!(tokens && (y || routed)) && !!tokens == !!table &&
                  !!routed == !!routed_w && !!routed == !!chosen &&
                  !!hist == !!coef && !(past && !hist) && !!shift == !!prev &&
                  !!shift == !!row_slot && !!shift == !!row_pos &&
                  !(next_w && shift) && (xn || (!next_w && !shift)),
              "stream_step: bad combination of operands");
  const torch::Tensor* act =
      y ? &*y : routed ? &*routed : xn ? &*xn : table ? &*table : nullptr;
  const int f32 = act ? act_type(*act, "activation") : 0;
  if (y) {
    check_like(*y, f32, "y");
    TORCH_CHECK(y->numel() == n * e, "y size");
    a.y = y->data_ptr();
  }
  if (xn) {
    check_like(*xn, f32, "xn");
    TORCH_CHECK(xn->numel() == n * e, "xn size");
    a.xn = xn->data_ptr();
  }
  if (table) {
    check_like(*table, f32, "table");
    TORCH_CHECK(table->dim() == 2 && table->size(1) == e, "table size");
    a.table = table->data_ptr();
    a.tokens = i32_ptr(*tokens, n, "tokens");
  }
  if (routed) {
    check_like(*routed, f32, "routed");
    TORCH_CHECK(routed->dim() == 3 && routed->size(0) == n &&
                    routed->size(2) == e,
                "routed must be [n, top, e]");
    a.top = (int)routed->size(1);
    a.routed = routed->data_ptr();
    a.routed_w = f32_ptr(*routed_w, n * (a.top + (y ? 1 : 0)), "routed_w");
    a.chosen = i32_ptr(*chosen, n * a.top, "chosen");
    a.experts = (int)experts;
  }
  if (post_w) a.post_w = f32_ptr(*post_w, e, "post_w");
  if (next_w) a.next_w = f32_ptr(*next_w, e, "next_w");
  if (hist) {
    TORCH_CHECK(hist->dim() == 3, "hist must be [depth, n, e]");
    a.depth = (int)hist->size(0);
    a.hist = f32_ptr(*hist, a.depth * n * e, "hist");
    a.coef = f32_ptr(*coef, a.depth + 1, "coef");
  }
  if (past) a.past = const_cast<float*>(f32_ptr(*past, n * e, "past"));
  if (keep) a.keep = const_cast<float*>(f32_ptr(*keep, n * e, "keep"));
  if (shift) {
    a.shift = f32_ptr(*shift, e, "shift");
    TORCH_CHECK(prev->dim() == 2 && prev->size(1) == e,
                "prev must be [slots, e]");
    a.prev = const_cast<float*>(f32_ptr(*prev, prev->numel(), "prev"));
    a.row_slot = i32_ptr(*row_slot, n, "row_slot");
    a.row_pos = i32_ptr(*row_pos, n, "row_pos");
  }
  a.groups = (int)groups;
  a.n = (int)n;
  a.e = (int)e;
  a.scale = (float)scale;
  a.eps = (float)eps;
  TORCH_CHECK(launch_stream_step(a, f32, cur_stream()) == 0,
              "stream_step: row of ", e, " elements");
}

void token_shift(torch::Tensor xn, torch::Tensor x, torch::Tensor shift,
                 torch::Tensor prev, torch::Tensor seg, int64_t max_len) {
  const int f32 = act_type(xn, "xn");
  TORCH_CHECK(x.dim() == 2 && xn.numel() == x.numel() && x.size(0) > 0,
              "token_shift: sizes");
  const int64_t n = x.size(0), e = x.size(1);
  TORCH_CHECK(prev.dim() == 2 && prev.size(1) == e, "prev must be [slots, e]");
  TORCH_CHECK(max_len > 0 && max_len <= n, "max_len");
  launch_token_shift(
      xn.data_ptr(), f32_ptr(x, n * e, "x"), f32_ptr(shift, e, "shift"),
      const_cast<float*>(f32_ptr(prev, prev.numel(), "prev")), seg_view(seg),
      (int)max_len, (int)e, f32, cur_stream());
}

void causal_conv(torch::Tensor out, torch::Tensor x, torch::Tensor w,
                 torch::Tensor bias, Opt in_bias, torch::Tensor state,
                 torch::Tensor seg, int64_t max_len, bool act) {
  const int f32 = act_type(out, "out");
  const Rows r = rows_of(x, f32, "x");
  check_like(state, f32, "state");
  ConvArgs a{};
  TORCH_CHECK(w.dim() == 2 && w.size(1) == r.cols && w.size(0) >= 1 &&
                  w.size(0) <= 16,
              "causal_conv: w must be [taps, channels], at most 16 taps");
  a.taps = (int)w.size(0);
  a.c = r.cols;
  TORCH_CHECK(out.numel() == (int64_t)r.n * r.cols && state.dim() == 3 &&
                  state.size(1) == std::max(1, a.taps - 1) &&
                  state.size(2) == r.cols && max_len > 0 && max_len <= r.n,
              "causal_conv: sizes");
  a.out = out.data_ptr();
  a.x = r.p;
  a.ld = r.ld;
  a.w = f32_ptr(w, w.numel(), "w");
  a.bias = f32_ptr(bias, r.cols, "bias");
  if (in_bias) a.in_bias = f32_ptr(*in_bias, r.cols, "in_bias");
  a.state = state.data_ptr();
  a.seg = seg_view(seg);
  a.max_len = (int)max_len;
  a.act = act ? 1 : 0;
  const int v = f32 ? 4 : 8;
  a.vec = r.cols % v == 0 && r.ld % v == 0 && (size_t)r.p % 16 == 0;
  launch_causal_conv(a, f32, cur_stream());
}

RgLruArgs rglru_args(const torch::Tensor& out, const torch::Tensor& u,
                     const torch::Tensor& y, const torch::Tensor& y_bias,
                     const torch::Tensor& gates,
                     const torch::Tensor& gate_bias,
                     const torch::Tensor& rate, const torch::Tensor& state,
                     const torch::Tensor& seg, int f32) {
  check_like(u, f32, "u");
  check_like(gates, f32, "gates");
  const Rows r = rows_of(y, f32, "y");
  RgLruArgs a{};
  TORCH_CHECK(u.dim() == 2 && u.size(0) == r.n && u.size(1) == r.cols &&
                  out.numel() == u.numel(),
              "rglru: rows");
  a.n = r.n;
  a.width = r.cols;
  TORCH_CHECK(gates.dim() == 3 && gates.size(0) % 2 == 0 &&
                  gates.size(1) == gates.size(2) &&
                  gates.size(0) / 2 * gates.size(1) == a.width,
              "rglru: gates must be [2 * blocks, part, part]");
  a.blocks = (int)gates.size(0) / 2;
  TORCH_CHECK(state.dim() == 2 && state.size(1) == a.width,
              "rglru: state must be [slots, width]");
  a.out = out.data_ptr();
  a.u = u.data_ptr();
  a.y = r.p;
  a.y_ld = r.ld;
  a.y_bias = f32_ptr(y_bias, a.width, "y_bias");
  a.gates = gates.data_ptr();
  a.gate_bias = f32_ptr(gate_bias, 2 * a.width, "gate_bias");
  a.rate = f32_ptr(rate, a.width, "rate");
  a.state = const_cast<float*>(f32_ptr(state, state.numel(), "state"));
  a.seg = seg_view(seg);
  return a;
}

void rglru_step(torch::Tensor out, torch::Tensor u, torch::Tensor y,
                torch::Tensor y_bias, torch::Tensor gates,
                torch::Tensor gate_bias, torch::Tensor rate,
                torch::Tensor state, torch::Tensor seg) {
  const int f32 = act_type(out, "out");
  const RgLruArgs a = rglru_args(out, u, y, y_bias, gates, gate_bias, rate,
                                 state, seg, f32);
  launch_rglru_step(a, f32, cur_stream());
}

void rglru_scan(torch::Tensor out, torch::Tensor u, torch::Tensor y,
                torch::Tensor y_bias, torch::Tensor gates,
                torch::Tensor gate_bias, torch::Tensor rate,
                torch::Tensor state, torch::Tensor seg, int64_t max_len) {
  const int f32 = act_type(out, "out");
  RgLruArgs a = rglru_args(out, u, y, y_bias, gates, gate_bias, rate, state,
                           seg, f32);
  TORCH_CHECK(max_len > 0 && max_len <= a.n, "max_len");
  a.max_len = (int)max_len;
  torch::Tensor work = torch::empty({2, a.n, a.width},
                                    out.options().dtype(torch::kFloat32));
  a.work = work.data_ptr<float>();
  launch_rglru_scan(a, f32, cur_stream());
}

Mamba2Args mamba2_args(const torch::Tensor& o, const torch::Tensor& xbc,
                       const torch::Tensor& dt, const torch::Tensor& state,
                       const torch::Tensor& dt_bias,
                       const torch::Tensor& rate, int64_t vdim,
                       const torch::Tensor& seg, int f32) {
  const Rows d = rows_of(dt, f32, "dt");
  Mamba2Args a{};
  TORCH_CHECK(state.dim() == 4, "state must be [slots, H, N, vstride]");
  a.heads = (int)state.size(1);
  a.dim = (int)state.size(2);
  a.vstride = (int)state.size(3);
  a.vdim = (int)vdim;
  TORCH_CHECK(a.vstride % 4 == 0 && vdim > 0 && vdim <= a.vstride &&
                  a.dim <= 256 && a.vstride <= 1024 && d.cols == a.heads,
              "mamba2: sizes");
  const int64_t inner = (int64_t)a.heads * vdim;
  TORCH_CHECK(xbc.dim() == 2 && xbc.size(0) == d.n && xbc.size(1) > inner &&
                  (xbc.size(1) - inner) % (2 * a.dim) == 0,
              "mamba2: xbc columns");
  a.groups = (int)((xbc.size(1) - inner) / (2 * a.dim));
  TORCH_CHECK(a.heads % a.groups == 0, "mamba2: groups");
  a.o = const_cast<float*>(f32_ptr(o, d.n * inner, "o"));
  a.xbc = xbc.data_ptr();
  a.dt = d.p;
  a.dt_ld = d.ld;
  a.state = const_cast<float*>(f32_ptr(state, state.numel(), "state"));
  a.dt_bias = f32_ptr(dt_bias, a.heads, "dt_bias");
  a.rate = f32_ptr(rate, a.heads, "rate");
  a.seg = seg_view(seg);
  return a;
}

void mamba2_step(torch::Tensor o, torch::Tensor xbc, torch::Tensor dt,
                 torch::Tensor state, torch::Tensor dt_bias,
                 torch::Tensor rate, int64_t vdim, torch::Tensor seg) {
  const int f32 = act_type(xbc, "xbc");
  launch_mamba2_step(mamba2_args(o, xbc, dt, state, dt_bias, rate, vdim, seg,
                                 f32), f32, cur_stream());
}

void mamba2_scan(torch::Tensor o, torch::Tensor xbc, torch::Tensor dt,
                 torch::Tensor state, torch::Tensor dt_bias,
                 torch::Tensor rate, int64_t vdim, torch::Tensor seg,
                 int64_t max_len) {
  const int f32 = act_type(xbc, "xbc");
  Mamba2Args a =
      mamba2_args(o, xbc, dt, state, dt_bias, rate, vdim, seg, f32);
  TORCH_CHECK(max_len > 0 && max_len <= xbc.size(0), "max_len");
  a.max_len = (int)max_len;
  torch::Tensor work = torch::empty(
      {hgrn2_work_floats((int)xbc.size(0), a.seg.n, a.heads, a.dim)},
      o.options());
  a.work = work.data_ptr<float>();
  TORCH_CHECK(launch_mamba2_scan(a, f32, cur_stream()) == 0,
              "mamba2_scan: unsupported state ", a.dim);
}

MLstmArgs mlstm_args(const torch::Tensor& out, const torch::Tensor& proj,
                     const torch::Tensor& state, const torch::Tensor& peak,
                     const torch::Tensor& gate_bias,
                     const torch::Tensor& norm_w, double cap, double q_scale,
                     double eps, const torch::Tensor& seg, int f32) {
  check_like(proj, f32, "proj");
  MLstmArgs a{};
  TORCH_CHECK(state.dim() == 4 && proj.dim() == 2 && proj.size(0) > 0,
              "mlstm: state must be [slots, H, dim, vstride]");
  a.n = (int)proj.size(0);
  a.heads = (int)state.size(1);
  a.dim = (int)state.size(2);
  a.vstride = (int)state.size(3);
  TORCH_CHECK(norm_w.numel() % a.heads == 0, "mlstm: norm_w");
  a.vdim = (int)(norm_w.numel() / a.heads);
  TORCH_CHECK(a.vstride % 4 == 0 && a.vdim > 0 && a.vdim < a.vstride &&
                  a.dim <= 256 && a.vstride <= 1024 && cap > 0.0,
              "mlstm: sizes");
  TORCH_CHECK(proj.size(1) == 2LL * a.heads * (a.dim + a.vdim + 1) &&
                  out.numel() == (int64_t)a.n * a.heads * a.vdim &&
                  (int64_t)a.n * a.heads < (int64_t)1 << 31,
              "mlstm: rows");
  TORCH_CHECK(peak.dim() == 2 && peak.size(0) == state.size(0) &&
                  peak.size(1) == a.heads,
              "mlstm: peak must be [slots, H]");
  a.out = out.data_ptr();
  a.proj = proj.data_ptr();
  a.state = const_cast<float*>(f32_ptr(state, state.numel(), "state"));
  a.peak = const_cast<float*>(f32_ptr(peak, peak.numel(), "peak"));
  a.gate_bias = f32_ptr(gate_bias, 2 * a.heads, "gate_bias");
  a.norm_w = f32_ptr(norm_w, a.heads * a.vdim, "norm_w");
  a.cap = (float)cap;
  a.q_scale = (float)q_scale;
  a.eps = (float)eps;
  a.seg = seg_view(seg);
  return a;
}

void mlstm_step(torch::Tensor out, torch::Tensor proj, torch::Tensor state,
                torch::Tensor peak, torch::Tensor gate_bias,
                torch::Tensor norm_w, double cap, double q_scale, double eps,
                torch::Tensor seg) {
  const int f32 = act_type(out, "out");
  launch_mlstm_step(mlstm_args(out, proj, state, peak, gate_bias, norm_w, cap,
                               q_scale, eps, seg, f32),
                    f32, cur_stream());
}

void mlstm_scan(torch::Tensor out, torch::Tensor proj, torch::Tensor state,
                torch::Tensor peak, torch::Tensor gate_bias,
                torch::Tensor norm_w, double cap, double q_scale, double eps,
                torch::Tensor seg, int64_t max_len) {
  const int f32 = act_type(out, "out");
  MLstmArgs a = mlstm_args(out, proj, state, peak, gate_bias, norm_w, cap,
                           q_scale, eps, seg, f32);
  TORCH_CHECK(max_len > 0 && max_len <= a.n, "max_len");
  a.max_len = (int)max_len;
  torch::Tensor work = torch::empty(
      {mlstm_work_floats(a.n, a.seg.n, a.heads, a.dim, a.vdim)},
      state.options());
  a.work = work.data_ptr<float>();
  TORCH_CHECK(launch_mlstm_scan(a, f32, cur_stream()) == 0,
              "mlstm_scan: unsupported dim ", a.dim);
}

MinGruArgs mingru_args(const torch::Tensor& out, const torch::Tensor& proj,
                       const torch::Tensor& bias, const torch::Tensor& state,
                       const torch::Tensor& seg, int f32) {
  const Rows r = rows_of(proj, f32, "proj");
  MinGruArgs a{};
  TORCH_CHECK(state.dim() == 2 && r.cols == 3 * state.size(1) &&
                  out.numel() == (int64_t)r.n * state.size(1),
              "mingru: proj must be [n, 3 * width], state [slots, width]");
  a.width = (int)state.size(1);
  a.out = out.data_ptr();
  a.proj = r.p;
  a.ld = r.ld;
  a.bias = f32_ptr(bias, 2 * a.width, "bias");
  a.state = const_cast<float*>(f32_ptr(state, state.numel(), "state"));
  a.seg = seg_view(seg);
  return a;
}

void mingru_step(torch::Tensor out, torch::Tensor proj, torch::Tensor bias,
                 torch::Tensor state, torch::Tensor seg) {
  const int f32 = act_type(out, "out");
  launch_mingru_step(mingru_args(out, proj, bias, state, seg, f32), f32,
                     cur_stream());
}

void mingru_scan(torch::Tensor out, torch::Tensor proj, torch::Tensor bias,
                 torch::Tensor state, torch::Tensor seg, int64_t max_len) {
  const int f32 = act_type(out, "out");
  MinGruArgs a = mingru_args(out, proj, bias, state, seg, f32);
  TORCH_CHECK(max_len > 0 && max_len <= proj.size(0), "max_len");
  a.max_len = (int)max_len;
  launch_mingru_scan(a, f32, cur_stream());
}

void mamba2_out(torch::Tensor out, torch::Tensor o, torch::Tensor xbc,
                torch::Tensor z, torch::Tensor skip, torch::Tensor w,
                int64_t groups, double eps) {
  const int f32 = act_type(out, "out");
  const Rows x = rows_of(xbc, f32, "xbc"), zr = rows_of(z, f32, "z");
  GatedNormArgs a{};
  a.n = zr.n;
  a.inner = zr.cols;
  const int heads = (int)skip.numel();
  TORCH_CHECK(x.n == a.n && x.cols >= a.inner && heads > 0 &&
                  a.inner % heads == 0 && groups > 0 &&
                  a.inner % groups == 0 &&
                  out.numel() == (int64_t)a.n * a.inner,
              "mamba2_out: sizes");
  a.vdim = a.inner / heads;
  a.groups = (int)groups;
  a.out = out.data_ptr();
  a.o = f32_ptr(o, (int64_t)a.n * a.inner, "o");
  a.x = x.p;
  a.z = zr.p;
  a.xld = x.ld;
  a.zld = zr.ld;
  a.skip = f32_ptr(skip, heads, "skip");
  a.w = f32_ptr(w, a.inner, "w");
  a.eps = (float)eps;
  const size_t bytes = f32 ? 16 : 8;
  a.vec = x.ld % 4 == 0 && zr.ld % 4 == 0 && (size_t)x.p % bytes == 0 &&
          (size_t)zr.p % bytes == 0;
  TORCH_CHECK(launch_gated_norm(a, f32, cur_stream()) == 0,
              "mamba2_out: row of ", a.inner, " elements");
}

void advance_batch(torch::Tensor slots, torch::Tensor sampled,
                   torch::Tensor pos, torch::Tensor tokens, int64_t spare) {
  const int n = (int)slots.numel();
  launch_advance_batch(i32_ptr(slots, n, "slots"),
                       i32_ptr(sampled, n, "sampled"),
                       const_cast<int*>(i32_ptr(pos, n, "pos")),
                       const_cast<int*>(i32_ptr(tokens, n, "tokens")),
                       (int)spare, n, cur_stream());
}

}  // namespace

void bind_hybrid(py::module_& m) {
  const auto none = c10::nullopt;
  m.def("residual_norm", &residual_norm,
        "float residual step (embed / add / post-norm add) + next norm",
        py::arg("x"), py::arg("y") = none, py::arg("post_w") = none,
        py::arg("xn") = none, py::arg("next_w") = none,
        py::arg("tokens") = none, py::arg("table") = none,
        py::arg("scale") = 1.0, py::arg("offset") = 0.0,
        py::arg("eps") = 1e-6, py::arg("mult") = 1.0,
        py::arg("pos_table") = none, py::arg("row_pos") = none,
        py::arg("routed") = none, py::arg("routed_w") = none,
        py::arg("gain") = none, py::arg("y2") = none,
        py::arg("post_w2") = none);
  m.def("relu2", &relu2, "in-place squared ReLU", py::arg("z"));
  m.def("xielu", &xielu, "in-place xIELU", py::arg("z"), py::arg("p"),
        py::arg("q"));
  m.def("gelu", &gelu, "in-place exact GELU", py::arg("z"));
  m.def("stream_step", &stream_step,
        "float residual step of blocks with output norms: embed / grouped "
        "norm + add of a sublayer and routed rows, average over depth, next "
        "operand",
        py::arg("x"), py::arg("y") = none, py::arg("post_w") = none,
        py::arg("xn") = none, py::arg("next_w") = none,
        py::arg("groups") = 1, py::arg("eps") = 1e-6,
        py::arg("tokens") = none, py::arg("table") = none,
        py::arg("scale") = 1.0, py::arg("routed") = none,
        py::arg("routed_w") = none, py::arg("chosen") = none,
        py::arg("experts") = 0, py::arg("hist") = none,
        py::arg("coef") = none, py::arg("keep") = none,
        py::arg("past") = none,
        py::arg("shift") = none, py::arg("prev") = none,
        py::arg("row_slot") = none, py::arg("row_pos") = none);
  m.def("token_shift", &token_shift, "mix with the row before",
        py::arg("xn"), py::arg("x"), py::arg("shift"), py::arg("prev"),
        py::arg("seg"), py::arg("max_len"));
  m.def("causal_conv", &causal_conv, "causal convolution per channel",
        py::arg("out"), py::arg("x"), py::arg("w"), py::arg("bias"),
        py::arg("in_bias"), py::arg("state"), py::arg("seg"),
        py::arg("max_len"), py::arg("act"));
  m.def("rglru_step", &rglru_step,
        "RG-LRU gates + recurrence + second branch, one token per segment",
        py::arg("out"), py::arg("u"), py::arg("y"), py::arg("y_bias"),
        py::arg("gates"), py::arg("gate_bias"), py::arg("rate"),
        py::arg("state"), py::arg("seg"));
  m.def("rglru_scan", &rglru_scan, "RG-LRU over token segments",
        py::arg("out"), py::arg("u"), py::arg("y"), py::arg("y_bias"),
        py::arg("gates"), py::arg("gate_bias"), py::arg("rate"),
        py::arg("state"), py::arg("seg"), py::arg("max_len"));
  m.def("mamba2_step", &mamba2_step,
        "Mamba-2 state update + read-out, one token per segment",
        py::arg("o"), py::arg("xbc"), py::arg("dt"), py::arg("state"),
        py::arg("dt_bias"), py::arg("rate"), py::arg("vdim"),
        py::arg("seg"));
  m.def("mamba2_scan", &mamba2_scan, "Mamba-2 over token segments",
        py::arg("o"), py::arg("xbc"), py::arg("dt"), py::arg("state"),
        py::arg("dt_bias"), py::arg("rate"), py::arg("vdim"), py::arg("seg"),
        py::arg("max_len"));
  m.def("mamba2_out", &mamba2_out, "skip + gate + grouped norm of the "
        "read-out", py::arg("out"), py::arg("o"), py::arg("xbc"),
        py::arg("z"), py::arg("skip"), py::arg("w"), py::arg("groups"),
        py::arg("eps"));
  m.def("mlstm_step", &mlstm_step,
        "mLSTM gates + state update + normalised, gated read-out, one token "
        "per segment",
        py::arg("out"), py::arg("proj"), py::arg("state"), py::arg("peak"),
        py::arg("gate_bias"), py::arg("norm_w"), py::arg("cap"),
        py::arg("q_scale"), py::arg("eps"), py::arg("seg"));
  m.def("mlstm_scan", &mlstm_scan, "mLSTM over token segments",
        py::arg("out"), py::arg("proj"), py::arg("state"), py::arg("peak"),
        py::arg("gate_bias"), py::arg("norm_w"), py::arg("cap"),
        py::arg("q_scale"), py::arg("eps"), py::arg("seg"),
        py::arg("max_len"));
  m.def("mingru_step", &mingru_step,
        "minGRU gates + recurrence + output gate, one token per segment",
        py::arg("out"), py::arg("proj"), py::arg("bias"), py::arg("state"),
        py::arg("seg"));
  m.def("mingru_scan", &mingru_scan, "minGRU over token segments",
        py::arg("out"), py::arg("proj"), py::arg("bias"), py::arg("state"),
        py::arg("seg"), py::arg("max_len"));
  m.def("hgrn2_step", &hgrn2_step,
        "HGRN2 gates + state update + read-out + head norm, one token per "
        "segment",
        py::arg("out"), py::arg("proj"), py::arg("state"),
        py::arg("f_bias"), py::arg("lower"), py::arg("norm_w"),
        py::arg("seg"), py::arg("eps"));
  m.def("hgrn2_scan", &hgrn2_scan, "HGRN2 over token segments",
        py::arg("out"), py::arg("proj"), py::arg("state"), py::arg("f_bias"), py::arg("lower"), py::arg("norm_w"),
        py::arg("seg"), py::arg("max_len"), py::arg("eps"));
  m.def("qk_norm_append", &qk_norm_append,
        "per-head q/k RMS norms + paged cache append", py::arg("q_out"),
        py::arg("kpages"), py::arg("vpages"), py::arg("proj"),
        py::arg("q_w"), py::arg("k_w"), py::arg("row_slot"),
        py::arg("row_pos"), py::arg("table"), py::arg("vdim"),
        py::arg("eps"), py::arg("rope") = none);
  m.def("row_norm_append", &row_norm_append,
        "q/k RMS norms over whole rows, query scale by position, values of "
        "unit size + paged cache append",
        py::arg("q_out"), py::arg("kpages"), py::arg("vpages"),
        py::arg("proj"), py::arg("q_w"), py::arg("k_w"), py::arg("row_slot"),
        py::arg("row_pos"), py::arg("table"), py::arg("vdim"), py::arg("eps"),
        py::arg("q_scale") = none, py::arg("unit_values") = true);
  m.def("kv_rows", &kv_rows, "cached keys and values <-> flat rows",
        py::arg("rows"), py::arg("kpages"), py::arg("vpages"),
        py::arg("row_slot"), py::arg("row_pos"), py::arg("table"),
        py::arg("dim"), py::arg("vdim"), py::arg("store"));
  m.def("paged_attn", &paged_attn,
        "paged attention: distance bias or slopes, sliding window, kept "
        "first tokens, capped scores, sink, output gate, one map or the "
        "difference of two",
        py::arg("out"), py::arg("q"), py::arg("kpages"), py::arg("vpages"),
        py::arg("bias"), py::arg("table"), py::arg("seg"),
        py::arg("max_len"), py::arg("window"), py::arg("keep_first"),
        py::arg("scale"), py::arg("splits"), py::arg("part_o") = none,
        py::arg("part_ml") = none, py::arg("softcap") = 0.0,
        py::arg("map_weight") = 0.0, py::arg("out_scale") = 1.0,
        py::arg("eps") = 0.0, py::arg("slopes") = none,
        py::arg("sink") = none, py::arg("gate") = none);
  m.def("latent_norm_append", &latent_norm_append,
        "norms of the query and key/value latents + paged cache append, and "
        "a gated activation in the same launch",
        py::arg("pages"), py::arg("kv"), py::arg("kv_w"),
        py::arg("row_slot"), py::arg("row_pos"), py::arg("table"),
        py::arg("eps"), py::arg("q_out") = none, py::arg("q") = none,
        py::arg("q_w") = none, py::arg("act_out") = none,
        py::arg("gate") = none, py::arg("up") = none, py::arg("act") = 0);
  m.def("latent_gather", &latent_gather, "cached latents as flat rows",
        py::arg("out"), py::arg("pages"), py::arg("table"), py::arg("seg"),
        py::arg("max_len"));
  m.def("gated_act", &gated_act, "act(gate) * up", py::arg("out"),
        py::arg("gate"), py::arg("up"), py::arg("act"));
  m.def("head_proj", &head_proj, "per-head product of a few rows",
        py::arg("out"), py::arg("x"), py::arg("w"), py::arg("x_rows") = none,
        py::arg("out_rows") = none, py::arg("gate") = none,
        py::arg("part_o") = none, py::arg("part_ml") = none);
  m.def("latent_attn", &latent_attn,
        "windowed attention of all heads over paged latents",
        py::arg("out"), py::arg("q"), py::arg("pages"), py::arg("table"),
        py::arg("seg"), py::arg("max_len"), py::arg("window"),
        py::arg("scale"), py::arg("splits"), py::arg("part_o") = none,
        py::arg("part_ml") = none);
  m.def("head_attn", &head_attn,
        "windowed attention per head over flat key/value rows, head gates",
        py::arg("out"), py::arg("q"), py::arg("kv"), py::arg("seg"),
        py::arg("ctx_seg"), py::arg("max_len"), py::arg("heads"),
        py::arg("dim"), py::arg("vdim"), py::arg("window"), py::arg("scale"),
        py::arg("gate") = none);
  m.def("moe_route", &moe_route,
        "float router, top experts, pairs ordered by expert",
        py::arg("weight"), py::arg("x"), py::arg("router"), py::arg("top"),
        py::arg("tile_rows") = 16, py::arg("correction") = none,
        py::arg("scale") = 1.0, py::arg("identity") = 0,
        py::arg("gated") = false);
  m.def("moe_up", &moe_up, "experts' gate and up products + activation",
        py::arg("mid"), py::arg("x"), py::arg("w"), py::arg("plan"),
        py::arg("act"), py::arg("tile_rows") = 16);
  m.def("moe_down", &moe_down, "experts' down products", py::arg("out"),
        py::arg("mid"), py::arg("w"), py::arg("plan"),
        py::arg("tile_rows") = 16);
  m.def("skinny_gemm", &skinny_gemm, "projection of up to 32 rows",
        py::arg("out"), py::arg("w"), py::arg("x"), py::arg("act") = 0,
        py::arg("act_p") = 0.0, py::arg("act_q") = 0.0);
  m.def("advance_batch", &advance_batch, "decode bookkeeping");
}
