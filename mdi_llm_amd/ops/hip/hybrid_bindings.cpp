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

void residual_norm(torch::Tensor x, Opt y, Opt post_w, Opt xn, Opt next_w,
                   Opt tokens, Opt table, double scale, double offset,
                   double eps) {
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
  const int rc = launch_residual_norm(
      xp, y ? y->data_ptr() : nullptr,
      post_w ? f32_ptr(*post_w, e, "post_w") : nullptr,
      xn ? xn->data_ptr() : nullptr,
      next_w ? f32_ptr(*next_w, e, "next_w") : nullptr,
      tokens ? i32_ptr(*tokens, n, "tokens") : nullptr,
      table ? table->data_ptr() : nullptr, (float)scale, (float)offset,
      (float)eps, n, e, f32, cur_stream());
  TORCH_CHECK(rc == 0, "residual_norm: row of ", e, " elements");
}

void xielu(torch::Tensor z, double p, double q) {
  const int f32 = act_type(z, "z");
  launch_xielu(z.data_ptr(), (long long)z.numel(), (float)p, (float)q, f32,
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
  int kv_heads, dpad, vpad;
};

Pages pages(const torch::Tensor& k, const torch::Tensor& v, int f32) {
  check_like(k, f32, "kpages");
  check_like(v, f32, "vpages");
  TORCH_CHECK(k.dim() == 3 && v.dim() == 3 && k.size(0) == v.size(0) &&
                  k.size(1) == v.size(1) && k.size(2) % (64 * 32) == 0 &&
                  v.size(2) % (64 * 32) == 0,
              "pages: expected k [P, G, 64 * dpad] and v [P, G, 64 * vpad]");
  return Pages{(int)k.size(1), (int)k.size(2) / 64, (int)v.size(2) / 64};
}

void qk_norm_append(torch::Tensor q_out, torch::Tensor kpages,
                    torch::Tensor vpages, torch::Tensor proj,
                    torch::Tensor q_w, torch::Tensor k_w,
                    torch::Tensor row_slot, torch::Tensor row_pos,
                    torch::Tensor table, int64_t vdim, double eps) {
  const int f32 = act_type(proj, "proj");
  const Pages pg = pages(kpages, vpages, f32);
  check_like(q_out, f32, "q_out");
  const int n = (int)proj.size(0), dim = (int)q_w.numel();
  TORCH_CHECK(q_out.dim() == 3 && q_out.size(0) == n &&
                  q_out.size(2) == pg.dpad && dim <= pg.dpad &&
                  vdim <= pg.vpad,
              "q_out must be [n, H, dpad]");
  const int heads = (int)q_out.size(1);
  TORCH_CHECK(proj.size(1) ==
                  (heads + pg.kv_heads) * dim + pg.kv_heads * vdim,
              "proj columns");
  TORCH_CHECK(table.dim() == 2, "table must be [slots, pages]");
  launch_qk_norm_append(
      q_out.data_ptr(), kpages.data_ptr(), vpages.data_ptr(),
      proj.data_ptr(), f32_ptr(q_w, dim, "q_w"), f32_ptr(k_w, dim, "k_w"),
      i32_ptr(row_slot, n, "row_slot"), i32_ptr(row_pos, n, "row_pos"),
      i32_ptr(table, table.numel(), "table"), (int)table.size(1), n, heads,
      pg.kv_heads, dim, (int)vdim, pg.dpad, pg.vpad, (float)eps, f32,
      cur_stream());
}

void paged_attn(torch::Tensor out, torch::Tensor q, torch::Tensor kpages,
                torch::Tensor vpages, torch::Tensor bias,
                torch::Tensor table, torch::Tensor seg, int64_t max_len,
                int64_t window, int64_t keep_first, double scale,
                int64_t splits, Opt part_o, Opt part_ml) {
  const int f32 = act_type(q, "q");
  const Pages pg = pages(kpages, vpages, f32);
  check_like(out, f32, "out");
  TORCH_CHECK(q.dim() == 3 && q.size(2) == pg.dpad, "q must be [n, H, dpad]");
  PagedAttnArgs a{};
  a.heads = (int)q.size(1);
  a.kv_heads = pg.kv_heads;
  TORCH_CHECK(a.heads % a.kv_heads == 0, "heads per kv head");
  TORCH_CHECK(out.dim() == 2 && out.size(0) == q.size(0) &&
                  out.size(1) % a.heads == 0,
              "out must be [n, H*vdim]");
  a.vdim = (int)out.size(1) / a.heads;
  a.dpad = pg.dpad;
  a.vpad = pg.vpad;
  TORCH_CHECK(a.vdim <= a.vpad, "vdim");
  TORCH_CHECK(bias.dim() == 2 && bias.size(0) == a.heads && bias.size(1) > 0,
              "bias must be [H, n]");
  a.bias = f32_ptr(bias, bias.numel(), "bias");
  a.bias_len = (int)bias.size(1);
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
  if (splits > 1) {
    TORCH_CHECK(max_len == 1, "split keys: one token per segment");
    TORCH_CHECK(part_o && part_ml, "split keys need scratch");
    const int64_t cells = (int64_t)a.seg.n * a.heads * splits;
    TORCH_CHECK(part_o->numel() >= cells * a.vpad &&
                    part_ml->numel() >= cells * 2,
                "split scratch too small");
    a.part_o = const_cast<float*>(
        f32_ptr(*part_o, part_o->numel(), "part_o"));
    a.part_ml = const_cast<float*>(
        f32_ptr(*part_ml, part_ml->numel(), "part_ml"));
  }
  const int rc = f32 ? launch_paged_attn_f32(a, cur_stream())
                     : launch_paged_attn_bf16(a, cur_stream());
  TORCH_CHECK(rc == 0, "paged_attn: unsupported padded sizes ", a.dpad, ", ",
              a.vpad);
}

void skinny_gemm(torch::Tensor out, torch::Tensor w, torch::Tensor x,
                 bool act, double act_p, double act_q) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && out.dim() == 2, "2-D operands");
  const int n = (int)x.size(0), m = (int)w.size(0), k = (int)x.size(1);
  for (const auto* t : {&out, &w, &x})
    TORCH_CHECK(act_type(*t, "operand") == 0, "skinny_gemm: bf16 operands");
  TORCH_CHECK(w.size(1) == k && out.size(0) == n && out.size(1) == m,
              "skinny_gemm: sizes");
  const int rc = launch_skinny_gemm(out.data_ptr(), w.data_ptr(),
                                    x.data_ptr(), n, m, k, act ? 1 : 0,
                                    (float)act_p, (float)act_q, cur_stream());
  TORCH_CHECK(rc == 0, "skinny_gemm: unsupported n ", n, " or k ", k);
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
        py::arg("eps") = 1e-6);
  m.def("xielu", &xielu, "in-place xIELU", py::arg("z"), py::arg("p"),
        py::arg("q"));
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
        py::arg("eps"));
  m.def("paged_attn", &paged_attn,
        "paged attention: distance bias, sliding window, kept first tokens",
        py::arg("out"), py::arg("q"), py::arg("kpages"), py::arg("vpages"),
        py::arg("bias"), py::arg("table"), py::arg("seg"),
        py::arg("max_len"), py::arg("window"), py::arg("keep_first"),
        py::arg("scale"), py::arg("splits"), py::arg("part_o") = none,
        py::arg("part_ml") = none);
  m.def("skinny_gemm", &skinny_gemm, "projection of up to 32 rows",
        py::arg("out"), py::arg("w"), py::arg("x"), py::arg("act") = false,
        py::arg("act_p") = 0.0, py::arg("act_q") = 0.0);
  m.def("advance_batch", &advance_batch, "decode bookkeeping");
}
