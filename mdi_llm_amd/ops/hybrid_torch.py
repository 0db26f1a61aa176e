"""The hybrid-stack operations in plain torch, for hosts without a GPU.

Same names, arguments and in-place behaviour as the HIP extension, over the
same cache layout, so that the engine, the cache, the scheduler and the ring
can be exercised on a CPU host.  On a GPU the engine never uses this module.
"""

from __future__ import annotations

import torch

from ..models.cache import PAGE, k_index, v_index

__all__ = ["residual_norm", "xielu", "hgrn2_step", "hgrn2_scan",
           "qk_norm_append", "paged_attn", "latent_norm_append",
           "latent_gather", "head_proj", "latent_attn", "head_attn",
           "gated_act", "moe_route", "moe_up", "moe_down", "advance_batch"]


def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def residual_norm(x, y=None, post_w=None, xn=None, next_w=None, tokens=None,
                  table=None, scale=1.0, offset=0.0, eps=1e-6, mult=1.0,
                  pos_table=None, row_pos=None, routed=None,
                  routed_w=None) -> None:
    if tokens is not None:
        x.copy_(table[tokens.long()].float() * scale)
        if pos_table is not None:
            x += pos_table[row_pos.long()].float()
    elif y is not None:
        a = y.float() if post_w is None else _rms(y, eps) * (offset + post_w)
        if routed is not None:
            a = a + (routed.float() * routed_w.unsqueeze(-1)).sum(1)
        x += a * mult
    if next_w is not None:
        xn.copy_(_rms(x, eps) * (offset + next_w))


def xielu(z, p, q) -> None:
    f = z.float()
    neg = f.clamp(max=0.0)
    z.copy_(torch.where(f > 0, p * f * f, (0.5 + q) * (neg.expm1() - neg))
            + 0.5 * f)


def _segments(seg):
    return seg.t().tolist()  # rows of (start, len, slot, pos0)


def hgrn2_scan(out, proj, state, f_bias, lower, norm_w, seg, max_len, eps) -> None:
    _, H, D, _ = state.shape
    E = norm_w.numel()
    q, f, v = proj.float().split((H * D, H * D, H * E), dim=1)
    q = torch.nn.functional.silu(q)
    f = lower + (1.0 - lower) * torch.sigmoid(f + f_bias)
    for start, n, slot, pos0 in _segments(seg):
        S = torch.zeros_like(state[slot]) if pos0 == 0 else state[slot]
        for t in range(start, start + n):
            ft = f[t].view(H, D, 1)
            S = ft * S
            S[..., :E] += (1.0 - ft) * v[t].view(H, 1, E)
            r = (S[..., :E] * q[t].view(H, D, 1)).sum(1)
            out[t] = (_rms(r, eps) * norm_w).view(-1).to(out.dtype)
        state[slot] = S


def hgrn2_step(out, proj, state, f_bias, lower, norm_w, seg, eps) -> None:
    hgrn2_scan(out, proj, state, f_bias, lower, norm_w, seg, 1, eps)


def qk_norm_append(q_out, kpages, vpages, proj, q_w, k_w, row_slot, row_pos,
                   table, vdim, eps) -> None:
    n, H, dpad = q_out.shape
    G = kpages.size(1)
    D = q_w.numel()
    q, k, v = proj.split((H * D, G * D, G * vdim), dim=1)
    q_out.zero_()
    q_out[..., :D] = (_rms(q.reshape(n, H, D), eps) * q_w).to(q_out.dtype)
    pos = row_pos.long()
    page = table[row_slot.long(), pos // PAGE].long().view(n, 1, 1)
    head = torch.arange(G).view(1, G, 1)
    at = k_index(dpad)[pos % PAGE, :D].view(n, 1, D)
    kpages[page, head, at] = (
        _rms(k.reshape(n, G, D), eps) * k_w).to(kpages.dtype)
    at = v_index(vpages.size(2) // PAGE)[pos % PAGE, :vdim].view(n, 1, vdim)
    vpages[page, head, at] = v.reshape(n, G, vdim)


def paged_attn(out, q, kpages, vpages, bias, table, seg, max_len, window,
               keep_first, scale, splits, part_o=None, part_ml=None) -> None:
    _, H, D = q.shape
    G = kpages.size(1)
    E = out.size(1) // H
    ki, vi = k_index(D), v_index(vpages.size(2) // PAGE)[:, :E]
    far = bias.size(1) - 1
    for start, n, slot, pos0 in _segments(seg):
        total = pos0 + n
        pages = table[slot, : -(-total // PAGE)].long()
        k, v = (t[pages][:, :, at].transpose(0, 1).flatten(1, 2)[:, :total]
                for t, at in ((kpages, ki), (vpages, vi)))
        k = k.float().repeat_interleave(H // G, 0)
        v = v.float().repeat_interleave(H // G, 0)
        i = torch.arange(pos0, total).view(-1, 1)
        j = torch.arange(total).view(1, -1)
        d = i - j
        ok = (d >= 0) & ((d < window) | (j < keep_first))
        s = q[start:start + n].float().transpose(0, 1) @ k.transpose(1, 2)
        # the bias table is in log2 units (see the HIP kernel)
        s = s * scale + bias[:, d.clamp(0, far)] * 0.6931471805599453
        p = s.masked_fill(~ok, float("-inf")).softmax(-1)
        out[start:start + n] = (p @ v).transpose(0, 1).reshape(n, -1)


def _rows(pages, table, slot, first, end, n_cols):
    """Cached rows first .. end-1 of a slot."""
    pos = torch.arange(first, end)
    page = table[slot, pos // PAGE].long()
    return pages[page, pos % PAGE, :n_cols]


def latent_norm_append(pages, kv, kv_w, row_slot, row_pos, table, eps,
                       q_out=None, q=None, q_w=None, act_out=None, gate=None,
                       up=None, act=0) -> None:
    if act_out is not None:
        gated_act(act_out, gate, up, act)
    if q is not None:
        q_out.copy_(_rms(q, eps) * q_w)
    if kv is None:
        return
    pos = row_pos.long()
    page = table[row_slot.long(), pos // PAGE].long()
    rows = kv if kv_w is None else _rms(kv, eps) * kv_w
    pages[page, pos % PAGE, :kv.size(1)] = rows.to(pages.dtype)


def latent_gather(out, pages, table, seg, max_len) -> None:
    for start, n, slot, first in _segments(seg):
        out[start:start + n] = _rows(pages, table, slot, first, first + n,
                                     out.size(1))


def head_proj(out, x, w, x_rows=None, out_rows=None, gate=None, part_o=None,
              part_ml=None) -> None:
    H, M, K = w.shape
    if part_o is not None:
        x = _combine(part_o, part_ml)
    if x_rows is not None:
        x = x[x_rows.long()]
    n = x.size(0)
    x = x.reshape(n, H, -1)
    y = torch.einsum("nhk,hmk->nhm", x.float(), w[..., :x.size(2)].float())
    rows = slice(None) if out_rows is None else out_rows.long()
    if gate is not None:
        y = y * torch.sigmoid(gate[rows].float()).unsqueeze(-1)
    out[rows] = y.reshape(n, -1).to(out.dtype)


def _combine(part_o, part_ml):
    m, l = part_ml.unbind(-1)
    e = torch.exp2(m - m.amax(-1, keepdim=True))
    e = e / (e * l).sum(-1, keepdim=True)
    o = torch.where(e.unsqueeze(-1) > 0, part_o * e.unsqueeze(-1), 0.0)
    return o.sum(2).flatten(1)


def _window_attn(q, k, v, pos0, first, window, scale):
    """q [n, H, D] at pos0.., k [t, H, D], v [t, H, E] at first.. ->
    [n, H, E]."""
    i = torch.arange(pos0, pos0 + q.size(0)).view(-1, 1)
    j = torch.arange(first, first + k.size(0)).view(1, -1)
    ok = (j <= i) & (i - j < window)
    s = torch.einsum("nhd,thd->hnt", q.float(), k.float()) * scale
    p = s.masked_fill(~ok, float("-inf")).softmax(-1)
    return torch.einsum("hnt,the->nhe", p, v.float())


def latent_attn(out, q, pages, table, seg, max_len, window, scale, splits,
                part_o=None, part_ml=None) -> None:
    n, H, R = q.shape
    for start, m, slot, pos0 in _segments(seg):
        first = max(0, pos0 - window + 1)
        c = _rows(pages, table, slot, first, pos0 + m, R)
        c = c.unsqueeze(1).expand(-1, H, -1)
        o = _window_attn(q[start:start + m], c, c, pos0, first, window, scale)
        if splits > 1:  # all of it in the first part
            part_ml[start:start + m] = torch.tensor([float("-inf"), 0.0])
            part_ml[start:start + m, :, 0] = torch.tensor([0.0, 1.0])
            part_o[start:start + m, :, 0] = o
        else:
            out[start:start + m] = o.reshape(m, -1).to(out.dtype)


def head_attn(out, q, kv, seg, ctx_seg, max_len, heads, dim, vdim, window,
              scale, gate=None) -> None:
    for (start, n, _, pos0), (at, t, _, first) in zip(_segments(seg),
                                                      _segments(ctx_seg)):
        k, v = kv[at:at + t].split((heads * dim, heads * vdim), 1)
        o = _window_attn(q[start:start + n].view(n, heads, dim),
                         k.reshape(t, heads, dim), v.reshape(t, heads, vdim),
                         pos0, first, window, scale)
        if gate is not None:
            o = o * torch.sigmoid(gate[start:start + n].float()).unsqueeze(-1)
        out[start:start + n] = o.reshape(n, -1).to(out.dtype)


def _act(z, act):
    return torch.nn.functional.gelu(z, approximate="tanh") if act == 1 \
        else torch.nn.functional.silu(z)


def gated_act(out, gate, up, act) -> None:
    out.copy_(_act(gate.float(), act) * up.float())


def moe_route(weight, x, router, top, tile_rows=16):
    """Fills the weights [n, top]; returns the plan of the expert products
    (here: the chosen experts [n, top])."""
    z, experts = (x.float() @ router.float().t()).topk(top, -1)
    weight.copy_(z.softmax(-1))
    return experts


def moe_up(out, x, w, plan, act, tile_rows=16) -> None:
    n, top = plan.shape
    for t in range(n):
        for k in range(top):
            gate, up = (w[plan[t, k]].float() @ x[t].float()).chunk(2)
            out[t * top + k] = (_act(gate, act) * up).to(out.dtype)


def moe_down(out, mid, w, plan, tile_rows=16) -> None:
    n, top = plan.shape
    for t in range(n):
        for k in range(top):
            out[t, k] = (w[plan[t, k]].float()
                         @ mid[t * top + k].float()).to(out.dtype)


def advance_batch(slots, sampled, pos, tokens, spare) -> None:
    live = slots != spare
    tokens[live] = sampled[live]
    pos[live] += 1
