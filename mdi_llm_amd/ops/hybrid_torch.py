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
           "gated_act", "moe_route", "moe_up", "moe_down", "advance_batch",
           "stream_step", "token_shift", "gelu", "causal_conv", "rglru_step",
           "rglru_scan", "mamba2_step", "mamba2_scan", "mamba2_out",
           "kv_rows", "row_norm_append", "relu2", "mlstm_step", "mlstm_scan",
           "mingru_step", "mingru_scan"]


def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def residual_norm(x, y=None, post_w=None, xn=None, next_w=None, tokens=None,
                  table=None, scale=1.0, offset=0.0, eps=1e-6, mult=1.0,
                  pos_table=None, row_pos=None, routed=None, routed_w=None,
                  gain=None, y2=None, post_w2=None) -> None:
    if tokens is not None:
        x.copy_(table[tokens.long()].float() * scale)
        if pos_table is not None:
            x += pos_table[row_pos.long()].float()
    elif y is not None:
        a = y.float() if post_w is None else _rms(y, eps) * (offset + post_w)
        if gain is not None:
            a = a * gain
        if y2 is not None:
            a = a + _rms(y2, eps) * (offset + post_w2)
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


def _rotate(x, rope, pos):
    """x [n, heads, D]: pairs of neighbours among the first rope dims."""
    if rope is None:
        return x
    c, s = rope[pos].unbind(-1)
    c, s = c.unsqueeze(1), s.unsqueeze(1)
    n = 2 * c.size(-1)
    u, v = x[..., :n:2], x[..., 1:n:2]
    r = torch.stack((u * c - v * s, v * c + u * s), -1).flatten(-2)
    return torch.cat((r, x[..., n:]), -1)


def qk_norm_append(q_out, kpages, vpages, proj, q_w, k_w, row_slot, row_pos,
                   table, vdim, eps, rope=None) -> None:
    n, H, dpad = q_out.shape
    D = q_w.numel()
    pos = row_pos.long()
    q = _rotate(_rms(proj[:, :H * D].reshape(n, H, D), eps) * q_w, rope, pos)
    q_out.zero_()
    q_out[..., :D] = q.to(q_out.dtype)
    if kpages is None:
        return
    G, GV = kpages.size(1), vpages.size(1)
    _, k, v = proj.split((H * D, G * D, GV * vdim), dim=1)
    k = _rotate(_rms(k.reshape(n, G, D), eps) * k_w, rope, pos)
    kv_rows(torch.cat((k.to(proj.dtype).flatten(1), v), 1), kpages, vpages,
            row_slot, row_pos, table, D, vdim, True)


def kv_rows(rows, kpages, vpages, row_slot, row_pos, table, dim, vdim,
            store) -> None:
    n, G, GV = rows.size(0), kpages.size(1), vpages.size(1)
    pos = row_pos.long()
    page = table[row_slot.long(), pos // PAGE].long().view(n, 1, 1)
    at = 0
    for pages, heads, size, index in (
            (kpages, G, dim, k_index(kpages.size(2) // PAGE)),
            (vpages, GV, vdim, v_index(vpages.size(2) // PAGE))):
        cols = rows[:, at:at + heads * size].view(n, heads, size)
        at += heads * size
        where = (page, torch.arange(heads).view(1, -1, 1),
                 index[pos % PAGE, :size].view(n, 1, size))
        if store:
            pages[where] = cols
        else:
            cols.copy_(pages[where])


def row_norm_append(q_out, kpages, vpages, proj, q_w, k_w, row_slot, row_pos,
                    table, vdim, eps, q_scale=None, unit_values=True) -> None:
    n, H, _ = q_out.shape
    G, D = kpages.size(1), q_w.numel() // H
    pos = row_pos.long()
    q, k, v = proj.split((H * D, G * D, G * vdim), dim=1)
    q = _rms(q, eps) * q_w
    if q_scale is not None:
        q = q * q_scale[pos].unsqueeze(1)
    q_out.zero_()
    q_out[..., :D] = q.view(n, H, D).to(q_out.dtype)
    k = _rms(k, eps) * k_w
    if unit_values:
        v = _rms(v.reshape(n, G, vdim), eps).flatten(1)
    kv_rows(torch.cat((k, v), 1).to(proj.dtype), kpages, vpages, row_slot,
            row_pos, table, D, vdim, True)


def paged_attn(out, q, kpages, vpages, bias, table, seg, max_len, window,
               keep_first, scale, splits, part_o=None, part_ml=None,
               softcap=0.0, map_weight=0.0, out_scale=1.0, eps=0.0,
               slopes=None, sink=None, gate=None) -> None:
    """Two key heads per value head: each query head has two maps, and what
    is stored is the unit-size difference of their outputs."""
    D = q.size(2)
    GV = vpages.size(1)
    maps = kpages.size(1) // GV
    H = q.size(1) // maps
    E = out.size(1) // H
    ki, vi = k_index(D), v_index(vpages.size(2) // PAGE)[:, :E]
    for start, n, slot, pos0 in _segments(seg):
        total = pos0 + n
        pages = table[slot, : -(-total // PAGE)].long()
        k, v = (t[pages][:, :, at].transpose(0, 1).flatten(1, 2)[:, :total]
                for t, at in ((kpages, ki), (vpages, vi)))
        k = k.float().view(GV, maps, total, D).repeat_interleave(H // GV, 0)
        v = v.float().repeat_interleave(H // GV, 0).unsqueeze(1)
        i = torch.arange(pos0, total).view(-1, 1)
        j = torch.arange(total).view(1, -1)
        d = i - j
        ok = (d >= 0) & ((d < window) | (j < keep_first))
        rows = q[start:start + n].float().view(n, H, maps, D)
        s = rows.permute(1, 2, 0, 3) @ k.transpose(2, 3) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        # bias table and slopes are in log2 units (see the HIP kernel)
        b = bias[:, d.clamp(0, bias.size(1) - 1)] if slopes is None \
            else -slopes.view(-1, 1, 1) * d
        s = s + b.unsqueeze(1) * 0.6931471805599453
        s = s.masked_fill(~ok, float("-inf"))
        if sink is None:
            p = s.softmax(-1)
        else:
            extra = sink.view(-1, 1, 1, 1).expand(-1, maps, n, 1)
            p = torch.cat((s, extra), -1).softmax(-1)[..., :-1]
        o = p @ v                                       # [H, maps, n, E]
        if maps == 2:
            o = _rms(o[:, 0] - map_weight * o[:, 1], eps) * out_scale
        else:
            o = o[:, 0]
        o = o.transpose(0, 1).reshape(n, -1)
        if gate is not None:
            o = o * torch.sigmoid(gate[start:start + n].float())
        out[start:start + n] = o.to(out.dtype)


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


def moe_route(weight, x, router, top, tile_rows=16, correction=None,
              scale=1.0, identity=0, gated=False):
    """Fills the weights [n, top]; returns the plan of the expert products
    (here: the chosen outputs [n, top])."""
    z = x.float() @ router.float().t()
    if gated:
        weight[:, top] = torch.sigmoid(z[:, -1])
        z = z[:, :-1]
    if correction is None:
        z, experts = z.topk(top, -1)
        weight.copy_(z.softmax(-1))
        return experts
    s = z.softmax(-1)
    experts = (s + correction).topk(top, -1).indices
    s = s.gather(1, experts)
    weight[:, :top] = s / (s.sum(-1, keepdim=True) + 1e-20) * scale
    return experts


def moe_up(out, x, w, plan, act, tile_rows=16) -> None:
    n, top = plan.shape
    for t in range(n):
        for k in range(top):
            if plan[t, k] < w.size(0):
                gate, up = (w[plan[t, k]].float() @ x[t].float()).chunk(2)
                out[t * top + k] = (_act(gate, act) * up).to(out.dtype)


def moe_down(out, mid, w, plan, tile_rows=16) -> None:
    n, top = plan.shape
    for t in range(n):
        for k in range(top):
            if plan[t, k] < w.size(0):
                out[t, k] = (w[plan[t, k]].float()
                             @ mid[t * top + k].float()).to(out.dtype)


def advance_batch(slots, sampled, pos, tokens, spare) -> None:
    live = slots != spare
    tokens[live] = sampled[live]
    pos[live] += 1


def _group_rms(x, groups, eps):
    return _rms(x.reshape(x.size(0), groups, -1), eps).flatten(1)


def stream_step(x, y=None, post_w=None, xn=None, next_w=None, groups=1,
                eps=1e-6, tokens=None, table=None, scale=1.0, routed=None,
                routed_w=None, chosen=None, experts=0, hist=None, coef=None,
                keep=None, past=None, shift=None, prev=None, row_slot=None,
                row_pos=None) -> None:
    if tokens is not None:
        x.copy_(table[tokens.long()].float() * scale)
    elif y is not None or routed is not None:
        a = torch.zeros_like(x) if y is None else y.float()
        if routed is not None:
            n, top, _ = routed.shape
            if y is not None:
                a = a * routed_w[:, top:]
            same = chosen.reshape(-1)[:n * top].view(n, top, 1) >= experts
            rows = torch.where(same, x.unsqueeze(1), routed.float())
            a = a + (rows * routed_w[:, :top].unsqueeze(-1)).sum(1)
        if post_w is not None:
            a = _group_rms(a, groups, eps) * post_w
        x += a
    if keep is not None:
        keep.copy_(x)
    if past is not None:
        past.copy_((hist * coef[:-1].view(-1, 1, 1)).sum(0))
    elif coef is not None:
        x.copy_((hist * coef[:-1].view(-1, 1, 1)).sum(0) + coef[-1] * x)
    if xn is None:
        return
    if next_w is not None:
        xn.copy_(_group_rms(x, groups, eps) * next_w)
    elif shift is not None:
        slot = row_slot.long()
        before = torch.where(row_pos.view(-1, 1) > 0, prev[slot], 0.0)
        xn.copy_(x + (before - x) * shift)
        prev[slot] = x
    else:
        xn.copy_(x)


def token_shift(xn, x, shift, prev, seg, max_len) -> None:
    for start, n, slot, pos0 in _segments(seg):
        h = x[start:start + n]
        first = prev[slot] if pos0 else torch.zeros_like(prev[slot])
        before = torch.cat((first.unsqueeze(0), h[:-1]))
        xn[start:start + n] = (h + (before - h) * shift).to(xn.dtype)
        prev[slot] = h[-1]


def gelu(z) -> None:
    z.copy_(torch.nn.functional.gelu(z.float()))


def relu2(z) -> None:
    z.copy_(z.float().clamp(min=0.0).square())


def causal_conv(out, x, w, bias, in_bias, state, seg, max_len, act) -> None:
    back = w.size(0) - 1
    for start, n, slot, pos0 in _segments(seg):
        raw = torch.cat((state[slot][:back], x[start:start + n]))
        rows = raw.float()
        if in_bias is not None:
            rows = rows + in_bias
        rows[:max(0, back - pos0)] = 0.0    # before the sequence's start
        y = bias + sum(w[k] * rows[k:k + n] for k in range(back + 1))
        if act:
            y = torch.nn.functional.silu(y)
        out[start:start + n] = y.to(out.dtype)
        if back:
            state[slot] = raw[-back:]


def rglru_scan(out, u, y, y_bias, gates, gate_bias, rate, state, seg,
               max_len) -> None:
    B = gates.size(0) // 2
    z = torch.einsum("nbk,gbmk->gnbm", u.float().unflatten(1, (B, -1)),
                     gates.float().unflatten(0, (2, B)))
    z = z + gate_bias.view(2, 1, B, -1)
    r, i = torch.sigmoid(z).flatten(2)
    log_a = rate * r
    a, x = log_a.exp(), (-(2 * log_a).expm1()).sqrt() * i * u.float()
    g = _act(y.float() + y_bias, 1)
    for start, n, slot, pos0 in _segments(seg):
        S = state[slot].clone() if pos0 else torch.zeros_like(state[slot])
        for t in range(start, start + n):
            S = a[t] * S + x[t]
            out[t] = (S * g[t]).to(out.dtype)
        state[slot] = S


def rglru_step(out, u, y, y_bias, gates, gate_bias, rate, state, seg) -> None:
    rglru_scan(out, u, y, y_bias, gates, gate_bias, rate, state, seg, 1)


def mamba2_scan(o, xbc, dt, state, dt_bias, rate, vdim, seg, max_len) -> None:
    _, H, N, _ = state.shape
    inner = H * vdim
    G = (xbc.size(1) - inner) // (2 * N)
    x, B, C = xbc.float().split((inner, G * N, G * N), 1)
    B, C = (t.reshape(-1, G, N).repeat_interleave(H // G, 1) for t in (B, C))
    dt = torch.nn.functional.softplus(dt.float() + dt_bias)
    decay = (rate * dt).exp()
    for start, n, slot, pos0 in _segments(seg):
        S = state[slot] if pos0 else torch.zeros_like(state[slot])
        for t in range(start, start + n):
            S = decay[t].view(H, 1, 1) * S
            S[..., :vdim] += (dt[t].view(H, 1) * B[t]).unsqueeze(-1) \
                * x[t].view(H, 1, vdim)
            o[t] = (S[..., :vdim] * C[t].unsqueeze(-1)).sum(1).view(-1)
        state[slot] = S


def mamba2_step(o, xbc, dt, state, dt_bias, rate, vdim, seg) -> None:
    mamba2_scan(o, xbc, dt, state, dt_bias, rate, vdim, seg, 1)


def mamba2_out(out, o, xbc, z, skip, w, groups, eps) -> None:
    n, inner = o.shape
    y = o + (xbc[:, :inner].float().view(n, skip.numel(), -1)
             * skip.view(1, -1, 1)).view(n, inner)
    out.copy_(_group_rms(y * _act(z.float(), 0), groups, eps) * w)


def mlstm_scan(out, proj, state, peak, gate_bias, norm_w, cap, q_scale, eps,
               seg, max_len) -> None:
    """The normaliser is the state's column behind the values."""
    _, H, D, _ = state.shape
    E = norm_w.numel() // H
    q, k, v, g, gates = proj.float().split(
        (H * D, H * D, H * E, H * E, 2 * H), 1)
    i, f = (cap * torch.tanh((gates + gate_bias) / cap)).split(H, 1)
    f = torch.nn.functional.logsigmoid(f)
    q = (q * q_scale).view(-1, H, D, 1)
    v = torch.cat((v.view(-1, H, E), torch.ones(len(v), H, 1)), -1)
    for start, n, slot, pos0 in _segments(seg):
        S, m = state[slot], peak[slot]
        if pos0 == 0:
            S, m = torch.zeros_like(S), torch.zeros_like(m)
        for t in range(start, start + n):
            new = torch.maximum(f[t] + m, i[t])
            S = torch.exp(f[t] + m - new).view(H, 1, 1) * S
            S[..., :E + 1] += torch.exp(i[t] - new).view(H, 1, 1) \
                * k[t].view(H, D, 1) * v[t].view(H, 1, E + 1)
            m = new
            r = (S[..., :E + 1] * q[t]).sum(1)
            size = torch.maximum(r[:, E:].abs(), torch.exp(-m).view(H, 1))
            r = _rms(r[:, :E] / (size + 1e-6), eps).view(-1) * norm_w
            out[t] = (r * torch.sigmoid(g[t])).to(out.dtype)
        state[slot], peak[slot] = S, m


def mlstm_step(*args) -> None:
    mlstm_scan(*args, 1)


def mingru_scan(out, proj, bias, state, seg, max_len) -> None:
    W = state.size(1)
    z, u, g = proj.float().split(W, 1)
    z = torch.sigmoid(z + bias[:W])
    u = u + bias[W:]
    c = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    g = torch.nn.functional.silu(g)
    for start, n, slot, pos0 in _segments(seg):
        S = state[slot].clone() if pos0 else torch.zeros_like(state[slot])
        for t in range(start, start + n):
            S = (1.0 - z[t]) * S + z[t] * c[t]
            out[t] = (S * g[t]).to(out.dtype)
        state[slot] = S


def mingru_step(out, proj, bias, state, seg) -> None:
    mingru_scan(out, proj, bias, state, seg, 1)
