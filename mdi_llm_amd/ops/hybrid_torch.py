"""The hybrid-stack operations in plain torch, for hosts without a GPU.

Same names, arguments and in-place behaviour as the HIP extension, over the
same cache layout, so that the engine, the cache, the scheduler and the ring
can be exercised on a CPU host.  On a GPU the engine never uses this module.
"""

from __future__ import annotations

import torch

from ..models.cache import PAGE, k_index, v_index

__all__ = ["residual_norm", "xielu", "hgrn2_step", "hgrn2_scan",
           "qk_norm_append", "paged_attn", "advance_batch"]


def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def residual_norm(x, y=None, post_w=None, xn=None, next_w=None, tokens=None,
                  table=None, scale=1.0, offset=0.0, eps=1e-6) -> None:
    if tokens is not None:
        x.copy_(table[tokens.long()].float() * scale)
    elif y is not None:
        x += y.float() if post_w is None else _rms(y, eps) * (offset + post_w)
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


def advance_batch(slots, sampled, pos, tokens, spare) -> None:
    live = slots != spare
    tokens[live] = sampled[live]
    pos[live] += 1
