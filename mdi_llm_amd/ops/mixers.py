"""Mixers with operands of their own (``HybridEngine`` dispatches to them):
what each kind needs and its step over a ragged batch."""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F

__all__ = ["RGLRU", "Mamba2", "MLSTM", "GatedAttention", "MinGRU", "Paired",
           "MIXERS"]


def _f32(t: torch.Tensor) -> torch.Tensor:
    return t.detach().float().contiguous()


class _Conv:
    """Causal convolution per channel; the cache holds each slot's last
    inputs as they come out of the projection."""

    def __init__(self, eng, i: int, m, act: bool, in_bias=None) -> None:
        self.eng, self.i, self.act = eng, i, act
        self.weight = _f32(m.conv.t())          # [taps, channels]
        self.bias = _f32(m.conv_bias)
        self.in_bias = in_bias
        if m.taps > 16:
            raise ValueError("convolutions have at most 16 taps")

    def __call__(self, b, x: torch.Tensor) -> torch.Tensor:
        e = self.eng
        out = torch.empty(b.n, self.weight.size(1), dtype=e.dtype,
                          device=e.device)
        e.ops.causal_conv(out, x, self.weight, self.bias, self.in_bias,
                          e.cache.conv[self.i], b.seg, b.max_len, self.act)
        return out


class RGLRU:
    """in_proj, convolution, block-diagonal gates with the recurrence and the
    second branch's activation, proj."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng, self.i, self.m = eng, i, m
        self.in_proj = m.in_proj.weight.detach()
        self.proj = m.proj.weight.detach()
        bias = _f32(m.in_proj.bias)
        self.y_bias = bias[:m.width].contiguous()
        self.conv = _Conv(eng, i, m, False, bias[m.width:].contiguous())
        self.gates = m.gates.detach().contiguous()
        self.gate_bias = _f32(m.gate_bias)
        # log a = rate * r
        self.rate = -8.0 * F.softplus(_f32(m.lam))

    def __call__(self, b, xn: torch.Tensor) -> torch.Tensor:
        e, m, n1 = self.eng, self.m, b.singles
        proj = e._linear(xn, self.in_proj)
        y = proj[:, :m.width]
        u = self.conv(b, proj[:, m.width:])
        out = torch.empty(b.n, m.width, dtype=e.dtype, device=e.device)
        state = e.cache.state[self.i]
        args = (self.y_bias, self.gates, self.gate_bias, self.rate, state)
        if n1:
            e.ops.rglru_step(out, u, y, *args, b.seg[:, :n1])
        if n1 < b.seg.size(1):
            e.ops.rglru_scan(out, u, y, *args, b.seg[:, n1:], b.max_len)
        return e._linear(out, self.proj)


class Mamba2:
    """in_proj, convolution, state update and read-out, gated group norm,
    proj."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng, self.i, self.m = eng, i, m
        if m.dim > 256 or m.vdim > 1024:
            raise ValueError("mamba2: state <= 256 and vdim <= 1024")
        self.in_proj = m.in_proj.weight.detach()
        self.proj = m.proj.weight.detach()
        self.conv = _Conv(eng, i, m, True)
        self.dt_bias = _f32(m.dt_bias)
        self.rate = -_f32(m.a_log).exp()        # log decay = rate * dt
        self.skip, self.norm = _f32(m.skip), _f32(m.norm.weight)

    def __call__(self, b, xn: torch.Tensor) -> torch.Tensor:
        e, m, n1 = self.eng, self.m, b.singles
        proj = e._linear(xn, self.in_proj)
        z = proj[:, :m.inner]
        dt = proj[:, m.inner + m.channels:]
        xbc = self.conv(b, proj[:, m.inner:m.inner + m.channels])
        o = torch.empty(b.n, m.inner, dtype=torch.float32, device=e.device)
        args = (xbc, dt, e.cache.state[self.i], self.dt_bias, self.rate,
                m.vdim)
        if n1:
            e.ops.mamba2_step(o, *args, b.seg[:, :n1])
        if n1 < b.seg.size(1):
            e.ops.mamba2_scan(o, *args, b.seg[:, n1:], b.max_len)
        y = torch.empty(b.n, m.inner, dtype=e.dtype, device=e.device)
        e.ops.mamba2_out(y, o, xbc, z, self.skip, self.norm, m.norm_groups,
                         e.config.norm_eps)
        return e._linear(y, self.proj)


class MLSTM:
    """in_proj, gates with state update and read-out (normalised, gated and
    of unit size per head), proj."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng, self.i, self.m = eng, i, m
        if m.dim > 256 or m.vdim > 1023:
            raise ValueError("mlstm: dim <= 256 and vdim < 1024")
        self.in_proj = m.in_proj.weight.detach()
        self.proj = m.proj.weight.detach()
        self.gate_bias = _f32(m.gate_bias)
        self.norm = _f32(m.norm.weight)

    def __call__(self, b, xn: torch.Tensor) -> torch.Tensor:
        e, m, n1 = self.eng, self.m, b.singles
        proj = e._linear(xn, self.in_proj)
        y = torch.empty(b.n, m.heads * m.vdim, dtype=e.dtype,
                        device=e.device)
        args = (y, proj, e.cache.state[self.i], e.cache.peak[self.i],
                self.gate_bias, self.norm, m.gate_cap, m.dim ** -0.5,
                e.config.norm_eps)
        if n1:
            e.ops.mlstm_step(*args, b.seg[:, :n1])
        if n1 < b.seg.size(1):
            e.ops.mlstm_scan(*args, b.seg[:, n1:], b.max_len)
        return e._linear(y, self.proj)


class GatedAttention:
    """Norms, query scale and cache append; attention with slopes, sinks and
    output gate; proj.  Reads its columns q | k | v | gate of a projection."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng, self.m = eng, m
        self.proj = m.proj.weight.detach()
        self.q_norm, self.k_norm = _f32(m.q_norm.weight), _f32(m.k_norm.weight)
        self.sink = _f32(m.sink)
        # in log2 units, as the scores are
        self.slopes = torch.tensor(
            [2.0 ** (-8.0 * (h + 1) / m.heads) * math.log2(math.e)
             for h in range(m.heads)], device=eng.device)
        t = m.q_temp
        self.q_scale = eng.query_scale_table(t["every"], t["coef"]) \
            if t else None

    def __call__(self, b, proj: torch.Tensor) -> torch.Tensor:
        e, m, c = self.eng, self.m, self.eng.cache
        k, v = c.k[m.source], c.v[m.source]
        q = torch.empty(b.n, m.heads, k.size(2) // 64, dtype=e.dtype,
                        device=e.device)
        at = proj.size(1) - m.inner
        e.ops.row_norm_append(q, k, v, proj[:, :at], self.q_norm, self.k_norm,
                              b.row_slot, b.row_pos, c.table, m.vdim,
                              e.config.norm_eps, self.q_scale)
        y = e.attend(m, b, q, slopes=self.slopes, sink=self.sink,
                     gate=proj[:, at:])
        return e._linear(y, self.proj)


class MinGRU:
    """Recurrence with its output gate, proj.  Reads its columns z | input |
    gate of a projection."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng, self.i = eng, i
        self.proj = m.proj.weight.detach()
        self.bias = _f32(m.bias)

    def __call__(self, b, proj: torch.Tensor) -> torch.Tensor:
        e, n1 = self.eng, b.singles
        y = torch.empty(b.n, proj.size(1) // 3, dtype=e.dtype,
                        device=e.device)
        args = (y, proj, self.bias, e.cache.state[self.i])
        if n1:
            e.ops.mingru_step(*args, b.seg[:, :n1])
        if n1 < b.seg.size(1):
            e.ops.mingru_scan(*args, b.seg[:, n1:], b.max_len)
        return e._linear(y, self.proj)


PARTS = {"gated_attention": GatedAttention, "mingru": MinGRU}


class Paired:
    """One projection for two mixers; returns both outputs."""

    def __init__(self, eng, i: int, m) -> None:
        self.eng = eng
        self.in_proj = m.in_proj.weight.detach()
        self.at = m.left.in_rows
        self.left, self.right = (PARTS[p.kind](eng, i, p) for p in m.parts)

    def __call__(self, b, xn: torch.Tensor):
        proj = self.eng._linear(xn, self.in_proj)
        return self.left(b, proj[:, :self.at]), \
            self.right(b, proj[:, self.at:])


MIXERS = {"rglru": RGLRU, "mamba2": Mamba2, "mlstm": MLSTM, "paired": Paired}
