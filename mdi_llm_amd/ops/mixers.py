"""Recurrent mixers with a short convolution (``HybridEngine`` dispatches to
them): the operands of each kind and its step over a ragged batch."""

from __future__ import annotations

import torch
import torch.nn.functional as F

__all__ = ["RGLRU", "Mamba2"]


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
