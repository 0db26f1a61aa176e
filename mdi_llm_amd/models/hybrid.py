"""Parameters of stacks whose layers differ (``ModelConfig.layers``).

These modules hold weights under the framework's key layout, so loading,
chunking and moving to a device work as for every other model; the layers
are computed by ``ops.hybrid_engine`` only.  Projections that read the same
input are stored stacked (``in_proj``), as the fused QKV of ``model.Block``
is, so that one matrix product serves all of them.  In a parallel block that
is every projection of the block's norm; the projections whose results are
added to the residual stream lie side by side in ``out_proj`` likewise.
"""

from __future__ import annotations

from typing import Dict, Tuple

import torch
import torch.nn as nn

from ..config import ModelConfig

__all__ = ["HybridBlock", "ParallelBlock", "make_block",
           "native_state_dict", "native_tensors"]


class Scale(nn.Module):
    """The weight of a norm; which norm it is, the engine knows."""

    def __init__(self, size: int) -> None:
        super().__init__()
        self.weight = nn.Parameter(torch.zeros(size))


class HGRN2Mixer(nn.Module):
    """Gated linear recurrence: in_proj rows are q | f | v."""

    kind = "hgrn2"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.heads, self.dim, self.vdim = (
            spec["heads"], spec["dim"], spec["vdim"])
        qk = self.heads * self.dim
        self.in_proj = nn.Linear(width, 2 * qk + self.heads * self.vdim,
                                 bias=False)
        self.f_bias = nn.Parameter(torch.zeros(qk))
        self.lower = nn.Parameter(torch.zeros(qk))
        self.norm = Scale(self.vdim)
        self.proj = nn.Linear(self.heads * self.vdim, width, bias=False)


class BiasedAttention(nn.Module):
    """Windowed attention with q/k norms and a distance-bucket bias:
    in_proj rows are q | k | v.  The table's row count is not part of the
    configuration; it follows the loaded tensor."""

    kind = "attention"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.heads, self.kv_heads = spec["heads"], spec["kv_heads"]
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.scale = float(spec["scale"])
        self.bias_max = spec["bias_max"]
        mask = spec.get("mask") or {}
        self.window = int(mask.get("size", 1 << 30))
        self.keep_first = int(mask.get("keep_first", 0))
        self.in_proj = nn.Linear(
            width,
            (self.heads + self.kv_heads) * self.dim
            + self.kv_heads * self.vdim,
            bias=False)
        self.q_norm = Scale(self.dim)
        self.k_norm = Scale(self.dim)
        self.rel = nn.Parameter(torch.zeros(32, self.heads))
        self.proj = nn.Linear(self.heads * self.vdim, width, bias=False)

    def _load_from_state_dict(self, state_dict, prefix, *args, **kwargs):
        t = state_dict.get(prefix + "rel")
        if t is not None and t.dim() == 2 and t.size(1) == self.heads:
            self.rel = nn.Parameter(self.rel.new_zeros(t.shape))
        super()._load_from_state_dict(state_dict, prefix, *args, **kwargs)


class XieluMLP(nn.Module):
    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.fc = nn.Linear(width, spec["ff"], bias=False)
        self.proj = nn.Linear(spec["ff"], width, bias=False)
        self.act = nn.Parameter(torch.zeros(2))


class LatentAttention(nn.Module):
    """Windowed attention over one cached latent row per token, from which
    every head has its keys and values (kv_up rows are k | v); its queries
    pass through a latent of their own.  A layer with ``kv_from`` has no
    latent: it reads that layer's.  Part of a ``ParallelBlock``: in_rows are
    its rows of the block's in_proj, out_cols its columns of out_proj."""

    kind = "latent_attention"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.heads = spec["heads"]
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.q_rank, self.rank = spec["q_rank"], spec["kv_rank"]
        self.scale = float(spec["scale"])
        self.window = int((spec.get("mask") or {}).get("size", 1 << 30))
        src = spec.get("kv_from")
        # model-wide index of the layer whose latent is read
        self.source = index if src is None else src
        self.owns_latent = src is None
        self.q_norm = Scale(self.q_rank)
        self.q_up = nn.Linear(self.q_rank, self.heads * self.dim, bias=False)
        self.kv_up = nn.Linear(
            self.rank, self.heads * (self.dim + self.vdim), bias=False)
        self.in_rows = [("dq", self.q_rank)]
        if self.owns_latent:
            self.kv_norm = Scale(self.rank)
            self.in_rows.append(("dkv", self.rank))
        self.gate_rows = [("g", self.heads)]
        self.out_cols = self.heads * self.vdim


class GatedMLP(nn.Module):
    """Dense gated feed-forward; its weights are in the block's in_proj and
    out_proj."""

    kind = "dense"
    act = "gelu_tanh"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.ff = spec["ff"]
        self.in_rows = [("gate", self.ff), ("up", self.ff)]


class RoutedMLP(nn.Module):
    """Gated experts, ``top`` of them for each token, and a gated shared
    expert, which lies in the block's in_proj and out_proj.  up holds every
    expert's gate rows, then its up rows."""

    kind = "moe"
    act = "silu"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.experts, self.top = (
            spec["router"]["experts"], spec["router"]["top"])
        self.expert_ff = spec["expert"]["ff"]
        self.ff = (spec.get("shared") or {}).get("ff", 0)
        self.in_rows = [("shared.gate", self.ff), ("shared.up", self.ff)] \
            if self.ff else []
        self.router = nn.Linear(width, self.experts, bias=False)
        self.up = nn.Linear(width, self.experts * 2 * self.expert_ff,
                            bias=False)
        self.down = nn.Linear(self.expert_ff, self.experts * width,
                              bias=False)


MIXERS = {m.kind: m for m in (HGRN2Mixer, BiasedAttention)}
PARALLEL_MIXERS = {m.kind: m for m in (LatentAttention,)}
PARALLEL_MLPS = {m.kind: m for m in (GatedMLP, RoutedMLP)}


class HybridBlock(nn.Module):
    """Layer ``index`` of the whole model (not of the stage)."""

    def __init__(self, config: ModelConfig, index: int) -> None:
        super().__init__()
        E = config.n_embd
        spec = config.layers[index]
        self.norm_1 = Scale(E)
        self.norm_1b = Scale(E) if config.post_norms else None
        self.mixer = MIXERS[spec["type"]](E, spec["mixer"])
        self.norm_2 = self.norm_2b = self.mlp = None
        if spec["mlp"] is not None:
            self.norm_2 = Scale(E)
            self.norm_2b = Scale(E) if config.post_norms else None
            self.mlp = XieluMLP(E, spec["mlp"])


class ParallelBlock(nn.Module):
    """Mixer and feed-forward that read one norm and are added together.

    in_proj rows: the feed-forward's gate | up, the mixer's rows, the head
    gates.  out_proj columns: the mixer's, then the feed-forward's."""

    def __init__(self, config: ModelConfig, index: int) -> None:
        super().__init__()
        E = config.n_embd
        spec = config.layers[index]
        self.norm_1 = Scale(E)
        self.mixer = PARALLEL_MIXERS[spec["type"]](E, spec["mixer"], index)
        self.mlp = None
        if spec["mlp"] is not None:
            self.mlp = PARALLEL_MLPS[spec["mlp"]["kind"]](E, spec["mlp"])
        rows = sum(n for _, n in self.in_rows())
        self.ff = self.mlp.ff if self.mlp is not None else 0
        self.in_proj = nn.Linear(E, rows, bias=False)
        self.out_proj = nn.Linear(self.mixer.out_cols + self.ff, E,
                                  bias=False)

    def in_rows(self):
        """(part, rows) of in_proj, in order."""
        mlp = self.mlp.in_rows if self.mlp is not None else []
        return mlp + self.mixer.in_rows + self.mixer.gate_rows


def make_block(config: ModelConfig, index: int) -> nn.Module:
    cls = ParallelBlock if config.parallel_residual else HybridBlock
    return cls(config, index)


# ---------------------------------------------------------------------------
# on-disk tensor names
# ---------------------------------------------------------------------------


def native_tensors(config: ModelConfig) -> Dict[str, Tuple[str, ...]]:
    """Framework key -> the on-disk tensors that are stacked to make it
    (``out_proj``: laid side by side)."""
    out = {
        "transformer.wte.weight": ("embed",),
        "transformer.ln_f.weight": ("final.norm",),
        "lm_head.weight": ("head",),
    }
    if config.pos_embedding == "learned":
        out["transformer.wpe.weight"] = ("pos",)
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"transformer.h.{i}."
        if config.parallel_residual:
            out.update(_parallel_tensors(spec, src, dst))
            continue
        norms = ["1", "1b"] if config.post_norms else ["1"]
        if spec["mlp"] is not None:
            norms += ["2", "2b"] if config.post_norms else ["2"]
        for n in norms:
            out[f"{dst}norm_{n}.weight"] = (f"{src}norm{n}",)
        mix, mixer = src + "mix.", dst + "mixer."
        if spec["type"] == "hgrn2":
            out[mixer + "in_proj.weight"] = (mix + "q", mix + "f", mix + "v")
            out[mixer + "f_bias"] = (mix + "f.b",)
            out[mixer + "lower"] = (mix + "lower",)
            out[mixer + "norm.weight"] = (mix + "norm",)
        else:
            out[mixer + "in_proj.weight"] = (mix + "q", mix + "k", mix + "v")
            out[mixer + "q_norm.weight"] = (mix + "q.norm",)
            out[mixer + "k_norm.weight"] = (mix + "k.norm",)
            out[mixer + "rel"] = (mix + "rel",)
        out[mixer + "proj.weight"] = (mix + "o",)
        if spec["mlp"] is not None:
            out[f"{dst}mlp.fc.weight"] = (f"{src}mlp.up",)
            out[f"{dst}mlp.proj.weight"] = (f"{src}mlp.down",)
            out[f"{dst}mlp.act"] = (f"{src}mlp.act",)
    return out


def _parallel_tensors(spec: dict, src: str, dst: str) -> dict:
    mix, mlp = src + "mix.", src + "mlp."
    rows, cols = [], [mix + "o"]
    out = {dst + "norm_1.weight": (src + "norm1",)}
    kind = spec["mlp"] and spec["mlp"]["kind"]
    if kind == "dense":
        rows += [mlp + "gate", mlp + "up"]
        cols.append(mlp + "down")
    elif kind == "moe":
        n = range(spec["mlp"]["router"]["experts"])
        if spec["mlp"].get("shared"):
            rows += [mlp + "shared.gate", mlp + "shared.up"]
            cols.append(mlp + "shared.down")
        out[dst + "mlp.router.weight"] = (mlp + "router",)
        out[dst + "mlp.up.weight"] = tuple(
            f"{mlp}e{e}.{part}" for e in n for part in ("gate", "up"))
        out[dst + "mlp.down.weight"] = tuple(f"{mlp}e{e}.down" for e in n)
    mixer = dst + "mixer."
    rows.append(mix + "dq")
    out[mixer + "q_norm.weight"] = (mix + "dq.norm",)
    out[mixer + "q_up.weight"] = (mix + "uq",)
    out[mixer + "kv_up.weight"] = (mix + "uk", mix + "uv")
    if spec["mixer"].get("kv_from") is None:
        rows.append(mix + "dkv")
        out[mixer + "kv_norm.weight"] = (mix + "dkv.norm",)
    rows.append(mix + "g")
    out[dst + "in_proj.weight"] = tuple(rows)
    out[dst + "out_proj.weight"] = tuple(cols)
    return out


def native_state_dict(config: ModelConfig, get) -> dict:
    """State dict in the framework's layout; ``get(name)`` reads one tensor
    (so that a file is read tensor by tensor)."""
    sd = {}
    for key, names in native_tensors(config).items():
        parts = [get(n) for n in names]
        dim = 1 if key.endswith(".out_proj.weight") else 0
        sd[key] = parts[0] if len(parts) == 1 else torch.cat(parts, dim)
    return sd
