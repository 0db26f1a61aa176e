"""Parameters of stacks whose layers differ (``ModelConfig.layers``).

These modules hold weights under the framework's key layout, so loading,
chunking and moving to a device work as for every other model; the layers
are computed by ``ops.hybrid_engine`` only.  Projections that read the same
input are stored stacked (``in_proj``), as the fused QKV of ``model.Block``
is, so that one matrix product serves all of them.
"""

from __future__ import annotations

from typing import Dict, Tuple

import torch
import torch.nn as nn

from ..config import ModelConfig

__all__ = ["HybridBlock", "native_state_dict", "native_tensors"]


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


MIXERS = {m.kind: m for m in (HGRN2Mixer, BiasedAttention)}


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


# ---------------------------------------------------------------------------
# on-disk tensor names
# ---------------------------------------------------------------------------


def native_tensors(config: ModelConfig) -> Dict[str, Tuple[str, ...]]:
    """Framework key -> the on-disk tensors that are stacked to make it."""
    out = {
        "transformer.wte.weight": ("embed",),
        "transformer.ln_f.weight": ("final.norm",),
        "lm_head.weight": ("head",),
    }
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"transformer.h.{i}."
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


def native_state_dict(config: ModelConfig, get) -> dict:
    """State dict in the framework's layout; ``get(name)`` reads one tensor
    (so that a file is read tensor by tensor)."""
    sd = {}
    for key, names in native_tensors(config).items():
        parts = [get(n) for n in names]
        sd[key] = parts[0] if len(parts) == 1 else torch.cat(parts)
    return sd
