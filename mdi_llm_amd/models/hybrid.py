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

__all__ = ["HybridBlock", "ParallelBlock", "make_block", "make_blocks",
           "native_state_dict", "native_tensors"]


class Scale(nn.Module):
    """The weight of a norm; which norm it is, the engine knows."""

    def __init__(self, size: int) -> None:
        super().__init__()
        self.weight = nn.Parameter(torch.zeros(size))


class HGRN2Mixer(nn.Module):
    """Gated linear recurrence: in_proj rows are q | f | v."""

    kind = "hgrn2"

    def __init__(self, width: int, spec: dict, index: int) -> None:
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

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.source = index     # model-wide index of the layer's K/V pages
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


class RGLRUMixer(nn.Module):
    """Two branches, in_proj rows y | x: x passes a causal convolution and a
    linear recurrence whose gates are block-diagonal products (gates: the
    recurrence gate's matrices, then the input gate's); the activated y
    multiplies what comes out."""

    kind = "rglru"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.width, self.blocks = spec["width"], spec["blocks"]
        if self.width % self.blocks:
            raise ValueError("rglru: width must be a multiple of blocks")
        self.taps, self.channels = spec["conv"], self.width
        W, part = self.width, self.width // self.blocks
        self.in_proj = nn.Linear(width, 2 * W, bias=True)
        self.conv = nn.Parameter(torch.zeros(W, self.taps))
        self.conv_bias = nn.Parameter(torch.zeros(W))
        self.gates = nn.Parameter(torch.zeros(2 * self.blocks, part, part))
        self.gate_bias = nn.Parameter(torch.zeros(2 * self.blocks, part))
        self.lam = nn.Parameter(torch.zeros(W))
        self.proj = nn.Linear(W, width, bias=False)


class Mamba2Mixer(nn.Module):
    """State-space duality with a scalar decay per head: in_proj rows are
    z | x | B | C | dt, of which x, B and C pass a causal convolution."""

    kind = "mamba2"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.heads, self.vdim = spec["heads"], spec["vdim"]
        self.dim, self.groups = spec["state"], spec["groups"]
        self.norm_groups, self.taps = spec["norm_groups"], spec["conv"]
        self.inner = self.heads * self.vdim
        if self.heads % self.groups or self.inner % self.norm_groups:
            raise ValueError("mamba2: heads must be a multiple of groups, "
                             "channels of norm_groups")
        self.channels = self.inner + 2 * self.groups * self.dim
        self.in_proj = nn.Linear(
            width, self.inner + self.channels + self.heads, bias=False)
        self.conv = nn.Parameter(torch.zeros(self.channels, self.taps))
        self.conv_bias = nn.Parameter(torch.zeros(self.channels))
        self.dt_bias = nn.Parameter(torch.zeros(self.heads))
        self.a_log = nn.Parameter(torch.zeros(self.heads))
        self.skip = nn.Parameter(torch.zeros(self.heads))
        self.norm = Scale(self.inner)
        self.proj = nn.Linear(self.inner, width, bias=False)


class DiffAttention(nn.Module):
    """Differential attention: every head has two attention maps over the
    same values and gives the first less ``lambda`` times the second.  in_proj
    rows are q | k | v, queries and keys as (head, map).  A layer with
    ``kv_from`` has queries only and reads that layer's keys and values.
    lambda is learned (exp(q1 k1) - exp(q2 k2) + diff, ``lam`` rows q1, k1,
    q2, k2)."""

    kind = "diff_attention"
    maps = 2

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.heads, self.kv_heads = spec["heads"], spec["kv_heads"]
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.scale, self.diff = float(spec["scale"]), float(spec["diff"])
        self.softcap = float(spec.get("softcap") or 0.0)
        self.rot = dict(spec["rot"])
        if self.rot["dims"] % 2 or self.rot["dims"] > self.dim:
            raise ValueError("rotated dimensions come in pairs within a head")
        self.window, self.keep_first = 1 << 30, 0
        src = spec.get("kv_from")
        self.source = index if src is None else src
        self.owns_kv = src is None
        rows = self.maps * self.heads * self.dim
        if self.owns_kv:
            rows += self.kv_heads * (self.maps * self.dim + self.vdim)
            self.k_norm = Scale(self.dim)
        self.in_proj = nn.Linear(width, rows, bias=False)
        self.q_norm = Scale(self.dim)
        self.lam = nn.Parameter(torch.zeros(4 * self.dim))
        self.proj = nn.Linear(self.heads * self.vdim, width, bias=False)

    def map_weight(self) -> float:
        q1, k1, q2, k2 = self.lam.detach().double().view(4, -1)
        return float((q1 * k1).sum().exp() - (q2 * k2).sum().exp()
                     + self.diff)


class MLSTMMixer(nn.Module):
    """Matrix memory per head with exponential input and forget gates, both
    capped: in_proj rows are q | k | v | output gate | input gate logits |
    forget gate logits."""

    kind = "mlstm"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.heads, self.dim, self.vdim = (
            spec["heads"], spec["dim"], spec["vdim"])
        self.gate_cap = float(spec["gate_cap"])
        H = self.heads
        self.in_proj = nn.Linear(
            width, 2 * H * (self.dim + self.vdim + 1), bias=False)
        self.gate_bias = nn.Parameter(torch.zeros(2 * H))
        self.norm = Scale(H * self.vdim)
        self.proj = nn.Linear(H * self.vdim, width, bias=False)


class GatedAttention(nn.Module):
    """Windowed attention with norms over all query and all key channels,
    queries that warm up with their position, values of unit size, a fixed
    slope by distance, a sink in the softmax and an element-wise output gate.
    Part of a ``PairedMixer``: in_rows are its rows of the pair's in_proj."""

    kind = "gated_attention"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.source = index     # model-wide index of the layer's K/V pages
        self.heads, self.kv_heads = spec["heads"], spec["kv_heads"]
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.scale = float(spec["scale"])
        self.q_temp = spec.get("q_temp")
        self.window = int((spec.get("mask") or {}).get("size", 1 << 30))
        self.keep_first = 0
        q, k = self.heads * self.dim, self.kv_heads * self.dim
        self.inner = self.heads * self.vdim
        self.in_rows = q + k + self.kv_heads * self.vdim + self.inner
        self.q_norm, self.k_norm = Scale(q), Scale(k)
        self.sink = nn.Parameter(torch.zeros(self.heads))
        self.proj = nn.Linear(self.inner, width, bias=False)


class MinGRU(nn.Module):
    """Recurrence per channel that blends its state with a candidate; blend
    and candidate depend on the token alone.  Part of a ``PairedMixer``: its
    rows of in_proj are blend z | input | output gate, of which the first two
    have a bias."""

    kind = "mingru"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.width = self.inner = spec["width"]
        self.in_rows = 3 * self.width
        self.bias = nn.Parameter(torch.zeros(2 * self.width))
        self.proj = nn.Linear(self.width, width, bias=False)


PARTS = {m.kind: m for m in (GatedAttention, MinGRU)}


class PairedMixer(nn.Module):
    """A pair of mixers over one input, the mean of whose normed outputs is
    the result.  in_proj rows: the left part's, then the right part's."""

    kind = "paired"

    def __init__(self, width: int, spec: dict, index: int) -> None:
        super().__init__()
        self.left, self.right = (
            PARTS[spec[side]["type"]](width, spec[side], index)
            for side in ("left", "right"))
        self.in_proj = nn.Linear(
            width, self.left.in_rows + self.right.in_rows, bias=False)
        self.left_norm, self.right_norm = Scale(width), Scale(width)

    @property
    def parts(self):
        return self.left, self.right


class XieluMLP(nn.Module):
    kind = "dense"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.fc = nn.Linear(width, spec["ff"], bias=False)
        self.proj = nn.Linear(spec["ff"], width, bias=False)
        self.act = nn.Parameter(torch.zeros(2))


class GeluMLP(nn.Module):
    """Up, exact GELU, down."""

    kind = "dense"

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.fc = nn.Linear(width, spec["ff"], bias=False)
        self.proj = nn.Linear(spec["ff"], width, bias=False)


class SquaredReluMLP(GeluMLP):
    """Up, squared ReLU, down."""


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
    gate_rows = 0           # router rows that are not a choice

    def __init__(self, width: int, spec: dict) -> None:
        super().__init__()
        self.experts, self.top = (
            spec["router"]["experts"], spec["router"]["top"])
        self.expert_ff = spec["expert"]["ff"]
        self.identity = spec["router"].get("identity", 0)
        self.ff = (spec.get("shared") or {}).get("ff", 0)
        self.in_rows = [("shared.gate", self.ff), ("shared.up", self.ff)] \
            if self.ff else []
        self.router = nn.Linear(width, self.experts + self.identity
                                + self.gate_rows, bias=False)
        self.up = nn.Linear(width, self.experts * 2 * self.expert_ff,
                            bias=False)
        self.down = nn.Linear(self.expert_ff, self.experts * width,
                              bias=False)


class CorrectedRoutedMLP(RoutedMLP):
    """Routed experts with weights of their own beside the choice: the
    softmax over all router outputs plus ``correction`` chooses, without it
    the weights are made (times ``scale``).  The last ``identity`` outputs
    stand for the input itself.  The shared expert is gated by the router's
    last row and has projections of its own (shared_in rows gate | up)."""

    gate_rows = 1

    def __init__(self, width: int, spec: dict) -> None:
        if not spec.get("shared"):
            self.gate_rows = 0
        super().__init__(width, spec)
        self.scale = float(spec["router"].get("scale", 1.0))
        self.correction = nn.Parameter(
            torch.zeros(self.experts + self.identity))
        if self.ff:
            self.shared_in = nn.Linear(width, 2 * self.ff, bias=False)
            self.shared_out = nn.Linear(self.ff, width, bias=False)


MIXERS = {m.kind: m for m in (HGRN2Mixer, BiasedAttention, RGLRUMixer,
                              Mamba2Mixer, DiffAttention, MLSTMMixer,
                              PairedMixer)}
MLPS = {"XieluMLP": {"dense": XieluMLP},
        "GeluMLP": {"dense": GeluMLP, "moe": CorrectedRoutedMLP},
        "SquaredReluMLP": {"dense": SquaredReluMLP}}
PARALLEL_MIXERS = {m.kind: m for m in (LatentAttention,)}
PARALLEL_MLPS = {m.kind: m for m in (GatedMLP, RoutedMLP)}


class HybridBlock(nn.Module):
    """Layer ``index`` of the whole model (not of the stage)."""

    def __init__(self, config: ModelConfig, index: int) -> None:
        super().__init__()
        E = config.n_embd
        spec = config.layers[index]

        def scale(wanted: bool):
            return Scale(E) if wanted else None

        self.norm_1 = scale(config.pre_norms)
        self.norm_1b = scale(config.post_norms)
        self.ls_1 = scale(config.layer_scale)
        self.mixer = MIXERS[spec["type"]](E, spec["mixer"], index)
        self.norm_2 = self.norm_2b = self.ls_2 = self.mlp = None
        if spec["mlp"] is not None:
            self.norm_2 = scale(config.pre_norms)
            self.norm_2b = scale(config.post_norms)
            self.ls_2 = scale(config.layer_scale)
            mlps = MLPS[config.mlp_class_name]
            self.mlp = mlps[spec["mlp"]["kind"]](E, spec["mlp"])
        self.shift = scale(config.token_shift)
        # coefficients of the embedding and of every result up to this one
        self.depth = Scale(index + 2) if config.depth_average else None


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


def make_blocks(config: ModelConfig, first: int, n: int) -> nn.ModuleList:
    """Layers ``first`` .. of the model.  Those that use another layer's
    weights hold its parameters, as long as it is one of them; else they have
    a copy."""
    blocks = nn.ModuleList(make_block(config, first + i) for i in range(n))
    seen: Dict[int, nn.Module] = {}
    for i, block in enumerate(blocks):
        owner = seen.setdefault(config.weights_of(first + i), block)
        if owner is not block:
            _share(block, owner)
    return blocks


def _share(block: nn.Module, owner: nn.Module) -> None:
    for name in owner._parameters:
        block._parameters[name] = owner._parameters[name]
    for name, part in owner._modules.items():
        if part is not None:
            _share(block._modules[name], part)


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
        src, dst = f"l{config.weights_of(i)}.", f"transformer.h.{i}."
        if config.parallel_residual:
            out.update(_parallel_tensors(spec, src, dst))
            continue
        out.update(_block_tensors(config, spec, src, dst))
    return out


_MIXER_TENSORS = {
    "hgrn2": {"in_proj.weight": ("q", "f", "v"), "f_bias": ("f.b",),
              "lower": ("lower",), "norm.weight": ("norm",)},
    "attention": {"in_proj.weight": ("q", "k", "v"),
                  "q_norm.weight": ("q.norm",), "k_norm.weight": ("k.norm",),
                  "rel": ("rel",)},
    "rglru": {"in_proj.weight": ("y", "x"), "in_proj.bias": ("y.b", "x.b"),
              "conv": ("conv",), "conv_bias": ("conv.b",),
              "gates": ("ra", "ri"), "gate_bias": ("ra.b", "ri.b"),
              "lam": ("lam",)},
    "mamba2": {"in_proj.weight": ("in",), "conv": ("conv",),
               "conv_bias": ("conv.b",), "dt_bias": ("dt_bias",),
               "a_log": ("A_log",), "skip": ("D",), "norm.weight": ("norm",)},
    "diff_attention": {"in_proj.weight": ("q", "k", "v"),
                       "q_norm.weight": ("q.norm",),
                       "k_norm.weight": ("k.norm",),
                       "lam": ("lq1", "lk1", "lq2", "lk2")},
    "mlstm": {"in_proj.weight": ("q", "k", "v", "g", "i", "f"),
              "gate_bias": ("i.b", "f.b"), "norm.weight": ("norm",)},
    "paired": {"in_proj.weight": ("left.q", "left.k", "left.v", "left.g",
                                  "right.z", "right.x", "right.g"),
               "left.q_norm.weight": ("left.q.norm",),
               "left.k_norm.weight": ("left.k.norm",),
               "left.sink": ("left.sink",),
               "left.proj.weight": ("left.o",),
               "right.bias": ("right.z.b", "right.x.b"),
               "right.proj.weight": ("right.o",),
               "left_norm.weight": ("left.out",),
               "right_norm.weight": ("right.out",)},
}


def _block_tensors(config: ModelConfig, spec: dict, src: str,
                   dst: str) -> dict:
    out, mlp = {}, spec["mlp"]
    for n in ("1",) if mlp is None else ("1", "2"):
        if config.pre_norms:
            out[f"{dst}norm_{n}.weight"] = (f"{src}norm{n}",)
        if config.post_norms:
            # a block's only norms go without the suffix
            b = "b" if config.pre_norms else ""
            out[f"{dst}norm_{n}b.weight"] = (f"{src}norm{n}{b}",)
        if config.layer_scale:
            out[f"{dst}ls_{n}.weight"] = (f"{src}ls{n}",)
    if config.token_shift:
        out[dst + "shift.weight"] = (src + "shift",)
    if config.depth_average:
        out[dst + "depth.weight"] = (src + "dwa",)
    mix, mixer = src + "mix.", dst + "mixer."
    for key, names in _MIXER_TENSORS[spec["type"]].items():
        if spec["mixer"].get("kv_from") is not None:
            if key == "k_norm.weight":
                continue
            names = tuple(n for n in names if n not in ("k", "v"))
        out[mixer + key] = tuple(mix + n for n in names)
    if spec["type"] != "paired":    # (whose parts have one each)
        out[mixer + "proj.weight"] = (mix + "o",)
    if mlp is None:
        return out
    pre, to = src + "mlp.", dst + "mlp."
    if mlp["kind"] == "dense":
        out[to + "fc.weight"] = (pre + "up",)
        out[to + "proj.weight"] = (pre + "down",)
        if config.mlp_class_name == "XieluMLP":
            out[to + "act"] = (pre + "act",)
        return out
    out[to + "router.weight"] = (pre + "router",)
    out[to + "correction"] = (pre + "correction",)
    out.update(_expert_tensors(mlp, pre, to))
    if mlp.get("shared"):
        out[to + "router.weight"] += (pre + "shared.sg",)
        out[to + "shared_in.weight"] = (pre + "shared.gate",
                                        pre + "shared.up")
        out[to + "shared_out.weight"] = (pre + "shared.down",)
    return out


def _expert_tensors(spec: dict, pre: str, to: str) -> dict:
    n = range(spec["router"]["experts"])
    return {to + "up.weight": tuple(f"{pre}e{e}.{part}" for e in n
                                    for part in ("gate", "up")),
            to + "down.weight": tuple(f"{pre}e{e}.down" for e in n)}


def _parallel_tensors(spec: dict, src: str, dst: str) -> dict:
    mix, mlp = src + "mix.", src + "mlp."
    rows, cols = [], [mix + "o"]
    out = {dst + "norm_1.weight": (src + "norm1",)}
    kind = spec["mlp"] and spec["mlp"]["kind"]
    if kind == "dense":
        rows += [mlp + "gate", mlp + "up"]
        cols.append(mlp + "down")
    elif kind == "moe":
        if spec["mlp"].get("shared"):
            rows += [mlp + "shared.gate", mlp + "shared.up"]
            cols.append(mlp + "shared.down")
        out[dst + "mlp.router.weight"] = (mlp + "router",)
        out.update(_expert_tensors(spec["mlp"], mlp, dst + "mlp."))
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
    sd, made = {}, {}
    for key, names in native_tensors(config).items():
        if names not in made:   # (layers may use the same tensors)
            parts = [get(n) for n in names]
            dim = 1 if key.endswith(".out_proj.weight") else 0
            made[names] = parts[0] if len(parts) == 1 \
                else torch.cat(parts, dim)
        sd[key] = made[names]
    return sd
