"""Step engine of hybrid stacks (``ModelConfig.layers``): every step is one
ragged batch, prompt pieces and decode tokens together.

Where ``DecodeEngine`` advances one sequence and ``GroupDecodeEngine`` a
fixed group, every step here takes any mix of sequences: the rows of all
entries lie flat in one activation matrix, so a projection is one matrix
product for the whole step, and the kernels that look at neighbours in time
(recurrence, attention) walk the entries as segments.  Steps in which every
entry is one token are captured as hipGraphs per batch size.

Blocks come in three forms: norms ahead of (and behind) each sublayer, or ahead
and behind the two parts of a mixer (``mixers.Paired``); one norm for parallel
sublayers (``latent_layer``); and norms on the sublayers' outputs only, with the
options of that form (``_run_output_normed``).

The residual stream, norms, gates, recurrent state and softmax are fp32; the
weights, matrix products and cached K/V have the stage's dtype (bf16, or
fp32 throughout).
"""

from __future__ import annotations

import math
import os
import warnings
from bisect import bisect_left
from dataclasses import dataclass, field
from fractions import Fraction
from typing import Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from ..config import ModelConfig
from ..models.cache import PAGE, HybridCache
from ..models.sampling import sample as sample_token
from ..models.model import build_pair_rope_table
from . import require_hip_ops
from .experts import RoutedExperts
from .mixers import MIXERS
from .latent_layer import LatentPlan, ParallelLayer, make_plan

__all__ = ["HybridEngine", "distance_bias"]


def distance_bucket_starts(rows: int, far) -> List[int]:
    """First distance of each bucket: one per distance below rows/2, then
    geometric up to ``far``, compared exactly (no logarithms)."""
    half = rows // 2
    m = rows - half
    starts = list(range(half))
    span = range(half, math.ceil(far) + 1)
    for k in range(m):
        # smallest n with (n / half)^m >= (far / half)^k
        bound = (Fraction(far) / half) ** k * half ** m
        starts.append(span[bisect_left(span, bound, key=lambda n: n ** m)])
    return starts


def distance_bias(rel: torch.Tensor, far) -> torch.Tensor:
    """[rows, heads] bucket table -> [heads, n] bias by distance in log2
    units; distances past the end share the last entry."""
    rows = rel.size(0)
    if rows < 2 or far <= rows // 2:
        raise ValueError("distance buckets: bias_max must exceed rows / 2")
    starts = distance_bucket_starts(rows, far)
    bucket = torch.zeros(starts[-1] + 1, dtype=torch.long)
    for b, s in enumerate(starts):
        bucket[s:] = b
    per = rel.detach().double()[bucket.to(rel.device)].t()
    return (per * math.log2(math.e)).float().contiguous()


@dataclass
class Batch:
    """Device view of one step."""

    n: int                   # rows
    seg: torch.Tensor        # [4, entries]: start, len, slot, pos0
    singles: int             # the first entries of seg are one token long
    max_len: int
    row_slot: torch.Tensor
    row_pos: torch.Tensor
    tokens: Optional[torch.Tensor]
    max_ctx: int             # longest sequence, this step included
    # the columns of seg on the host; None: single tokens, known only there
    entries: Optional[List[Tuple[int, int, int, int]]] = None
    plans: dict = field(default_factory=dict)
    contexts: dict = field(default_factory=dict)  # gathered latents

    def latent_plan(self, m, device, form: Optional[str]) -> LatentPlan:
        if self.entries is None:
            return LatentPlan(seg=self.seg, n_rows=self.n)
        key = (m.dim, m.vdim, m.rank, m.window)
        if key not in self.plans:
            self.plans[key] = make_plan(self.entries, self.n, m, device, form)
        return self.plans[key]


FEW_ROWS = 64           # rows whose residual steps are bound by latency
XIELU, GELU, RELU2 = 1, 2, 3    # activations that a projection can end with


class _LayerWeights:
    """One layer's operands: matrices as they are, the rest in fp32."""

    def __init__(self, eng: "HybridEngine", i: int, block) -> None:
        def f(t):
            return None if t is None else t.detach().float().contiguous()

        def w(norm):
            return None if norm is None else f(norm.weight)

        self.norm1, self.norm1b = w(block.norm_1), w(block.norm_1b)
        self.norm2, self.norm2b = w(block.norm_2), w(block.norm_2b)
        m = block.mixer
        self.norm1c = None      # of a second output beside the first
        if m.kind == "paired":
            self.norm1b = 0.5 * w(m.left_norm)
            self.norm1c = 0.5 * w(m.right_norm)
        # a factor on a sublayer's output joins the weight of its norm
        self.gain1, self.gain2 = w(block.ls_1), w(block.ls_2)
        if self.norm1b is not None and self.gain1 is not None:
            self.norm1b = self.norm1b * self.gain1
            if self.norm1c is not None:
                self.norm1c = self.norm1c * self.gain1
            self.gain1 = None
        if self.norm2b is not None and self.gain2 is not None:
            self.norm2b, self.gain2 = self.norm2b * self.gain2, None
        self.shift, self.depth = w(block.shift), w(block.depth)
        if self.depth is not None:  # for a sum over earlier results
            self.depth_end = torch.stack((torch.ones_like(self.depth[-1]),
                                          self.depth[-1]))
        self.mixer, self.mix = m, None
        if m.kind in MIXERS:
            self.mix = MIXERS[m.kind](eng, i, m)
        else:
            self.in_proj = m.in_proj.weight.detach()
            self.proj = m.proj.weight.detach()
        if m.kind == "hgrn2":
            self.f_bias, self.lower = f(m.f_bias), f(m.lower)
            self.norm = f(m.norm.weight)
        elif m.kind == "attention":
            self.q_norm, self.k_norm = f(m.q_norm.weight), f(m.k_norm.weight)
            self.bias = distance_bias(m.rel, m.bias_max)
            self.rotate, self.two_maps = {}, {}
        elif m.kind == "diff_attention":
            self.q_norm = f(m.q_norm.weight)
            self.k_norm = f(m.k_norm.weight) if m.owns_kv else None
            self.bias = torch.zeros(m.heads, 1, device=eng.device)
            self.rotate = dict(rope=eng.rope_table(m.rot))
            self.two_maps = dict(softcap=m.softcap, map_weight=m.map_weight(),
                                 out_scale=1.0 - m.diff,
                                 eps=eng.config.norm_eps)
        mlp = block.mlp
        self.mlp = mlp is not None
        self.experts = self.act = None
        if not self.mlp:
            return
        if mlp.kind == "moe":
            self.experts = RoutedExperts(eng, mlp)
            self.shared_ff = mlp.ff
            if mlp.ff:
                self.shared_in = mlp.shared_in.weight.detach()
                self.shared_out = mlp.shared_out.weight.detach()
            return
        self.fc = mlp.fc.weight.detach()
        self.down = mlp.proj.weight.detach()
        if hasattr(mlp, "act"):
            self.act = (XIELU, *F.softplus(mlp.act.detach().float()).tolist())
        else:
            squared = eng.config.mlp_class_name == "SquaredReluMLP"
            self.act = (RELU2 if squared else GELU, 0.0, 0.0)


class _DecodeStep:
    """Static buffers and graphs of single-token steps of one batch size."""

    def __init__(self, eng: "HybridEngine", size: int) -> None:
        dev = eng.device
        # start, len, slot, pos0 | token, sampling key
        self.io = torch.zeros(6, size, dtype=torch.int32, device=dev)
        self.load([], [], [], [], eng.cache.spare)
        io = self.io
        self.batch = Batch(size, io[:4], size, 1, io[2], io[3], io[4],
                           eng.max_ctx)
        self.sampled = torch.zeros(size, dtype=torch.int32, device=dev)
        self.scratch = torch.zeros(520 * size, dtype=torch.int32, device=dev)
        self.logits: Optional[torch.Tensor] = None
        self.forward = self.forward_graph = None
        self.sample_graphs: dict = {}
        self.slots: List[int] = []

    def load(self, slots, pos, tokens, keys, spare: int) -> None:
        size = self.io.size(1)
        pad = [0] * (size - len(slots))
        rows = [list(range(size)), [1] * size,
                list(slots) + [spare] * len(pad), list(pos) + pad,
                list(tokens) + pad, list(keys) + pad]
        self.io.copy_(torch.tensor(rows, dtype=torch.int32))
        self.slots = list(slots)


class HybridEngine:
    """Drives one stage (starter or secondary) of a hybrid stack."""

    supports_hip_prefill = True

    def __init__(self, stage, cache: HybridCache,
                 use_graphs: bool = True) -> None:
        self.config: ModelConfig = stage.config
        self.stage = stage
        self.cache = cache
        p = next(stage.parameters())
        self.device, self.dtype = p.device, p.dtype
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid stacks run in bfloat16 or float32")
        for var in ("MDI_WEIGHT_DTYPE", "MDI_KV_DTYPE"):
            if os.environ.get(var, "bf16") != "bf16":
                warnings.warn(f"{var}={os.environ[var]} ignored: hybrid "
                              "stacks keep weights and K/V in the stage's "
                              "dtype")
        self.hip = self.device.type == "cuda"
        if self.hip:
            self.ops = require_hip_ops()
        else:
            from . import hybrid_torch

            self.ops = hybrid_torch
        self.use_graphs = use_graphs and self.hip
        self.is_starter = hasattr(stage, "lm_head")
        self.parallel = self.config.parallel_residual
        self.latent_form: Optional[str] = None  # "absorbed" or "expanded"
        # longest sequence that can occur
        self.max_ctx = min(cache.n_pages * PAGE, stage.max_seq_length)
        self._tables: Dict[str, torch.Tensor] = {}  # by position
        if self.parallel:
            self.layers = [ParallelLayer(self, b) for b in stage.transformer.h]
        else:
            self.layers = [_LayerWeights(self, i, b)
                           for i, b in enumerate(stage.transformer.h)]
        for lw in self.layers:
            m = lw.mixer
            if m.kind == "hgrn2" and (m.dim > 256 or m.vdim > 1024):
                raise ValueError("hgrn2: dim <= 256 and vdim <= 1024")
        if self.is_starter:
            self.wte = stage.transformer.wte.weight.detach()
            # (a factor on the logits joins the last norm's weight)
            self.final = stage.transformer.ln_f.weight.detach().float() \
                * self.config.logit_scale
            self.head = stage.lm_head.weight.detach()
            wpe = getattr(stage.transformer, "wpe", None)
            self.wpe = None if wpe is None else wpe.weight.detach()
        self._ring_columns(stage)
        self._steps: Dict[int, _DecodeStep] = {}

    def _ring_columns(self, stage) -> None:
        """Columns of the rows between stages that hold shared cache rows:
        those that local layers read from an earlier stage, those made
        here."""
        first, cfg = stage.first_layer, self.config
        self.first_layer = first
        shared = cfg.shared_rows()
        at = cfg.ring_width - sum(shared.values())
        self.ring_in, self.ring_out = {}, {}
        for src, n in shared.items():
            cols = slice(at, at + n)
            at += n
            if first <= src < first + len(self.layers):
                self.ring_out[src] = cols
            elif src in self.cache.latent or src in self.cache.k:
                self.ring_in[src] = cols

    def rope_table(self, rot: dict) -> torch.Tensor:
        """cos and sin by position, one table for all layers that rotate
        alike."""
        key = repr(sorted(rot.items(), key=str))
        if key not in self._tables:
            self._tables[key] = build_pair_rope_table(self.max_ctx, rot,
                                                      self.device)
        return self._tables[key]

    def query_scale_table(self, every, coef: float) -> torch.Tensor:
        """Factors on queries that grow with the logarithm of the position,
        a step every ``every`` tokens."""
        key = repr(("query scale", every, coef))
        if key not in self._tables:
            p = torch.arange(1, self.max_ctx + 1, dtype=torch.float64)
            f = 1.0 + coef * torch.log(torch.floor(p / every) + 1.0)
            self._tables[key] = f.float().to(self.device)
        return self._tables[key]

    # ------------------------------------------------------------------
    # building blocks
    # ------------------------------------------------------------------
    def _norm_step(self, x, y=None, post_w=None, next_w=None, tokens=None,
                   row_pos=None, routed=None, gain=None, post_w2=None):
        """x <- embed(tokens) or x + post-norm(y) (+ routed experts); the
        next pre-norm.  ``gain``: factors on y without a norm; a pair of
        outputs in y has two post-norms."""
        xn, extra = None, {}
        if isinstance(y, tuple):
            y, y2 = y
            extra.update(y2=y2, post_w2=post_w2)
        if gain is not None:
            extra.update(gain=gain)
        if tokens is not None and self.wpe is not None:
            extra.update(pos_table=self.wpe, row_pos=row_pos)
        if routed is not None:
            extra.update(routed=routed[0], routed_w=routed[1])
        if next_w is not None:
            xn = torch.empty(x.shape, dtype=self.dtype, device=self.device)
        self.ops.residual_norm(
            x, y=y, post_w=post_w, xn=xn, next_w=next_w, tokens=tokens,
            table=None if tokens is None else self.wte,
            scale=self.config.embedding_scale,
            offset=self.config.norm_offset, eps=self.config.norm_eps,
            mult=self.config.residual_mult, **extra)
        return xn

    def _linear(self, x: torch.Tensor, w: torch.Tensor, act=None):
        (M, K), n = w.shape, x.size(0)
        if self.hip and self.dtype == torch.bfloat16 and n <= 32:
            # few rows: the weight stream decides.  Past 16 rows, and for
            # the widest outputs, the library's kernels stream as well,
            # except along a very long K.
            kind, p, q = act or (0, 0.0, 0.0)
            out = torch.empty(n, M, dtype=self.dtype, device=self.device)
            if n == 1 and K % 8 == 0:
                self.ops.gemv(out, w, x, None, None, kind and kind + 3,
                              rows=4 if M >= 65536 else 1, act_p=p, act_q=q)
                return out
            if K % 64 == 0 and M < 65536 and (n <= 16 or K >= 16384):
                self.ops.skinny_gemm(out, w, x, kind, p, q)
                return out
        out = F.linear(x, w)
        if act is not None and act[0] == XIELU:
            self.ops.xielu(out, *act[1:])
        elif act is not None and act[0] == GELU:
            self.ops.gelu(out)
        elif act is not None:
            self.ops.relu2(out)
        return out

    def _hgrn2(self, i: int, lw: _LayerWeights, b: Batch, xn: torch.Tensor):
        m, eps = lw.mixer, self.config.norm_eps
        proj = self._linear(xn, lw.in_proj)
        y = torch.empty(b.n, m.heads * m.vdim, dtype=self.dtype,
                        device=self.device)
        state = self.cache.state[i]
        if b.singles:
            self.ops.hgrn2_step(y, proj, state, lw.f_bias, lw.lower, lw.norm,
                                b.seg[:, :b.singles], eps)
        if b.singles < b.seg.size(1):
            self.ops.hgrn2_scan(y, proj, state, lw.f_bias, lw.lower,
                                lw.norm, b.seg[:, b.singles:], b.max_len, eps)
        return self._linear(y, lw.proj)

    def _splits(self, m, n_seg: int, max_ctx: int) -> int:
        """Blocks that share the keys of one (sequence, kv head): enough of
        them to fill the chip, none with less than two tiles a wave."""
        tiles = min(-(-max_ctx // 32),
                    -(-m.window // 32) + -(-m.keep_first // 32) + 1)
        want = -(-512 // (n_seg * m.kv_heads))
        return max(1, min(want, -(-tiles // 8), 256))

    def _attention(self, i: int, lw: _LayerWeights, b: Batch,
                   xn: torch.Tensor):
        m, eps, c = lw.mixer, self.config.norm_eps, self.cache
        proj = self._linear(xn, lw.in_proj)
        k, v = c.k[m.source], c.v[m.source]
        maps = k.size(1) // m.kv_heads
        q = torch.empty(b.n, m.heads * maps, k.size(2) // PAGE,
                        dtype=self.dtype, device=self.device)
        owns = lw.k_norm is not None    # else an earlier layer's are read
        self.ops.qk_norm_append(q, k if owns else None, v if owns else None,
                                proj, lw.q_norm, lw.k_norm, b.row_slot,
                                b.row_pos, c.table, m.vdim, eps, **lw.rotate)
        return self._linear(self.attend(m, b, q, lw.bias, **lw.two_maps),
                            lw.proj)

    def attend(self, m, b: Batch, q: torch.Tensor, bias=None, **kw):
        """Heads' outputs [n, heads * vdim] of padded queries over the cached
        keys and values, this step's included."""
        c = self.cache
        k, v = c.k[m.source], c.v[m.source]
        maps = k.size(1) // m.kv_heads
        y = torch.empty(b.n, m.heads * m.vdim, dtype=self.dtype,
                        device=self.device)

        def attend(seg, max_len, splits, part=(None, None)):
            self.ops.paged_attn(y, q, k, v, bias, c.table, seg, max_len,
                                m.window, m.keep_first, m.scale, splits,
                                *part, **kw)

        if b.singles:
            splits = self._splits(m, b.singles, b.max_ctx)
            part = (None, None)
            if splits > 1 or maps > 1:
                cells = b.singles * m.heads * maps * splits
                part = (torch.empty(cells * v.size(2) // PAGE, dtype=torch.float32,
                                    device=self.device),
                        torch.empty(cells * 2, dtype=torch.float32,
                                    device=self.device))
            attend(b.seg[:, :b.singles], 1, splits, part)
        if b.singles < b.seg.size(1):
            attend(b.seg[:, b.singles:], b.max_len, 0)
        return y

    def _mix(self, i: int, lw: _LayerWeights, b: Batch, xn: torch.Tensor):
        if lw.mix is not None:
            return lw.mix(b, xn)
        if lw.mixer.kind == "hgrn2":
            return self._hgrn2(i, lw, b, xn)
        return self._attention(i, lw, b, xn)

    # -- blocks with norms on the sublayers' outputs only ---------------
    def _stream_step(self, b: Optional[Batch], x, y=None, post_w=None,
                     reader=None, final=False, rows=False, **kw):
        """x <- embed(tokens) or x + norm(y), with routed experts and the
        average over depth if asked for; returns what reads the stream next:
        layer ``reader``'s mixer (its token shift applied), the head
        (``final``), a feed-forward (``rows``) or nothing."""
        xn, shift = None, None
        if reader is not None:
            shift = self.layers[reader].shift
        if reader is not None or final or rows:
            xn = torch.empty(x.shape, dtype=self.dtype, device=self.device)
        single = b is not None and b.singles == b.seg.size(1)
        if shift is not None and single:    # the previous row is in the slot
            kw.update(shift=shift, prev=self.cache.prev[reader],
                      row_slot=b.row_slot, row_pos=b.row_pos)
        later = shift is not None and not single
        self.ops.stream_step(
            x, y=y, post_w=post_w, xn=None if later else xn,
            next_w=self.final if final else None,
            groups=self.config.norm_groups, eps=self.config.norm_eps, **kw)
        if later:
            self.ops.token_shift(xn, x, shift, self.cache.prev[reader],
                                 b.seg, b.max_len)
        return xn

    def _shared_expert(self, lw: _LayerWeights, xn: torch.Tensor):
        F = lw.shared_ff
        if not F:
            return None
        mid = torch.empty(xn.size(0), F, dtype=self.dtype, device=self.device)
        if self.hip and self.dtype == torch.bfloat16 and xn.size(0) == 1 \
                and 8 <= xn.size(1) <= 32768 and xn.size(1) % 8 == 0:
            self.ops.gemv_swiglu(mid, lw.shared_in[:F], lw.shared_in[F:], xn,
                                 False)
        else:
            h = self._linear(xn, lw.shared_in)
            self.ops.gated_act(mid, h[:, :F], h[:, F:], lw.experts.act)
        return self._linear(mid, lw.shared_out)

    def _run_output_normed(self, b: Batch, rows: Optional[torch.Tensor],
                           final: bool, layers_out: Optional[list] = None):
        """All local layers.  Returns (rows [n, streams * width], final-normed
        rows or None); ``rows`` are the stream, then what the layers average:
        the embedding and every layer's result, where later layers exist."""
        cfg, first, n = self.config, self.first_layer, b.n
        L, E = len(self.layers), cfg.n_embd
        states = None
        if cfg.depth_average:
            states = torch.empty(min(first + L + 1, cfg.n_layer), n, E,
                                 dtype=torch.float32, device=self.device)
        reader = 0 if L else None
        if rows is None:
            x = torch.empty(n, E, dtype=torch.float32, device=self.device)
            xn = self._stream_step(
                b, x, reader=reader, final=final and not L, tokens=b.tokens,
                table=self.wte, scale=cfg.embedding_scale,
                keep=None if states is None else states[0])
        else:
            x = rows[:, :E].contiguous()
            for j in range(0 if states is None else first + 1):
                states[j] = rows[:, (j + 1) * E:(j + 2) * E]
            xn = self._stream_step(b, x, reader=reader, final=final and not L)
        for i, lw in enumerate(self.layers):
            last = i + 1 == L
            end = dict(reader=None if last else i + 1, final=final and last)
            if states is not None:
                seen = first + i + 1
                end.update(hist=states[:seen], coef=lw.depth)
                if seen < states.size(0):
                    end.update(keep=states[seen])
            y = self._mix(i, lw, b, xn)
            if not lw.mlp:
                xn = self._stream_step(b, x, y, lw.norm1b, **end)
            else:
                ahead = {}
                if states is not None and n <= FEW_ROWS:
                    # other blocks of this launch sum up what is there
                    ahead.update(hist=end["hist"], coef=lw.depth,
                                 past=torch.empty_like(x))
                    end.update(hist=ahead["past"].unsqueeze(0),
                               coef=lw.depth_end)
                xn = self._stream_step(b, x, y, lw.norm1b, rows=True, **ahead)
                if lw.experts is not None:
                    out, weight, plan = lw.experts(xn)
                    y = self._shared_expert(lw, xn)
                    end.update(routed=out, routed_w=weight, chosen=plan,
                               experts=lw.experts.experts)
                else:
                    y = self._linear(self._linear(xn, lw.fc, lw.act), lw.down)
                xn = self._stream_step(b, x, y, lw.norm2b, **end)
            if layers_out is not None:
                layers_out.append(x.clone())
        return (x, states), xn

    def _run(self, b: Batch, x: Optional[torch.Tensor], final: bool,
             layers_out: Optional[list] = None):
        """All local layers.  Returns (x, final-normed rows or None)."""
        if not self.config.pre_norms:
            return self._run_output_normed(b, x, final, layers_out)
        norms = [lw.norm1 for lw in self.layers[1:]]
        norms.append(self.final if final else None)
        first = self.layers[0].norm1 if self.layers else norms[0]
        if x is None:
            x = torch.empty(b.n, self.config.n_embd, dtype=torch.float32,
                            device=self.device)
            xn = self._norm_step(x, next_w=first, tokens=b.tokens,
                                 row_pos=b.row_pos)
        else:
            xn = self._norm_step(x, next_w=first)
        for i, (lw, after) in enumerate(zip(self.layers, norms)):
            if self.parallel:
                y, routed = lw.step(b, xn)
                xn = self._norm_step(x, y, None, after, routed=routed)
                if layers_out is not None:
                    layers_out.append(x.clone())
                continue
            y = self._mix(i, lw, b, xn)
            if lw.mlp:
                xn = self._norm_step(x, y, lw.norm1b, lw.norm2,
                                     gain=lw.gain1, post_w2=lw.norm1c)
                y = self._linear(self._linear(xn, lw.fc, lw.act), lw.down)
                xn = self._norm_step(x, y, lw.norm2b, after, gain=lw.gain2)
            else:
                xn = self._norm_step(x, y, lw.norm1b, after, gain=lw.gain1,
                                     post_w2=lw.norm1c)
            if layers_out is not None:
                layers_out.append(x.clone())
        return x, xn

    # ------------------------------------------------------------------
    # batches
    # ------------------------------------------------------------------
    def _batch(self, entries: Sequence[Tuple[int, int]],
               tokens: Optional[Sequence[int]]) -> Tuple[Batch, List[int]]:
        """entries: (slot, rows).  Takes the cache rows and returns the
        device batch and each entry's first row."""
        c = self.cache
        if len({s for s, _ in entries}) != len(entries):
            raise ValueError("a sequence can be in a step only once")
        for slot, n in entries:
            if n < 1:
                raise ValueError("an entry needs at least one token")
            if c.length[slot] + n > self.max_ctx:
                raise ValueError(
                    f"sequence of {c.length[slot] + n} tokens, at most "
                    f"{self.max_ctx} fit")
        pos0 = [c.length[slot] for slot, _ in entries]
        c.extend({slot: n for slot, n in entries})
        starts, at = [], 0
        for _, n in entries:
            starts.append(at)
            at += n
        order = sorted(range(len(entries)), key=lambda e: entries[e][1] > 1)
        cols = [(starts[e], entries[e][1], entries[e][0], pos0[e])
                for e in order]
        seg = list(map(list, zip(*cols)))
        row_slot = [s for s, n in entries for _ in range(n)]
        row_pos = [p + t for p, (_, n) in zip(pos0, entries)
                   for t in range(n)]
        flat = torch.tensor(row_slot + row_pos + sum(seg, [])
                            + list(tokens or ()), dtype=torch.int32)
        flat = flat.to(self.device)
        S = len(entries)
        b = Batch(
            n=at,
            seg=flat[2 * at:2 * at + 4 * S].view(4, S),
            singles=sum(n == 1 for _, n in entries),
            max_len=max(n for _, n in entries),
            row_slot=flat[:at], row_pos=flat[at:2 * at],
            tokens=flat[2 * at + 4 * S:] if tokens is not None else None,
            max_ctx=max(p + n for p, (_, n) in zip(pos0, entries)),
            entries=cols,
        )
        return b, starts

    def _check_tokens(self, tokens) -> None:
        V = self.wte.size(0)
        if tokens and not (0 <= min(tokens) and max(tokens) < V):
            raise ValueError(f"token ids must be in [0, {V})")

    # ------------------------------------------------------------------
    # public steps
    # ------------------------------------------------------------------
    @torch.no_grad()
    def step(self, entries: Sequence[Tuple[int, Sequence[int]]],
             want: Optional[Sequence[Sequence[int]]] = None,
             layers_out: Optional[list] = None) -> Optional[torch.Tensor]:
        """Run the given tokens of each entry's sequence; ``want[e]`` are the
        places among entry ``e``'s tokens whose logits are returned (default:
        the last), in order, as [wanted, vocab]; None if none is wanted."""
        if want is None:
            want = [[len(t) - 1] for _, t in entries]
        tokens = [int(t) for _, ts in entries for t in ts]
        self._check_tokens(tokens)
        if (self.use_graphs and layers_out is None
                and all(len(t) == 1 for _, t in entries)):
            logits = self.decode([s for s, _ in entries], tokens)
            rows = [e for e, w in enumerate(want) for _ in w]
            if not rows:
                return None
            return logits if rows == list(range(len(entries))) \
                else logits[rows]
        b, starts = self._batch([(s, len(t)) for s, t in entries], tokens)
        rows = [s + k for s, w in zip(starts, want) for k in w]
        _, xn = self._run(b, None, bool(rows), layers_out)
        if not rows:
            return None
        if rows != list(range(b.n)):
            xn = xn[torch.tensor(rows, device=self.device)]
        return self._linear(xn, self.head)

    @torch.no_grad()
    def hidden(self, slot: int, tokens: Optional[Sequence[int]] = None,
               x: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Pipeline stages: one sequence's tokens (starter) or the rows of
        the stage before (secondary) -> rows after the local layers, fp32:
        the residual stream (with the results that later layers average),
        then the cached rows that later stages may read."""
        rows = None
        if tokens is not None:
            self._check_tokens(tokens)
            n = len(tokens)
        else:
            rows = x.reshape(-1, self.config.ring_width).float()
            n, x = rows.size(0), rows[:, :self.ring_streams()].clone()
        b, _ = self._batch([(slot, n)], tokens)
        for src, cols in self.ring_in.items():
            self._ring_rows(src, b, rows[:, cols].to(self.dtype).contiguous(),
                            store=True)
        x = self._run(b, x, False)[0]
        if isinstance(x, tuple):        # the stream and what layers average
            x = x[0] if x[1] is None else torch.cat((x[0], *x[1]), 1)
        if self.config.ring_width == x.size(1):
            return x
        out = torch.zeros(n, self.config.ring_width, device=self.device) \
            if rows is None else rows.clone()
        out[:, :x.size(1)] = x
        for src, cols in self.ring_out.items():
            c = torch.empty(n, cols.stop - cols.start, dtype=self.dtype,
                            device=self.device)
            self._ring_rows(src, b, c, store=False)
            out[:, cols] = c
        return out

    def ring_streams(self) -> int:
        """Columns of a ring row ahead of the shared cache rows."""
        return self.config.ring_width - sum(
            self.config.shared_rows().values())

    def _ring_rows(self, src: int, b: Batch, rows: torch.Tensor,
                   store: bool) -> None:
        """This step's rows of layer ``src``'s latents, or keys and values:
        into the pages, or out of them."""
        c, ops = self.cache, self.ops
        if src in c.k:
            m = self.config.layers[src]["mixer"]
            ops.kv_rows(rows, c.k[src], c.v[src], b.row_slot, b.row_pos,
                        c.table, m["dim"], m["vdim"], store)
        elif store:
            ops.latent_norm_append(c.latent[src], rows, None, b.row_slot,
                                   b.row_pos, c.table, self.config.norm_eps)
        else:
            ops.latent_gather(rows, c.latent[src], c.table, b.seg, b.n)

    @torch.no_grad()
    def logits(self, x: torch.Tensor) -> torch.Tensor:
        """Rows of the last stage -> logits."""
        x = x.reshape(-1, self.config.ring_width)[:, :self.config.n_embd]
        x = x.float().contiguous()
        if self.config.pre_norms:
            xn = self._norm_step(x, next_w=self.final)
        else:
            xn = self._stream_step(None, x, final=True)
        return self._linear(xn, self.head)

    # ------------------------------------------------------------------
    # single-token steps (hipGraph per batch size)
    # ------------------------------------------------------------------
    def _decode_step(self, n: int) -> _DecodeStep:
        size = 1
        while size < n:
            size *= 2
        st = self._steps.get(size)
        if st is not None:
            return st
        st = _DecodeStep(self, size)

        def forward():
            _, xn = self._run(st.batch, None, True)
            return self._linear(xn, self.head)

        if self.use_graphs:
            # warm-up and capture run on the spare slot only
            s = torch.cuda.Stream()
            s.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(s):
                forward()
            torch.cuda.current_stream().wait_stream(s)
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                st.logits = forward()
            st.forward_graph = g
        st.forward = forward
        self._steps[size] = st
        return st

    @torch.no_grad()
    def decode(self, slots: Sequence[int],
               tokens: Optional[Sequence[int]] = None,
               keys: Optional[Sequence[int]] = None) -> torch.Tensor:
        """One token for each slot; logits [len(slots), vocab], valid until
        the next call.  Without ``tokens`` the step continues from what
        ``sample_decoded`` drew for the same slots, on the device."""
        c = self.cache
        slots = list(slots)
        for s in slots:
            if c.length[s] + 1 > self.max_ctx:
                raise ValueError(f"at most {self.max_ctx} tokens fit")
        st = self._decode_step(len(slots))
        if tokens is None:
            if st.slots != slots:
                raise ValueError("the batch changed: pass its tokens")
            c.extend({s: 1 for s in slots})
        else:
            if len(set(slots)) != len(slots):
                raise ValueError("a sequence can be in a step only once")
            pos = [c.length[s] for s in slots]
            c.extend({s: 1 for s in slots})
            st.load(slots, pos, [int(t) for t in tokens], keys or slots,
                    c.spare)
        if st.forward_graph is not None:
            st.forward_graph.replay()
        else:
            st.logits = st.forward()
        self._last = st
        return st.logits[:len(slots)]

    @torch.no_grad()
    def sample_decoded(self, temperature: float, top_k, seed: int,
                       top_p: float = 1.0) -> torch.Tensor:
        """Draw from the logits of the last ``decode`` on the device (bf16
        stages) and make the drawn tokens its next input; int32 tokens."""
        st = self._last
        key = (float(temperature), int(top_k or 0), int(seed), float(top_p))

        def draw():
            self._hip_sample(st.sampled, st.logits, st.scratch, key,
                             st.io[3], st.io[5], 1)
            self.ops.advance_batch(st.io[2], st.sampled, st.io[3], st.io[4],
                                   self.cache.spare)

        if not self.use_graphs:
            draw()
        else:
            g = st.sample_graphs.get(key)
            if g is None:
                torch.cuda.synchronize()
                g = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g):
                    draw()
                st.sample_graphs[key] = g
            g.replay()
        return st.sampled[:len(st.slots)]

    @property
    def samples_on_device(self) -> bool:
        return self.hip and self.dtype == torch.bfloat16

    def _hip_sample(self, out, logits, scratch, key, pos, keys,
                    pos_bias: int) -> None:
        t, k, seed, p = key
        self.ops.sample(out, logits, scratch, t, k, t > 0.0,
                        seed & 0x7FFFFFFF, pos, keys, logits.size(0), p,
                        pos_bias=pos_bias)

    @torch.no_grad()
    def sample(self, logits: torch.Tensor, temperature: float, top_k, seed,
               top_p: float, pos: Sequence[int], keys: Sequence[int],
               generators=None) -> List[int]:
        """Draw one token per row.  On the device the draw is keyed by
        (seed, key, position of the drawn token), so it does not depend on
        the schedule; elsewhere each row has a torch generator."""
        if self.samples_on_device:
            n = logits.size(0)
            pk = torch.tensor([list(pos), list(keys)], dtype=torch.int32)
            pk = pk.to(self.device)
            out = torch.zeros(n, dtype=torch.int32, device=self.device)
            scratch = torch.zeros(520 * n, dtype=torch.int32,
                                  device=self.device)
            self._hip_sample(out, logits.contiguous(), scratch,
                             (float(temperature), int(top_k or 0),
                              int(seed or 0), float(top_p)), pk[0], pk[1], 0)
            return out.tolist()
        return [int(sample_token(
            row, temperature=temperature, top_k=top_k, top_p=top_p,
            generator=generators[i] if generators else None))
            for i, row in enumerate(logits)]

    # ------------------------------------------------------------------
    # what chat and the runners share with DecodeEngine
    # ------------------------------------------------------------------
    def prefill_prompt(self, tokens: torch.Tensor, slot: int,
                       pos0: int = 0) -> torch.Tensor:
        c = self.cache
        if pos0 == 0:
            if c.is_live(slot):
                c.release(slot)
            c.admit(slot)
        if c.length[slot] != pos0:
            raise ValueError(
                f"slot {slot} holds {c.length[slot]} tokens, not {pos0}")
        return self.hidden(slot, tokens=tokens.reshape(-1).tolist())

    def set_slot_pos(self, slot: int, pos: int) -> None:
        """Positions live in the cache; nothing to stage."""
