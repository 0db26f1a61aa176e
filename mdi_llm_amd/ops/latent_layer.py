"""Parallel blocks of ``HybridEngine``: latent attention beside a dense or
routed gated feed-forward.

One matrix product makes everything that reads the block's norm (query and
key/value latents, head gates, the feed-forward's gate and up halves); the
attention output and the activated feed-forward lie side by side in one
buffer, so that one more product gives what both add to the residual stream.

Attention over latents has two forms with the same result:

* absorbed: every head's query is taken into the latent space
  (q' = W_uk^T q), all heads attend to the cached rows themselves, and the
  weighted latent is brought to the value space afterwards.  Nothing is
  expanded, so this is the form of decoding and of short portions.
* expanded: the visible context becomes keys and values once, then attention
  runs per head at its own, smaller sizes: the form of prompts.

Each entry of a step takes the cheaper one.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch

from ..models.cache import PAGE
from .experts import ACTS, RoutedExperts

__all__ = ["LatentPlan", "ParallelLayer"]

MAX_EXPANDED = 256      # head sizes of the expanded form


def _round_up(n: int, k: int) -> int:
    return -(-n // k) * k


def prefers_absorbed(n: int, pos0: int, m) -> bool:
    """Multiply-adds of either form for ``n`` tokens after ``pos0``."""
    if n == 1 or max(m.dim, m.vdim) > MAX_EXPANDED:
        return True
    per_head = m.dim + m.vdim
    seen = sum(min(m.window, p) for p in (pos0 + 1, pos0 + n)) / 2
    ctx = n + min(pos0, m.window - 1)
    absorbed = n * m.rank * (per_head + 2 * seen)
    return absorbed < per_head * (m.rank * ctx + n * seen)


@dataclass
class LatentPlan:
    """How the entries of one step attend, for one geometry of layers."""

    # absorbed: seg [4, s] over the compact rows; rows maps them to the
    # step's rows (None: all of them, in order)
    seg: Optional[torch.Tensor] = None
    rows: Optional[torch.Tensor] = None
    n_rows: int = 0
    max_len: int = 1
    # expanded: seg [4, s] over the step's rows, context segments [4, s]
    # (start, len, slot, first position) over the gathered rows
    long_seg: Optional[torch.Tensor] = None
    ctx_seg: Optional[torch.Tensor] = None
    long_max: int = 0
    ctx_rows: int = 0
    ctx_max: int = 0


def make_plan(entries: List[Tuple[int, int, int, int]], n_rows: int, m,
              device, force: Optional[str] = None) -> LatentPlan:
    """``entries``: (start, len, slot, pos0) of every segment."""
    short, rows, long, ctx = [], [], [], []
    p = LatentPlan()
    for start, n, slot, pos0 in entries:
        absorbed = prefers_absorbed(n, pos0, m) if force is None \
            else force == "absorbed"
        if absorbed:
            short.append((len(rows), n, slot, pos0))
            rows.extend(range(start, start + n))
            p.max_len = max(p.max_len, n)
        else:
            first = max(0, pos0 - m.window + 1)
            ctx.append((p.ctx_rows, pos0 + n - first, slot, first))
            long.append((start, n, slot, pos0))
            p.ctx_rows += ctx[-1][1]
            p.ctx_max = max(p.ctx_max, ctx[-1][1])
            p.long_max = max(p.long_max, n)
    p.n_rows = len(rows)
    if rows == list(range(n_rows)):
        rows = []
    parts = [[x for col in zip(*t) for x in col] for t in (short, long, ctx)]
    flat = torch.tensor(sum(parts, []) + rows, dtype=torch.int32).to(device)
    at = 0
    segs = []
    for t in (short, long, ctx):
        segs.append(flat[at:at + 4 * len(t)].view(4, -1) if t else None)
        at += 4 * len(t)
    p.seg, p.long_seg, p.ctx_seg = segs
    if rows:
        p.rows = flat[at:]
    return p


class ParallelLayer:
    """Operands of one ``ParallelBlock`` and its step."""

    def __init__(self, eng, block) -> None:
        def f(norm):
            return norm.weight.detach().float().contiguous()

        self.eng, self.mixer, m = eng, block.mixer, block.mixer
        self.norm1 = f(block.norm_1)
        self.in_proj = block.in_proj.weight.detach()
        self.out_proj = block.out_proj.weight.detach()
        at, self.part = 0, {}
        for name, n in block.in_rows():
            self.part[name] = slice(at, at + n)
            at += n
        self.q_norm = f(m.q_norm)
        self.kv_norm = f(m.kv_norm) if m.owns_latent else None
        self.q_up = m.q_up.weight.detach()
        self.kv_up = m.kv_up.weight.detach()
        # absorbed form, padded to whole MFMA steps: uk as [H, rpad, dim],
        # uv as [H, vdim, rpad]
        H, D, V, R = m.heads, m.dim, m.vdim, m.rank
        self.rpad = eng.cache.latent[m.source].size(2)
        self.uk = self.kv_up.new_zeros(H, self.rpad, _round_up(D, 32))
        self.uk[:, :R, :D] = self.kv_up[:H * D].view(H, D, R).transpose(1, 2)
        self.uv = self.kv_up.new_zeros(H, V, self.rpad)
        self.uv[..., :R] = self.kv_up[H * D:].view(H, V, R)
        # feed-forward
        mlp = block.mlp
        self.ff = block.ff
        if self.ff:
            pre = "shared." if mlp.kind == "moe" else ""
            self.gate, self.up = self.part[pre + "gate"], self.part[pre + "up"]
        self.act = ACTS[mlp.act] if mlp is not None else 0
        self.experts = RoutedExperts(eng, mlp) \
            if mlp is not None and mlp.kind == "moe" else None

    # ------------------------------------------------------------------
    def _new(self, *shape, dtype=None) -> torch.Tensor:
        e = self.eng
        return torch.empty(*shape, dtype=dtype or e.dtype, device=e.device)

    def step(self, b, xn: torch.Tensor):
        """The block's sum before the residual multiplier, and the routed
        experts' rows with their weights (None without experts)."""
        m = self.mixer
        proj = self.eng._linear(xn, self.in_proj)
        y = self._new(b.n, m.out_cols + self.ff)
        branch = {}
        if self.ff:
            branch = dict(act_out=y[:, m.out_cols:], gate=proj[:, self.gate],
                          up=proj[:, self.up], act=self.act)
        self._attend(b, proj, y[:, :m.out_cols], branch)
        routed = self.experts(xn)[:2] if self.experts else None
        return self.eng._linear(y, self.out_proj), routed

    # -- attention ------------------------------------------------------
    def _attend(self, b, proj: torch.Tensor, y: torch.Tensor,
                branch: dict) -> None:
        """``branch``: the feed-forward's activation, which shares a launch
        with the latents' norms."""
        m, e = self.mixer, self.eng
        c, eps = e.cache, e.config.norm_eps
        pages = c.latent[m.source]
        cq = self._new(b.n, m.q_rank)
        kv = proj[:, self.part["dkv"]] if m.owns_latent else None
        e.ops.latent_norm_append(
            pages, kv, self.kv_norm, b.row_slot, b.row_pos, c.table, eps,
            q_out=cq, q=proj[:, self.part["dq"]], q_w=self.q_norm, **branch)
        q = e._linear(cq, self.q_up)
        gate = proj[:, self.part["g"]]
        plan = b.latent_plan(m, e.device, e.latent_form)
        if plan.seg is not None:
            self._absorbed(b, plan, q, gate, y, pages)
        if plan.long_seg is not None:
            self._expanded(b, plan, q, gate, y, pages)

    def _splits(self, plan: LatentPlan, max_ctx: int) -> int:
        """Blocks that share the pages of one group of query rows: enough of
        them to fill the chip, none without a page."""
        m = self.mixer
        pages = min(-(-max_ctx // PAGE), (m.window + plan.max_len - 2) // PAGE
                    + 2)
        blocks = plan.seg.size(1) * -(-plan.max_len * m.heads // 64)
        return max(1, min(-(-256 // blocks), pages, 256))

    def _absorbed(self, b, plan, q, gate, y, pages) -> None:
        m, e, R = self.mixer, self.eng, self.rpad
        n, H = plan.n_rows, m.heads
        qc = self._new(n, H, R)
        e.ops.head_proj(qc.view(n, H * R), q, self.uk, x_rows=plan.rows)
        splits = self._splits(plan, b.max_ctx)
        part_o = part_ml = out = None
        if splits > 1:
            part_o = self._new(n, H, splits, R, dtype=torch.float32)
            part_ml = self._new(n, H, splits, 2, dtype=torch.float32)
        else:
            out = self._new(n, H * R)
        e.ops.latent_attn(out, qc, pages, e.cache.table, plan.seg,
                          plan.max_len, m.window, m.scale, splits,
                          part_o, part_ml)
        e.ops.head_proj(y, out, self.uv, out_rows=plan.rows, gate=gate,
                        part_o=part_o, part_ml=part_ml)

    def _expanded(self, b, plan, q, gate, y, pages) -> None:
        m, e = self.mixer, self.eng
        key = (m.source, id(plan))
        ctx = b.contexts.get(key)
        if ctx is None:
            ctx = self._new(plan.ctx_rows, m.rank)
            e.ops.latent_gather(ctx, pages, e.cache.table, plan.ctx_seg,
                                plan.ctx_max)
            b.contexts[key] = ctx
        kv = e._linear(ctx, self.kv_up)
        e.ops.head_attn(y, q, kv, plan.long_seg, plan.ctx_seg, plan.long_max,
                        m.heads, m.dim, m.vdim, m.window, m.scale, gate)
