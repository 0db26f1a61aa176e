"""Routed experts of hybrid stacks, shared by every block form that has them.
"""

from __future__ import annotations

import torch

__all__ = ["ACTS", "RoutedExperts"]

ACTS = {"silu": 0, "gelu_tanh": 1}
BIG_TILE = 128          # pairs of one expert in a tile of large batches


class RoutedExperts:
    """Operands of a ``RoutedMLP``'s router and experts."""

    def __init__(self, eng, mlp) -> None:
        self.eng = eng
        self.experts, self.top = mlp.experts, mlp.top
        self.identity, self.gated = mlp.identity, mlp.gate_rows
        self.ff, self.act = mlp.expert_ff, ACTS[mlp.act]
        self.router = mlp.router.weight.detach()
        self.choice = {}
        if getattr(mlp, "correction", None) is not None:
            self.choice = dict(
                correction=mlp.correction.detach().float().contiguous(),
                scale=mlp.scale, identity=self.identity,
                gated=bool(self.gated))
        self.up = mlp.up.weight.detach().view(self.experts, 2 * self.ff, -1)
        self.down = mlp.down.weight.detach().view(self.experts, -1, self.ff)
        width = self.router.size(1)
        self.big_tiles = eng.dtype == torch.bfloat16 \
            and self.ff % 64 == 0 and self.ff >= 128 \
            and width % 64 == 0 and width >= 256

    def __call__(self, xn: torch.Tensor):
        """xn [n, width] -> (rows [n, top, width], their weights [n, top],
        the plan).  A last column of the weights is the shared expert's gate,
        if the router has one.  Rows of identity outputs are not written; the
        plan begins with the chosen outputs [n, top]."""
        e, n = self.eng, xn.size(0)

        def new(*shape, dtype=e.dtype):
            return torch.empty(*shape, dtype=dtype, device=e.device)

        # pairs (row, choice) per expert decide the tile
        tile = BIG_TILE if self.big_tiles and \
            n * self.top >= BIG_TILE // 2 * self.experts and \
            n * max(xn.size(1), self.top * self.ff) < 1 << 30 else 16
        weight = new(n, self.top + self.gated, dtype=torch.float32)
        plan = e.ops.moe_route(weight, xn, self.router, self.top, tile,
                               **self.choice)
        mid = new(n * self.top, self.ff)
        e.ops.moe_up(mid, xn, self.up, plan, self.act, tile)
        out = new(n, self.top, xn.size(1))
        e.ops.moe_down(out, mid, self.down, plan, tile)
        return out, weight, plan
