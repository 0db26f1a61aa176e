"""Continuous batching for runners whose engine takes ragged steps.

Requests wait until a sequence slot and enough cache pages for their whole
length are free, enter in portions of at most ``budget`` tokens a step
beside the requests that already decode, and leave their slot and pages to
the next one as soon as they end.
"""

from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List, Optional, Sequence, Tuple

import torch

from ..models.cache import CacheFull

__all__ = ["BatchScheduler", "Request"]


@dataclass
class Request:
    rid: int
    prompt: List[int]
    max_new: int
    output: List[int] = field(default_factory=list)
    fed: int = 0                    # prompt tokens already in the cache
    slot: Optional[int] = None
    generator: Optional[torch.Generator] = None

    @property
    def decoding(self) -> bool:
        return self.fed == len(self.prompt)


class BatchScheduler:
    def __init__(self, runner, sampling, stop_tokens: Sequence = (),
                 budget: int = 4096) -> None:
        self.engine = runner.engine
        self.cache = runner.cache
        self.pos = runner.pos
        self.sampling = sampling
        self.stop_tokens = [list(s) for s in stop_tokens]
        self.budget = max(1, budget)
        self.requests: List[Request] = []
        self.waiting: Deque[Request] = deque()
        self.live: List[Request] = []
        self._chained: List[int] = []   # slots whose draw is on the device

    @property
    def idle(self) -> bool:
        return not self.waiting and not self.live

    def add(self, prompt: Sequence[int], max_new: int) -> Request:
        r = Request(len(self.requests), list(prompt), max_new)
        if not r.prompt or max_new < 1:
            raise ValueError("a request has a prompt and asks for tokens")
        if len(r.prompt) > self.engine.max_ctx:
            raise CacheFull(
                f"prompt of {len(r.prompt)} tokens, the cache holds "
                f"{self.engine.max_ctx}")
        if self.sampling.seed is not None:
            r.generator = torch.Generator(device=self.engine.device)
            r.generator.manual_seed(self.sampling.seed + r.rid)
        self.requests.append(r)
        self.waiting.append(r)
        return r

    def _rows(self, r: Request) -> int:
        """Cache rows the request can come to hold (its last token is never
        fed back)."""
        return min(len(r.prompt) + r.max_new - 1, self.engine.max_ctx)

    def _admit(self) -> None:
        c = self.cache
        while self.waiting and c.free_slots:
            r = self.waiting[0]
            promised = sum(c.pages_for(self._rows(q)) for q in self.live)
            if promised + c.pages_for(self._rows(r)) > c.n_pages:
                return
            self.waiting.popleft()
            r.slot = c.admit()
            self.live.append(r)

    def _finish(self, r: Request) -> None:
        self.live.remove(r)
        self.cache.release(r.slot)
        r.slot = None

    def _ended(self, r: Request) -> bool:
        if len(r.output) >= r.max_new:
            return True
        if len(r.prompt) + len(r.output) > self.engine.max_ctx:
            return True
        return any(s and r.output[-len(s):] == s for s in self.stop_tokens)

    def step(self) -> List[Tuple[int, int]]:
        """One engine step; the (request id, token) pairs it produced."""
        self._admit()
        if not self.live:
            raise CacheFull("nothing can be admitted")
        if all(r.decoding for r in self.live):
            drawn = self._decode_step()
        else:
            drawn = self._mixed_step()
        out = []
        for r, tok in drawn:
            r.output.append(tok)
            self.pos[r.slot] = self.cache.length[r.slot]
            out.append((r.rid, tok))
            if self._ended(r):
                self._finish(r)
        return out

    def _draw(self, logits, rs: List[Request]) -> List[int]:
        s = self.sampling
        return self.engine.sample(
            logits, s.temperature, s.top_k, s.seed, s.top_p,
            [self.cache.length[r.slot] for r in rs], [r.rid for r in rs],
            [r.generator for r in rs])

    def _decode_step(self):
        rs, s, eng = list(self.live), self.sampling, self.engine
        slots = [r.slot for r in rs]
        if self._chained == slots:
            logits = eng.decode(slots)
        else:
            logits = eng.decode(slots, [r.output[-1] for r in rs],
                                [r.rid for r in rs])
        if eng.samples_on_device:
            toks = eng.sample_decoded(s.temperature, s.top_k, s.seed or 0,
                                      s.top_p).tolist()
            self._chained = slots
        else:
            toks = self._draw(logits, rs)
        return list(zip(rs, toks))

    def _mixed_step(self):
        self._chained = []
        entries, want, ready = [], [], []
        left = self.budget
        for r in self.live:
            if r.decoding:
                entries.append((r.slot, r.output[-1:]))
                want.append([0])
                ready.append(r)
                left -= 1
        for r in [r for r in self.live if not r.decoding]:
            if left <= 0:
                break
            part = r.prompt[r.fed:r.fed + left]
            r.fed += len(part)
            left -= len(part)
            entries.append((r.slot, part))
            want.append([len(part) - 1] if r.decoding else [])
            if r.decoding:
                ready.append(r)
        logits = self.engine.step(entries, want)
        if not ready:
            return []
        return list(zip(ready, self._draw(logits, ready)))
