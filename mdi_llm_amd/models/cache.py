"""Sequence cache of hybrid stacks: paged K/V and latents, and recurrent
state slots.

``model.KVCachePool`` gives every slot ``max_seq`` rows.  Here the K/V rows
of all sequences share one pool of 64-token pages, taken as a sequence grows
and given back when it ends, and each recurrent layer has one fixed-size
state per slot.  One page table serves all attention layers of the stage:
page ``p`` is row ``p`` of every layer's arena.

Layout (what the kernels in ``paged_attn.inc``, ``row_attn.inc`` and
``hybrid_kernels.hip`` read): K pages ``[pages, kv_heads, 64 * dpad]`` and V
pages ``[pages, kv_heads, 64 * vpad]`` in MFMA operand order (``k_index``,
``v_index``), latent pages ``[pages, 64, rpad]`` with one zero-padded row per
token, states ``[slots, heads, dim, vstride]`` (or ``[slots, channels]``) in
fp32.  Differential attention has a K page per map and kv head, ``[pages,
kv_heads * 2, 64 * dpad]``.  Layers that read one latent, or one layer's keys
and values, share its pages (``latent``, ``k`` and ``v`` are keyed by the layer
that makes them).  A matrix memory with exponential gates keeps its
normaliser as one more column and the exponent of both in ``peak`` (``[slots,
heads]``, fp32).  A short convolution's last inputs (``conv``, ``[slots, taps
- 1, channels]``) and the previous token's row of a layer with token shift
(``prev``, fp32) are part of a slot as well.

Nothing needs clearing when a page or slot is taken again: keys past a
sequence's end are masked, and a recurrence, a convolution and a shift start
from zeros at position 0.
"""

from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

__all__ = ["HybridCache", "CacheFull", "PAGE", "k_index", "v_index"]

PAGE = 64


class CacheFull(RuntimeError):
    """No free slot, or not enough free pages."""


def _pad_to(n: int, sizes: Sequence[int], what: str) -> int:
    for s in sizes:
        if n <= s:
            return s
    raise ValueError(f"{what} {n} is larger than {sizes[-1]}")


def _in_block(row: torch.Tensor, step: torch.Tensor) -> torch.Tensor:
    """Place in a 16 x 32 block: lane (quad of steps, row) holds four steps
    of either half."""
    return ((step % 16 // 4) * 16 + row) * 8 + step // 16 * 4 + step % 4


def k_index(dpad: int) -> torch.Tensor:
    """[64 keys, dpad channels] -> place in a K page."""
    key = torch.arange(PAGE).view(-1, 1)
    d = torch.arange(dpad).view(1, -1)
    return (key // 16 * (dpad // 32) + d // 32) * 512 \
        + _in_block(key % 16, d % 32)


def v_index(vpad: int) -> torch.Tensor:
    """[64 keys, vpad columns] -> place in a V page."""
    key = torch.arange(PAGE).view(-1, 1)
    c = torch.arange(vpad).view(1, -1)
    return (key // 32 * (vpad // 16) + c // 16) * 512 \
        + _in_block(c % 16, key % 32)


class HybridCache:
    """``n_tokens`` bounds the rows of all live sequences together, each
    rounded up to whole pages.  One further slot with a page of its own (the
    spare) absorbs the padding entries of fixed-size decode batches."""

    fp8 = False

    def __init__(self, mixers, n_slots: int, n_tokens: int,
                 device: torch.device, dtype: torch.dtype,
                 shift_width: int = 0) -> None:
        self.n_slots = n_slots
        self.n_pages = max(1, -(-n_tokens // PAGE))
        self.spare = n_slots
        self.device = device
        self.dtype = dtype
        self.k: Dict[int, torch.Tensor] = {}
        self.v: Dict[int, torch.Tensor] = {}
        self.state: Dict[int, torch.Tensor] = {}
        self.latent: Dict[int, torch.Tensor] = {}
        self.conv: Dict[int, torch.Tensor] = {}
        self.prev: Dict[int, torch.Tensor] = {}
        self.peak: Dict[int, torch.Tensor] = {}
        # (a mixer that is made of parts caches what they cache)
        parts = [(i, p) for i, m in enumerate(mixers)
                 for p in getattr(m, "parts", (m,))]
        for i, m in parts:
            if shift_width:
                self.prev[i] = torch.zeros(n_slots + 1, shift_width,
                                           device=device,
                                           dtype=torch.float32)
            if m.kind in ("rglru", "mamba2"):
                self.conv[i] = torch.zeros(n_slots + 1, max(1, m.taps - 1),
                                           m.channels, device=device,
                                           dtype=dtype)
            if m.kind in ("attention", "diff_attention", "gated_attention"):
                if m.source in self.k:
                    continue
                dpad = _pad_to(m.dim, (32, 64, 128, 256), "attention dim")
                vpad = _pad_to(m.vdim, (32, 64, 128, 256), "attention vdim")
                P, G = self.n_pages + 1, m.kv_heads
                maps = getattr(m, "maps", 1)
                self.k[m.source] = torch.zeros(
                    P, G * maps, PAGE * dpad, device=device, dtype=dtype)
                self.v[m.source] = torch.zeros(
                    P, G, PAGE * vpad, device=device, dtype=dtype)
            elif m.kind == "latent_attention":
                if m.source not in self.latent:
                    rpad = _pad_to(m.rank, (64, 128, 256, 512),
                                   "latent size")
                    self.latent[m.source] = torch.zeros(
                        self.n_pages + 1, PAGE, rpad, device=device,
                        dtype=dtype)
            elif m.kind in ("rglru", "mingru"):
                self.state[i] = torch.zeros(n_slots + 1, m.width,
                                            device=device,
                                            dtype=torch.float32)
            else:
                cols = m.vdim
                if m.kind == "mlstm":
                    cols += 1
                    self.peak[i] = torch.zeros(n_slots + 1, m.heads,
                                               device=device,
                                               dtype=torch.float32)
                vstride = -(-cols // 4) * 4
                self.state[i] = torch.zeros(
                    n_slots + 1, m.heads, m.dim, vstride, device=device,
                    dtype=torch.float32)
        # the spare slot's only page is the last one
        self.table = torch.zeros(n_slots + 1, self.n_pages, device=device,
                                 dtype=torch.int32)
        self.table[self.spare] = self.n_pages
        self._free_pages: List[int] = list(range(self.n_pages))[::-1]
        self._free_slots: List[int] = list(range(n_slots))[::-1]
        self._pages: List[Optional[List[int]]] = [None] * n_slots
        self.length = [0] * n_slots

    # -- slots ------------------------------------------------------------
    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    @property
    def free_pages(self) -> int:
        return len(self._free_pages)

    @staticmethod
    def pages_for(n_tokens: int) -> int:
        return -(-n_tokens // PAGE)

    def is_live(self, slot: int) -> bool:
        return self._pages[slot] is not None

    def admit(self, slot: Optional[int] = None) -> int:
        """Start a sequence in a free slot (a given one, if asked)."""
        if slot is None:
            if not self._free_slots:
                raise CacheFull("no free sequence slot")
            slot = self._free_slots.pop()
        else:
            if self.is_live(slot):
                raise ValueError(f"slot {slot} is in use")
            self._free_slots.remove(slot)
        self._pages[slot] = []
        self.length[slot] = 0
        return slot

    def release(self, slot: int) -> None:
        """End the slot's sequence; its pages can be used again."""
        if not self.is_live(slot):
            raise ValueError(f"slot {slot} is not in use")
        self._free_pages.extend(reversed(self._pages[slot]))
        self._pages[slot] = None
        self.length[slot] = 0
        self._free_slots.append(slot)

    def reset(self, slot: Optional[int] = None) -> None:
        for s in range(self.n_slots) if slot is None else (slot,):
            if self.is_live(s):
                self.release(s)

    def missing_pages(self, slot: int, n_new: int) -> int:
        return max(0, self.pages_for(self.length[slot] + n_new)
                   - len(self._pages[slot]))

    def extend(self, extra: Dict[int, int]) -> None:
        """Make room for ``extra[slot]`` more tokens in each slot, all or
        nothing, and count them as stored."""
        need = {s: self.missing_pages(s, n) for s, n in extra.items()}
        if sum(need.values()) > len(self._free_pages):
            raise CacheFull(
                f"{sum(need.values())} pages needed, "
                f"{len(self._free_pages)} free")
        rows, cols, pages = [], [], []
        for s, n in need.items():
            for _ in range(n):
                page = self._free_pages.pop()
                rows.append(s)
                cols.append(len(self._pages[s]))
                pages.append(page)
                self._pages[s].append(page)
            self.length[s] += extra[s]
        if pages:
            idx = torch.tensor([rows, cols, pages]).to(self.device)
            self.table[idx[0], idx[1]] = idx[2].to(torch.int32)

    def memory_bytes(self) -> int:
        return sum(t.numel() * t.element_size()
                   for d in (self.k, self.v, self.state, self.latent,
                             self.conv, self.prev, self.peak)
                   for t in d.values())
