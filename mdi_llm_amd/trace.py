"""Replay of recorded token streams, for comparing logits across builds.

The input is JSON lines, one engine step each: which requests take part, the
ids they continue with, the places whose logits are kept (``want``), and the
requests that end.  Steps go through ``HybridEngine.step``, as generation
does, over a ``HybridCache`` whose pool the caller bounds; no token is drawn.
"""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path
from typing import Dict, IO, Iterable

import torch

from .models.stages import StarterStage
from .parallel.runner import make_runner
from .utils.checkpoint import load_from_pt

__all__ = ["load_runner", "replay", "main"]

SLOTS = 4


def load_runner(model_dir, dtype: torch.dtype, device: torch.device,
                max_tokens: int):
    """The checkpoint as one whole-model stage, ``SLOTS`` sequences at a time
    in ``max_tokens`` cache rows."""
    config, sd = load_from_pt(model_dir)
    if not config.is_hybrid:
        raise ValueError(
            f"{config.name!r}: only batch-step (hybrid) models are replayed")
    stage = StarterStage(config, config.n_layer)
    stage.load_state_dict(sd)
    stage = stage.to(device=device, dtype=dtype).eval()
    if config.pos_embedding != "learned":  # a table ends where it ends
        config.block_size = max(config.block_size, max_tokens)
    stage.max_seq_length = config.block_size
    return make_runner(stage, SLOTS, device, n_tokens=max_tokens)


def replay(runner, lines: Iterable[str], out_dir: Path,
           report: IO[str]) -> None:
    engine, cache = runner.engine, runner.cache
    slots: Dict[str, int] = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries, want = [], []
        for e in step["entries"]:
            if e["id"] not in slots:
                slots[e["id"]] = cache.admit()
            entries.append((slots[e["id"]], e["tokens"]))
            want.append(e["want"])
        if entries:
            logits = engine.step(entries, want)
            if logits is not None:
                (out_dir / f"{step['step']}.f32").write_bytes(
                    logits.float().cpu().numpy().astype("<f4").tobytes())
        for rid in step.get("end", ()):
            cache.release(slots.pop(rid))
        print(f"done {step['step']}", file=report, flush=True)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(
        prog="trace_run", description="Replay token traces, write logits")
    ap.add_argument("--model", type=Path, required=True,
                    help="checkpoint folder")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"],
                    default="bfloat16")
    ap.add_argument("--out", type=Path, required=True,
                    help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="cache rows of all live requests together, each "
                         "rounded up to whole pages of 64")
    args = ap.parse_args(argv)
    if not torch.cuda.is_available():
        raise RuntimeError("trace_run needs an AMD GPU")
    args.out.mkdir(parents=True, exist_ok=True)
    runner = load_runner(args.model, getattr(torch, args.dtype),
                         torch.device("cuda"), args.max_tokens)
    replay(runner, sys.stdin, args.out, sys.stdout)
    return 0
