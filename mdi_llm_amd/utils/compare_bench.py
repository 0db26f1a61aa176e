"""Throughput of a hybrid stack beside the existing model of equal size:
prefill of one prompt, decode of one sequence and of a batch, both models in
turn in one process (random weights, synthetic tokens)."""

from __future__ import annotations

import sys
import time
from typing import Callable, Dict

import torch

from ..config import ModelConfig
from ..models.stages import StarterStage
from ..parallel.runner import make_runner

__all__ = ["PAIRS", "compare"]

# hybrid -> existing model of equal width, depth and weights per token
PAIRS = {
    "nerozen-1b": "tiny-llama-1.1b-chat",
    "nerozen-8b": "Meta-Llama-3-8B-Instruct",
    "resolorn-1b": "tiny-llama-1.1b-chat",
    "resolorn-8b": "Meta-Llama-3-8B-Instruct",
    "dinuzen-1b": "tiny-llama-1.1b-chat",
    "dinuzen-8b": "Meta-Llama-3-8B-Instruct",
    # the closest one: matrix states and windowed attention
    "sosutar-1b": "nerozen-1b",
    "sosutar-8b": "nerozen-8b",
}
SAMPLING = dict(temperature=0.8, top_k=200, seed=1234)


def _stage(cfg: ModelConfig, device, max_seq: int) -> StarterStage:
    torch.manual_seed(1234)
    torch.set_default_dtype(torch.bfloat16)
    with torch.device(device):
        stage = StarterStage(cfg, cfg.n_layer)
    torch.set_default_dtype(torch.float32)
    with torch.no_grad():
        for p in stage.parameters():
            p.normal_(0.0, 0.02)
    stage.max_seq_length = min(max_seq, cfg.block_size)
    return stage.eval()


def _weights(cfg: ModelConfig) -> int:
    """Matrix weights that one token uses."""
    return sum(cfg.layer_weights(i, active=True) for i in range(cfg.n_layer))


def _timed(run: Callable[[], None], n: int) -> float:
    """Seconds per call, after one untimed call."""
    run()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(n):
        run()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / n


def _hybrid(cfg, device, prompt: int, batch: int, steps: int) -> dict:
    max_seq = prompt + 64
    stage = _stage(cfg, device, max_seq)
    short = 128
    r = make_runner(stage, batch, device,
                    n_tokens=max(max_seq, batch * (short + 4 * steps)) + 4096)
    eng, c = r.engine, r.cache
    out = {"weights": _weights(cfg)}
    toks = torch.randint(0, cfg.vocab_size, (max_seq,)).tolist()

    def prefill():
        c.reset()
        eng.step([(c.admit(), toks[:prompt])])

    out["prefill_tok_s"] = prompt / _timed(prefill, 5)

    for name, n, ctx in (("decode1", 1, short), ("decode1_long", 1, prompt),
                         (f"decode{batch}", batch, short)):
        c.reset()
        slots = [c.admit() for _ in range(n)]
        for s in slots:
            eng.step([(s, toks[:ctx])])
        steps_ = steps if ctx == short else 16
        eng.decode(slots, [1] * n)
        eng.sample_decoded(**SAMPLING)

        def step():
            eng.decode(slots)
            eng.sample_decoded(**SAMPLING)

        out[name + "_tok_s"] = n / _timed(step, steps_)
    return out


def _existing(cfg, device, prompt: int, batch: int, steps: int) -> dict:
    from ..ops.group_engine import GroupDecodeEngine

    short = 128
    stage = _stage(cfg, device, prompt + 64)
    r = make_runner(stage, batch, device)
    eng = r.engine
    eng.ensure_fused_graphs(0.8, 200, 1234)
    geng = GroupDecodeEngine(stage, stage.kv_pool, batch)
    geng.ensure_graphs(0.8, 200, 1234)
    r.reset()
    toks = torch.randint(0, cfg.vocab_size, (stage.max_seq_length,),
                         device=device)
    out = {"weights": _weights(cfg)}

    def prefill():
        r.tail(r.prefill_head(toks[:prompt], 0)[-1])

    out["prefill_tok_s"] = prompt / _timed(prefill, 5)
    for name, ctx in (("decode1", short), ("decode1_long", prompt)):
        r.prefill_head(toks[:ctx], 0)
        out[name + "_tok_s"] = 1 / _timed(
            lambda: eng.standalone_step(0), steps if ctx == short else 16)
    for s in range(batch):
        r.prefill_head(toks[:short], s)
        geng.set_slot_pos(s, short)
    geng.set_group(torch.arange(batch, dtype=torch.int32, device=device))
    out[f"decode{batch}_tok_s"] = batch / _timed(geng.standalone_step, steps)
    return out


def compare(name: str, prompt: int = 4096, batch: int = 32,
            steps: int = 64) -> Dict[str, dict]:
    """Measure ``name`` and its counterpart; tokens/s by phase."""
    device = torch.device("cuda:0")
    res = {}
    for model in (name, PAIRS[name]):
        cfg = ModelConfig.from_name(model)
        run = _hybrid if cfg.is_hybrid else _existing
        # the counterpart's position limit does not bound its kernels
        cfg.block_size = max(cfg.block_size, prompt + 64)
        res[model] = {k: round(v, 1) if k != "weights" else v
                      for k, v in run(cfg, device, prompt, batch,
                                      steps).items()}
        print(f"[compare] {model}: {res[model]}", file=sys.stderr,
              flush=True)
        torch.cuda.empty_cache()
    return res
