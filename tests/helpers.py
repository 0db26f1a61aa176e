"""Shared test fixtures: build a complete toy litGPT checkpoint dir
(model_config.yaml + lit_model.pth + tokenizer.json) on the fly; operations,
inputs and comparison of the kernel tests; runs of a sequence in portions."""

from pathlib import Path

import pytest
import torch


def make_toy_tokenizer(out_dir: Path, vocab_size: int = 256) -> Path:
    """Train a tiny byte-level BPE tokenizer and save tokenizer.json."""
    from tokenizers import Tokenizer, models, pre_tokenizers, trainers
    from tokenizers.processors import TemplateProcessing

    tok = Tokenizer(models.BPE(unk_token="<unk>"))
    tok.pre_tokenizer = pre_tokenizers.ByteLevel(add_prefix_space=False)
    trainer = trainers.BpeTrainer(
        vocab_size=vocab_size,
        special_tokens=["<unk>", "<s>", "</s>"],
    )
    corpus = [
        "the quick brown fox jumps over the lazy dog",
        "hello world this is a tiny tokenizer for tests",
        "who are you? I am a language model running on MI355X",
        "0123456789 abcdefghijklmnopqrstuvwxyz",
    ] * 8
    tok.train_from_iterator(corpus, trainer)
    out_dir.mkdir(parents=True, exist_ok=True)
    tok.save(str(out_dir / "tokenizer.json"))
    (out_dir / "tokenizer_config.json").write_text(
        '{"bos_token": "<s>", "eos_token": "</s>", "add_bos_token": false}'
    )
    return out_dir / "tokenizer.json"


def make_toy_checkpoint(out_dir: Path, name: str = "nano-test",
                        seed: int = 0) -> Path:
    from mdi_llm_amd import GPT, ModelConfig
    from mdi_llm_amd.utils.checkpoint import save_checkpoint

    torch.manual_seed(seed)
    cfg = ModelConfig.from_name(name)
    m = GPT(cfg)
    m.apply_init()
    save_checkpoint(out_dir, cfg, m.state_dict())
    make_toy_tokenizer(out_dir)
    return out_dir


# -- kernel tests: where an operation runs, and in which precision
CPU = pytest.param("cpu", torch.float32, id="cpu-f32")
GPU32 = pytest.param("cuda", torch.float32, id="gpu-f32",
                     marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda", torch.bfloat16, id="gpu-bf16",
                     marks=pytest.mark.gpu)
everywhere = pytest.mark.parametrize("device,dtype", [CPU, GPU32, GPU16])


def ops_for(device):
    if device == "cuda":
        from mdi_llm_amd.ops import require_hip_ops

        return require_hip_ops()
    from mdi_llm_amd.ops import hybrid_torch

    return hybrid_torch


def close(got, want, dtype, scale=None):
    want = want.double().cpu()
    got = got.double().cpu()
    tol = 1e-5 if dtype == torch.float32 else 1.2e-2
    scale = float(want.abs().max()) if scale is None else scale
    err = float((got - want).abs().max())
    assert err <= tol * max(scale, 1e-3), (err, scale)


def rand(*shape, seed=0, dtype=torch.float32, device="cpu"):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(dtype).to(device)


def seg(rows, device):
    return torch.tensor(list(map(list, zip(*rows))), dtype=torch.int32,
                        device=device)


def run_portions(runner, toks, portions, slot=None):
    """All logits of one sequence cut into the given portions (the last one
    repeats)."""
    c = runner.cache
    slot = c.admit() if slot is None else slot
    at, out, portions = 0, [], list(portions)
    while at < len(toks):
        n = portions.pop(0) if len(portions) > 1 else portions[0]
        part = toks[at:at + n]
        out.append(runner.engine.step([(slot, part)],
                                      [range(len(part))]).float().clone())
        at += n
    c.release(slot)
    return torch.cat(out)
