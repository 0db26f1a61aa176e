"""Nerozen in the rest of the framework: configuration, checkpoints, cache
bookkeeping, pipeline stages, command lines and trace replay."""

import io
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch
import torch.multiprocessing as mp

import nerozen_oracle as oracle
from helpers import make_toy_tokenizer
from mdi_llm_amd.config import ModelConfig, is_native_checkpoint
from mdi_llm_amd.models.cache import CacheFull, HybridCache
from nerozen_models import (MODELS, deviation, make_runner, save, tokens,
                            weights)

ROOT = Path(__file__).resolve().parent.parent
device_param = pytest.mark.parametrize(
    "device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])


def model(name="mixed", seed=0):
    cfg, rows = MODELS[name]
    return cfg, weights(cfg, rows, seed)


# ---------------------------------------------------------------------------
def test_config_round_trips(tmp_path):
    cfg, w = model()
    c = ModelConfig.from_native(cfg)
    assert c.is_hybrid and c.n_layer == 4 and c.padded_vocab_size == 133
    assert ModelConfig.from_dict(c.to_dict()).to_dict() == c.to_dict()
    c.save(tmp_path / "model_config.yaml")
    assert ModelConfig.from_file(
        tmp_path / "model_config.yaml").to_dict() == c.to_dict()
    save(tmp_path / "m", cfg, w)
    assert is_native_checkpoint(tmp_path / "m")
    assert ModelConfig.from_checkpoint(tmp_path / "m").layers == cfg["layers"]
    (tmp_path / "m" / "config.json").write_text(
        json.dumps({"architectures": ["LlamaForCausalLM"]}))
    assert not is_native_checkpoint(tmp_path / "m")


@pytest.mark.parametrize("name", ["nerozen-nano", "nerozen-1b", "nerozen-8b"])
def test_registry(name):
    c = ModelConfig.from_name(name)
    assert c.is_hybrid
    assert {l["type"] for l in c.layers} == {"hgrn2", "attention"}


def test_unknown_parts_are_refused():
    cfg, _ = model()
    for path, value in ((("layers", 0, "type"), "convolution"),
                        (("layers", 1, "mlp", "kind"), "routed")):
        bad = json.loads(json.dumps(cfg))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            ModelConfig.from_native(bad)


def test_gpt_module_refuses_hybrid_stacks():
    from mdi_llm_amd import GPT

    with pytest.raises(ValueError, match="stages"):
        GPT(ModelConfig.from_name("nerozen-nano"))


@pytest.mark.parametrize("name", list(MODELS))
def test_checkpoint_loads_every_tensor(name, tmp_path):
    from mdi_llm_amd.models.stages import StarterStage
    from mdi_llm_amd.utils.checkpoint import (has_weights, load_from_pt,
                                              save_checkpoint)

    cfg, w = model(name)
    save(tmp_path / "a", cfg, w)
    assert has_weights(tmp_path / "a") and not has_weights(tmp_path)
    config, sd = load_from_pt(tmp_path / "a")
    stage = StarterStage(config, config.n_layer)
    stage.load_state_dict(sd)  # strict
    n = sum(p.numel() for p in stage.parameters())
    assert n == sum(t.numel() for t in w.values())
    # and through the framework's own checkpoint form
    save_checkpoint(tmp_path / "b", config, sd)
    config2, sd2 = load_from_pt(tmp_path / "b")
    assert config2.to_dict() == config.to_dict()
    assert all(torch.equal(sd[k], sd2[k]) for k in sd)


def test_balanced_split_of_a_hybrid_stack():
    from mdi_llm_amd.utils.partition import balanced_split, layer_split

    c = ModelConfig.from_name("nerozen-8b")
    for n in (2, 4, 8):
        for s in (balanced_split(c, n), layer_split(c.n_layer, n)):
            assert sum(s) == c.n_layer and len(s) == n


# ---------------------------------------------------------------------------
def cache(n_slots=3, n_tokens=300):
    r = make_runner(*model(), "cpu", torch.float32, n_slots, n_tokens)
    assert isinstance(r.cache, HybridCache)
    return r.cache


def test_pages_are_taken_and_given_back():
    c = cache()
    assert c.n_pages == 5
    a, b = c.admit(), c.admit()
    c.extend({a: 64, b: 65})
    assert c.free_pages == 2 and c.length[a] == 64 and c.length[b] == 65
    assert c.missing_pages(a, 1) == 1 and c.missing_pages(b, 63) == 0
    used = c.table[a, :1].tolist() + c.table[b, :2].tolist()
    assert len(set(used)) == 3
    with pytest.raises(CacheFull):
        c.extend({a: 64, b: 128})
    assert c.free_pages == 2 and c.length[a] == 64  # nothing was taken
    c.release(a)
    assert c.free_pages == 3 and c.free_slots == 2
    with pytest.raises(ValueError):
        c.release(a)
    assert c.admit(a) == a
    with pytest.raises(ValueError):
        c.admit(a)
    c.reset()
    assert c.free_pages == 5 and c.free_slots == 3
    for _ in range(3):
        c.admit()
    with pytest.raises(CacheFull):
        c.admit()


@device_param
def test_bad_steps_are_refused(device):
    cfg, w = model()
    r = make_runner(cfg, w, device, torch.float32, 2, 128)
    a = r.cache.admit()
    for bad in ([(a, [cfg["vocab"]])], [(a, [-1])], [(a, [])],
                [(a, [1]), (a, [2])], [(a, [1] * 129)]):
        with pytest.raises(ValueError):
            r.engine.step(bad)
    assert r.cache.length[a] == 0
    r.engine.step([(a, [1] * 128)])
    with pytest.raises((ValueError, CacheFull)):
        r.engine.step([(a, [1])])


def test_requests_that_never_fit_are_refused():
    from mdi_llm_amd.parallel.runtime import SamplingParams
    from mdi_llm_amd.parallel.scheduler import BatchScheduler

    r = make_runner(*model(), "cpu", torch.float32, 2, 128)
    s = BatchScheduler(r, SamplingParams(temperature=0.0))
    with pytest.raises(CacheFull):
        s.add([1] * 129, 1)
    q = s.add([1] * 120, 50)  # ends where the cache does
    while not s.idle:
        s.step()
    assert len(q.output) == 9


# ---------------------------------------------------------------------------
def _ring_worker(rank, world, tmp, port, device):
    import torch.distributed as dist

    from mdi_llm_amd.models.stages import build_stage
    from mdi_llm_amd.parallel.ring import RingComm
    from mdi_llm_amd.parallel.runner import make_runner
    from mdi_llm_amd.parallel.runtime import PipelineRuntime, SamplingParams
    from mdi_llm_amd.utils import layer_split, split_parameters
    from mdi_llm_amd.utils.checkpoint import load_from_pt

    dist.init_process_group("gloo", init_method=f"tcp://127.0.0.1:{port}",
                            rank=rank, world_size=world)
    cfg, sd = load_from_pt(tmp)
    split = layer_split(cfg.n_layer, world)
    stage = build_stage(cfg, rank, split[rank], sum(split[:rank]))
    stage.load_state_dict(split_parameters(sd, world)[rank])
    dev = torch.device(device)
    stage = stage.to(device=dev, dtype=torch.float32)
    stage.max_seq_length = 256
    stage.eval()
    prompts = [torch.tensor(p) for p in torch.load(
        os.path.join(tmp, "prompts.pt"), weights_only=True)]
    runner = make_runner(stage, len(prompts), dev)
    comm = RingComm(cfg.ring_width, stage.max_seq_length, dev, len(prompts),
                    dtype=cfg.residual_dtype(torch.float32))
    rt = PipelineRuntime(runner, rank=rank, world=world, comm=comm,
                         device=dev)
    if rank == 0:
        res = rt.generate(prompts, 8, SamplingParams(temperature=0.0))
        torch.save([s.tolist() for s in res.sequences],
                   os.path.join(tmp, "out.pt"))
    else:
        rt.serve(n_samples=len(prompts))
    dist.barrier()
    dist.destroy_process_group()


@device_param
@pytest.mark.parametrize("world", [2, 3])
def test_ring_pipeline_matches_standalone(world, device, tmp_path):
    """Stages in processes of their own; on a GPU they share it, and the
    activations go through host memory."""
    from mdi_llm_amd.parallel.runtime import PipelineRuntime, SamplingParams

    cfg, w = model()
    save(tmp_path, cfg, w)
    prompts = [tokens(cfg, n, n) for n in (70, 5, 33)]
    torch.save(prompts, tmp_path / "prompts.pt")
    r = make_runner(cfg, w, device, torch.float32)
    ref = PipelineRuntime(r, device=torch.device(device)).generate([torch.tensor(p) for p in prompts], 8,
                                      SamplingParams(temperature=0.0))
    mp.spawn(_ring_worker,
             args=(world, str(tmp_path), 29930 + world, device),
             nprocs=world, join=True)
    got = torch.load(tmp_path / "out.pt", weights_only=True)
    assert got == [s.tolist() for s in ref.sequences]


# ---------------------------------------------------------------------------
@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    d = tmp_path_factory.mktemp("nerozen") / "toy"
    tok = make_toy_tokenizer(d)
    cfg, rows = MODELS["mixed"]
    cfg = dict(cfg, vocab=max(json.loads(tok.read_text())["model"]["vocab"]
                              .values()) + 1)
    save(d, cfg, weights(cfg, rows))
    return d


def run(args):
    return subprocess.run([sys.executable] + args, cwd=ROOT,
                          capture_output=True, text=True, timeout=240)


@device_param
def test_sample_cli(checkpoint, device):
    r = run(["sample.py", "--ckpt", str(checkpoint), "--n-samples", "3",
             "--n-tokens", "6", "--device", device, "--sequence-length",
             "512"])
    assert r.returncode == 0, r.stderr[-2000:]
    assert "sample 2" in r.stdout and "18 tokens" in r.stdout
    assert f"backend={'hip' if device == 'cuda' else 'torch'}" in r.stdout


def test_prepare_model_cli(checkpoint):
    r = run(["prepare_model.py", "--ckpt", str(checkpoint), "--n-nodes", "2"])
    assert r.returncode == 0, r.stderr[-2000:]
    assert (checkpoint / "chunks" / "2nodes" / "model_secondary0.pth"
            ).is_file()


@device_param
def test_chat_cli(checkpoint, device):
    r = subprocess.run(
        [sys.executable, "chat.py", "--ckpt", str(checkpoint), "--device",
         device, "--max-new-tokens", "5", "--sequence-length", "512"],
        cwd=ROOT, input="hello\nwho are you\n", capture_output=True,
        text=True, timeout=240)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.count(">>") == 3


@device_param
def test_trace_replay(device, tmp_path):
    from mdi_llm_amd.trace import load_runner, replay

    cfg, w = model()
    save(tmp_path / "m", cfg, w)
    a, b = tokens(cfg, 90, 1), tokens(cfg, 10, 2)
    steps = [
        dict(entries=[dict(id="a", tokens=a[:70], want=[0, 69]),
                      dict(id="b", tokens=b[:1], want=[])], end=[]),
        dict(entries=[dict(id="b", tokens=b[1:9], want=[7])], end=[]),
        dict(entries=[dict(id="b", tokens=b[9:], want=[0]),
                      dict(id="a", tokens=a[70:71], want=[0])], end=["b"]),
        dict(entries=[dict(id="a", tokens=a[71:], want=[])], end=["a"]),
    ]
    lines = [json.dumps(dict(step=n, **s)) + "\n"
             for n, s in enumerate(steps)]
    runner = load_runner(tmp_path / "m", torch.float32, torch.device(device),
                         192)
    report = io.StringIO()
    replay(runner, lines, tmp_path, report)
    assert report.getvalue().split("\n")[:4] == [f"done {n}"
                                                 for n in range(4)]
    assert runner.cache.free_pages == 3 and runner.cache.free_slots == 4
    wa, wb = (oracle.forward(cfg, w, t) for t in (a, b))
    want = {0: wa[[0, 69]], 1: wb[[8]], 2: torch.stack([wb[9], wa[70]])}
    for n, x in want.items():
        got = np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(x.shape)
        assert deviation(torch.from_numpy(got), x) < 5e-5
    assert not (tmp_path / "3.f32").exists()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(dtype, tmp_path):
    cfg, w = model("odd")
    save(tmp_path / "m", cfg, w)
    t = tokens(cfg, 12)
    line = json.dumps(dict(step=0, entries=[dict(id="x", tokens=t,
                                                 want=[11])], end=["x"]))
    r = subprocess.run(
        [str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path / "m"),
         "--dtype", dtype, "--out", str(tmp_path / "out"), "--max-tokens",
         "64"], input=line + "\n", capture_output=True, text=True,
        timeout=240)
    assert r.returncode == 0, r.stderr[-2000:]
    assert "done 0" in r.stdout
    got = torch.from_numpy(np.fromfile(tmp_path / "out" / "0.f32", "<f4"))
    want = oracle.forward(cfg, w, t)[11]
    assert deviation(got, want) < (5e-5 if dtype == "float32" else 0.06)


@pytest.mark.timeout(180)
def test_two_node_http_bootstrap(checkpoint, tmp_path):
    """Starter and secondary over the control plane: chunks are split from
    the checkpoint folder, each stage builds its own part of the layers."""
    import multiprocessing

    from test_orchestrator_e2e import _secondary_proc, _starter_proc, _topo

    topo = tmp_path / "topo.json"
    topo.write_text(json.dumps(_topo(tmp_path, 18795, 18797, 29841)))
    ctx = multiprocessing.get_context("spawn")
    q = ctx.Queue()
    procs = [ctx.Process(target=_secondary_proc, args=(str(topo), q)),
             ctx.Process(target=_starter_proc,
                         args=(str(topo), str(checkpoint), q))]
    for p in procs:
        p.start()
    procs[1].join(timeout=150)
    procs[0].join(timeout=30)
    if procs[0].is_alive():
        procs[0].terminate()
    assert procs[1].exitcode == 0
    seqs = next(r for r in (q.get(timeout=5), q.get(timeout=5))
                if isinstance(r, list))
    assert len(seqs) == 2 and all(len(s) > 6 for s in seqs)
