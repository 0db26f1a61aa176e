"""Sosutar in the rest of the framework: configuration, checkpoints, cache,
pipeline stages, command lines and trace replay."""

import copy
import io
import json
import re
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch
import torch.multiprocessing as mp

import sosutar_oracle as oracle
from sosutar_models import MODELS, weights
from helpers import make_toy_tokenizer
from mdi_llm_amd.config import ModelConfig, is_native_checkpoint
from nerozen_models import make_runner, save, tokens
from test_sosutar import errors
from test_nerozen_serving import _ring_worker, run

ROOT = Path(__file__).resolve().parent.parent
device_param = pytest.mark.parametrize(
    "device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])


def model(name="mixed", seed=0):
    cfg = MODELS[name]
    return cfg, weights(cfg, seed)


# ---------------------------------------------------------------------------
def test_config_round_trips(tmp_path):
    cfg, w = model()
    c = ModelConfig.from_native(cfg)
    assert c.is_hybrid and c.n_layer == 8 and c.padded_vocab_size == 133
    assert c.block_size == 700 and c.pos_embedding == "learned"
    assert c.layer_scale and c.pre_norms and not c.post_norms
    assert (c.logit_scale, c.embedding_scale) == (0.7, 1.5)
    assert c.shared_rows() == {} and c.ring_width == 72
    assert (c.n_head, c.n_query_groups, c.head_size) == (6, 2, 24)
    # a repeat of a repeat uses the layer with the tensors
    assert [c.weights_of(i) for i in range(8)] == [0, 1, 2, 3, 0, 2, 6, 2]
    assert ModelConfig.from_dict(c.to_dict()).to_dict() == c.to_dict()
    c.save(tmp_path / "model_config.yaml")
    assert ModelConfig.from_file(
        tmp_path / "model_config.yaml").to_dict() == c.to_dict()
    save(tmp_path / "m", cfg, w)
    assert is_native_checkpoint(tmp_path / "m")
    got = ModelConfig.from_checkpoint(tmp_path / "m").layers
    assert [l["mixer"] for l in got] == [l["mixer"] for l in c.layers]
    assert cfg["layers"][0]["type"] == "parallel"   # left as it was


@pytest.mark.parametrize("name", ["sosutar-nano", "sosutar-1b", "sosutar-8b"])
def test_registry(name):
    c = ModelConfig.from_name(name)
    assert c.is_hybrid and c.layer_scale
    assert {l["type"] for l in c.layers} == {"mlstm", "paired"}
    assert all(l["mlp"]["kind"] == "dense" for l in c.layers)


def test_weight_counts_follow_the_tensors():
    """Matrix weights of each layer, its own or another's."""
    for name in MODELS:
        cfg, w = model(name)
        c = ModelConfig.from_native(cfg)
        for i in range(c.n_layer):
            p = f"l{c.weights_of(i)}."
            n = sum(t.numel() for k, t in w.items()
                    if k.startswith(p) and t.dim() == 2)
            assert c.layer_weights(i) == c.layer_weights(i, active=True) == n


def test_unknown_parts_are_refused():
    cfg, _ = model()
    for path, value in ((("layers", 0, "type"), "convolution"),
                        (("layers", 1, "mlp", "kind"), "sparse"),
                        (("layers", 4, "mixer", "left", "dim"), 32),
                        (("layers", 5, "mlp"), dict(kind="dense", ff=8)),
                        (("layers", 7, "weights_of"), 1),
                        (("layers", 2, "weights_of"), 5)):
        bad = json.loads(json.dumps(cfg))   # (some layers share parts)
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            ModelConfig.from_native(bad)


def test_gpt_module_refuses_the_stack():
    from mdi_llm_amd import GPT

    with pytest.raises(ValueError, match="stages"):
        GPT(ModelConfig.from_name("sosutar-nano"))


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
    # layers with the same weights hold them once
    n = sum(p.numel() for p in stage.parameters())
    assert n == sum(t.numel() for t in w.values())
    stage.load_state_dict(sd, assign=True)
    n = {t.data_ptr(): t.numel() for t in stage.parameters()}
    assert sum(n.values()) == sum(t.numel() for t in w.values())
    # and through the framework's own checkpoint form
    save_checkpoint(tmp_path / "b", config, sd)
    config2, sd2 = load_from_pt(tmp_path / "b")
    assert config2.to_dict() == config.to_dict()
    assert all(torch.equal(sd[k], sd2[k]) for k in sd)


def test_balanced_split():
    from mdi_llm_amd.utils.partition import balanced_split, layer_split

    c = ModelConfig.from_name("sosutar-8b")
    for n in (2, 4, 8):
        for s in (balanced_split(c, n), layer_split(c.n_layer, n)):
            assert sum(s) == c.n_layer and len(s) == n


def test_what_a_sequence_holds():
    """Pages and states by layer, whoever's weights it uses; a matrix memory
    has a column for its normaliser and an exponent."""
    c = make_runner(*model(), "cpu", torch.float32, 2, 200).cache
    assert sorted(c.k) == sorted(c.v) == [0, 3, 4]
    assert c.k[0].shape == (5, 2, 64 * 32) and c.v[0].shape == (5, 2, 64 * 64)
    assert c.k[0] is not c.k[4]
    assert {i: tuple(t.shape) for i, t in c.state.items()} == {
        0: (3, 80), 1: (3, 3, 28, 24), 2: (3, 2, 16, 52), 3: (3, 52),
        4: (3, 80), 5: (3, 2, 16, 52), 6: (3, 5, 8, 12), 7: (3, 2, 16, 52)}
    assert {i: tuple(t.shape) for i, t in c.peak.items()} == {
        1: (3, 3), 2: (3, 2), 5: (3, 2), 6: (3, 5), 7: (3, 2)}
    assert all(t.dtype == torch.float32
               for d in (c.state, c.peak) for t in d.values())
    assert c.memory_bytes() == sum(
        4 * t.numel() for d in (c.k, c.v, c.state, c.peak)
        for t in d.values())


@pytest.mark.parametrize("i,part,value,match", [
    (0, "dim", 300, "attention dim"), (0, "vdim", 260, "attention vdim"),
    (1, "dim", 300, "mlstm"), (1, "vdim", 1024, "mlstm")])
def test_sizes_beyond_the_kernels_are_refused(i, part, value, match):
    cfg = copy.deepcopy(MODELS["mixed"])
    for layer in cfg["layers"]:
        if layer["type"] == cfg["layers"][i]["type"]:
            layer["mixer"].get("left", layer["mixer"])[part] = value
    with pytest.raises(ValueError, match=match):
        make_runner(cfg, weights(cfg), "cpu", torch.float32, max_seq=256)


# ---------------------------------------------------------------------------
@device_param
@pytest.mark.parametrize("world", [2, 3])
def test_ring_pipeline_matches_standalone(world, device, tmp_path):
    """Stages in processes of their own; on a GPU they share it, and the rows
    go through host memory."""
    from mdi_llm_amd.parallel.runtime import PipelineRuntime, SamplingParams

    cfg, w = model("mixed")
    save(tmp_path, cfg, w)
    prompts = [tokens(cfg, n, n) for n in (70, 5, 33)]
    torch.save(prompts, tmp_path / "prompts.pt")
    r = make_runner(cfg, w, device, torch.float32, max_seq=512)
    ref = PipelineRuntime(r, device=torch.device(device)).generate(
        [torch.tensor(p) for p in prompts], 8,
        SamplingParams(temperature=0.0))
    mp.spawn(_ring_worker,
             args=(world, str(tmp_path), 29990 + world, device),
             nprocs=world, join=True)
    got = torch.load(tmp_path / "out.pt", weights_only=True)
    assert got == [s.tolist() for s in ref.sequences]


# ---------------------------------------------------------------------------
@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    d = tmp_path_factory.mktemp("sosutar") / "toy"
    tok = make_toy_tokenizer(d)
    cfg = dict(MODELS["mixed"],
               vocab=max(json.loads(tok.read_text())["model"]["vocab"]
                         .values()) + 1)
    save(d, cfg, weights(cfg))
    return d


@device_param
def test_sample_cli(checkpoint, device):
    r = run(["sample.py", "--ckpt", str(checkpoint), "--n-samples", "3",
             "--n-tokens", "6", "--device", device, "--sequence-length",
             "512"])
    assert r.returncode == 0, r.stderr[-2000:]
    # (a random model may draw the end token)
    n = int(re.search(r"(\d+) tokens in", r.stdout)[1])
    assert "sample 2" in r.stdout and 3 <= n <= 18
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
         device, "--max-new-tokens", "5"],
        cwd=ROOT, input="hello\nwho are you\n", capture_output=True,
        text=True, timeout=240)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.count(">>") == 3


@pytest.mark.timeout(180)
def test_two_node_http_bootstrap(checkpoint, tmp_path):
    """Starter and secondary over the control plane."""
    import multiprocessing

    from test_orchestrator_e2e import _secondary_proc, _starter_proc, _topo

    topo = tmp_path / "topo.json"
    topo.write_text(json.dumps(_topo(tmp_path, 18835, 18837, 29881)))
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


# ---------------------------------------------------------------------------
@device_param
def test_trace_replay(device, tmp_path):
    """Requests that pause, end and give back what they hold."""
    from mdi_llm_amd.trace import load_runner, replay

    cfg, w = model("mixed")
    save(tmp_path / "m", cfg, w)
    a, b, c = (tokens(cfg, n, n) for n in (90, 10, 70))
    steps = [
        dict(entries=[dict(id="a", tokens=a[:70], want=[0, 69]),
                      dict(id="b", tokens=b[:1], want=[])], end=[]),
        dict(entries=[dict(id="b", tokens=b[1:9], want=[7])], end=[]),
        dict(entries=[dict(id="b", tokens=b[9:], want=[0]),
                      dict(id="a", tokens=a[70:71], want=[0])], end=["b"]),
        dict(entries=[dict(id="a", tokens=a[71:], want=[])], end=["a"]),
        # only fits in the pages of the two
        dict(entries=[dict(id="c", tokens=c, want=[0, 69])], end=["c"]),
    ]
    lines = [json.dumps(dict(step=n, **s)) + "\n"
             for n, s in enumerate(steps)]
    runner = load_runner(tmp_path / "m", torch.float32, torch.device(device),
                         192)
    report = io.StringIO()
    replay(runner, lines, tmp_path, report)
    assert report.getvalue().split("\n")[:5] == [f"done {n}"
                                                 for n in range(5)]
    assert runner.cache.free_pages == 3 and runner.cache.free_slots == 4
    wa, wb, wc = (oracle.forward(cfg, w, t) for t in (a, b, c))
    want = {0: wa[[0, 69]], 1: wb[[8]], 2: torch.stack([wb[9], wa[70]]),
            4: wc[[0, 69]]}
    for n, x in want.items():
        got = np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(x.shape)
        assert float(errors(torch.from_numpy(got), x).max()) < 1e-4
    assert not (tmp_path / "3.f32").exists()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(dtype, tmp_path):
    cfg, w = model("pairs")
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
    want = oracle.forward(cfg, w, t)[11:12]
    assert float(errors(got.view(1, -1), want).max()) < (
        1e-4 if dtype == "float32" else 0.08)
