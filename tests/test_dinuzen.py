"""Dinuzen through the framework's engine, cache and scheduler against the
plain implementation in ``dinuzen_oracle``: on a CPU host over the torch
operations, on a GPU over the HIP kernels."""

import random

import pytest
import torch

import dinuzen_oracle as oracle
from dinuzen_models import (MODELS, attention, config, dense, mamba2, moe,
                            rglru, rotation, weights)
from helpers import everywhere, run_portions
from nerozen_models import make_runner, tokens

LENGTH = 90     # past a page (64) and several chunks (16)

_cache = {}


def model(name, seed=0):
    if (name, seed) not in _cache:
        cfg = MODELS[name]
        _cache[name, seed] = (cfg, weights(cfg, seed))
    return _cache[name, seed]


def expected(name, toks):
    """Oracle logits; shorter prefixes of a sequence are cut from it."""
    toks = tuple(toks)
    for key, out in _cache.items():
        if key[0] == name and isinstance(key[1], tuple) \
                and key[1][:len(toks)] == toks:
            return out[:len(toks)]
    cfg, w = model(name)
    _cache[name, toks] = oracle.forward(cfg, w, list(toks))
    return _cache[name, toks]


def errors(got, want):
    """Per position: rms difference of the mean-free rows over the rms of
    the wanted ones."""
    want = want.double().cpu()
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def agrees(got, want, dtype):
    """Everywhere in fp32 (norms of a few elements enlarge the rounding of
    single positions).  In bf16 a token whose router is nearly undecided may
    take another expert, so a few positions are let go."""
    e = errors(got, want).sort().values
    n = e.numel()
    if dtype == torch.float32:
        return float(e[-1]) < 1e-3 and float(e[int(0.9 * (n - 1))]) < 4e-5
    return float(e[int(0.8 * (n - 1))]) < 0.12 \
        and (n < 8 or float(e[n // 2]) < 0.06)


def runner(name, device, dtype, **kw):
    return make_runner(*model(name), device, dtype, **{"max_seq": 512, **kw})


@everywhere
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt(name, device, dtype):
    r = runner(name, device, dtype)
    toks = tokens(MODELS[name], LENGTH)
    want = expected(name, toks)
    for n in (LENGTH, 1, 2, 17):
        assert agrees(run_portions(r, toks[:n], [n]), want[:n], dtype), n
    assert r.cache.free_pages == r.cache.n_pages


@everywhere
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_residual_stream_after_every_layer(name, device, dtype):
    cfg, w = model(name)
    toks = tokens(cfg, 21)
    want, got = [], []
    oracle.forward(cfg, w, toks, want)
    r = runner(name, device, dtype)
    r.engine.step([(r.cache.admit(), toks)], layers_out=got)
    assert len(got) == len(want)
    for g, x in zip(got, want):
        assert g.dtype == torch.float32
        assert agrees(g, x, dtype)


@everywhere
@pytest.mark.parametrize("portions", [[2], [1], [63, 2, 1, 1, 20],
                                      [3, 61, 5, 1, 7], [89, 1],
                                      [15, 2, 16, 31, 17]])
@pytest.mark.parametrize("name", list(MODELS))
def test_portions_and_decoding(name, portions, device, dtype):
    """Cuts down to two tokens and one, across page and chunk edges."""
    r = runner(name, device, dtype)
    toks = tokens(MODELS[name], LENGTH)
    got = run_portions(r, toks, portions)
    assert agrees(got, expected(name, toks), dtype)


@everywhere
@pytest.mark.parametrize("name", ["odd", "plain"])
def test_long_decoding(name, device, dtype):
    toks = tokens(MODELS[name], 260)
    r = runner(name, device, dtype)
    got = run_portions(r, toks, [130, 1])
    assert agrees(got, expected(name, toks), dtype)


@everywhere
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_unequal_batches(name, device, dtype):
    """Portions beside single tokens; slots and pages taken over by later
    requests; a pool that only just holds the live ones."""
    cfg, w = model(name)
    lengths = [90, 1, 67, 40, 64, 80, 2]
    seqs = [tokens(cfg, n, seed=i) for i, n in enumerate(lengths)]
    r = runner(name, device, dtype, n_slots=4, n_tokens=512)
    rng = random.Random(5)
    waiting, live = list(range(len(seqs))), {}
    got = [[] for _ in seqs]
    taken, both = set(), 0
    while waiting or live:
        while waiting and len(live) < 4:
            i = waiting.pop(0)
            live[i] = (r.cache.admit(), 0)
            taken.add(live[i][0])
        step = [i for i in live if rng.random() < 0.8] or list(live)
        rng.shuffle(step)
        entries = []
        for i in step:
            slot, at = live[i]
            n = rng.choice([1, 1, 2, 9, 33, 50])
            entries.append((slot, seqs[i][at:at + n]))
        sizes = {len(t) for _, t in entries}
        both += 1 in sizes and max(sizes) > 30
        out = r.engine.step(entries, [range(len(t)) for _, t in entries])
        out = out.float().clone()
        at0 = 0
        for i, (slot, t) in zip(step, entries):
            got[i].append(out[at0:at0 + len(t)])
            at0 += len(t)
            at = live[i][1] + len(t)
            live[i] = (slot, at)
            if at == len(seqs[i]):
                r.cache.release(slot)
                del live[i]
    assert len(taken) < len(seqs) and both  # slots were used again
    for i, s in enumerate(seqs):
        assert agrees(torch.cat(got[i]), expected(name, s), dtype), i
    assert r.cache.free_pages == r.cache.n_pages


@everywhere
@pytest.mark.parametrize("name", ["mixed", "ones"])
def test_a_reused_slot_starts_clean(name, device, dtype):
    """The same slot and pages, with another sequence and no clearing: first
    tokens alone, in pairs and in a prompt."""
    cfg, w = model(name)
    r = runner(name, device, dtype, n_slots=1, n_tokens=128)
    run_portions(r, tokens(cfg, 100, 9), [100])
    for seed, n, cut in ((1, 5, [1]), (2, 66, [66]), (3, 7, [2]), (4, 3, [3]),
                         (5, 70, [65, 1])):
        toks = tokens(cfg, n, seed)
        assert agrees(run_portions(r, toks, cut), expected(name, toks),
                      dtype), (n, cut)


@everywhere
def test_an_entry_does_not_depend_on_its_company(device, dtype):
    """The same portions alone and beside other sequences' prompts."""
    cfg, w = model("mixed")
    toks, other = tokens(cfg, 80, 1), tokens(cfg, 160, 2)
    r = runner("mixed", device, dtype)
    alone = run_portions(r, toks, [40, 40])
    s, o = r.cache.admit(), r.cache.admit()
    got = []
    for a, b, cut in ((0, 40, slice(0, 95)), (40, 80, slice(95, 160))):
        out = r.engine.step([(o, other[cut]), (s, toks[a:b])],
                            [[], range(b - a)])
        got.append(out.float().clone())
    e = errors(torch.cat(got), alone)
    assert float(e.median()) < (1e-5 if dtype == torch.float32 else 0.03)
    assert agrees(torch.cat(got), expected("mixed", toks), dtype)


# ---------------------------------------------------------------------------
def marked_model():
    """Token 1 is what every query of the first map looks for; its value
    appears in logit 0.  Ahead of it and after it stand recurrent layers that
    add nothing, and the keys are read through a second layer."""
    E, D = 16, 16
    rot = dict(dims=2, base=10.0)   # dimension 2 and on do not turn
    kw = dict(heads=1, kv_heads=1, dim=D, vdim=16, rot=rot, mlp=None,
              diff=0.5, softcap=60.0)
    cfg = config([attention(**kw), mamba2(1, 8, 4, 1, 1, 2, None),
                  attention(**kw, kv_from=0)], width=E, vocab=8, groups=1)
    for i in (0, 2):
        cfg["layers"][i]["mixer"]["scale"] = 1.0
    w = {k: torch.zeros_like(t) for k, t in weights(cfg).items()}
    w["embed"][:, 0] = 1.0               # what every token shares
    w["embed"][:, 1] = -1.0              # the mark's sign
    w["embed"][1, 1] = 1.0
    w["final.norm"] += 1.0
    for i in (0, 1, 2):
        w[f"l{i}.dwa"][-1] = 1.0
        w[f"l{i}.norm1"] += 1.0
        w[f"l{i}.mix.norm" if i == 1 else f"l{i}.mix.q.norm"] += 1.0
    w["l0.mix.k.norm"] += 1.0
    w["l0.mix.q"][4, 0] = w["l2.mix.q"][4, 0] = 4.0     # map 1
    w["l0.mix.k"][4, 1] = 4.0
    w["l0.mix.v"][0, 0] = 1.0            # every key
    w["l0.mix.v"][1, 1] = 1.0            # the mark, or not
    w["l2.mix.o"][3, 1] = 1.0
    w["l2.ls1"] += 1.0
    w["head"][0, 3] = 1.0
    return cfg, w


@everywhere
@pytest.mark.parametrize("at", [0, 1, 63, 64, 100])
def test_a_far_key_in_the_whole_model(at, device, dtype):
    """One key among hundreds, from its own place on and as far as the
    sequence goes, in a prompt, in portions and in decoding."""
    cfg, w = marked_model()
    n = 330
    toks = [0] * n
    toks[at] = 1
    r = make_runner(cfg, w, device, dtype, max_seq=400)
    plain = oracle.forward(cfg, w, toks[:140])[:, 0]
    for cut in ([n], [100, 2, 1, 64], [60, 1]):
        got = run_portions(r, toks, cut)[:, 0].double().cpu()
        assert float((got[:140] - plain).abs().max()) < 0.05, cut
        low, high = got[:at], got[at:]
        if at:
            assert float(low.max()) < 0 < 0.2 < float(high.min()), cut
        else:
            assert float(high.min()) > 0.2, cut


# ---------------------------------------------------------------------------
def greedy_agrees(name, prompt, out, dtype):
    """Each token is the oracle's choice, or close to it."""
    logits = expected(name, prompt + out)
    slack = 2e-4 if dtype == torch.float32 else 0.3
    good = [float(logits[len(prompt) - 1 + k].max()
                  - logits[len(prompt) - 1 + k, tok]) <= slack
            for k, tok in enumerate(out)]
    need = len(out) if dtype == torch.float32 else 0.9 * len(out)
    return sum(good) >= need


@everywhere
def test_greedy_generation(device, dtype):
    """The runtime's entry point and scheduler, more requests than slots and
    a pool that makes them wait."""
    from mdi_llm_amd.parallel.runtime import PipelineRuntime, SamplingParams

    cfg, w = model("odd")
    prompts = [tokens(cfg, n, 20 + n) for n in (3, 100, 1, 64, 31, 7)]
    r = runner("odd", device, dtype, n_slots=3, n_tokens=384)
    rt = PipelineRuntime(r, device=torch.device(device))
    seen = []
    res = rt.generate([torch.tensor(p) for p in prompts], 20,
                      SamplingParams(temperature=0.0),
                      token_callback=lambda i, t: seen.append((i, t)))
    assert len(seen) == res.total_new_tokens == 20 * len(prompts)
    for i, (p, seq) in enumerate(zip(prompts, res.sequences)):
        seq = seq.tolist()
        assert seq[:len(p)] == p and len(seq) == len(p) + 20
        assert [t for j, t in seen if j == i] == seq[len(p):]
        assert greedy_agrees("odd", p, seq[len(p):], dtype), i
    assert r.cache.free_pages == r.cache.n_pages
    # and once more over used pages: same tokens
    again = rt.generate([torch.tensor(p) for p in prompts], 20,
                        SamplingParams(temperature=0.0))
    if dtype == torch.float32:
        assert [s.tolist() for s in again.sequences] == \
            [s.tolist() for s in res.sequences]


@everywhere
def test_small_prefill_budget(device, dtype):
    """Prompts cut by the scheduler's step budget; stop sequences."""
    from mdi_llm_amd.parallel.runtime import SamplingParams
    from mdi_llm_amd.parallel.scheduler import BatchScheduler

    cfg, w = model("mixed")
    r = runner("mixed", device, dtype, n_slots=3, n_tokens=512)
    s = BatchScheduler(r, SamplingParams(temperature=0.0), budget=10)
    prompts = [tokens(cfg, n, 40 + n) for n in (45, 4, 23, 70)]
    reqs = [s.add(p, 7) for p in prompts]
    while not s.idle:
        s.step()
    for p, q in zip(prompts, reqs):
        assert len(q.output) == 7
        assert greedy_agrees("mixed", p, q.output, dtype)
    stop = reqs[0].output[3:5]
    s = BatchScheduler(r, SamplingParams(temperature=0.0), [stop])
    q = s.add(prompts[0], 9)
    while not s.idle:
        s.step()
    assert q.output[-2:] == stop and len(q.output) <= 5


@everywhere
@pytest.mark.parametrize("split", [(8,), (1, 7), (3, 5), (2, 2, 4)])
def test_stages(split, device, dtype):
    """The calls of the pipeline runtime.  A stack cut anywhere: the rows
    between stages carry the earlier layers' results, which later layers
    average, and the keys and values that they read."""
    from mdi_llm_amd.config import ModelConfig
    from mdi_llm_amd.models.hybrid import native_state_dict
    from mdi_llm_amd.models.stages import build_stage
    from mdi_llm_amd.parallel.runner import make_runner as make

    cfg, w = model("mixed")
    conf = ModelConfig.from_native(cfg)
    sd = native_state_dict(conf, w.__getitem__)
    rs = []
    for k, n in enumerate(split):
        first = sum(split[:k])
        stage = build_stage(conf, k, n, first)
        part = {}
        for key, t in sd.items():
            bits = key.split(".")
            if bits[1] == "h":
                if first <= int(bits[2]) < first + n:
                    bits[2] = str(int(bits[2]) - first)
                    part[".".join(bits)] = t
            elif k == 0:
                part[key] = t
        stage.load_state_dict(part)
        rs.append(make(stage.to(device=device, dtype=dtype).eval(), 2,
                       torch.device(device)))
    toks = tokens(cfg, 75)
    for _ in range(2):  # the second prefill takes the slot over
        x = rs[0].prefill_head(torch.tensor(toks[:68]), 1)
        assert x.shape == (68, conf.ring_width) and x.dtype == torch.float32
        for r in rs[1:]:
            x = r.prefill_mid(x, 1)
        got = [rs[0].tail(x[-1])]
        for t in toks[68:]:
            x = rs[0].decode_head(torch.tensor([t]), 1)
            for r in rs[1:]:
                x = r.decode_mid(x, 1)
            got.append(rs[0].tail(x))
        assert agrees(torch.stack(got).float(),
                      expected("mixed", toks)[67:], dtype)


# ---------------------------------------------------------------------------
@pytest.mark.gpu
@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
@pytest.mark.parametrize("n", [1, 3, 4])
def test_decode_graph_replays(n, name):
    """Replays between other work of the program, each against the eager
    step of the same tokens."""
    cfg, w = model(name)
    r = runner(name, "cuda", torch.bfloat16, n_tokens=2048)
    e = runner(name, "cuda", torch.bfloat16, n_tokens=2048)
    e.engine.use_graphs = False
    prompts = [tokens(cfg, 60 + 70 * i, i) for i in range(n)]
    for q in (r, e):
        for p in prompts:
            q.engine.step([(q.cache.admit(), p)])
    slots = sorted(s for s in range(4) if r.cache.is_live(s))
    for k in range(12):
        toks = [tokens(cfg, 12, 50 + i)[k] for i in range(n)]
        got = r.engine.decode(slots, toks).float().clone()
        want = e.engine.step([(s, [t]) for s, t in zip(slots, toks)])
        err = errors(got, want.float())
        assert float(err.max()) < 0.03, k
        torch.randn(1000, device="cuda").sum().item()
        if k % 4 == 3:
            torch.cuda.synchronize()


@pytest.mark.gpu
def test_sampled_tokens_do_not_depend_on_the_schedule():
    """Device draws are keyed by request and position: the same request
    alone and among others, chained on the device and fed from the host."""
    from mdi_llm_amd.parallel.runtime import PipelineRuntime, SamplingParams

    cfg, w = model("plain")
    prompts = [torch.tensor(tokens(cfg, n, n)) for n in (12, 70, 5)]
    sp = SamplingParams(temperature=0.7, top_k=20, seed=11)

    def run(n_slots):
        r = runner("plain", "cuda", torch.bfloat16, n_slots=n_slots)
        res = PipelineRuntime(r, device=torch.device("cuda")).generate(
            prompts, 12, sp)
        return [s.tolist() for s in res.sequences]

    one, three = run(1), run(3)
    # batch sizes round differently; a draw flips only at a near tie
    same = sum(a == b for x, y in zip(one, three) for a, b in zip(x, y))
    assert same >= 0.8 * sum(map(len, one))
    assert run(3) == three


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_large_prompt(dtype):
    """Long enough for the tiles of 128 pairs, in vectorised sizes, whole and
    in portions that stay below them."""
    cfg = config([rglru(256, 2, 4, moe(4, 3, 128, 64, 2, 1.5)),
                  mamba2(4, 64, 128, 2, 2, 4, dense(192)),
                  attention(4, 2, 64, 128, rotation(64), moe(3, 2, 192, 128)),
                  attention(4, 2, 64, 128, rotation(64), dense(512),
                            kv_from=2)], width=256, vocab=97, groups=4)
    w = weights(cfg, 3)
    r = make_runner(cfg, w, "cuda", dtype, max_seq=512)
    toks = tokens(cfg, 400)
    want = oracle.forward(cfg, w, toks)
    assert agrees(run_portions(r, toks, [400]), want, dtype)
    assert agrees(run_portions(r, toks, [40]), want, dtype)
    assert agrees(run_portions(r, toks, [380, 1]), want, dtype)
