"""Resolorn through the framework's engine, cache and scheduler against the
plain implementation in ``resolorn_oracle``: on a CPU host over the torch
operations, on a GPU over the HIP kernels."""

import random

import pytest
import torch

import resolorn_oracle as oracle
from helpers import everywhere, run_portions
from nerozen_models import make_runner, tokens
from resolorn_models import MODELS, att, config, dense, weights

forms = pytest.mark.parametrize("form", [None, "absorbed", "expanded"])

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
    """Everywhere in fp32.  In bf16 a token whose router is nearly undecided
    may take another expert, so a few positions are let go."""
    e = errors(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 5e-5
    return float(e.kthvalue(-(-9 * e.numel() // 10)).values) < 0.06


def runner(name, device, dtype, form=None, **kw):
    r = make_runner(*model(name), device, dtype,
                    **{"max_seq": 512, **kw})
    r.engine.latent_form = form
    return r


@everywhere
@forms
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt(name, form, device, dtype):
    if name == "narrow" and form == "expanded":
        pytest.skip("heads of this size are absorbed only")
    r = runner(name, device, dtype, form)
    toks = tokens(MODELS[name], 150)
    want = expected(name, toks)
    for n in (1, 2, 17, 150):
        assert agrees(run_portions(r, toks[:n], [n]), want[:n], dtype), n
    assert r.cache.free_pages == r.cache.n_pages


@everywhere
@pytest.mark.parametrize("name", ["mixed", "shared"])
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
@forms
@pytest.mark.parametrize("name", list(MODELS))
def test_portions_and_decoding(name, form, device, dtype):
    """Cuts down to two tokens and one, across page (64) and window edges."""
    if name == "narrow" and form == "expanded":
        pytest.skip("heads of this size are absorbed only")
    r = runner(name, device, dtype, form)
    toks = tokens(MODELS[name], 150)
    want = expected(name, toks)
    for portions in ([2], [1], [63, 2, 1, 1, 64], [3, 61, 5, 1, 7],
                     [149, 1], [31, 33, 16, 17]):
        got = run_portions(r, toks, portions)
        assert agrees(got, want, dtype), portions


@everywhere
def test_long_decoding(device, dtype):
    """Most of the sequence decoded, far past every window but one, up to
    the last learned position."""
    cfg, w = model("mixed")
    toks = tokens(cfg, 512)
    r = runner("mixed", device, dtype)
    got = run_portions(r, toks, [130, 1])
    assert agrees(got, expected("mixed", toks), dtype)
    slot = r.cache.admit()
    r.engine.step([(slot, toks)])
    with pytest.raises(ValueError):
        r.engine.step([(slot, toks[:1])])


@everywhere
@pytest.mark.parametrize("name", ["mixed", "odd", "shared"])
def test_unequal_batches(name, device, dtype):
    """Portions beside single tokens; slots and pages taken over by later
    requests; a pool that only just holds the live ones."""
    cfg, w = model(name)
    lengths = [150, 1, 97, 40, 64, 129, 66, 2]
    seqs = [tokens(cfg, n, seed=i) for i, n in enumerate(lengths)]
    r = runner(name, device, dtype, n_slots=4, n_tokens=600)
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
            n = rng.choice([1, 1, 2, 9, 33, 70])
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
def test_a_reused_slot_starts_clean(device, dtype):
    """The same slot and pages, with another sequence and no clearing."""
    cfg, w = model("mixed")
    r = runner("mixed", device, dtype, n_slots=1, n_tokens=192)
    for seed, n in ((1, 190), (2, 64), (3, 65), (4, 3), (5, 130)):
        toks = tokens(cfg, n, seed)
        for cut in ([n], [1]):
            got = run_portions(r, toks, cut)
            assert agrees(got, expected("mixed", toks), dtype), (n, cut)


@everywhere
def test_an_entry_does_not_depend_on_its_company(device, dtype):
    """The same portions alone and beside other sequences' prompts."""
    cfg, w = model("mixed")
    toks, other = tokens(cfg, 100, 1), tokens(cfg, 300, 2)
    r = runner("mixed", device, dtype)
    alone = run_portions(r, toks, [40, 60])
    s, o = r.cache.admit(), r.cache.admit()
    got = []
    for a, b, cut in ((0, 40, slice(0, 170)), (40, 100, slice(170, 300))):
        out = r.engine.step([(o, other[cut]), (s, toks[a:b])],
                            [[], range(b - a)])
        got.append(out.float().clone())
    e = errors(torch.cat(got), alone)
    assert float(e.median()) < (1e-5 if dtype == torch.float32 else 0.02)
    assert agrees(torch.cat(got), expected("mixed", toks), dtype)


@everywhere
def test_wanted_rows(device, dtype):
    cfg, w = model("shared")
    a, b = tokens(cfg, 30), tokens(cfg, 9, 1)
    r = runner("shared", device, dtype)
    sa, sb = r.cache.admit(), r.cache.admit()
    got = r.engine.step([(sa, a), (sb, b)], [[29, 0], [4]])
    want = torch.stack([expected("shared", a)[29], expected("shared", a)[0],
                        expected("shared", b)[4]])
    assert float(errors(got.float(), want).median()) < (
        5e-5 if dtype == torch.float32 else 0.06)
    assert r.engine.step([(sa, a[:2]), (sb, b[:1])], [[], []]) is None
    assert r.cache.length[sa] == 32 and r.cache.length[sb] == 10


# ---------------------------------------------------------------------------
def window_model(size, mult=1.0):
    """One layer whose attention copies the value of the one key that
    matches, so that a single wrong key shows: token 1 is what queries look
    for, every other key repels."""
    E = 16
    cfg = config([att(2, 16, 16, 16, 16, size, None)], width=E, vocab=8,
                 mult=mult, positions=400)
    w = {k: torch.zeros_like(t) for k, t in weights(cfg).items()}
    w["embed"][:, 0] = 1.0               # what every token shares
    w["embed"][1, 1] = 1.0               # the mark
    w["embed"][:, 2] = -1.0
    w["embed"][1, 2] = 1.0
    for n in ("l0.norm1", "final.norm", "l0.mix.dq.norm", "l0.mix.dkv.norm"):
        w[n] += 1.0
    w["l0.mix.dq"][0, 0] = 1.0
    for h in (0, 1):
        w["l0.mix.uq"][h * 16, 0] = 16.0
        w["l0.mix.uk"][h * 16, 2] = 16.0
        w["l0.mix.uv"][h * 16, 1] = 4.0
    w["l0.mix.dkv"] += torch.eye(E)
    w["l0.mix.g"][:, 0] = 8.0            # gates open
    w["l0.mix.o"][3, 0] = w["l0.mix.o"][3, 16] = 1.0
    w["head"][0, 3] = 1.0
    return cfg, w


@everywhere
@forms
@pytest.mark.parametrize("size", [1, 2, 63, 64, 65, 150])
def test_window_edges_in_the_whole_model(size, form, device, dtype):
    """The marked token is seen up to exactly the window's last place, in a
    prompt, in portions and in decoding."""
    cfg, w = window_model(size)
    n, at = 230, 37
    toks = [0] * n
    toks[at] = 1
    r = make_runner(cfg, w, device, dtype, max_seq=400)
    r.engine.latent_form = form
    for cut in ([n], [100, 2, 1, 64], [60, 1]):
        got = run_portions(r, toks, cut)[:, 0].cpu()
        seen = torch.zeros(n, dtype=torch.bool)
        seen[at:at + size] = True
        # alone in sight, the mark has all the weight; elsewhere none
        low, high = got[~seen], got[seen]
        assert float(low.abs().max()) < 0.05 < 0.5 < float(high.min()), cut


# ---------------------------------------------------------------------------
def greedy_agrees(name, prompt, out, dtype):
    """Each token is the oracle's choice, or close to it."""
    logits = expected(name, prompt + out)
    slack = 2e-4 if dtype == torch.float32 else 0.25
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

    cfg, w = model("mixed")
    prompts = [tokens(cfg, n, 20 + n) for n in (3, 100, 1, 64, 31, 7)]
    r = runner("mixed", device, dtype, n_slots=3, n_tokens=384)
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
        assert greedy_agrees("mixed", p, seq[len(p):], dtype), i
    assert r.cache.free_pages == r.cache.n_pages
    # and once more over used pages: same tokens
    again = rt.generate([torch.tensor(p) for p in prompts], 20,
                        SamplingParams(temperature=0.0))
    if dtype == torch.float32:
        assert [s.tolist() for s in again.sequences] == \
            [s.tolist() for s in res.sequences]


@everywhere
def test_small_prefill_budget(device, dtype):
    """Prompts cut by the scheduler's step budget, stop sequences, and the
    end of the learned positions."""
    from mdi_llm_amd.parallel.runtime import SamplingParams
    from mdi_llm_amd.parallel.scheduler import BatchScheduler

    cfg, w = model("mixed")
    r = runner("mixed", device, dtype, n_slots=3, n_tokens=2048)
    s = BatchScheduler(r, SamplingParams(temperature=0.0), budget=10)
    prompts = [tokens(cfg, n, 40 + n) for n in (45, 4, 23, 80)]
    reqs = [s.add(p, 9) for p in prompts]
    while not s.idle:
        s.step()
    for p, q in zip(prompts, reqs):
        assert len(q.output) == 9
        assert greedy_agrees("mixed", p, q.output, dtype)
    stop = reqs[0].output[3:5]
    s = BatchScheduler(r, SamplingParams(temperature=0.0), [stop])
    q = s.add(prompts[0], 9)
    while not s.idle:
        s.step()
    assert q.output[-2:] == stop and len(q.output) <= 5
    s = BatchScheduler(r, SamplingParams(temperature=0.0))
    q = s.add(tokens(cfg, 508, 3), 50)
    while not s.idle:
        s.step()
    assert len(q.output) == 5  # the last one is not fed back


@everywhere
def test_runner_roles_match_steps(device, dtype):
    """The calls of the pipeline runtime: head, middle, tail.  Rows between
    stages carry the latents that later stages may read."""
    cfg, w = model("mixed")
    toks = tokens(cfg, 40)
    r = runner("mixed", device, dtype)
    want = expected("mixed", toks)
    for _ in range(2):  # the second prefill takes the slot over
        x = r.prefill_head(torch.tensor(toks[:30]), 2)
        assert x.shape == (30, cfg["width"] + 56 + 88)
        assert x.dtype == torch.float32
        got = [r.tail(x[-1])]
        for t in toks[30:]:
            got.append(r.tail(r.decode_head(torch.tensor([t]), 2)))
        assert r.pos[2] == 40
        assert agrees(torch.stack(got).float(), want[29:], dtype)


@everywhere
@pytest.mark.parametrize("split", [(1, 4), (2, 3), (3, 2), (1, 1, 3)])
def test_stages_share_latents(split, device, dtype):
    """A stack cut between a latent and the layers that read it."""
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
    toks = tokens(cfg, 90)
    x = rs[0].prefill_head(torch.tensor(toks[:80]), 1)
    for r in rs[1:]:
        x = r.prefill_mid(x, 1)
    got = [rs[0].tail(x[-1])]
    for t in toks[80:]:
        x = rs[0].decode_head(torch.tensor([t]), 1)
        for r in rs[1:]:
            x = r.decode_mid(x, 1)
        got.append(rs[0].tail(x))
    assert agrees(torch.stack(got).float(), expected("mixed", toks)[79:],
                  dtype)


# ---------------------------------------------------------------------------
@pytest.mark.gpu
@pytest.mark.parametrize("name", ["mixed", "wide"])
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

    cfg, w = model("mixed")
    prompts = [torch.tensor(tokens(cfg, n, n)) for n in (12, 70, 5)]
    sp = SamplingParams(temperature=0.7, top_k=20, seed=11)

    def run(n_slots):
        r = runner("mixed", "cuda", torch.bfloat16, n_slots=n_slots)
        res = PipelineRuntime(r, device=torch.device("cuda")).generate(
            prompts, 12, sp)
        return [s.tolist() for s in res.sequences]

    one, three = run(1), run(3)
    # batch sizes round differently; a draw flips only at a near tie
    same = sum(a == b for x, y in zip(one, three) for a, b in zip(x, y))
    assert same >= 0.8 * sum(map(len, one))
    assert run(3) == three


@pytest.mark.gpu
def test_large_expert_tiles_in_a_prompt():
    """A prompt long enough for the tiles of 128 pairs, against the same
    prompt in portions that stay below them."""
    from resolorn_models import moe

    cfg = config([att(4, 32, 32, 64, 64, 90, moe(4, 2, 128, 64)),
                  att(4, 32, 32, 64, 64, 30, dense(192), 0),
                  att(4, 32, 32, 64, 64, 300, moe(3, 3, 192))],
                 width=256, vocab=97)
    w = weights(cfg, 3)
    r = make_runner(cfg, w, "cuda", torch.bfloat16, max_seq=512)
    toks = tokens(cfg, 500)
    want = oracle.forward(cfg, w, toks)
    assert agrees(run_portions(r, toks, [500]), want, torch.bfloat16)
    assert agrees(run_portions(r, toks, [40]), want, torch.bfloat16)
