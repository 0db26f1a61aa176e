"""Each mechanism of Resolorn alone against its oracle: the HIP kernels on a
GPU, the torch operations of the CPU path elsewhere.  Inputs are made so that
one wrong key, expert or edge changes the result visibly."""

import math

import pytest
import torch

import resolorn_oracle as oracle
from helpers import close, everywhere, ops_for, rand, seg
from mdi_llm_amd.ops.latent_layer import (ACTS, make_plan, prefers_absorbed)

PAGE = 64


def up(n, k):
    return -(-n // k) * k


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("e", [8, 27, 300, 1501, 4096])
def test_embedding_with_positions(e, device, dtype):
    ops, eps = ops_for(device), 1e-5
    table = rand(11, e, seed=1, dtype=dtype, device=device)
    pos = rand(9, e, seed=2, dtype=dtype, device=device)
    w = rand(e, seed=3, device=device)
    toks = torch.tensor([3, 10, 0, 3], dtype=torch.int32, device=device)
    at = torch.tensor([8, 0, 5, 1], dtype=torch.int32, device=device)
    x = torch.empty(4, e, device=device)
    xn = torch.empty(4, e, dtype=dtype, device=device)
    ops.residual_norm(x, tokens=toks, table=table, scale=1.0, xn=xn,
                      next_w=w, eps=eps, pos_table=pos, row_pos=at)
    want = table.double().cpu()[toks.long().cpu()] \
        + pos.double().cpu()[at.long().cpu()]
    close(x, want, torch.float32)
    close(xn, oracle.rms_norm(want, w.double().cpu(), eps), dtype)


@everywhere
@pytest.mark.parametrize("e,top", [(8, 1), (27, 3), (300, 2), (1501, 6),
                                   (4096, 4), (9000, 2)])
def test_residual_with_multiplier_and_experts(e, top, device, dtype):
    ops, eps, mult, n = ops_for(device), 1e-5, -0.7, 5
    x = rand(n, e, seed=1, device=device)
    y = rand(n, e, seed=2, dtype=dtype, device=device)
    z = rand(n, top, e, seed=3, dtype=dtype, device=device)
    p = rand(n, top, seed=4, device=device).softmax(-1)
    w = rand(e, seed=5, device=device)
    xn = torch.empty_like(y)
    want = x.double().cpu() + mult * (
        y.double().cpu()
        + (z.double().cpu() * p.double().cpu().unsqueeze(-1)).sum(1))
    ops.residual_norm(x, y=y, xn=xn, next_w=w, eps=eps, mult=mult, routed=z,
                      routed_w=p)
    close(x, want, torch.float32)
    close(xn, oracle.rms_norm(want, w.double().cpu(), eps), dtype)


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("act", list(ACTS))
@pytest.mark.parametrize("cols,skew", [(64, 0), (33, 1), (2048, 0), (200, 3)])
def test_gated_act(cols, skew, act, device, dtype):
    """Views into wider rows, with and without vector alignment."""
    n = 6
    proj = rand(n, 2 * cols + 16, seed=1, dtype=dtype, device=device) * 4
    proj[0, :] *= 10
    out = torch.zeros(n, cols + 8, dtype=dtype, device=device)
    gate, upper = proj[:, skew:skew + 2 * cols].split(cols, 1)
    ops_for(device).gated_act(out[:, 8:], gate, upper, ACTS[act])
    f = getattr(oracle, act)
    want = f(gate.double().cpu()) * upper.double().cpu()
    err = (out[:, 8:].double().cpu() - want).abs()
    assert bool((err <= (1e-5 if dtype == torch.float32 else 8e-3)
                 * (1 + want.abs())).all())
    assert float(out[:, :8].abs().max()) == 0


def scattered(slots, per, seed=3):
    perm = torch.randperm(slots * per,
                          generator=torch.Generator().manual_seed(seed))
    return perm.view(slots, per).to(torch.int32)


@everywhere
@pytest.mark.parametrize("rank,rpad,q_rank", [(56, 64, 40), (11, 64, 13),
                                              (300, 512, 1536), (128, 128, 8)])
def test_latent_norm_append_and_gather(rank, rpad, q_rank, device, dtype):
    """Two sequences' rows among each other; nothing else changes; rows come
    back from any position; the same launch may activate a feed-forward."""
    ops, eps, n = ops_for(device), 1e-5, 140
    table = scattered(3, 3).to(device)
    pages = rand(9, PAGE, rpad, seed=9, dtype=dtype, device=device)
    before = pages.clone()
    ff = 24
    proj = rand(n, q_rank + rank + 2 * ff, seed=1, dtype=dtype,
                device=device) * 3
    q, kv = proj[:, :q_rank], proj[:, q_rank:q_rank + rank]
    gate, upper = proj[:, -2 * ff:-ff], proj[:, -ff:]
    qw, kw = rand(q_rank, seed=2, device=device), rand(rank, seed=3,
                                                       device=device)
    slot = torch.tensor([2, 0] * (n // 2), dtype=torch.int32, device=device)
    pos = torch.arange(n, dtype=torch.int32, device=device) // 2 + 50
    q_out = torch.empty(n, q_rank, dtype=dtype, device=device)
    acted = torch.empty(n, ff, dtype=dtype, device=device)
    ops.latent_norm_append(pages, kv, kw, slot, pos, table, eps, q_out=q_out,
                           q=q, q_w=qw, act_out=acted, gate=gate, up=upper,
                           act=ACTS["silu"])
    close(q_out, oracle.rms_norm(q.double().cpu(), qw.double().cpu(), eps),
          dtype)
    close(acted, oracle.silu(gate.double().cpu()) * upper.double().cpu(),
          dtype)
    want = oracle.rms_norm(kv.double().cpu(), kw.double().cpu(), eps)
    out = torch.zeros(45, rank, dtype=dtype, device=device)
    # slot 0 from position 55, slot 2 from 100, with rows between them free
    segs = [(0, 30, 0, 55), (33, 12, 2, 100)]
    ops.latent_gather(out, pages, table, seg(segs, device), 30)
    close(out[:30], want[1::2][5:35], dtype)
    close(out[33:], want[0::2][50:62], dtype)
    assert float(out[30:33].abs().max()) == 0
    # only these rows were written, and only their first columns
    touched = torch.zeros(9, PAGE, rpad, dtype=torch.bool)
    for s, p in zip(slot.tolist(), pos.tolist()):
        touched[table[s, p // PAGE], p % PAGE, :rank] = True
    same = (pages == before).cpu()
    assert bool(same[~touched].all())
    # without a norm: as it is; without a latent: only the queries
    ops.latent_norm_append(pages, kv, None, slot, pos, table, eps)
    ops.latent_gather(out, pages, table, seg(segs, device), 30)
    assert torch.equal(out[:30], kv[1::2][5:35])
    kept = pages.clone()
    q_out.zero_()
    ops.latent_norm_append(pages, None, None, slot, pos, table, eps,
                           q_out=q_out, q=q, q_w=qw)
    close(q_out, oracle.rms_norm(q.double().cpu(), qw.double().cpu(), eps),
          dtype)
    assert torch.equal(pages, kept)


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("n,H,K,M", [(1, 4, 64, 128), (5, 3, 7, 64),
                                     (17, 2, 300, 20), (40, 5, 520, 9),
                                     (3, 40, 24, 256)])
def test_head_proj(n, H, K, M, device, dtype):
    """Row maps in and out, gates of the output's rows, odd sizes."""
    ops = ops_for(device)
    x = rand(n + 4, H * K + 3, seed=1, dtype=dtype, device=device)[:, :H * K]
    w = torch.zeros(H, M, up(K, 32), dtype=dtype, device=device)
    w[..., :K] = rand(H, M, K, seed=2, dtype=dtype) * K ** -0.5
    gate = rand(n + 4, H, seed=3, dtype=dtype, device=device) * 2
    want = torch.einsum("nhk,hmk->nhm",
                        x.double().cpu().reshape(n + 4, H, K),
                        w[..., :K].double().cpu())
    rows = torch.randperm(n + 4, generator=torch.Generator().manual_seed(5)
                          )[:n].to(torch.int32).to(device)
    out = torch.zeros(n + 4, H * M, dtype=dtype, device=device)
    ops.head_proj(out, x, w)
    close(out, want.reshape(n + 4, -1), dtype)
    # gather the rows, then put them back gated
    part = torch.zeros(n, H * M, dtype=dtype, device=device)
    ops.head_proj(part, x, w, x_rows=rows)
    at = rows.long().cpu()
    close(part, want[at].reshape(n, -1), dtype)
    out.fill_(7.0)
    compact = x[rows.long()].contiguous()
    ops.head_proj(out, compact, w, out_rows=rows, gate=gate)
    g = torch.sigmoid(gate.double().cpu()).unsqueeze(-1)
    close(out[rows.long()], (want * g)[at].reshape(n, -1), dtype)
    rest = [r for r in range(n + 4) if r not in set(at.tolist())]
    assert bool((out[rest] == 7.0).all())


# ---------------------------------------------------------------------------
class Latents:
    """Sequences of latent rows in scattered pages that were used before."""

    def __init__(self, device, dtype, H, R, n_pages=30, slots=3):
        self.ops, self.device, self.dtype = ops_for(device), device, dtype
        self.H, self.R = H, R
        self.rpad = next(p for p in (64, 128, 256, 512) if R <= p)
        self.pages = rand(n_pages, PAGE, self.rpad, seed=91, dtype=dtype,
                          device=device)
        self.pages[..., R:] = 0
        self.table = scattered(slots, n_pages // slots).to(device)

    def store(self, slot, pos0, c):
        n = c.size(0)
        self.ops.latent_norm_append(
            self.pages, c, None,
            torch.full((n,), slot, dtype=torch.int32, device=self.device),
            torch.arange(pos0, pos0 + n, dtype=torch.int32,
                         device=self.device), self.table, 1e-6)

    def attend(self, q, segs, window, scale, splits):
        """q [rows, H, R] -> the weighted latents [rows, H, R]; partial
        results are merged by the projection, here with the identity."""
        n, H, P = q.size(0), self.H, self.rpad
        qp = torch.zeros(n, H, P, dtype=self.dtype, device=self.device)
        qp[..., :self.R] = q
        out = torch.zeros(n, H * P, dtype=self.dtype, device=self.device)
        part = (None, None)
        if splits > 1:
            part = (torch.full((n, H, splits, P), math.nan,
                               device=self.device),
                    torch.full((n, H, splits, 2), math.nan,
                               device=self.device))
        self.ops.latent_attn(out if splits == 1 else None, qp, self.pages,
                             self.table, seg(segs, self.device),
                             max(s[1] for s in segs), window, scale, splits,
                             *part)
        eye = torch.eye(P, dtype=self.dtype, device=self.device)
        y = torch.zeros(n, H * P, dtype=self.dtype, device=self.device)
        if splits > 1:
            rows = torch.cat([torch.arange(s[0], s[0] + s[1]) for s in segs])
            rows = rows.to(self.device)
            self.ops.head_proj(
                y, None, eye.expand(H, P, P).contiguous(),
                out_rows=rows.to(torch.int32),
                part_o=part[0][rows].contiguous(),
                part_ml=part[1][rows].contiguous())
        else:
            y = out
        return y.view(n, H, P)[..., :self.R]


@everywhere
@pytest.mark.parametrize("H,R,window", [(6, 56, 37), (3, 64, 64), (16, 100, 1),
                                        (20, 128, 500), (33, 200, 90),
                                        (70, 30, 65), (32, 512, 130),
                                        (1, 300, 2)])
def test_latent_attention(H, R, window, device, dtype):
    """A prompt whole, in portions, and its tokens one by one (with the pages
    split in several ways), in scattered pages that were used before."""
    T, scale = 200, 2.0 * R ** -0.5
    L = Latents(device, dtype, H, R)
    c = rand(T, R, seed=8, dtype=dtype, device=device)
    q = rand(T, H, R, seed=9, dtype=dtype, device=device)
    cd = c.double().cpu().unsqueeze(1).expand(T, H, R)
    want = oracle.attend(q.double().cpu(), cd, cd, scale, window)
    peak = float(want.abs().max())
    L.store(1, 0, c)
    close(L.attend(q, [(0, T, 1, 0)], window, scale, 1), want, dtype, peak)
    # portions inside a larger batch, as they come in
    at = 0
    for n in (2, 63, 1, 31, 64, 39):
        L.store(0, at, c[at:at + n])
        some = torch.cat([torch.zeros_like(q[:1]), q[at:at + n]])
        for splits in (1, 3):
            o = L.attend(some, [(1, n, 0, at)], window, scale, splits)
            close(o[1:], want[at:at + n], dtype, peak)
        at += n
    # one by one; later keys are in the pages already and must not be seen
    ts = list(range(0, T, 7)) + [63, 64, 65, window - 1, window, T - 1]
    ts = sorted({t for t in ts if 0 <= t < T})
    for splits in (1, 2, 5):
        o = L.attend(q, [(t, 1, 1, t) for t in ts], window, scale, splits)
        close(o[ts], want[ts], dtype, peak)


@everywhere
@pytest.mark.parametrize("H,D,E,window", [(2, 64, 64, 64), (3, 24, 40, 50),
                                          (1, 7, 9, 1), (2, 128, 128, 500),
                                          (2, 200, 96, 33), (1, 96, 256, 70),
                                          (4, 256, 256, 129)])
def test_head_attention(H, D, E, window, device, dtype):
    """Two prompts at once, one of which goes on after a context of which
    only the visible part is there; gates; views of wider rows."""
    ops, scale = ops_for(device), 2.0 * D ** -0.5
    T, pos0 = 170, 90
    k, v = rand(2, T, H, D, seed=1, dtype=dtype), rand(2, T, H, E, seed=2,
                                                       dtype=dtype)
    q = rand(2, T, H, D, seed=3, dtype=dtype)
    want = torch.stack([oracle.attend(*(t[b].double() for t in (q, k, v)),
                                      scale, window) for b in (0, 1)])
    first = max(0, pos0 - window + 1)
    n0, n1 = T, T - pos0
    pad = rand(3, H * (D + E), seed=5, dtype=dtype)
    kv = torch.cat([pad, torch.cat([k[0].flatten(1), v[0].flatten(1)], 1),
                    pad, torch.cat([k[1].flatten(1), v[1].flatten(1)],
                                   1)[first:]]).to(device)
    rows = torch.cat([q[1, pos0:].flatten(1), q[0].flatten(1)]).to(device)
    segs = [(n1, n0, 0, 0), (0, n1, 1, pos0)]
    ctx = [(3, T, 0, 0), (T + 6, T - first, 1, first)]
    wide = rand(n0 + n1, H + 5, seed=6, dtype=dtype, device=device)
    gate = wide[:, 5:]
    for g in (None, gate):
        out = torch.zeros(n0 + n1, H * E + 7, dtype=dtype, device=device)
        ops.head_attn(out[:, :H * E], rows, kv, seg(segs, device),
                      seg(ctx, device), n0, H, D, E, window, scale, g)
        full = torch.cat([want[1, pos0:], want[0]])
        if g is not None:
            full = full * torch.sigmoid(g.double().cpu()).unsqueeze(-1)
        close(out[:, :H * E], full.flatten(1), dtype)
        assert float(out[:, H * E:].abs().max()) == 0


@everywhere
@pytest.mark.parametrize("window", [1, 2, 40, 63, 64, 65, 128, 130, 300])
def test_one_key_stands_out(window, device, dtype):
    """All keys repel the query but one; its value must come through exactly
    where the window lets it, at page borders, just inside and just outside
    of the window, whichever way the step is computed."""
    H, R, T = 2, 48, 260
    ops = ops_for(device)
    L = Latents(device, dtype, H, R)
    queries = [255, 256, 259, 128, 191, 192]
    spots = {0, 1, 63, 64, 65, 127, 128}
    for i in queries:
        spots |= {i, i - 1, i - window + 1, i - window, i - window - 1}
    for j in sorted(s for s in spots if 0 <= s < T):
        c = torch.zeros(T, R, dtype=dtype, device=device)
        c[:, 0] = -1.0
        c[j, 0] = 1.0
        c[:, 1] = 0.01
        c[j, 1] = 1.0
        q = torch.zeros(T, H, R, dtype=dtype, device=device)
        q[..., 0] = 8.0
        L.store(2, 0, c)
        segs = [(i, 1, 2, i) for i in queries]
        got = [L.attend(q, [(0, T, 2, 0)], window, 1.0, 1)[..., 1]]
        got += [L.attend(q, segs, window, 1.0, s)[..., 1] for s in (1, 3)]
        kv = torch.cat([c, c, c[:, 1:2], c[:, 1:2]], 1)
        out = torch.zeros(T, H, dtype=dtype, device=device)
        one = seg([(0, T, 2, 0)], device)
        ops.head_attn(out, q.flatten(1), kv, one, one, T, H, R, 1, window,
                      1.0)
        for o in got + [out]:
            for i in queries:
                # alone in sight, any key has all the weight
                seen = oracle.visible(i, j, window)
                low = float(o[i].float().min())
                assert abs(low - (1.0 if seen else 0.01)) < 0.02, (i, j)


@everywhere
def test_a_far_key_among_hundreds(device, dtype):
    """One sharp key far back counts as much as hundreds of dull ones."""
    H, R, T, window = 3, 64, 710, 690
    L = Latents(device, dtype, H, R, n_pages=36)
    c = rand(T, R, seed=1, dtype=dtype, device=device) * 0.1
    q = rand(T, H, R, seed=2, dtype=dtype, device=device) * 0.1
    c[:, 0] = 0.0
    c[15, 0] = 2.0
    q[..., 0] = 4.0
    cd = c.double().cpu().unsqueeze(1).expand(T, H, R)
    ts = [16, 300, 640, 15 + window - 1, 15 + window]
    qd = q.double().cpu()
    want = torch.stack([one_query(qd[t], cd, t, 0.75, window) for t in ts])
    L.store(0, 0, c)
    for splits in (1, 4, 11):
        o = L.attend(q, [(t, 1, 0, t) for t in ts], window, 0.75, splits)
        close(o[ts], want, dtype)
    whole = L.attend(q, [(0, T, 0, 0)], window, 0.75, 1)
    close(whole[ts], want, dtype)


def one_query(q, c, t, scale, window):
    js = [j for j in range(t + 1) if oracle.visible(t, j, window)]
    p = ((c[js] * q).sum(-1) * scale).softmax(0)
    return (p[:, :, None] * c[js]).sum(0)


# ---------------------------------------------------------------------------
class Geometry:
    def __init__(self, dim, vdim, rank, window):
        self.dim, self.vdim, self.rank, self.window = dim, vdim, rank, window


def test_the_form_of_an_entry():
    m = Geometry(128, 128, 512, 2048)
    assert prefers_absorbed(1, 0, m) and prefers_absorbed(1, 10 ** 5, m)
    assert prefers_absorbed(2, 4000, m)
    assert not prefers_absorbed(4096, 0, m)
    assert not prefers_absorbed(512, 4096, m)
    assert prefers_absorbed(4096, 0, Geometry(264, 16, 512, 2048))


def test_plan_separates_the_forms():
    m = Geometry(64, 64, 96, 33)
    entries = [(0, 1, 3, 70), (201, 1, 1, 0), (1, 200, 0, 50)]
    p = make_plan(entries, 202, m, "cpu")
    assert p.seg.t().tolist() == [[0, 1, 3, 70], [1, 1, 1, 0]]
    assert p.rows.tolist() == [0, 201] and p.n_rows == 2 and p.max_len == 1
    assert p.long_seg.t().tolist() == [[1, 200, 0, 50]]
    assert p.ctx_seg.t().tolist() == [[0, 232, 0, 18]]
    assert (p.ctx_rows, p.ctx_max, p.long_max) == (232, 232, 200)
    p = make_plan(entries, 202, m, "cpu", "absorbed")
    assert p.long_seg is None and p.n_rows == 202 and p.max_len == 200
    assert p.seg.t().tolist() == [[0, 1, 3, 70], [1, 1, 1, 0],
                                  [2, 200, 0, 50]]
    assert p.rows.tolist() == [0, 201] + list(range(1, 201))
    p = make_plan([(0, 2, 0, 0), (2, 3, 1, 0)], 5, m, "cpu", "absorbed")
    assert p.rows is None


# ---------------------------------------------------------------------------
def expert_weights(E, F, W, dtype, device):
    upper = rand(E, 2 * F, W, seed=11, dtype=dtype, device=device) * W ** -0.5
    down = rand(E, W, F, seed=12, dtype=dtype, device=device) * F ** -0.5
    return upper, down


def check_experts(n, top, E, W, F, tile, device, dtype, router=None):
    ops = ops_for(device)
    x = rand(n, W, seed=1, dtype=dtype, device=device)
    if router is None:
        router = rand(E, W, seed=2) * 4 * W ** -0.5
    router = router.to(dtype).to(device)
    upper, down = expert_weights(E, F, W, dtype, device)
    weight = torch.full((n, top), math.nan, device=device)
    plan = ops.moe_route(weight, x, router, top, tile)
    mid = torch.full((n * top, F), math.nan, dtype=dtype, device=device)
    ops.moe_up(mid, x, upper, plan, ACTS["silu"], tile)
    out = torch.full((n, top, W), math.nan, dtype=dtype, device=device)
    ops.moe_down(out, mid, down, plan, tile)
    xd, ud, dd = (t.double().cpu() for t in (x, upper, down))
    z = xd @ router.double().cpu().t()
    got, want, weights = [], [], []
    for t in range(n):
        chosen = oracle.route(z[t], top)
        weights.append(sorted(float(p) for _, p in chosen))
        want.append(sum(
            p * (dd[e] @ (oracle.silu(ud[e, :F] @ xd[t])
                          * (ud[e, F:] @ xd[t]))) for e, p in chosen))
        got.append((weight[t].double().cpu()[:, None]
                    * out[t].double().cpu()).sum(0))
    close(weight.sort(-1).values, torch.tensor(weights), torch.float32, 4.0)
    close(torch.stack(got), torch.stack(want), dtype)


@everywhere
@pytest.mark.parametrize("n,top,E,W,F", [(1, 2, 5, 72, 24), (37, 3, 7, 64, 40),
                                         (5, 1, 1, 27, 5), (70, 4, 4, 33, 9),
                                         (9, 6, 64, 2048, 16),
                                         (90, 2, 130, 40, 8)])
def test_experts(n, top, E, W, F, device, dtype):
    check_experts(n, top, E, W, F, 16, device, dtype)


@everywhere
def test_all_tokens_to_one_expert(device, dtype):
    """The most unequal load, and experts that nobody chose."""
    n, W = 40, 48
    x = rand(n, W, seed=1, dtype=dtype)  # what check_experts takes
    router = torch.zeros(6, W)
    router[4] = torch.linalg.pinv(x.double()).sum(1).float() * 3
    check_experts(n, 1, 6, W, 24, 16, device, dtype, router)


@pytest.mark.gpu
@pytest.mark.parametrize("n,top,E,W,F", [(400, 2, 3, 256, 128),
                                         (130, 3, 5, 320, 192),
                                         (257, 1, 2, 448, 320)])
def test_large_expert_tiles(n, top, E, W, F):
    """Short last tiles, outputs that no tile divides, both plan sizes."""
    check_experts(n, top, E, W, F, 128, "cuda", torch.bfloat16)


@pytest.mark.gpu
def test_operations_refuse_what_they_cannot_hold():
    ops, d = ops_for("cuda"), "cuda"
    x = torch.zeros(4, 64, device=d)
    w = torch.zeros(4, 65, device=d)
    for call in (
            lambda: ops.moe_route(w, x, torch.zeros(80, 64, device=d), 65),
            lambda: ops.moe_route(w[:, :2].contiguous(), x,
                                  torch.zeros(300, 64, device=d), 2),
            lambda: ops.moe_route(w[:, :2].contiguous(), x,
                                  torch.zeros(4, 64, device=d), 2, 128),
            lambda: ops.head_attn(torch.zeros(4, 300, device=d),
                                  torch.zeros(4, 300, device=d),
                                  torch.zeros(4, 600, device=d),
                                  seg([(0, 4, 0, 0)], d),
                                  seg([(0, 4, 0, 0)], d), 4, 1, 300, 300, 9,
                                  1.0),
            lambda: ops.gated_act(x, x[:, :32], x, 0)):
        with pytest.raises(RuntimeError):
            call()
