"""Each mechanism of Dinuzen alone against its oracle: the HIP kernels on a
GPU, the torch operations of the CPU path elsewhere.  Inputs are made so that
one wrong key, tap, state, expert or edge changes the result visibly."""

import math

import pytest
import torch

import dinuzen_oracle as oracle
from dinuzen_models import rotation
from helpers import close, everywhere, ops_for, rand, seg
from mdi_llm_amd.models.model import build_pair_rope_table, scaled_rope_angles

PAGE = 64


def f64(t):
    return t.double().cpu()


# ---------------------------------------------------------------------------
ROWS = [(8, 1), (8, 4), (27, 9), (300, 3), (1501, 1), (4096, 8), (9000, 2)]


@everywhere
@pytest.mark.parametrize("e,groups", ROWS)
def test_residual_step(e, groups, device, dtype):
    """Embedding, a sublayer's normed output, the final norm."""
    ops, n, eps = ops_for(device), 5, 1e-3
    table = rand(11, e, seed=1, dtype=dtype, device=device)
    toks = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32, device=device)
    x = torch.empty(n, e, device=device)
    xn = torch.empty(n, e, dtype=dtype, device=device)
    kept = torch.zeros(n, e, device=device)
    ops.stream_step(x, tokens=toks, table=table, xn=xn, keep=kept)
    want = f64(table)[toks.long().cpu()]
    close(x, want, torch.float32)
    close(xn, want, dtype)
    assert torch.equal(kept, x)
    # parts of unequal sizes, so that a norm over the whole row shows
    y = rand(n, e, seed=2, dtype=dtype, device=device)
    y = (y.view(n, groups, -1) * torch.logspace(
        -1, 1, groups, device=device).view(1, -1, 1).to(dtype)).flatten(1)
    w, wn = rand(e, seed=3, device=device), rand(e, seed=4, device=device)
    want = want + oracle.group_norm(f64(y), f64(w), groups, eps)
    ops.stream_step(x, y, w, xn=xn, groups=groups, eps=eps)
    close(x, want, torch.float32)
    close(xn, want, dtype)
    ops.stream_step(x, xn=xn, next_w=wn, groups=groups, eps=eps)
    close(x, want, torch.float32)
    close(xn, oracle.group_norm(want, f64(wn), groups, eps), dtype)


@everywhere
@pytest.mark.parametrize("e,groups", ROWS)
@pytest.mark.parametrize("depth", [1, 2, 9, 35])
def test_average_over_depth(e, groups, depth, device, dtype):
    """The layer's own result is kept as it is before the average."""
    ops, n, eps = ops_for(device), 3, 1e-5
    x = rand(n, e, seed=1, device=device)
    y = rand(n, e, seed=2, dtype=dtype, device=device)
    w = rand(e, seed=3, device=device)
    hist = rand(depth + 1, n, e, seed=4, device=device)
    coef = rand(depth + 1, seed=5, device=device)
    # ahead of time, beside another step that only adds
    z, x0 = torch.zeros_like(y), x.clone()
    past = torch.full((n, e), 5.0, device=device)
    ops.stream_step(x, z, w, groups=groups, eps=eps, hist=hist[:depth],
                    coef=coef, past=past)
    assert torch.equal(x, x0)
    close(past, oracle.depth_average(list(f64(hist[:depth])),
                                     f64(coef[:-1])), torch.float32)
    xn = torch.empty(n, e, dtype=dtype, device=device)
    own = f64(x) + oracle.group_norm(f64(y), f64(w), groups, eps)
    want = oracle.depth_average(list(f64(hist[:depth])) + [own], f64(coef))
    ops.stream_step(x, y, w, xn=xn, groups=groups, eps=eps,
                    hist=hist[:depth], coef=coef, keep=hist[depth])
    close(x, want, torch.float32)
    close(xn, want, dtype)
    close(hist[depth], own, torch.float32)


@everywhere
@pytest.mark.parametrize("shared", [False, True])
@pytest.mark.parametrize("e,top", [(8, 1), (27, 3), (300, 2), (4096, 6)])
def test_residual_step_with_experts(e, top, shared, device, dtype):
    """Identity outputs give the float stream itself and their rows are never
    read; the shared expert has a weight of its own."""
    ops, n, eps, experts = ops_for(device), 6, 1e-5, 4
    x = rand(n, e, seed=1, device=device)
    y = rand(n, e, seed=2, dtype=dtype, device=device) if shared else None
    rows = rand(n, top, e, seed=3, dtype=dtype, device=device)
    p = rand(n, top + shared, seed=4, device=device)
    chosen = (torch.arange(n * top, dtype=torch.int32) * 5 % 7).view(n, top)
    for t, k in (chosen >= experts).nonzero().tolist():
        rows[t, k] = math.nan
    w = rand(e, seed=5, device=device)
    xn = torch.empty(n, e, dtype=dtype, device=device)
    add = torch.zeros(n, e, dtype=torch.float64)
    for t in range(n):
        for k in range(top):
            add[t] += f64(p[t, k]) * f64(
                x[t] if chosen[t, k] >= experts else rows[t, k])
        if shared:
            add[t] += f64(p[t, top]) * f64(y[t])
    want = f64(x) + oracle.group_norm(add, f64(w), 1, eps)
    ops.stream_step(x, y, w, xn=xn, eps=eps, routed=rows, routed_w=p,
                    chosen=chosen.to(device), experts=experts)
    close(x, want, torch.float32)
    close(xn, want, dtype)


@everywhere
@pytest.mark.parametrize("e", [8, 27, 300, 4096])
def test_token_shift(e, device, dtype):
    """A sequence whole, in portions beside another, and token by token
    within the residual step; slots hold leftovers."""
    ops, T = ops_for(device), 20
    x = rand(2, T, e, seed=1, device=device)
    mu = rand(e, seed=2, device=device)
    want = [oracle.token_shift(f64(s), f64(mu)) for s in x]
    prev = torch.full((5, e), 50.0, device=device)

    def rows(*parts):
        flat = torch.cat(parts)
        return flat.contiguous(), torch.empty(*flat.shape, dtype=dtype,
                                              device=device)

    flat, out = rows(x[0])
    ops.token_shift(out, flat, mu, prev, seg([(0, T, 3, 0)], device), T)
    close(out, want[0], dtype)
    at = 0
    for n in (2, 1, 5, 12):
        flat, out = rows(x[1][at:at + n], x[0][at:at + n])
        ops.token_shift(out, flat, mu, prev, seg(
            [(0, n, 0, at), (n, n, 2, at)], device), n)
        close(out, torch.cat([want[1][at:at + n], want[0][at:at + n]]),
              dtype)
        at += n
    slot = torch.tensor([2, 0], dtype=torch.int32, device=device)
    for t in range(6):
        flat, out = rows(x[0, t:t + 1], x[1, t:t + 1])
        pos = torch.full((2,), t, dtype=torch.int32, device=device)
        ops.stream_step(flat, xn=out, shift=mu, prev=prev, row_slot=slot,
                        row_pos=pos)
        close(out, torch.stack([want[0][t], want[1][t]]), dtype)
    assert torch.equal(prev[2], x[0, 5]) and torch.equal(prev[3], x[0, -1])
    assert float(prev[1].min()) == 50.0  # nobody's slot


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("c,bias,act", [(5, True, False), (64, False, True),
                                        (300, True, True),
                                        (2056, False, False)])
def test_causal_conv(c, bias, act, taps, device, dtype):
    """Two sequences in portions, down to one token, in columns of a wider
    row; what a slot held before does not count."""
    ops, T = ops_for(device), 60
    x = rand(2, T, c, seed=1, dtype=dtype, device=device)
    w = rand(taps, c, seed=2, device=device)
    b = rand(c, seed=3, device=device)
    ib = rand(c, seed=4, device=device) if bias else None
    want = []
    for s in x:
        h = f64(s) + (f64(ib) if bias else 0.0)
        h = oracle.causal_conv(h, f64(w).T, f64(b))
        want.append(oracle.silu(h) if act else h)
    peak = float(torch.stack(want).abs().max())
    state = torch.full((4, max(1, taps - 1), c), 30.0, dtype=dtype,
                       device=device)
    for cuts in ((60,), (2, 17, 1, 1, 33, 1, 5), (1,) * 20):
        at = 0
        for n in cuts:
            wide = rand(2 * n + 1, c + 24, seed=9, dtype=dtype,
                        device=device)
            wide[1:1 + n, 16:16 + c] = x[0, at:at + n]
            wide[1 + n:, 16:16 + c] = x[1, at:at + n]
            out = torch.zeros(2 * n + 1, c, dtype=dtype, device=device)
            ops.causal_conv(out, wide[:, 16:16 + c], w, b, ib, state, seg(
                [(1, n, 3, at), (1 + n, n, 0, at)], device), n, act)
            for rows, s in ((out[1:1 + n], 0), (out[1 + n:], 1)):
                close(rows, want[s][at:at + n], dtype, peak)
            assert float(out[0].abs().max()) == 0
            at += n
    assert float(state[1:3].min()) == 30.0


# ---------------------------------------------------------------------------
def drive(T, run):
    """A sequence whole, one in portions and one token by token:
    run(which, slot, first, count, by the one-token operation)."""
    run(0, 2, 0, T, False)
    at = 0
    for n in (2, 1, 16, 17, 31, 1, 130):
        n = min(n, T - at)
        if n:
            run(1, 0, at, n, n == 1)
        at += n
    if at < T:
        run(1, 0, at, T - at, False)
    for t in range(T):
        run(2, 3, t, 1, True)


@everywhere
@pytest.mark.parametrize("W,blocks", [(5, 1), (21, 3), (64, 64), (80, 5),
                                      (320, 2), (96, 1), (512, 2)])
def test_rglru(W, blocks, device, dtype):
    """Channels from ones that forget at once to ones that hold on."""
    ops, T, part = ops_for(device), 200, W // blocks
    u = rand(3, T, W, seed=1, dtype=dtype, device=device)
    y = rand(3, T, W, seed=2, dtype=dtype, device=device) * 2
    y_bias = rand(W, seed=3, device=device)
    gates = (rand(2 * blocks, part, part, seed=4) * part ** -0.5).to(
        dtype).to(device)
    gb = rand(2 * blocks, part, seed=5, device=device)
    lam = (rand(W, seed=6) * 3 - 3).to(device)
    rate = -8.0 * torch.nn.functional.softplus(lam)
    w = {"ra": f64(gates[:blocks]), "ri": f64(gates[blocks:]),
         "ra.b": f64(gb[:blocks]), "ri.b": f64(gb[blocks:])}
    want = []
    for s in range(3):
        r, i = oracle.rglru_gates(f64(u[s]), w, "", blocks)
        want.append(oracle.decayed_sum(f64(u[s]), r, i, f64(lam))
                    * oracle.gelu_tanh(f64(y[s]) + f64(y_bias)))
    state = torch.full((5, W), 9.0, device=device)
    got = torch.zeros(3, T, W, dtype=dtype, device=device)

    def run(s, slot, at, n, step):
        # in the middle of a larger batch, y in columns of a wider row
        uu = torch.zeros(n + 3, W, dtype=dtype, device=device)
        yy = torch.zeros(n + 3, 2 * W + 1, dtype=dtype, device=device)
        uu[2:2 + n], yy[2:2 + n, :W] = u[s, at:at + n], y[s, at:at + n]
        out = torch.zeros_like(uu)
        args = (out, uu, yy[:, :W], y_bias, gates, gb, rate, state,
                seg([(2, n, slot, at)], device))
        ops.rglru_step(*args) if step else ops.rglru_scan(*args, n)
        assert float(out[:2].abs().max()) == float(out[2 + n:].abs().max()) \
            == 0
        got[s, at:at + n] = out[2:2 + n]

    drive(T, run)
    for s in range(3):
        close(got[s], want[s], dtype)
    assert float(state[1].min()) == float(state[4].min()) == 9.0


@everywhere
def test_rglru_holds_a_far_token(device, dtype):
    """Input gates open at the first token only, no decay: what it wrote
    comes back hundreds of tokens later."""
    ops, W, T = ops_for(device), 16, 700
    u = torch.ones(T, W, dtype=dtype, device=device)
    u[1:] = -1.0
    # input gate sigmoid(40 u); log a = -8 softplus(-16) r, about -1e-6 r
    gates = torch.zeros(2, W, W, dtype=dtype, device=device)
    gates[1] = 40 * torch.eye(W)
    gb = torch.zeros(2, W, device=device)
    rate = torch.full((W,), -8 * math.log1p(math.exp(-16.0)), device=device)
    y = torch.full((T, W), 6.0, dtype=dtype, device=device)
    zero = torch.zeros(W, device=device)
    state = torch.full((1, W), 3.0, device=device)
    out = torch.zeros(T, W, dtype=dtype, device=device)
    ops.rglru_scan(out, u, y, zero, gates, gb, rate, state,
                   seg([(0, T, 0, 0)], device), T)
    a = math.exp(float(rate[0]) / 2)    # r = 1/2
    want = math.sqrt(1 - a * a) * a ** (T - 1) * 6.0
    got = float(out[-1].float().min())
    assert abs(got - want) < 0.01 * want, (got, want)
    ops.rglru_step(out, u, y, zero, gates, gb, rate, state,
                   seg([(T - 1, 1, 0, T)], device))
    assert abs(float(out[-1].float().max()) - want * a) < 0.01 * want


@everywhere
@pytest.mark.parametrize("H,N,E,G", [(1, 1, 1, 1), (3, 9, 7, 3), (6, 28, 20, 3),
                                     (4, 16, 32, 1), (2, 200, 136, 2),
                                     (2, 100, 72, 1), (2, 64, 16, 2),
                                     (4, 128, 64, 2)])
def test_mamba2(H, N, E, G, device, dtype):
    """Update and read-out, then skip, gate and grouped norm."""
    ops, T, eps = ops_for(device), 100, 1e-5
    inner = H * E
    cols = inner + 2 * G * N
    xbc = rand(3, T, cols, seed=1, dtype=dtype, device=device)
    dt = rand(3, T, H, seed=2, dtype=dtype, device=device) * 2
    z = rand(3, T, inner, seed=3, dtype=dtype, device=device) * 2
    dt_bias = rand(H, seed=4, device=device) - 1
    a_log = rand(H, seed=5, device=device) * 2 - 1
    skip = rand(H, seed=6, device=device)
    w = rand(inner, seed=7, device=device)
    groups = next(g for g in (7, 5, 4, 2, 1) if inner % g == 0)
    head = torch.arange(H) // (H // G)
    reads, want = [], []
    for s in range(3):
        x, B, C = f64(xbc[s]).split((inner, G * N, G * N), 1)
        args = (x.view(T, H, E), B.view(T, G, N)[:, head],
                C.view(T, G, N)[:, head],
                oracle.softplus(f64(dt[s]) + f64(dt_bias)),
                f64(a_log).exp())
        reads.append(oracle.ssd(*args, torch.zeros(H).double()).flatten(1))
        full = oracle.ssd(*args, f64(skip)).flatten(1)
        want.append(oracle.group_norm(full * oracle.silu(f64(z[s])), f64(w),
                                      groups, eps))
    state = torch.full((5, H, N, -(-E // 4) * 4), 7.0, device=device)
    got = torch.zeros(3, T, inner, device=device)
    normed = torch.zeros(3, T, inner, dtype=dtype, device=device)

    def run(s, slot, at, n, step):
        wide = torch.zeros(n + 3, inner + H, dtype=dtype, device=device)
        rows = torch.zeros(n + 3, cols, dtype=dtype, device=device)
        rows[2:2 + n] = xbc[s, at:at + n]
        wide[2:2 + n, :inner] = z[s, at:at + n]
        wide[2:2 + n, inner:] = dt[s, at:at + n]
        o = torch.zeros(n + 3, inner, device=device)
        args = (o, rows, wide[:, inner:], state, dt_bias, -a_log.exp(), E,
                seg([(2, n, slot, at)], device))
        ops.mamba2_step(*args) if step else ops.mamba2_scan(*args, n)
        assert float(o[:2].abs().max()) == float(o[2 + n:].abs().max()) == 0
        out = torch.empty(n + 3, inner, dtype=dtype, device=device)
        ops.mamba2_out(out, o, rows, wide[:, :inner], skip, w, groups, eps)
        got[s, at:at + n], normed[s, at:at + n] = o[2:2 + n], out[2:2 + n]

    drive(T, run)
    for s in range(3):
        # the read-out itself is float whatever the activations are
        close(got[s], reads[s], torch.float32, 4 * float(
            reads[s].abs().max()))
        if E > 1:
            close(normed[s], want[s], dtype)
    assert float(state[1].min()) == float(state[4].min()) == 7.0


@everywhere
def test_mamba2_holds_a_far_token(device, dtype):
    """Steps near zero after the first token: it is read unchanged hundreds
    of tokens later, and two heads of one group keep states of their own."""
    ops, H, N, E, T = ops_for(device), 2, 16, 16, 600
    xbc = torch.zeros(T, H * E + 2 * N, dtype=dtype, device=device)
    xbc[:, :H * E] = rand(T, H * E, seed=1, dtype=dtype, device=device)
    xbc[:, H * E] = 1.0                 # write row 0
    xbc[:, H * E + N] = 1.0             # read row 0
    dt = torch.full((T, H), -60.0, dtype=dtype, device=device)
    dt[0, 0], dt[0, 1] = 1.0, 2.0
    state = torch.full((1, H, N, E), 3.0, device=device)
    zero = torch.zeros(H, device=device)
    rate = torch.tensor([-0.5, -2.0], device=device)
    o = torch.zeros(T, H * E, device=device)
    ops.mamba2_scan(o, xbc, dt, state, zero, rate, E,
                    seg([(0, T, 0, 0)], device), T)
    size = oracle.softplus(torch.tensor([1.0, 2.0]).double())
    want = (f64(xbc[0, :H * E]).view(H, E) * size.view(H, 1)).flatten()
    close(o[-1], want, torch.float32)
    ops.mamba2_step(o, xbc, dt, state, zero, rate, E,
                    seg([(T - 1, 1, 0, T)], device))
    close(o[-1], want, torch.float32)


# ---------------------------------------------------------------------------
@pytest.mark.parametrize("rot", [
    dict(dims=16, base=10000.0), rotation(2, 10.0), rotation(16),
    rotation(64, 5e5, 16.0, 4096, 32.0, 1.0), rotation(40, 100.0, 1.0),
    rotation(128, 1e4, 4.0, 64, 64.0, 0.01), rotation(8, 7.0, 2.0, 9, 2, 2)])
def test_stretched_angles(rot):
    f, mult = scaled_rope_angles(rot)
    want, factor = oracle.yarn_frequencies(rot)
    assert torch.allclose(f, torch.tensor(want, dtype=torch.float64),
                          rtol=1e-12)
    assert mult == pytest.approx(factor, rel=1e-12)
    table = build_pair_rope_table(3000, rot)
    a = 2999 * torch.tensor(want, dtype=torch.float64)
    assert torch.allclose(table[-1].double(), torch.stack(
        (a.cos(), a.sin()), -1) * factor, atol=1e-6)


class Paged:
    """Sequences in scattered pages that were used before, two maps."""

    def __init__(self, device, dtype, H, G, D, E, rot, n_pages=60, slots=3):
        def pad(n):
            return next(p for p in (32, 64, 128, 256) if n <= p)

        self.ops, self.device, self.dtype = ops_for(device), device, dtype
        self.H, self.G, self.D, self.E, self.rot = H, G, D, E, rot
        self.k = rand(n_pages, 2 * G, PAGE * pad(D), seed=91, dtype=dtype,
                      device=device)
        self.v = rand(n_pages, G, PAGE * pad(E), seed=92, dtype=dtype,
                      device=device)
        per = n_pages // slots
        perm = torch.randperm(per * slots,
                              generator=torch.Generator().manual_seed(3))
        self.table = perm.view(slots, per).to(torch.int32).to(device)
        self.qw = rand(D, seed=93, device=device) * 0.2 + 1
        self.kw = rand(D, seed=94, device=device) * 0.2 + 1
        self.rope = None if rot is None else build_pair_rope_table(
            per * PAGE, rot, device)
        self.eps = 1e-5

    def rows(self, slot, pos0, n):
        return (torch.full((n,), slot, dtype=torch.int32, device=self.device),
                torch.arange(pos0, pos0 + n, dtype=torch.int32,
                             device=self.device))

    def append(self, slot, pos0, proj, store=True):
        n = proj.size(0)
        q = torch.empty(n, 2 * self.H, self.k.size(2) // PAGE,
                        dtype=self.dtype, device=self.device)
        if not store:
            proj = proj[:, :2 * self.H * self.D].contiguous()
        pages = (self.k, self.v) if store else (None, None)
        self.ops.qk_norm_append(
            q, *pages, proj, self.qw, self.kw if store else None,
            *self.rows(slot, pos0, n), self.table, self.E, self.eps,
            rope=self.rope)
        return q

    def attend(self, q, segs, scale, cap, lam, diff, splits):
        out = torch.zeros(q.size(0), self.H * self.E, dtype=self.dtype,
                          device=self.device)
        part = ()
        if splits:
            cells = len(segs) * 2 * self.H * splits
            part = (torch.full((cells * self.v.size(2) // PAGE,), math.nan,
                               device=self.device),
                    torch.full((cells * 2,), math.nan, device=self.device))
        bias = torch.zeros(self.H, 1, device=self.device)
        self.ops.paged_attn(out, q, self.k, self.v, bias, self.table,
                            seg(segs, self.device), max(s[1] for s in segs),
                            1 << 30, 0, scale, splits, *part, softcap=cap,
                            map_weight=lam, out_scale=1.0 - diff,
                            eps=self.eps)
        return out

    def oracle(self, proj, scale, cap, lam, diff):
        T, p = proj.size(0), f64(proj)
        H, G, D, E = self.H, self.G, self.D, self.E
        q, k, v = p.split((2 * H * D, 2 * G * D, G * E), 1)
        q = oracle.unit(q.reshape(T, H, 2, D), self.eps) * f64(self.qw)
        k = oracle.unit(k.reshape(T, G, 2, D), self.eps) * f64(self.kw)
        if self.rot is not None:
            q, k = oracle.rotate(q, self.rot), oracle.rotate(k, self.rot)
        v, out = v.reshape(T, G, E), []
        for h in range(H):
            g = h // (H // G)
            a1, a2 = (oracle.attend(q[:, h, m], k[:, g, m], v[:, g], scale,
                                    cap) for m in (0, 1))
            out.append(oracle.difference(a1, a2, lam, diff, self.eps))
        return torch.cat(out, 1)


@everywhere
@pytest.mark.parametrize("H,G,D,E,rot,cap", [
    (4, 2, 32, 32, rotation(32), 5.0), (6, 2, 24, 40, rotation(16), 0.0),
    (3, 1, 10, 9, rotation(6, 50.0), 2.0), (1, 1, 2, 3, rotation(2), 9.0),
    (20, 1, 16, 24, None, 30.0), (2, 2, 64, 130, rotation(64), 50.0),
    (4, 4, 120, 100, rotation(8), 3.0), (3, 1, 200, 256, rotation(200), 8.0)])
def test_differential_attention(H, G, D, E, rot, cap, device, dtype):
    """A prompt whole, in portions, its tokens one by one with the keys split
    in several ways, and queries over keys that another layer stored."""
    T, scale, lam, diff = 150, 0.35, 0.55, 0.3
    P = Paged(device, dtype, H, G, D, E, rot)
    proj = rand(T, 2 * (H + G) * D + G * E, seed=8, dtype=dtype,
                device=device)
    want = P.oracle(proj, scale, cap, lam, diff)
    peak = float(want.abs().max())
    # the difference of two rounded averages is brought to unit size
    if dtype == torch.bfloat16:
        peak *= 2

    def check(q, segs, splits, rows, expect):
        o = P.attend(q, segs, scale, cap, lam, diff, splits)
        close(o[rows], expect, dtype, peak)

    q = P.append(1, 0, proj)
    check(q, [(0, T, 1, 0)], 0, slice(None), want)
    kept = P.k.clone(), P.v.clone()
    assert torch.equal(P.append(1, 0, proj, store=False), q)
    assert torch.equal(P.k, kept[0]) and torch.equal(P.v, kept[1])
    at = 0
    for n in (2, 62, 1, 3, 61, 21):
        q2 = P.append(0, at, proj[at:at + n])
        q2 = torch.cat([torch.zeros_like(q2[:1]), q2])
        check(q2, [(1, n, 0, at)], 0, slice(1, None), want[at:at + n])
        at += n
    # later keys are in the pages already and must not be seen
    ts = sorted({*range(0, T, 7), 62, 63, 64, 65, 127, 128, T - 1})
    for splits in (1, 2, 5):
        check(q, [(t, 1, 1, t) for t in ts], splits, ts, want[ts])


@everywhere
@pytest.mark.parametrize("which", [0, 1])
def test_one_key_of_one_map_stands_out(which, device, dtype):
    """One map's queries meet one key among hundreds, the other map's weights
    are even: the value comes out with the map's sign, wherever the key is."""
    H, G, D, E, T, lam = 2, 1, 32, 32, 700, 0.5
    P = Paged(device, dtype, H, G, D, E, None)
    P.qw.fill_(3.0)
    P.kw.fill_(3.0)
    queries = [1, 63, 64, 65, 255, 256, 639, 640, 699]
    for j in (0, 1, 62, 63, 64, 65, 127, 128, 255, 256, 640):
        proj = torch.zeros(T, 2 * (H + G) * D + G * E, dtype=dtype,
                           device=device)
        proj[:, which * D] = proj[:, (2 + which) * D] = 1.0
        k0 = 2 * H * D
        proj[:, k0 + which * D] = -1.0
        proj[j, k0 + which * D] = 1.0
        v0 = 2 * (H + G) * D
        proj[:, v0] = 1.0           # the other keys' value
        proj[j, v0] = 0.0
        proj[j, v0 + 1] = 1.0
        q = P.append(2, 0, proj)
        segs = [(i, 1, 2, i) for i in queries]
        for o in (P.attend(q, [(0, T, 2, 0)], 1.0, 0.0, lam, 0.0, 0),
                  P.attend(q, segs, 1.0, 0.0, lam, 0.0, 1),
                  P.attend(q, segs, 1.0, 0.0, lam, 0.0, 4)):
            for i in queries:
                share = 1.0 / (i + 1) if j <= i else 0.0
                even = torch.tensor([1.0 - share, share]).double()
                sharp = torch.tensor([0.0, 1.0] if j <= i else [1.0, 0.0]
                                     ).double()
                a = (sharp, even) if which == 0 else (even, sharp)
                d = torch.zeros(E).double()
                d[:2] = a[0] - lam * a[1]
                want = oracle.unit(d, P.eps)[:2]
                got = f64(o[i]).view(H, E)[:, :2]
                assert float((got - want).abs().max()) < 0.06, (i, j)


@everywhere
def test_capped_scores(device, dtype):
    """Scores far past the cap: what is left is the cap's own difference."""
    H, G, D, E, T, cap = 1, 1, 32, 32, 40, 1.5
    P = Paged(device, dtype, H, G, D, E, None)
    P.qw.fill_(4.0)
    P.kw.fill_(4.0)
    proj = torch.zeros(T, 4 * D + E, dtype=dtype, device=device)
    proj[:, 0] = proj[:, D] = 1.0
    proj[:, 2 * D] = -1.0           # map 1: key 7 attracts, the rest repel
    proj[7, 2 * D] = 1.0
    proj[:, 3 * D:4 * D:2] = 1.0    # map 2: even
    proj[:, 4 * D] = 1.0
    proj[7, 4 * D] = 0.0
    proj[7, 4 * D + 1] = 1.0
    want = P.oracle(proj, 1.0, cap, 0.3, 0.2)
    hot = math.exp(2 * cap) / (math.exp(2 * cap) + T - 1)
    d = torch.zeros(E).double()
    d[0], d[1] = 1 - hot - 0.3 * (1 - 1 / T), hot - 0.3 / T
    assert torch.allclose(want[-1], oracle.unit(d, P.eps) * 0.8, atol=1e-3)
    q = P.append(0, 0, proj)
    close(P.attend(q, [(0, T, 0, 0)], 1.0, cap, 0.3, 0.2, 0), want, dtype)
    o = P.attend(q, [(T - 1, 1, 0, T - 1)], 1.0, cap, 0.3, 0.2, 2)
    close(o[-1], want[-1], dtype)


@everywhere
@pytest.mark.parametrize("G,D,E", [(2, 24, 40), (1, 10, 9), (3, 64, 128)])
def test_cached_rows_come_back(G, D, E, device, dtype):
    """Keys and values between stages: out of one cache into another."""
    n = 100
    a, b = (Paged(device, dtype, G, G, D, E, None) for _ in "ab")
    rows = rand(n, 2 * G * D + G * E, seed=4, dtype=dtype, device=device)
    where = a.rows(1, 30, n)
    a.ops.kv_rows(rows, a.k, a.v, *where, a.table, D, E, True)
    back = torch.zeros_like(rows)
    a.ops.kv_rows(back, a.k, a.v, *where, a.table, D, E, False)
    assert torch.equal(back, rows)
    # the same pages as an append makes
    proj = rand(n, 4 * G * D + G * E, seed=5, dtype=dtype, device=device)
    a.append(2, 7, proj)
    b.k.copy_(a.k), b.v.copy_(a.v)
    where = a.rows(2, 7, n)
    a.ops.kv_rows(rows, a.k, a.v, *where, a.table, D, E, False)
    assert torch.equal(rows[:, 2 * G * D:], proj[:, 4 * G * D:])
    b.ops.kv_rows(rows, b.k, b.v, *where, b.table, D, E, True)
    assert torch.equal(a.k, b.k) and torch.equal(a.v, b.v)


# ---------------------------------------------------------------------------
def routed(n, top, experts, identity, W, F, tile, gated, device, dtype,
           correction=None):
    ops, scale = ops_for(device), 1.7
    outputs = experts + identity
    x = rand(n, W, seed=1, dtype=dtype, device=device)
    router = (rand(outputs + gated, W, seed=2) * 3 * W ** -0.5).to(
        dtype).to(device)
    if correction is None:
        correction = rand(outputs, seed=3) * 0.4
    upper = (rand(experts, 2 * F, W, seed=11) * W ** -0.5).to(dtype)
    down = (rand(experts, W, F, seed=12) * F ** -0.5).to(dtype)
    weight = torch.full((n, top + gated), math.nan, device=device)
    plan = ops.moe_route(weight, x, router, top, tile,
                         correction=correction.to(device), scale=scale,
                         identity=identity, gated=bool(gated))
    mid = torch.full((n * top, F), math.nan, dtype=dtype, device=device)
    ops.moe_up(mid, x, upper.to(device), plan, 0, tile)
    rows = torch.full((n, top, W), math.nan, dtype=dtype, device=device)
    ops.moe_down(rows, mid, down.to(device), plan, tile)
    stream = f64(x).float().to(device)
    before = f64(stream)
    y = rand(n, W, seed=5, dtype=dtype, device=device) if gated else None
    ops.stream_step(stream, y, routed=rows, routed_w=weight, chosen=plan,
                    experts=experts)
    xd, z = f64(x), f64(x) @ f64(router).T
    want, picks = [], []
    for t in range(n):
        add = torch.zeros(W).double()
        for e, p in oracle.route(z[t, :outputs], f64(correction), top, scale):
            picks.append(e)
            if e >= experts:
                add += p * xd[t]
                continue
            ud, dd = f64(upper[e]), f64(down[e])
            add += p * (dd @ (oracle.silu(ud[:F] @ xd[t])
                              * (ud[F:] @ xd[t])))
        if gated:
            g = oracle.sigmoid(z[t, -1])
            assert abs(float(weight[t, top]) - float(g)) < 1e-5
            add += g * f64(y[t])
        want.append(add)
    close(f64(stream) - before, torch.stack(want), dtype)
    return picks


@everywhere
@pytest.mark.parametrize("gated", [0, 1])
@pytest.mark.parametrize("n,top,experts,identity,W,F", [
    (1, 2, 5, 2, 72, 24), (37, 3, 7, 1, 64, 40), (5, 1, 1, 0, 27, 5),
    (30, 4, 2, 5, 33, 9), (9, 6, 64, 4, 512, 16), (50, 2, 130, 20, 40, 8)])
def test_corrected_routing(n, top, experts, identity, W, F, gated, device,
                           dtype):
    picks = routed(n, top, experts, identity, W, F, 16, gated, device, dtype)
    if n > 20 and identity:
        assert max(picks) >= experts > min(picks)


@everywhere
def test_correction_chooses_but_does_not_weigh(device, dtype):
    """A correction past every score decides alone; weights stay those of the
    scores, whose sum is scaled."""
    experts, identity = 6, 2
    correction = torch.zeros(experts + identity)
    correction[3], correction[7] = 5.0, 4.0
    picks = routed(20, 2, experts, identity, 64, 16, 16, 1, device, dtype,
                   correction)
    assert picks == [3, 7] * 20
    # and all tokens to the identity outputs
    correction[6] = 9.0
    correction[3] = 0.0
    assert set(routed(20, 2, experts, identity, 64, 16, 16, 1, device, dtype,
                      correction)) == {6, 7}


@pytest.mark.gpu
@pytest.mark.parametrize("n,top,experts,identity", [(400, 3, 3, 2),
                                                    (257, 1, 2, 1)])
def test_large_expert_tiles_with_identity_outputs(n, top, experts, identity):
    routed(n, top, experts, identity, 256, 128, 128, 1, "cuda",
           torch.bfloat16)


# ---------------------------------------------------------------------------
@everywhere
def test_gelu(device, dtype):
    z = torch.cat([torch.linspace(-9, 9, 4001),
                   torch.tensor([0.0, -1e-4, 1e-4, -30.0])]).to(dtype)
    want = oracle.gelu_erf(z.double())
    for n in (z.numel(), 8, 1):
        g = z[:n].clone().to(device)
        ops_for(device).gelu(g)
        err = (f64(g) - want[:n]).abs()
        assert bool((err <= (2e-6 if dtype == torch.float32 else 8e-3)
                     * (want[:n].abs() + 1)).all())


@pytest.mark.gpu
@pytest.mark.parametrize("n,m,k", [(1, 300, 4096), (5, 50, 192),
                                   (16, 1000, 4160), (32, 33, 20480)])
def test_gelu_at_the_end_of_a_projection(n, m, k):
    ops = ops_for("cuda")
    x = rand(n, k, seed=1, dtype=torch.bfloat16, device="cuda")
    w = rand(m, k, seed=2, dtype=torch.bfloat16, device="cuda") * k ** -0.5
    want = oracle.gelu_erf(f64(x) @ f64(w).T)
    out = torch.full((n, m), math.nan, dtype=torch.bfloat16, device="cuda")
    ops.skinny_gemm(out, w, x, 2, 0.0, 0.0)
    close(out, want, torch.bfloat16)
    if n == 1:
        out.fill_(math.nan)
        ops.gemv(out, w, x, None, None, 5, rows=1, act_p=0.0, act_q=0.0)
        close(out, want, torch.bfloat16)


@pytest.mark.gpu
def test_operations_refuse_what_they_cannot_hold():
    """Errors from the host's checks, ahead of any launch."""
    ops, d = ops_for("cuda"), "cuda"
    x = torch.zeros(4, 64, device=d)
    v = torch.zeros(64, device=d)
    s = seg([(0, 4, 0, 0)], d)
    state = torch.zeros(2, 64, device=d)
    for call in (
            lambda: ops.stream_step(x, x, v, groups=5),
            lambda: ops.stream_step(x, xn=x, next_w=v, shift=v, prev=state,
                                    row_slot=s[0], row_pos=s[0]),
            lambda: ops.causal_conv(x, x, torch.zeros(17, 64, device=d), v,
                                    None, torch.zeros(2, 16, 64, device=d),
                                    s, 4, False),
            lambda: ops.rglru_scan(x, x, x, v, torch.zeros(2, 32, 32,
                                                           device=d), v, v,
                                   state, s, 4),
            lambda: ops.mamba2_scan(x, x, x[:, :2],
                                    torch.zeros(2, 2, 300, 16, device=d), v,
                                    v, 16, s, 4),
            lambda: ops.mamba2_out(x, x, x, x, v[:3], v, 1, 1e-5),
            lambda: ops.moe_route(x, x, torch.zeros(8, 64, device=d), 2, 16,
                                  correction=v, identity=8)):
        with pytest.raises(RuntimeError):
            call()
