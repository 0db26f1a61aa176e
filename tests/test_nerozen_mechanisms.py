"""Each mechanism of Nerozen alone against its oracle: the HIP kernels on a
GPU, the torch operations of the CPU path elsewhere.  Inputs are made so
that one wrong key, gate or edge changes the result visibly."""

import math

import pytest
import torch

import nerozen_oracle as oracle
from helpers import close, everywhere, ops_for, rand, seg
from mdi_llm_amd.ops.hybrid_engine import distance_bias

PAGE = 64


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("e", [8, 27, 300, 1024, 1501, 4096, 5000, 9000])
def test_residual_norm(e, device, dtype):
    ops, n, eps = ops_for(device), 5, 1e-5
    x = rand(n, e, seed=1, device=device) * 3
    y = rand(n, e, seed=2, dtype=dtype, device=device) * 0.01
    wb, wn = rand(e, seed=3, device=device), rand(e, seed=4, device=device)
    # add with post-norm, then pre-norm
    x1, xn = x.clone(), torch.empty_like(y)
    ops.residual_norm(x1, y=y, post_w=wb, xn=xn, next_w=wn, offset=1.0,
                      eps=eps)
    want = x.double().cpu() + oracle.zero_centred_norm(
        y.double().cpu(), wb.double().cpu(), eps)
    close(x1, want, torch.float32)
    close(xn, oracle.zero_centred_norm(want, wn.double().cpu(), eps), dtype)
    # plain add, no further norm; plain weights (offset 0)
    x2 = x.clone()
    ops.residual_norm(x2, y=y)
    close(x2, x.double().cpu() + y.double().cpu(), torch.float32)
    ops.residual_norm(x2.copy_(x), xn=xn, next_w=wn, eps=eps)
    close(x2, x, torch.float32)
    close(xn, oracle.rms(x.double().cpu(), eps) * wn.double().cpu(), dtype)
    # embedding
    table = rand(11, e, seed=5, dtype=dtype, device=device)
    toks = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32, device=device)
    ops.residual_norm(x2, tokens=toks, table=table, scale=0.5, xn=xn,
                      next_w=wn, offset=1.0, eps=eps)
    want = table.double().cpu()[toks.long().cpu()] * 0.5
    close(x2, want, torch.float32)
    close(xn, oracle.zero_centred_norm(want, wn.double().cpu(), eps), dtype)


@everywhere
def test_xielu(device, dtype):
    p, q = 0.3, 1.7
    z = torch.cat([torch.linspace(-30, 12, 4001),
                   torch.tensor([0.0, -1e-4, 1e-4, -1e-2])]).to(dtype)
    act = torch.tensor([math.log(math.expm1(p)), math.log(math.expm1(q))],
                       dtype=torch.float64)
    want = oracle.xielu(z.double(), act)
    for n in (z.numel(), 8, 1):
        g = z[:n].clone().to(device)
        ops_for(device).xielu(g, p, q)
        err = (g.double().cpu() - want[:n]).abs()
        assert bool((err <= (1e-6 if dtype == torch.float32 else 8e-3)
                     * (1 + want[:n].abs())).all())


# ---------------------------------------------------------------------------
def recurrence_case(H, D, E, n, seed, dtype, device):
    proj = rand(n, H * (2 * D + E), seed=seed, dtype=dtype, device=device)
    fb = rand(H * D, seed=seed + 1, device=device) * 3 + 2
    lower = torch.rand(H * D, generator=torch.Generator().manual_seed(seed))
    lower = (lower * 0.95).to(device)
    w = rand(E, seed=seed + 2, device=device) * 0.2 + 1
    return proj, fb, lower, w


def recurrence_oracle(proj, fb, lower, w, H, D, E, eps):
    p = proj.double().cpu()
    n = p.size(0)
    q, f, v = p.split((H * D, H * D, H * E), 1)
    f = oracle.forget_gate(f, fb.double().cpu(), lower.double().cpu())
    o = oracle.gated_scan(oracle.silu(q).view(n, H, D), f.view(n, H, D),
                          v.view(n, H, E))
    return (oracle.rms(o, eps) * w.double().cpu()).reshape(n, H * E)


@everywhere
@pytest.mark.parametrize("H,D,E", [(2, 32, 72), (3, 16, 16), (1, 1, 3),
                                   (2, 100, 30), (1, 256, 8), (2, 8, 130),
                                   (2, 64, 48), (2, 128, 128)])
def test_hgrn2_scan_and_step(H, D, E, device, dtype):
    """Three sequences: a prompt, a prompt in uneven portions, and one that
    is decoded; states in slots that hold leftovers."""
    ops, eps = ops_for(device), 1e-5
    n = 70
    cases = [recurrence_case(H, D, E, n, 10 * s, dtype, device)
             for s in range(3)]
    _, fb, lower, w = cases[0]
    projs = [c[0] for c in cases]
    wants = [recurrence_oracle(p, fb, lower, w, H, D, E, eps) for p in projs]
    state = torch.full((4, H, D, -(-E // 4) * 4), 7.0, device=device)
    got = [torch.zeros(n, H * E, dtype=dtype, device=device)
           for _ in projs]

    def run(seq, slot, at, m, step):
        # the segment lies in the middle of a larger batch
        flat = torch.zeros(m + 3, projs[seq].size(1), dtype=dtype,
                           device=device)
        flat[2:2 + m] = projs[seq][at:at + m]
        y = torch.zeros(m + 3, H * E, dtype=dtype, device=device)
        s = seg([(2, m, slot, at)], device)
        if step:
            ops.hgrn2_step(y, flat, state, fb, lower, w, s, eps)
        else:
            ops.hgrn2_scan(y, flat, state, fb, lower, w, s, m, eps)
        assert float(y[:2].abs().max()) == float(y[2 + m:].abs().max()) == 0
        got[seq][at:at + m] = y[2:2 + m]

    run(0, 2, 0, n, False)
    at = 0
    for m in (2, 1, 16, 17, 31, 3):
        run(1, 0, at, m, m == 1)
        at += m
    for t in range(n):
        run(2, 3, t, 1, True)
    for g, x in zip(got, wants):
        close(g, x, dtype)
    assert float(state[1].min()) == 7.0  # nobody's slot


@everywhere
def test_hgrn2_holds_a_far_token(device, dtype):
    """Gates shut after the first token: its value comes back unchanged
    hundreds of tokens later, from a prompt and from decoding."""
    ops, H, D, E, n = ops_for(device), 1, 16, 16, 600
    fb = torch.full((D,), 30.0, device=device)   # keep everything
    lower = torch.zeros(D, device=device)
    w = torch.ones(E, device=device)
    proj = torch.zeros(n, 2 * D + E, dtype=dtype, device=device)
    proj[:, 0] = 4.0                       # read channel 0
    proj[0, D] = -60.0                     # f = 0: write the first value
    proj[:, 2 * D:] = rand(n, E, seed=3, dtype=dtype, device=device)
    first = oracle.rms(proj[0, 2 * D:].double().cpu(), 1e-5)
    state = torch.zeros(2, H, D, E, device=device)
    y = torch.zeros(n, E, dtype=dtype, device=device)
    ops.hgrn2_scan(y, proj, state, fb, lower, w, seg([(0, n, 0, 0)], device), n, 1e-5)
    close(y[n - 1], first, dtype)
    ops.hgrn2_step(y, proj, state, fb, lower, w,
                   seg([(n - 1, 1, 0, n)], device), 1e-5)
    close(y[n - 1], first, dtype)


# ---------------------------------------------------------------------------
@pytest.mark.parametrize("rows,far", [(16, 200), (8, 64), (20, 320),
                                      (2, 9), (32, 128), (10, 7), (6, 1000)])
def test_distance_buckets(rows, far):
    rel = torch.arange(rows * 3, dtype=torch.float64).view(rows, 3)
    b = distance_bias(rel, far) / math.log2(math.e)
    for n in range(2 * far + 5):
        want = rel[oracle.distance_bucket(n, rows, far)]
        got = b[:, min(n, b.size(1) - 1)].double()
        assert torch.allclose(got, want, rtol=1e-6), n


class Paged:
    """Sequences in scattered pages, filled through the append operation."""

    def __init__(self, device, dtype, H, G, D, E, n_pages=40, slots=3):
        pad = lambda n: next(p for p in (32, 64, 128, 256) if n <= p)
        self.ops, self.device, self.dtype = ops_for(device), device, dtype
        self.H, self.G, self.D, self.E = H, G, D, E
        # what earlier owners of the pages left behind
        self.k = rand(n_pages, G, PAGE * pad(D), seed=91, dtype=dtype,
                      device=device)
        self.v = rand(n_pages, G, PAGE * pad(E), seed=92, dtype=dtype,
                      device=device)
        perm = torch.randperm(n_pages,
                              generator=torch.Generator().manual_seed(3))
        per = n_pages // slots
        self.table = perm[:per * slots].view(slots, per).to(
            torch.int32).to(device)
        self.qw = rand(D, seed=93, device=device) * 0.1 + 1
        self.kw = rand(D, seed=94, device=device) * 0.1 + 1
        self.eps = 1e-6

    def append(self, slot, pos0, proj):
        n = proj.size(0)
        q = torch.empty(n, self.H, self.k.size(2) // PAGE, dtype=self.dtype,
                        device=self.device)
        rs = torch.full((n,), slot, dtype=torch.int32, device=self.device)
        rp = torch.arange(pos0, pos0 + n, dtype=torch.int32,
                          device=self.device)
        self.ops.qk_norm_append(q, self.k, self.v, proj, self.qw, self.kw,
                                rs, rp, self.table, self.E, self.eps)
        return q

    def attend(self, q, segs, bias, window, keep, scale, splits):
        out = torch.zeros(q.size(0), self.H * self.E, dtype=self.dtype,
                          device=self.device)
        part = ()
        if splits > 1:
            cells = len(segs) * self.H * splits
            part = (torch.full((cells * self.v.size(2) // PAGE,), math.nan,
                               device=self.device),
                    torch.full((cells * 2,), math.nan, device=self.device))
        self.ops.paged_attn(out, q, self.k, self.v, bias, self.table,
                            seg(segs, self.device), max(s[1] for s in segs),
                            window, keep, scale, splits, *part)
        return out

    def oracle(self, proj, rel, far, window, keep, scale):
        T = proj.size(0)
        p = proj.double().cpu()
        H, G, D, E = self.H, self.G, self.D, self.E
        q, k, v = p.split((H * D, G * D, G * E), 1)
        q = oracle.rms(q.reshape(T, H, D), self.eps) * self.qw.double().cpu()
        k = oracle.rms(k.reshape(T, G, D), self.eps) * self.kw.double().cpu()
        a = oracle.attention_weights(q, k, scale, rel.double(), far, window,
                                     keep)
        o = torch.einsum("htj,jhe->the", a, v.reshape(
            T, G, E).repeat_interleave(H // G, 1))
        return o.reshape(T, H * E)


SHAPES = [(4, 2, 32, 32, 50, 3), (6, 2, 48, 20, 37, 0), (5, 1, 64, 64, 64, 1),
          (3, 3, 100, 130, 1, 4), (20, 1, 16, 24, 33, 40),
          (8, 8, 128, 128, 500, 2), (2, 1, 200, 256, 90, 33)]


@everywhere
@pytest.mark.parametrize("H,G,D,E,window,keep", SHAPES)
def test_attention(H, G, D, E, window, keep, device, dtype):
    """A prompt whole, in portions, and its tokens one by one (with the keys
    split in several ways), in scattered pages that were used before."""
    T, far, scale = 200, 70, 0.3
    P = Paged(device, dtype, H, G, D, E)
    rel = rand(10, H, seed=7)
    bias = distance_bias(rel, far).to(device)
    proj = rand(T, (H + G) * D + G * E, seed=8, dtype=dtype, device=device)
    want = P.oracle(proj, rel, far, window, keep, scale)
    tol_scale = float(want.abs().max())
    # whole
    q = P.append(1, 0, proj)
    close(P.attend(q, [(0, T, 1, 0)], bias, window, keep, scale, 0), want,
          dtype, tol_scale)
    # portions, rows inside a larger batch
    at = 0
    for n in (2, 63, 1, 31, 64, 39):
        q = P.append(0, at, proj[at:at + n])
        q = torch.cat([torch.zeros_like(q[:1]), q])
        o = P.attend(q, [(1, n, 0, at)], bias, window, keep, scale, 0)
        close(o[1:], want[at:at + n], dtype, tol_scale)
        at += n
    # one by one; every position of the prompt's cache is there already, the
    # later ones must not be seen
    q = P.append(1, 0, proj)
    for splits in (1, 2, 5):
        ts = list(range(0, T, 7)) + [63, 64, 65, window - 1, window, T - 1]
        ts = sorted({t for t in ts if 0 <= t < T})
        o = P.attend(q, [(t, 1, 1, t) for t in ts], bias, window, keep,
                     scale, splits)
        close(o[ts], want[ts], dtype, tol_scale)


@everywhere
@pytest.mark.parametrize("window,keep", [(40, 0), (40, 5), (64, 33), (1, 2),
                                         (130, 64), (300, 1)])
def test_one_key_stands_out(window, keep, device, dtype):
    """All keys repel the query but one; its value must come through exactly
    where the mask lets it, at page borders, just inside and just outside of
    the window and of the kept tokens."""
    H, G, D, E, T = 2, 1, 32, 32, 260
    P = Paged(device, dtype, H, G, D, E)
    P.qw.fill_(3.0)
    P.kw.fill_(3.0)
    bias = torch.zeros(H, 2, device=device)
    queries = [255, 256, 259, 128, 191, 192]
    spots = {0, 1, keep - 1, keep, keep + 1, 63, 64, 65, 127, 128}
    for i in queries:
        spots |= {i, i - 1, i - window + 1, i - window, i - window - 1}
    for j in sorted(s for s in spots if 0 <= s < T):
        proj = torch.zeros(T, (H + G) * D + G * E, dtype=dtype,
                           device=device)
        proj[:, 0] = proj[:, D] = 1.0          # both query heads
        proj[:, H * D] = -1.0                  # keys
        proj[j, H * D] = 1.0
        proj[:, (H + G) * D:] = 0.01
        proj[j, (H + G) * D:] = 1.0
        q = P.append(2, 0, proj)
        segs = [(i, 1, 2, i) for i in queries]
        whole = P.attend(q, [(0, T, 2, 0)], bias, window, keep, 1.0, 0)
        for o in (whole, P.attend(q, segs, bias, window, keep, 1.0, 1),
                  P.attend(q, segs, bias, window, keep, 1.0, 3)):
            for i in queries:
                # alone in sight, any key has all the weight
                seen = oracle.visible(i, j, window, keep)
                got = float(o[i].float().min())
                assert abs(got - (1.0 if seen else 0.01)) < 0.02, (i, j)


@everywhere
def test_bias_counts_beside_the_score(device, dtype):
    """Equal scores: the weights are the softmax of the bias alone, whatever
    the score scale; distances in every bucket and past the last."""
    H, G, D, E, T, rows, far = 3, 1, 16, 8, 150, 8, 60
    P = Paged(device, dtype, H, G, D, E)
    rel = rand(rows, H, seed=5) * 2
    bias = distance_bias(rel, far).to(device)
    proj = torch.zeros(T, (H + G) * D + G * E, dtype=dtype, device=device)
    proj[:, :(H + G) * D] = 1.0
    proj[:, (H + G) * D:] = rand(T, E, seed=6, dtype=dtype, device=device)
    for scale in (0.125, 1.0):
        q = P.append(0, 0, proj)
        o = P.attend(q, [(0, T, 0, 0)], bias, 1000, 0, scale, 0)
        want = P.oracle(proj, rel, far, 1000, 0, scale)
        close(o, want, dtype)


# ---------------------------------------------------------------------------
@pytest.mark.gpu
@pytest.mark.parametrize("m,k", [(16, 64), (50, 192), (300, 4096),
                                 (1000, 4160), (33, 20480)])
@pytest.mark.parametrize("n", [1, 2, 5, 16, 17, 32])
def test_few_row_projection(n, m, k):
    """Odd output widths, K with and without whole unrolled stretches; the
    activation in the epilogue; a row does not depend on its companions."""
    ops = ops_for("cuda")
    x = rand(n, k, seed=1, dtype=torch.bfloat16, device="cuda")
    w = rand(m, k, seed=2, dtype=torch.bfloat16, device="cuda") * k ** -0.5
    want = x.double().cpu() @ w.double().cpu().T
    out = torch.full((n, m), math.nan, dtype=torch.bfloat16, device="cuda")
    ops.skinny_gemm(out, w, x)
    close(out, want, torch.bfloat16)
    act = torch.tensor([0.2, -0.4], dtype=torch.float64)
    p, q = torch.nn.functional.softplus(act).tolist()
    ops.skinny_gemm(out, w, x, True, p, q)
    close(out, oracle.xielu(want, act), torch.bfloat16)
    one = torch.empty(1, m, dtype=torch.bfloat16, device="cuda")
    ops.skinny_gemm(one, w, x[-1:].contiguous(), True, p, q)
    if n <= 16:
        assert torch.equal(one[0], out[-1])
