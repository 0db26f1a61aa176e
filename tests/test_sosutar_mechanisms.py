"""Each mechanism of Sosutar alone against its oracle: the HIP kernels on a
GPU, the torch operations of the CPU path elsewhere.  Inputs are made so that
one wrong key, state, sink or edge changes the result visibly."""

import math

import pytest
import torch

import sosutar_oracle as oracle
from helpers import close, everywhere, ops_for, rand, seg
from test_dinuzen_mechanisms import drive

PAGE = 64


def f64(t):
    return t.double().cpu()


# ---------------------------------------------------------------------------
ROWS = [8, 27, 300, 1024, 1501, 4096, 9000]


@everywhere
@pytest.mark.parametrize("e", ROWS)
def test_layer_scale(e, device, dtype):
    """A sublayer's output times its factors, without a norm, then the norm
    of the sum."""
    ops, n, eps = ops_for(device), 5, 1e-3
    x, y = rand(n, e, seed=1, device=device), rand(
        n, e, seed=2, dtype=dtype, device=device)
    g, w = rand(e, seed=3, device=device), rand(e, seed=4, device=device)
    xn = torch.empty(n, e, dtype=dtype, device=device)
    want = f64(x) + f64(g) * f64(y)
    ops.residual_norm(x, y=y, gain=g, xn=xn, next_w=w, eps=eps)
    close(x, want, torch.float32)
    close(xn, oracle.rms_norm(want, f64(w), eps), dtype)


@everywhere
@pytest.mark.parametrize("e", ROWS)
def test_sum_of_two_normed_outputs(e, device, dtype):
    """Outputs of very different size: each has a norm of its own."""
    ops, n, eps = ops_for(device), 5, 1e-3
    x = rand(n, e, seed=1, device=device)
    y = rand(n, e, seed=2, dtype=dtype, device=device) * 20
    z = rand(n, e, seed=3, dtype=dtype, device=device) * 0.05
    wy, wz = rand(e, seed=4, device=device), rand(e, seed=5, device=device)
    w = rand(e, seed=6, device=device)
    xn = torch.empty(n, e, dtype=dtype, device=device)
    want = f64(x) + oracle.rms_norm(f64(y), f64(wy), eps) \
        + oracle.rms_norm(f64(z), f64(wz), eps)
    ops.residual_norm(x, y=y, post_w=wy, y2=z, post_w2=wz, xn=xn, next_w=w,
                      eps=eps)
    close(x, want, torch.float32)
    close(xn, oracle.rms_norm(want, f64(w), eps), dtype)


@everywhere
def test_scaled_embedding_with_positions(device, dtype):
    """The position's vector is not scaled."""
    ops, e = ops_for(device), 72
    table = rand(11, e, seed=1, dtype=dtype, device=device)
    pos = rand(9, e, seed=2, dtype=dtype, device=device)
    toks = torch.tensor([3, 10, 0], dtype=torch.int32, device=device)
    at = torch.tensor([8, 0, 5], dtype=torch.int32, device=device)
    x = torch.empty(3, e, device=device)
    ops.residual_norm(x, tokens=toks, table=table, scale=2.5, pos_table=pos,
                      row_pos=at)
    close(x, f64(table)[[3, 10, 0]] * 2.5 + f64(pos)[[8, 0, 5]],
          torch.float32)


@everywhere
def test_squared_relu(device, dtype):
    z = torch.cat([torch.linspace(-9, 9, 4001),
                   torch.tensor([0.0, -1e-4, 1e-4, -30.0])]).to(dtype)
    want = f64(z).clamp(min=0.0).square()
    for n in (z.numel(), 8, 1):
        g = z[:n].clone().to(device)
        ops_for(device).relu2(g)
        close(g, want[:n], dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("n,m,k", [(1, 300, 4096), (5, 50, 192),
                                   (16, 1000, 4160), (32, 33, 20480)])
def test_squared_relu_at_the_end_of_a_projection(n, m, k):
    ops = ops_for("cuda")
    x = rand(n, k, seed=1, dtype=torch.bfloat16, device="cuda")
    w = rand(m, k, seed=2, dtype=torch.bfloat16, device="cuda") * k ** -0.5
    want = (f64(x) @ f64(w).T).clamp(min=0.0).square()
    out = torch.full((n, m), math.nan, dtype=torch.bfloat16, device="cuda")
    ops.skinny_gemm(out, w, x, 3, 0.0, 0.0)
    close(out, want, torch.bfloat16)
    if n == 1:
        out.fill_(math.nan)
        ops.gemv(out, w, x, None, None, 6, rows=1, act_p=0.0, act_q=0.0)
        close(out, want, torch.bfloat16)


# ---------------------------------------------------------------------------
def memory_oracle(proj, gate_bias, norm_w, H, D, E, cap, eps):
    p = f64(proj)
    T = p.shape[0]
    q, k, v, g, i, f = p.split((H * D, H * D, H * E, H * E, H, H), 1)
    q, k, v = q.view(T, H, D) * D ** -0.5, k.view(T, H, D), v.view(T, H, E)
    bi, bf = f64(gate_bias).split(H)
    i = oracle.capped(i + bi, cap)
    f = oracle.log_sigmoid(oracle.capped(f + bf, cap))
    o = torch.cat([oracle.unit(oracle.matrix_memory(
        q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]), eps)
        for a in range(H)], 1)
    return o * f64(norm_w) * oracle.sigmoid(g)


class Memory:
    """Sequences in slots that hold leftovers; segments lie in the middle of
    a larger batch."""

    def __init__(self, device, dtype, H, D, E, cap, norm_w=None, bias=None):
        self.ops, self.device, self.dtype = ops_for(device), device, dtype
        self.H, self.D, self.E, self.cap, self.eps = H, D, E, cap, 1e-5
        self.state = torch.full((5, H, D, -(-(E + 1) // 4) * 4), 7.0,
                                device=device)
        self.peak = torch.full((5, H), 3.0, device=device)
        self.norm_w = rand(H * E, seed=71, device=device) * 0.2 + 1 \
            if norm_w is None else norm_w
        self.bias = bias if bias is not None else torch.cat(
            (rand(H, seed=72) * 2, rand(H, seed=73) * 3 + 1)).to(device)

    def run(self, part, slot, at, step):
        n = part.size(0)
        flat = torch.zeros(n + 3, part.size(1), dtype=self.dtype,
                           device=self.device)
        flat[2:2 + n] = part
        y = torch.zeros(n + 3, self.H * self.E, dtype=self.dtype,
                        device=self.device)
        args = (y, flat, self.state, self.peak, self.bias, self.norm_w,
                self.cap, self.D ** -0.5, self.eps,
                seg([(2, n, slot, at)], self.device))
        self.ops.mlstm_step(*args) if step else self.ops.mlstm_scan(*args, n)
        assert float(y[:2].abs().max()) == float(y[2 + n:].abs().max()) == 0
        return y[2:2 + n]

    def oracle(self, proj):
        return memory_oracle(proj, self.bias, self.norm_w, self.H, self.D,
                             self.E, self.cap, self.eps)


@everywhere
@pytest.mark.parametrize("H,D,E,cap", [
    (1, 1, 1, 5.0), (3, 7, 9, 2.0), (2, 16, 16, 15.0), (4, 32, 20, 8.0),
    (2, 100, 30, 15.0), (1, 256, 8, 6.0), (2, 200, 136, 9.0),
    (3, 64, 130, 12.0), (2, 128, 128, 20.0), (1, 24, 301, 7.0),
    (1, 40, 260, 7.0)])
def test_matrix_memory(H, D, E, cap, device, dtype):
    """A prompt whole, one in portions, and one token by token."""
    T = 150
    mem = Memory(device, dtype, H, D, E, cap)
    projs = [rand(T, 2 * H * (D + E + 1), seed=s, dtype=dtype, device=device)
             * 1.5 for s in range(3)]
    got = [torch.zeros(T, H * E, dtype=dtype, device=device) for _ in projs]

    def run(s, slot, at, n, step):
        got[s][at:at + n] = mem.run(projs[s][at:at + n], slot, at, step)

    drive(T, run)
    for g, p in zip(got, projs):
        want = mem.oracle(p)
        if E == 1:      # a sign, times its weight and gate
            keep = ((f64(g) - want).abs() < 0.02).all(1)
            assert float(keep.double().mean()) > 0.95
            continue
        close(g, want, dtype, 2 * float(want.abs().max()))
    for slot in (1, 4):     # nobody's
        assert float(mem.state[slot].min()) == 7.0
        assert float(mem.peak[slot].min()) == 3.0


@everywhere
@pytest.mark.parametrize("lengths", [(1100, 40, 17), (16, 1500, 2)])
def test_matrix_memory_of_unequal_segments(lengths, device, dtype):
    """Segments of very different length in one launch, gates over more than
    one tile of tokens, continued by one more portion each."""
    H, D, E, cap = 2, 16, 24, 10.0
    mem = Memory(device, dtype, H, D, E, cap)
    projs = [rand(n + 5, 2 * H * (D + E + 1), seed=s, dtype=dtype,
                  device=device) for s, n in enumerate(lengths)]
    wants = [mem.oracle(p) for p in projs]
    at = [0] * 3
    for cut in (lengths, (5, 5, 5)):
        flat = torch.cat([p[a:a + n] for p, a, n in zip(projs, at, cut)])
        y = torch.empty(flat.size(0), H * E, dtype=dtype, device=device)
        segs, start = [], 0
        for s, n in enumerate(cut):
            segs.append((start, n, 3 - s, at[s]))
            start += n
        mem.ops.mlstm_scan(y, flat.contiguous(), mem.state, mem.peak,
                           mem.bias, mem.norm_w, cap, D ** -0.5, mem.eps,
                           seg(segs, device), max(cut))
        for s, (start, n, _, a) in enumerate(segs):
            close(y[start:start + n], wants[s][a:a + n], dtype,
                  2 * float(wants[s].abs().max()))
            at[s] += n


def gates(H, D, E, T, device, dtype, i, f):
    """Rows of zeros but the gates' logits [T] of all heads."""
    p = torch.zeros(T, 2 * H * (D + E + 1), dtype=dtype, device=device)
    p[:, -2 * H:-H] = i.view(T, 1).to(dtype)
    p[:, -H:] = f.view(T, 1).to(dtype)
    return p


@everywhere
def test_memory_holds_a_far_token(device, dtype):
    """One token writes, the others hardly do and forget nothing: its value
    is read hundreds of tokens later, from a prompt and in decoding."""
    H, D, E, T, cap = 1, 16, 16, 700, 12.0
    one, zero = torch.ones(E, device=device), torch.zeros(2, device=device)
    mem = Memory(device, dtype, H, D, E, cap, one, zero)
    for at in (0, 1, 15, 16, 17, 63, 300):
        i = torch.full((T,), -200.0, device=device)
        i[at] = 200.0
        p = gates(H, D, E, T, device, dtype, i,
                  torch.full((T,), 200.0, device=device))
        p[:, 0] = p[:, D] = 4.0
        p[:, 2 * D:2 * D + E] = rand(T, E, seed=3, dtype=dtype,
                                     device=device)
        p[:, 2 * D + E:2 * D + 2 * E] = 20.0        # open output gates
        want = oracle.unit(f64(p[at, 2 * D:2 * D + E]), 1e-5)
        y = mem.run(p, 2, 0, False)
        close(y[-1], want, dtype)
        close(y[at], want, dtype)
        close(mem.run(p[-1:], 2, T, True)[0], want, dtype)
        # and decoded from the start
        for t in range(0, at + 3 if at < 70 else 0):
            y = mem.run(p[t:t + 1], 0, t, True)
            if t >= at:
                close(y[0], want, dtype)


@everywhere
def test_running_maximum_starts_at_zero(device, dtype):
    """Input gates far below 0 leave the maximum to decay from 0, and the
    read-out is small against exp(-m): it shows in the unit norm's eps.  Heads
    that write strongly are normalised by what they read."""
    H, D, E, T, cap = 2, 4, 4, 40, 30.0
    one = torch.ones(H * E, device=device)
    bias = torch.tensor([-9.0, 3.0, 2.0, -1.0], device=device)
    mem = Memory(device, dtype, H, D, E, cap, one, bias)
    p = gates(H, D, E, T, device, dtype, torch.zeros(T, device=device),
              torch.zeros(T, device=device))
    body = rand(T, 2 * H * (D + E), seed=5, dtype=dtype, device=device)
    p[:, :2 * H * (D + E)] = body
    want = mem.oracle(p)
    # against a maximum that starts at minus infinity
    i = oracle.capped(f64(bias[:1]).expand(T), cap)
    f = oracle.log_sigmoid(oracle.capped(f64(bias[2:3]).expand(T), cap))
    m, free = torch.zeros(()).double(), i[0]
    for t in range(T):
        m = torch.maximum(f[t] + m, i[t])
        free = torch.maximum(f[t] + free, i[t])
    assert float(m) - float(free) > 2
    for y in (mem.run(p, 2, 0, False),
              torch.cat([mem.run(p[t:t + 1], 3, t, True)
                         for t in range(T)])):
        close(y, want, dtype, float(want.abs().max()))
        small = f64(y)[:, :E] - want[:, :E]
        assert float(small.abs().max()) < 0.03 * float(
            want[:, :E].abs().max())
    assert abs(float(mem.peak[2, 0]) - float(m)) < 1e-4


@everywhere
def test_input_gates_are_capped(device, dtype):
    """Logits beyond the cap all count as the cap: two values written with
    logits of 3 and 9 caps are read with nearly equal weights."""
    H, D, E, cap = 1, 4, 4, 2.0
    mem = Memory(device, dtype, H, D, E, cap, torch.ones(E, device=device),
                 torch.zeros(2, device=device))
    p = gates(H, D, E, 2, device, dtype, torch.tensor([6.0, 18.0]),
              torch.tensor([1000.0, 1000.0]))
    p[:, 0] = p[:, D] = 2.0
    p[0, 2 * D] = p[1, 2 * D + 1] = 1.0
    p[:, 2 * D + E:2 * D + 2 * E] = 20.0
    y = mem.run(p, 1, 0, False)
    close(y, mem.oracle(p), dtype)
    ratio = float(y[1, 1]) / float(y[1, 0])
    forget = math.log1p(math.exp(-cap))
    assert abs(ratio - math.exp(cap * (1 - math.tanh(3.0)) + forget)) < 0.02


# ---------------------------------------------------------------------------
@everywhere
@pytest.mark.parametrize("W", [1, 5, 21, 64, 130, 300, 512])
def test_mingru(W, device, dtype):
    """Channels that hold on and channels that follow the input; columns of a
    wider row."""
    ops, T = ops_for(device), 200
    x = rand(3, T, 3 * W, seed=1, dtype=dtype, device=device) * 2
    bias = torch.cat((rand(W, seed=2) * 4 - 2, rand(W, seed=3))).to(device)
    want = []
    for s in range(3):
        z, u, g = f64(x[s]).split(W, 1)
        bz, bu = f64(bias).split(W)
        want.append(oracle.blend(oracle.sigmoid(z + bz),
                                 oracle.candidate(u + bu)) * oracle.silu(g))
    state = torch.full((5, W), 9.0, device=device)
    got = torch.zeros(3, T, W, dtype=dtype, device=device)

    def run(s, slot, at, n, step):
        wide = torch.zeros(n + 3, 3 * W + 9, dtype=dtype, device=device)
        wide[2:2 + n, 8:8 + 3 * W] = x[s, at:at + n]
        out = torch.zeros(n + 3, W, dtype=dtype, device=device)
        args = (out, wide[:, 8:8 + 3 * W], bias, state,
                seg([(2, n, slot, at)], device))
        ops.mingru_step(*args) if step else ops.mingru_scan(*args, n)
        assert float(out[:2].abs().max()) == float(out[2 + n:].abs().max()) \
            == 0
        got[s, at:at + n] = out[2:2 + n]

    drive(T, run)
    for s in range(3):
        close(got[s], want[s], dtype)
    assert float(state[1].min()) == float(state[4].min()) == 9.0


@everywhere
def test_mingru_holds_a_far_token(device, dtype):
    """Gates open at one token only: what it wrote comes back hundreds of
    tokens later; candidates on both sides of 0."""
    ops, W, T = ops_for(device), 16, 700
    for at, u in ((0, 3.0), (127, -3.0), (128, 0.0), (300, -0.5)):
        x = torch.zeros(T, 3 * W, dtype=dtype, device=device)
        x[:, :W] = -40.0
        x[at, :W] = 40.0
        x[:, W:2 * W] = 9.0
        x[at, W:2 * W] = u
        x[:, 2 * W:] = 6.0
        state = torch.full((1, W), 3.0, device=device)
        out = torch.zeros(T, W, dtype=dtype, device=device)
        bias = torch.zeros(2 * W, device=device)
        ops.mingru_scan(out, x, bias, state, seg([(0, T, 0, 0)], device), T)
        want = u + 0.5 if u >= 0 else 1 / (1 + math.exp(-u))
        want *= 6.0 / (1 + math.exp(-6.0))
        got = f64(out)[-1]
        assert float((got - want).abs().max()) < 0.01 * want, (at, u)
        assert float(f64(out)[:at].abs().sum()) < 1e-3
        ops.mingru_step(out, x, bias, state,
                        seg([(T - 1, 1, 0, T)], device))
        assert float((f64(out)[-1] - want).abs().max()) < 0.01 * want


# ---------------------------------------------------------------------------
class Paged:
    """Sequences in scattered pages that were used before."""

    def __init__(self, device, dtype, H, G, D, E, temp=None, n_pages=60,
                 slots=3):
        def pad(n):
            return next(p for p in (32, 64, 128, 256) if n <= p)

        self.ops, self.device, self.dtype = ops_for(device), device, dtype
        self.H, self.G, self.D, self.E = H, G, D, E
        self.k = rand(n_pages, G, PAGE * pad(D), seed=91, dtype=dtype,
                      device=device)
        self.v = rand(n_pages, G, PAGE * pad(E), seed=92, dtype=dtype,
                      device=device)
        per = n_pages // slots
        perm = torch.randperm(per * slots,
                              generator=torch.Generator().manual_seed(3))
        self.table = perm.view(slots, per).to(torch.int32).to(device)
        self.qw = rand(H * D, seed=93, device=device) * 0.2 + 1
        self.kw = rand(G * D, seed=94, device=device) * 0.2 + 1
        self.temp, self.eps = temp, 1e-4
        self.q_scale = None if temp is None else torch.tensor(
            [oracle.temperature(p, temp) for p in range(per * PAGE)],
            device=device)
        self.slopes = torch.tensor(oracle.slopes(H), device=device) \
            * math.log2(math.e)

    def rows(self, slot, pos0, n):
        return (torch.full((n,), slot, dtype=torch.int32, device=self.device),
                torch.arange(pos0, pos0 + n, dtype=torch.int32,
                             device=self.device))

    def append(self, slot, pos0, proj, unit_values=True):
        q = torch.empty(proj.size(0), self.H, self.k.size(2) // PAGE,
                        dtype=self.dtype, device=self.device)
        self.ops.row_norm_append(
            q, self.k, self.v, proj, self.qw, self.kw,
            *self.rows(slot, pos0, proj.size(0)), self.table, self.E,
            self.eps, self.q_scale, unit_values)
        return q

    def attend(self, q, segs, window, scale, splits, sink=None, gate=None,
               slopes=True):
        out = torch.zeros(q.size(0), self.H * self.E, dtype=self.dtype,
                          device=self.device)
        part = ()
        if splits > 1:
            cells = len(segs) * self.H * splits
            part = (torch.full((cells * self.v.size(2) // PAGE,), math.nan,
                               device=self.device),
                    torch.full((cells * 2,), math.nan, device=self.device))
        bias = None if slopes else torch.zeros(self.H, 1, device=self.device)
        self.ops.paged_attn(out, q, self.k, self.v, bias, self.table,
                            seg(segs, self.device), max(s[1] for s in segs),
                            window, 0, scale, splits, *part,
                            slopes=self.slopes if slopes else None,
                            sink=sink, gate=gate)
        return out

    def oracle(self, proj, window, scale, sink, gate):
        p = f64(proj)
        T, H, G, D, E = p.shape[0], self.H, self.G, self.D, self.E
        q, k, v = p.split((H * D, G * D, G * E), 1)
        q = oracle.rms_norm(q, f64(self.qw), self.eps)
        if self.temp is not None:
            q = q * torch.tensor([oracle.temperature(i, self.temp)
                                  for i in range(T)]).double()[:, None]
        q = q.view(T, H, D)
        k = oracle.rms_norm(k, f64(self.kw), self.eps).view(T, G, D)
        v = oracle.unit(v.reshape(T, G, E), self.eps)
        o = torch.cat([oracle.attend(
            q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], scale, s,
            window, f64(sink)[h]) for h, s in enumerate(oracle.slopes(H))], 1)
        return o if gate is None else o * oracle.sigmoid(f64(gate))


@everywhere
@pytest.mark.parametrize("H,G,D,E", [(4, 2, 32, 32), (6, 2, 24, 40),
                                     (3, 1, 10, 9), (1, 1, 1, 1),
                                     (2, 2, 64, 130), (12, 3, 200, 256),
                                     (32, 8, 128, 128)])
@pytest.mark.parametrize("n", [1, 5, 64, 65, 150])
def test_row_norms_and_append(H, G, D, E, n, device, dtype):
    """Heads of very different size: the norms are over the whole row, and
    the values' over each head.  Rows lie in a wider projection."""
    P = Paged(device, dtype, H, G, D, E, dict(coef=0.7, every=9), n_pages=12)
    proj = rand(n, (H + G) * D + G * E, seed=8, dtype=dtype, device=device)
    loud = torch.logspace(-1, 1, H + 2 * G, device=device)
    proj = proj * torch.cat((loud[:H + G].repeat_interleave(D),
                             loud[H + G:].repeat_interleave(E))).to(dtype)
    wide = torch.zeros(n, proj.size(1) + 24, dtype=dtype, device=device)
    wide[:, 8:8 + proj.size(1)] = proj
    q = P.append(1, 30, wide[:, 8:8 + proj.size(1)])
    heat = torch.tensor([oracle.temperature(30 + i, P.temp)
                         for i in range(n)]).double()[:, None]
    a, b, v = f64(proj).split((H * D, G * D, G * E), 1)
    close(q[..., :D].reshape(n, -1),
          oracle.rms_norm(a, f64(P.qw), P.eps) * heat, dtype)
    assert float(q[..., D:].abs().sum()) == 0
    back = torch.zeros(n, G * (D + E), dtype=dtype, device=device)
    P.ops.kv_rows(back, P.k, P.v, *P.rows(1, 30, n), P.table, D, E, False)
    close(back[:, :G * D], oracle.rms_norm(b, f64(P.kw), P.eps), dtype)
    close(back[:, G * D:],
          oracle.unit(v.reshape(n, G, E), P.eps).flatten(1), dtype)
    # values as they are
    P.append(1, 30, proj, unit_values=False)
    P.ops.kv_rows(back, P.k, P.v, *P.rows(1, 30, n), P.table, D, E, False)
    assert torch.equal(back[:, G * D:], proj[:, (H + G) * D:])


@everywhere
@pytest.mark.parametrize("H,G,D,E,window", [
    (4, 2, 32, 32, 37), (6, 2, 24, 40, 64), (3, 1, 10, 9, 1),
    (1, 1, 2, 3, 2), (20, 1, 16, 24, 500), (2, 2, 64, 130, 90),
    (4, 4, 120, 100, 33), (3, 1, 200, 256, 128)])
def test_attention(H, G, D, E, window, device, dtype):
    """A prompt whole, in portions, its tokens one by one with the keys split
    in several ways."""
    T, scale, temp = 150, 2 * (D + 30) ** -0.5, dict(coef=0.3, every=20)
    P = Paged(device, dtype, H, G, D, E, temp)
    proj = rand(T, (H + G) * D + G * E, seed=8, dtype=dtype, device=device)
    gate = rand(T, H * E + 8, seed=9, dtype=dtype, device=device)[:, 8:] * 2
    sink = rand(H, seed=10, device=device) * 2
    want = P.oracle(proj, window, scale, sink, gate)
    peak = float(want.abs().max())
    q = P.append(1, 0, proj)
    close(P.attend(q, [(0, T, 1, 0)], window, scale, 0, sink, gate), want,
          dtype, peak)
    at = 0
    for n in (2, 62, 1, 3, 61, 21):
        q2 = P.append(0, at, proj[at:at + n])
        q2 = torch.cat([torch.zeros_like(q2[:1]), q2])
        g2 = torch.cat([gate[:1], gate[at:at + n]])
        o = P.attend(q2, [(1, n, 0, at)], window, scale, 0, sink, g2)
        close(o[1:], want[at:at + n], dtype, peak)
        at += n
    # later keys are in the pages already and must not be seen
    ts = sorted({*range(0, T, 7), 62, 63, 64, 65, 127, 128, T - 1,
                 *(t for t in (window - 1, window, window + 1) if t < T)})
    for splits in (1, 2, 5):
        o = P.attend(q, [(t, 1, 1, t) for t in ts], window, scale, splits,
                     sink, gate)
        close(o[ts], want[ts], dtype, peak)


@everywhere
@pytest.mark.parametrize("window", [1, 2, 40, 64, 65, 130, 300])
def test_one_key_stands_out(window, device, dtype):
    """Every key repels the query but one, so strongly that no slope helps;
    its value comes through exactly where the window lets it, else the sink
    takes all the weight."""
    H, G, D, E, T = 2, 1, 32, 32, 320
    P = Paged(device, dtype, H, G, D, E)
    P.qw.fill_(20.0)
    P.kw.fill_(20.0)
    P.slopes = P.slopes / 50
    sink = torch.zeros(H, device=device)
    queries = [255, 256, 259, 128, 191, 192, 319]
    spots = {0, 1, 63, 64, 65, 127, 128}
    for i in queries:
        spots |= {i, i - 1, i - window + 1, i - window, i - window - 1}
    for j in sorted(s for s in spots if 0 <= s < T):
        proj = torch.zeros(T, (H + G) * D + G * E, dtype=dtype,
                           device=device)
        proj[:, 0] = proj[:, D] = 1.0
        proj[:, H * D] = -1.0
        proj[j, H * D] = 1.0
        proj[:, (H + G) * D:] = 1.0     # of unit size, whatever the key
        q = P.append(2, 0, proj)
        segs = [(i, 1, 2, i) for i in queries]
        for o in (P.attend(q, [(0, T, 2, 0)], window, 0.1, 0, sink),
                  P.attend(q, segs, window, 0.1, 1, sink),
                  P.attend(q, segs, window, 0.1, 3, sink)):
            for i in queries:
                want = 1.0 if 0 <= i - j < window else 0.0
                assert abs(float(o[i].float().min()) - want) < 0.02, (i, j)


@everywhere
def test_sink_takes_its_share(device, dtype):
    """Equal scores: n keys have n / (n + e^sink) of the weight, whatever the
    score's scale; without a sink, all of it, also beside a bias table."""
    H, G, D, E, T = 3, 1, 16, 8, 150
    P = Paged(device, dtype, H, G, D, E)
    P.slopes, P.eps = P.slopes * 0, 1e-9
    proj = torch.zeros(T, (H + G) * D + G * E, dtype=dtype, device=device)
    proj[:, (H + G) * D:] = 1.0
    sink = torch.tensor([-3.0, 0.0, 4.0], device=device)
    q = P.append(0, 0, proj)
    for window in (1, 20, 400):
        seen = torch.arange(1, T + 1).clamp(max=window).double().view(T, 1)
        want = seen / (seen + f64(sink).exp())
        want = want.repeat_interleave(E, 1)
        segs = [(t, 1, 0, t) for t in range(T)]
        for scale, splits, slopes in ((0.125, 0, True), (1.0, 0, False),
                                      (1.0, 1, True), (0.5, 4, True),
                                      (0.5, 3, False)):
            s = [(0, T, 0, 0)] if splits == 0 else segs
            o = P.attend(q, s, window, scale, splits, sink, slopes=slopes)
            close(o, want, dtype)
            o = P.attend(q, s, window, scale, splits, slopes=slopes)
            close(o, torch.ones_like(want), dtype)


@everywhere
def test_slopes_are_taken_off_after_the_scale(device, dtype):
    """Equal scores: weights fall by the slope per token, by the same factor
    for any score scale, next to a sink that does not fall."""
    H, G, D, E, T = 8, 2, 16, 8, 200
    P = Paged(device, dtype, H, G, D, E)
    proj = torch.ones(T, (H + G) * D + G * E, dtype=dtype, device=device)
    proj[:, (H + G) * D:] = rand(T, G * E, seed=6, dtype=dtype,
                                 device=device)
    sink = rand(H, seed=7, device=device)
    for scale in (0.01, 0.2):
        q = P.append(0, 0, proj)
        want = P.oracle(proj, 1000, scale, sink, None)
        close(P.attend(q, [(0, T, 0, 0)], 1000, scale, 0, sink), want, dtype)


@everywhere
def test_queries_warm_up(device, dtype):
    """The factor steps up where a run of positions begins: the scores of
    the tokens on both sides of the step differ by it."""
    H, G, D, E, T = 1, 1, 32, 32, 100
    temp = dict(coef=3.0, every=10)
    P = Paged(device, dtype, H, G, D, E, temp)
    P.slopes = P.slopes * 0
    P.qw.fill_(1.0)
    P.kw.fill_(1.0)
    proj = torch.ones(T, 3 * 32, dtype=dtype, device=device)
    sink = torch.full((1,), 5.0, device=device)
    q = P.append(0, 0, proj)
    for i in (0, 8, 9, 10, 18, 19, 20, 99):
        warm = 1 + 3.0 * math.log((i + 1) // 10 + 1)
        assert abs(float(q[i, 0, 0]) - warm) < 0.01 * warm
    want = P.oracle(proj, 1, 1 / 32, sink, None)
    assert float(want[9, 0]) > 2 * float(want[8, 0])
    close(P.attend(q, [(0, T, 0, 0)], 1, 1 / 32, 0, sink), want, dtype)


def test_the_engines_tables_by_position():
    from types import SimpleNamespace

    from mdi_llm_amd.ops.hybrid_engine import HybridEngine

    e = SimpleNamespace(_tables={}, max_ctx=500, device="cpu")
    for every, coef in ((1, 0.3), (7, 0.0), (64, 2.0), (1000, 1.0)):
        got = HybridEngine.query_scale_table(e, every, coef)
        want = torch.tensor([oracle.temperature(
            p, dict(every=every, coef=coef)) for p in range(500)])
        assert torch.allclose(got, want, rtol=1e-6)


@pytest.mark.gpu
def test_operations_refuse_what_they_cannot_hold():
    """Errors from the host's checks, ahead of any launch."""
    ops, d = ops_for("cuda"), "cuda"
    x = torch.zeros(4, 64, device=d)
    v = torch.zeros(64, device=d)
    s = seg([(0, 4, 0, 0)], d)
    state = torch.zeros(2, 2, 300, 16, device=d)
    P = Paged(d, torch.float32, 2, 1, 32, 32)
    q = torch.zeros(4, 2, 32, device=d)
    for call in (
            lambda: ops.residual_norm(x, y=x, gain=v, post_w=v),
            lambda: ops.residual_norm(x, y=x, y2=x, post_w2=v),
            lambda: ops.residual_norm(x, y=x, post_w=v, y2=x),
            lambda: ops.mingru_scan(x, x, v, torch.zeros(2, 64, device=d), s,
                                    4),
            lambda: ops.mlstm_scan(x, x, state, state[0, :, 0], v[:4], v[:30],
                                   1.0, 1.0, 1e-5, s, 4),
            lambda: P.append(0, 0, x),
            lambda: ops.paged_attn(x, q, P.k, P.v, None, P.table, s, 4, 9, 0,
                                   1.0, 0),
            lambda: P.attend(q, [(0, 4, 0, 0)], 9, 1.0, 0, sink=v),
            lambda: P.attend(q, [(0, 4, 0, 0)], 9, 1.0, 0, gate=x[:3])):
        with pytest.raises(RuntimeError):
            call()
