"""Plain, slow Dinuzen: one function per mechanism, whole sequences in
float64, no cache, no batching.  Shares no code with ``mdi_llm_amd``.

``cfg`` is the parsed config.json, ``w`` a dict of tensors under their
on-disk names.
"""

import math

import torch


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    inner = math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)
    return 0.5 * z * (1.0 + torch.tanh(inner))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def unit(x, eps):
    return x / torch.sqrt(x.square().mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    parts = x.reshape(*x.shape[:-1], groups, -1)
    return unit(parts, eps).reshape(x.shape) * weight


def token_shift(h, mu):
    before = torch.zeros_like(h)
    before[1:] = h[:-1]
    return h + (before - h) * mu


def causal_conv(x, taps, bias):
    """x [T, C], taps [C, K]: the last tap meets the current token."""
    T, K = x.shape[0], taps.shape[1]
    out = []
    for t in range(T):
        y = bias.clone()
        for k in range(K):
            s = t - (K - 1) + k
            if s >= 0:
                y = y + taps[:, k] * x[s]
        out.append(y)
    return torch.stack(out)


# -- recurrent block with a gated linear unit -------------------------------
def rglru_gates(u, w, pre, blocks):
    """u [T, width] -> recurrence and input gates, [T, width] each."""
    T = u.shape[0]
    parts = u.view(T, blocks, -1)
    out = []
    for name in ("ra", "ri"):
        z = torch.stack([parts[:, b] @ w[pre + name][b].T
                         + w[pre + name + ".b"][b] for b in range(blocks)], 1)
        out.append(sigmoid(z).reshape(T, -1))
    return out


def decayed_sum(u, r, i, lam):
    """The recurrence itself, over time."""
    S, out = torch.zeros_like(u[0]), []
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = torch.exp(log_a) * S \
            + torch.sqrt(-torch.expm1(2.0 * log_a)) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru(h, w, pre, m):
    y = gelu_tanh(h @ w[pre + "y"].T + w[pre + "y.b"])
    u = causal_conv(h @ w[pre + "x"].T + w[pre + "x.b"], w[pre + "conv"],
                    w[pre + "conv.b"])
    r, i = rglru_gates(u, w, pre, m["blocks"])
    S = decayed_sum(u, r, i, w[pre + "lam"])
    return (S * y) @ w[pre + "o"].T


# -- state-space duality ----------------------------------------------------
def ssd(x, B, C, dt, A, D):
    """x [T, H, E], B, C [T, H, N] (already by head), dt [T, H]."""
    T, H, E = x.shape
    S, out = x.new_zeros(H, B.shape[-1], E), []
    for t in range(T):
        S = torch.exp(-A * dt[t])[:, None, None] * S \
            + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out.append((S * C[t][:, :, None]).sum(1) + D[:, None] * x[t])
    return torch.stack(out)


def mamba2(h, w, pre, m, eps):
    T, H, E = h.shape[0], m["heads"], m["vdim"]
    N, G = m["state"], m["groups"]
    inner = H * E
    z, xbc, dt = (h @ w[pre + "in"].T).split(
        (inner, inner + 2 * G * N, H), 1)
    xbc = silu(causal_conv(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    x, B, C = xbc.split((inner, G * N, G * N), 1)
    head_group = torch.arange(H) // (H // G)
    y = ssd(x.view(T, H, E), B.view(T, G, N)[:, head_group],
            C.view(T, G, N)[:, head_group],
            softplus(dt + w[pre + "dt_bias"]), torch.exp(w[pre + "A_log"]),
            w[pre + "D"])
    y = y.reshape(T, inner) * silu(z)
    y = group_norm(y, w[pre + "norm"], m["norm_groups"], eps)
    return y @ w[pre + "o"].T


# -- differential attention -------------------------------------------------
def yarn_frequencies(rot):
    """(one angle per position for each pair, the factor on cos and sin)"""
    n, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if s is None:
        return f, 1.0

    def where(turns):
        return n * math.log(s["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(where(s["fast"])), 0)
    hi = min(math.ceil(where(s["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, rot):
    """x [T, ..., dim]: pairs (2i, 2i + 1) of the first ``dims``."""
    freqs, mult = yarn_frequencies(rot)
    at = torch.arange(x.shape[0], dtype=torch.float64)
    out = x.clone()
    for i, f in enumerate(freqs):
        a = (at * f).view(-1, *[1] * (x.dim() - 2))
        c, s = torch.cos(a) * mult, torch.sin(a) * mult
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def attend(q, k, v, scale, softcap):
    """One map: q, k [T, D], v [T, E]."""
    out = []
    for i in range(q.shape[0]):
        s = (k[:i + 1] @ q[i]) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        p = torch.exp(s - s.max())
        out.append((p / p.sum()) @ v[:i + 1])
    return torch.stack(out)


def keys_values(h, w, pre, m, eps):
    T, G = h.shape[0], m["kv_heads"]
    k = (h @ w[pre + "k"].T).view(T, G, 2, m["dim"])
    k = rotate(unit(k, eps) * w[pre + "k.norm"], m["rot"])
    return k, (h @ w[pre + "v"].T).view(T, G, m["vdim"])


def map_weight(w, pre, diff):
    return float(torch.exp((w[pre + "lq1"] * w[pre + "lk1"]).sum())
                 - torch.exp((w[pre + "lq2"] * w[pre + "lk2"]).sum()) + diff)


def difference(a1, a2, lam, diff, eps):
    return unit(a1 - lam * a2, eps) * (1.0 - diff)


def diff_attention(h, kv, w, pre, m, eps):
    """``kv``: this layer's keys and values, or an earlier layer's."""
    T, H, rep = h.shape[0], m["heads"], m["heads"] // m["kv_heads"]
    k, v = kv
    q = (h @ w[pre + "q"].T).view(T, H, 2, m["dim"])
    q = rotate(unit(q, eps) * w[pre + "q.norm"], m["rot"])
    lam, cap = map_weight(w, pre, m["diff"]), m.get("softcap")
    out = []
    for a in range(H):
        g = a // rep
        a1, a2 = (attend(q[:, a, j], k[:, g, j], v[:, g], m["scale"], cap)
                  for j in (0, 1))
        out.append(difference(a1, a2, lam, m["diff"], eps))
    return torch.cat(out, 1) @ w[pre + "o"].T


# -- feed-forwards ----------------------------------------------------------
def gated(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) \
        @ w[pre + "down"].T


def route(logits, correction, top, scale):
    """One token's logits -> [(output, weight)]."""
    e = torch.exp(logits - logits.max())
    s = e / e.sum()
    rank = s + correction
    best = sorted(range(len(s)), key=lambda j: -float(rank[j]))[:top]
    total = sum(float(s[j]) for j in best) + 1e-20
    return [(j, float(s[j]) / total * scale) for j in best]


def mixture(h, w, pre, spec):
    r = spec["router"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        z = w[pre + "router"] @ h[t]
        for j, p in route(z, w[pre + "correction"], r["top"], r["scale"]):
            out[t] += p * (gated(h[t], w, f"{pre}e{j}.")
                           if j < r["experts"] else h[t])
    if spec.get("shared"):
        out = out + sigmoid(h @ w[pre + "shared.sg"].T) \
            * gated(h, w, pre + "shared.")
    return out


def feed_forward(h, w, pre, spec):
    if spec["kind"] == "dense":
        return gelu_erf(h @ w[pre + "up"].T) @ w[pre + "down"].T
    return mixture(h, w, pre, spec)


def depth_average(states, coefficients):
    out = torch.zeros_like(states[0])
    for c, x in zip(coefficients, states):
        out = out + c * x
    return out


def forward(cfg, w, tokens, layers_out=None):
    """tokens (list of ints) -> logits [T, vocab], float64."""
    w = {k: t.double() for k, t in w.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = w["embed"][torch.as_tensor(tokens)]
    states, kept = [x], {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        mix = p + "mix."
        h = token_shift(x, w[p + "shift"])
        if layer["type"] == "rglru":
            y = rglru(h, w, mix, m)
        elif layer["type"] == "mamba2":
            y = mamba2(h, w, mix, m, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                src = i
                kept[i] = keys_values(h, w, mix, m, eps)
            y = diff_attention(h, kept[src], w, mix, m, eps)
        x = x + w[p + "ls1"] * group_norm(y, w[p + "norm1"], groups, eps)
        if layer["mlp"] is not None:
            y = feed_forward(x, w, p + "mlp.", layer["mlp"])
            x = x + w[p + "ls2"] * group_norm(y, w[p + "norm2"], groups, eps)
        states.append(x)
        x = depth_average(states, w[p + "dwa"])
        if layers_out is not None:
            layers_out.append(x)
    return group_norm(x, w["final.norm"], groups, eps) @ w["head"].T
