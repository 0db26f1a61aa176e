"""Plain, slow Nerozen: one function per mechanism, whole sequences in
float64, no cache, no batching.  Shares no code with ``mdi_llm_amd``.

``cfg`` is the parsed config.json, ``w`` a dict of tensors under their
on-disk names.
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def silu(x):
    return x * torch.sigmoid(x)


def xielu(z, act):
    """Two quadratic/exponential branches meeting at 0 with slope 1/2."""
    p, q = torch.nn.functional.softplus(act[0]), torch.nn.functional.softplus(act[1])
    pos = p * z * z + 0.5 * z
    zn = torch.clamp(z, max=0.0)
    neg = (0.5 + q) * (torch.exp(zn) - 1.0 - zn) + 0.5 * zn
    return torch.where(z > 0, pos, neg)


def forget_gate(raw, bias, lower):
    return lower + (1.0 - lower) * torch.sigmoid(raw + bias)


def gated_scan(q, f, v):
    """q, f [T, H, D], v [T, H, E] -> o [T, H, E]:
    S <- f * S + (1 - f) v^T, o = S^T q, one token after another."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(T):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def hgrn2(h, w, pre, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[pre + "q"].T).view(T, H, D)
    v = (h @ w[pre + "v"].T).view(T, H, E)
    f = forget_gate(h @ w[pre + "f"].T, w[pre + "f.b"],
                    w[pre + "lower"]).view(T, H, D)
    o = rms(gated_scan(q, f, v), eps) * w[pre + "norm"]
    return o.reshape(T, H * E) @ w[pre + "o"].T


def distance_bucket(n, rows, far):
    """Exact for the first half of the table, logarithmic up to ``far``."""
    half = rows // 2
    if n < half:
        return n
    # largest k with (n/half) >= (far/half)^(k/(rows-half)), in integers
    k, m = 0, rows - half
    while k < m and n ** m * half ** (k + 1) >= far ** (k + 1) * half ** m:
        k += 1
    return min(rows - 1, half + k)


def visible(i, j, size, keep):
    return j <= i and (i - j < size or j < keep)


def attention_weights(q, k, scale, rel, far, size, keep):
    """q [T, H, D], k [T, G, D] -> softmax weights [H, T, T]."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    s = torch.einsum("thd,jhd->htj", q, k.repeat_interleave(rep, 1)) * scale
    ok = torch.zeros(T, T, dtype=torch.bool)
    buckets = [distance_bucket(n, rel.shape[0], far) for n in range(T)]
    b = torch.zeros(H, T, T, dtype=q.dtype)
    for i in range(T):
        for j in range(i + 1):
            b[:, i, j] = rel[buckets[i - j]]
            ok[i, j] = visible(i, j, size, keep)
    return torch.softmax((s + b).masked_fill(~ok, -math.inf), -1)


def attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[pre + "q"].T).view(T, H, D), eps) * w[pre + "q.norm"]
    k = rms((h @ w[pre + "k"].T).view(T, G, D), eps) * w[pre + "k.norm"]
    v = (h @ w[pre + "v"].T).view(T, G, E)
    p = attention_weights(q, k, m["scale"], w[pre + "rel"], m["bias_max"],
                          m["mask"]["size"], m["mask"]["keep_first"])
    o = torch.einsum("htj,jhe->the", p, v.repeat_interleave(H // G, 1))
    return o.reshape(T, H * E) @ w[pre + "o"].T


MIXERS = {"hgrn2": hgrn2, "attention": attention}


def feed_forward(h, w, pre):
    return xielu(h @ w[pre + "up"].T, w[pre + "act"]) @ w[pre + "down"].T


def forward(cfg, w, tokens, layers_out=None):
    """tokens (list of ints) -> logits [T, vocab], float64."""
    w = {k: t.double() for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = zero_centred_norm(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        x = x + zero_centred_norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            h = zero_centred_norm(x, w[p + "norm2"], eps)
            y = feed_forward(h, w, p + "mlp.")
            x = x + zero_centred_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return zero_centred_norm(x, w["final.norm"], eps) @ w["head"].T
