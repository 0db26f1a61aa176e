"""Plain, slow Sosutar: one function per mechanism, whole sequences in
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


def log_sigmoid(z):
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def unit(x, eps):
    return x / torch.sqrt(x.square().mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit(x, eps) * weight


def embed(w, tokens, scale):
    return w["embed"][torch.as_tensor(tokens)] * scale \
        + w["pos"][:len(tokens)]


# -- matrix memory with exponential gates ------------------------------------
def capped(z, cap):
    return cap * torch.tanh(z / cap)


def matrix_memory(q, k, v, i, log_f):
    """One head: q, k [T, D], v [T, E], gates [T] -> [T, E]."""
    S = q.new_zeros(q.shape[1], v.shape[1])
    n = q.new_zeros(q.shape[1])
    m, out = q.new_zeros(()), []
    for t in range(q.shape[0]):
        new = torch.maximum(log_f[t] + m, i[t])
        keep, write = torch.exp(log_f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = keep * S + write * k[t][:, None] * v[t][None, :]
        n = keep * n + write * k[t]
        size = torch.maximum((n @ q[t]).abs(), torch.exp(-m))
        out.append((S.T @ q[t]) / (size + 1e-6))
    return torch.stack(out)


def mlstm(h, w, pre, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).view(T, H, D)
    v = (h @ w[pre + "v"].T).view(T, H, E)
    i = capped(h @ w[pre + "i"].T + w[pre + "i.b"], m["gate_cap"])
    f = log_sigmoid(capped(h @ w[pre + "f"].T + w[pre + "f.b"],
                           m["gate_cap"]))
    heads = [unit(matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]),
                  eps) for a in range(H)]
    y = torch.cat(heads, 1) * w[pre + "norm"] * sigmoid(h @ w[pre + "g"].T)
    return y @ w[pre + "o"].T


# -- gated attention ---------------------------------------------------------
def temperature(pos, spec):
    return 1.0 + spec["coef"] * math.log((pos + 1) // spec["every"] + 1)


def slopes(heads):
    return [2.0 ** (-8.0 * (a + 1) / heads) for a in range(heads)]


def attend(q, k, v, scale, slope, window, sink):
    """One head: q, k [T, D], v [T, E]."""
    out = []
    for i in range(q.shape[0]):
        first = max(0, i - window + 1)
        at = torch.arange(first, i + 1)
        s = (k[at] @ q[i]) * scale - slope * (i - at)
        top = torch.maximum(s.max(), sink)
        p = torch.exp(s - top)
        out.append((p / (p.sum() + torch.exp(sink - top))) @ v[at])
    return torch.stack(out)


def gated_attention(h, w, pre, m, eps):
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rms_norm(h @ w[pre + "q"].T, w[pre + "q.norm"], eps)
    k = rms_norm(h @ w[pre + "k"].T, w[pre + "k.norm"], eps).view(T, G, D)
    v = unit((h @ w[pre + "v"].T).view(T, G, m["vdim"]), eps)
    warm = torch.tensor([temperature(p, m["q_temp"]) for p in range(T)],
                        dtype=h.dtype)
    q = (q * warm[:, None]).view(T, H, D)
    heads = [attend(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)],
                    m["scale"], slope, m["mask"]["size"],
                    w[pre + "sink"][a]) for a, slope in enumerate(slopes(H))]
    y = torch.cat(heads, 1) * sigmoid(h @ w[pre + "g"].T)
    return y @ w[pre + "o"].T


# -- blend of a state and a candidate, per channel ---------------------------
def candidate(u):
    return torch.where(u >= 0, u + 0.5, sigmoid(u))


def blend(z, c):
    S, out = torch.zeros_like(c[0]), []
    for t in range(c.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        out.append(S)
    return torch.stack(out)


def mingru(h, w, pre):
    z = sigmoid(h @ w[pre + "z"].T + w[pre + "z.b"])
    c = candidate(h @ w[pre + "x"].T + w[pre + "x.b"])
    return (blend(z, c) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def paired(h, w, pre, m, eps):
    a = gated_attention(h, w, pre + "left.", m["left"], eps)
    b = mingru(h, w, pre + "right.")
    return 0.5 * (rms_norm(a, w[pre + "left.out"], eps)
                  + rms_norm(b, w[pre + "right.out"], eps))


# ---------------------------------------------------------------------------
def feed_forward(h, w, pre):
    return torch.clamp(h @ w[pre + "up"].T, min=0.0).square() \
        @ w[pre + "down"].T


def owner(layers, i):
    """The layer whose tensors layer ``i`` uses."""
    while "weights_of" in layers[i]:
        i = layers[i]["weights_of"]
    return i


def forward(cfg, w, tokens, layers_out=None):
    """tokens (list of ints) -> logits [T, vocab], float64."""
    w = {k: t.double() for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = embed(w, tokens, cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{owner(cfg['layers'], i)}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        y = mlstm(h, w, p + "mix.", m, eps) if layer["type"] == "mlstm" \
            else paired(h, w, p + "mix.", m, eps)
        x = x + w[p + "ls1"] * y
        if layer["mlp"] is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            x = x + w[p + "ls2"] * feed_forward(h, w, p + "mlp.")
        if layers_out is not None:
            layers_out.append(x)
    return (rms_norm(x, w["final.norm"], eps) @ w["head"].T) \
        * cfg["logit_scale"]
