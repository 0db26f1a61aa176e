"""Plain, slow Resolorn: one function per mechanism, whole sequences in
float64, no cache, no batching.  Shares no code with ``mdi_llm_amd``.

``cfg`` is the parsed config.json, ``w`` a dict of tensors under their
on-disk names.
"""

import math

import torch


def rms_norm(x, weight, eps):
    return weight * x / torch.sqrt(x.square().mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    inner = math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)
    return 0.5 * z * (1.0 + torch.tanh(inner))


def visible(i, j, window):
    return j <= i and i - j < window


def attend(q, k, v, scale, window):
    """q, k [T, H, D], v [T, H, E] -> [T, H, E], one query at a time."""
    out = []
    for i in range(q.shape[0]):
        js = [j for j in range(k.shape[0]) if visible(i, j, window)]
        s = (k[js] * q[i]).sum(-1) * scale                 # [J, H]
        p = torch.exp(s - s.max(0).values)
        p = p / p.sum(0)
        out.append((p[:, :, None] * v[js]).sum(0))
    return torch.stack(out)


def latent(h, w, pre, eps):
    """The row that a layer keeps of every token."""
    return rms_norm(h @ w[pre + "dkv"].T, w[pre + "dkv.norm"], eps)


def latent_attention(h, c, w, pre, m, eps):
    """``c`` [T, kv_rank]: this layer's latent, or an earlier layer's."""
    T, H = h.shape[0], m["heads"]
    cq = rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps)
    q = (cq @ w[pre + "uq"].T).view(T, H, m["dim"])
    k = (c @ w[pre + "uk"].T).view(T, H, m["dim"])
    v = (c @ w[pre + "uv"].T).view(T, H, m["vdim"])
    o = attend(q, k, v, m["scale"], m["mask"]["size"])
    o = o * torch.sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * m["vdim"]) @ w[pre + "o"].T


def gated(h, w, pre, act):
    return (act(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) \
        @ w[pre + "down"].T


def route(logits, top):
    """One token's logits [experts] -> [(expert, weight)]."""
    best = sorted(range(len(logits)), key=lambda e: -float(logits[e]))[:top]
    e = torch.exp(logits[best] - logits[best].max())
    return list(zip(best, e / e.sum()))


def mixture(h, w, pre, spec):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in route(w[pre + "router"] @ h[t], spec["router"]["top"]):
            out[t] += p * gated(h[t], w, f"{pre}e{e}.", silu)
    if spec.get("shared"):
        out = out + gated(h, w, pre + "shared.", silu)
    return out


def feed_forward(h, w, pre, spec):
    if spec["kind"] == "dense":
        return gated(h, w, pre, gelu_tanh)
    return mixture(h, w, pre, spec)


def forward(cfg, w, tokens, layers_out=None):
    """tokens (list of ints) -> logits [T, vocab], float64."""
    w = {k: t.double() for k, t in w.items()}
    eps, scale = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens)] + w["pos"][:len(tokens)]
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        src = m.get("kv_from")
        if src is None:
            src = i
            latents[i] = latent(h, w, p + "mix.", eps)
        y = latent_attention(h, latents[src], w, p + "mix.", m, eps)
        if layer["mlp"] is not None:
            y = y + feed_forward(h, w, p + "mlp.", layer["mlp"])
        x = x + scale * y
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
