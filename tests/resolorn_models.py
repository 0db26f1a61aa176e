"""Small random Resolorn models in their on-disk form, for the tests."""

import torch


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared=None):
    out = dict(kind="moe", router=dict(experts=experts, top=top),
               expert=dict(ff=ff))
    if shared is not None:
        out["shared"] = dict(ff=shared)
    return out


def att(heads, dim, vdim, q_rank, kv_rank, size, mlp, kv_from=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
             scale=1.6 * dim ** -0.5, mask=dict(size=size))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=m, mlp=mlp)


def config(layers, width=64, vocab=120, eps=1e-5, mult=0.6, positions=512):
    return dict(architecture="Resolorn", vocab=vocab, width=width,
                max_positions=positions, norm=dict(eps=eps),
                residual_mult=mult, layers=layers)


MODELS = {
    # unequal query and value sizes, both feed-forwards, an own latent after
    # shared ones, a latent read across another latent's layer
    "mixed": config([att(6, 48, 20, 40, 56, 37, moe(5, 2, 24, 40)),
                     att(3, 16, 72, 33, 56, 70, dense(96), 0),
                     att(5, 24, 24, 24, 88, 9, None),
                     att(4, 32, 40, 48, 88, 130, moe(3, 1, 32), 2),
                     att(2, 16, 16, 16, 56, 21, dense(50), 0)],
                    width=72, vocab=133),
    # sizes that no vector load divides, every expert chosen
    "odd": config([att(3, 7, 9, 13, 11, 12, dense(33)),
                   att(5, 5, 3, 9, 11, 50, moe(4, 4, 5, 3), 0)],
                  width=27, vocab=61, mult=1.0),
    # large latents and heads, more than 32 rows a token, all in sight
    "wide": config([att(4, 160, 136, 72, 300, 4096, dense(64)),
                    att(40, 16, 8, 40, 70, 100, moe(9, 3, 16, 24))],
                   width=48),
    # heads beyond the expanded form; a window of one token; no feed-forward
    "narrow": config([att(1, 264, 270, 24, 500, 1, None),
                      att(1, 1, 1, 1, 1, 33, moe(1, 1, 8, 8))],
                     width=40, mult=-0.8),
    # one latent for the whole stack
    "shared": config([att(2, 32, 32, 32, 64, 45, dense(80))]
                     + [att(2 + i, 32, 16, 24, 64, 20 + 30 * i,
                            moe(4, 2, 20, 12), 0) for i in range(3)],
                     width=64),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).bfloat16()

    def mlp(pre, E, F):
        w[pre + "gate"] = r(F, E, std=1.5 * E ** -0.5)
        w[pre + "up"] = r(F, E, std=E ** -0.5)
        w[pre + "down"] = r(E, F, std=1.5 * F ** -0.5)

    E = cfg["width"]
    w = {"embed": r(cfg["vocab"], E), "pos": r(cfg["max_positions"], E,
                                               std=0.5),
         "final.norm": r(E, std=0.2, mean=1.0),
         "head": r(cfg["vocab"], E, std=E ** -0.5)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        w[p + "norm1"] = r(E, std=0.2, mean=1.0)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        Q, R = m["q_rank"], m["kv_rank"]
        q = p + "mix."
        w[q + "dq"] = r(Q, E, std=E ** -0.5)
        w[q + "dq.norm"] = r(Q, std=0.2, mean=1.0)
        w[q + "uq"] = r(H * D, Q, std=Q ** -0.5)
        if "kv_from" not in m:
            w[q + "dkv"] = r(R, E, std=E ** -0.5)
            w[q + "dkv.norm"] = r(R, std=0.2, mean=1.0)
        w[q + "uk"] = r(H * D, R, std=R ** -0.5)
        w[q + "uv"] = r(H * V, R, std=R ** -0.5)
        w[q + "g"] = r(H, E, std=2.0 * E ** -0.5)
        w[q + "o"] = r(E, H * V, std=2.0 * (H * V) ** -0.5)
        if f is None:
            continue
        if f["kind"] == "dense":
            mlp(p + "mlp.", E, f["ff"])
            continue
        w[p + "mlp.router"] = r(f["router"]["experts"], E, std=2 * E ** -0.5)
        for e in range(f["router"]["experts"]):
            mlp(f"{p}mlp.e{e}.", E, f["expert"]["ff"])
        if "shared" in f:
            mlp(p + "mlp.shared.", E, f["shared"]["ff"])
    return w
