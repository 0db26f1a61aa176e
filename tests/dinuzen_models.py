"""Small random Dinuzen models in their on-disk form, for the tests."""

import torch


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared, identity=0, scale=1.0):
    return dict(kind="moe", router=dict(experts=experts, top=top,
                                        identity=identity, scale=scale),
                expert=dict(ff=ff), shared=dict(ff=shared))


def rglru(width, blocks, conv, mlp):
    return dict(type="rglru", mixer=dict(width=width, blocks=blocks,
                                         conv=conv), mlp=mlp)


def mamba2(heads, vdim, state, groups, norm_groups, conv, mlp):
    return dict(type="mamba2",
                mixer=dict(heads=heads, vdim=vdim, state=state, groups=groups,
                           norm_groups=norm_groups, conv=conv), mlp=mlp)


def rotation(dims, base=1000.0, factor=3.0, original=90, fast=4.0, slow=0.5):
    return dict(dims=dims, base=base,
                scaling=dict(factor=factor, original=original, fast=fast,
                             slow=slow))


def attention(heads, kv_heads, dim, vdim, rot, mlp, diff=0.4, softcap=9.0,
              kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=rot,
             diff=diff, softcap=softcap, scale=1.5 * dim ** -0.5)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m, mlp=mlp)


def config(layers, width=64, vocab=120, eps=1e-5, groups=2):
    return dict(architecture="Dinuzen", vocab=vocab, width=width,
                norm=dict(eps=eps, groups=groups), layers=layers)


SHARED = dict(heads=6, kv_heads=2, dim=24, vdim=40, rot=rotation(16))

MODELS = {
    # every mixer with every feed-forward; keys and values shared across
    # other mixers; two layers that read the same ones
    "mixed": config([attention(**SHARED, mlp=moe(5, 2, 24, 40, 2, 1.7)),
                     rglru(80, 5, 4, dense(96)),
                     mamba2(6, 20, 28, 3, 4, 3, None),
                     attention(**SHARED, mlp=dense(50), kv_from=0, diff=0.7,
                               softcap=4.0),
                     mamba2(4, 32, 16, 1, 1, 2, moe(3, 3, 32, 16, 1)),
                     rglru(48, 1, 2, None),
                     attention(4, 4, 32, 32, rotation(32, 500.0), None),
                     attention(**SHARED, mlp=moe(4, 1, 16, 24), kv_from=0)],
                    width=72, vocab=133, groups=3),
    # sizes that no vector load divides; more identity outputs than experts
    "odd": config([rglru(21, 3, 5, moe(2, 4, 5, 3, 3, 0.6)),
                   mamba2(3, 7, 9, 3, 7, 6, dense(33)),
                   attention(3, 1, 10, 9, rotation(6, 50.0), dense(19)),
                   attention(3, 1, 10, 9, rotation(6, 50.0),
                             moe(3, 2, 7, 9, 1), kv_from=2)],
                  width=27, vocab=61, groups=9),
    # large heads and states
    "wide": config([mamba2(2, 136, 200, 2, 2, 4, dense(64)),
                    attention(4, 2, 120, 160, rotation(64), dense(64)),
                    rglru(320, 2, 3, moe(9, 3, 16, 24, 1, 2.5)),
                    attention(8, 1, 40, 64, rotation(40), dense(64)),
                    mamba2(1, 72, 100, 1, 8, 4, None)], width=48, groups=4),
    # what can be 1 is 1: heads, groups, blocks, taps, choices, dims / 2
    "ones": config([attention(1, 1, 2, 1, rotation(2, 10.0), dense(8)),
                    rglru(5, 5, 1, moe(1, 1, 8, 8)),
                    mamba2(1, 1, 1, 1, 1, 1, None),
                    rglru(24, 1, 16, None),
                    mamba2(2, 8, 4, 2, 16, 16, dense(1))],
                   width=40, groups=1, eps=0.02),
    # no recurrence; plain and stretched angles; wide groups
    "plain": config([attention(8, 2, 32, 32, dict(dims=16, base=100.0),
                               dense(80)),
                     attention(2, 2, 64, 24, rotation(64, 100.0, 8.0, 40),
                               dense(80), diff=0.05, softcap=50.0),
                     attention(8, 2, 32, 32, dict(dims=16, base=100.0),
                               moe(4, 2, 20, 12, 1), kv_from=0)], width=64),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).bfloat16()

    def lin(key, out, size, std=1.0):
        w[key] = r(out, size, std=std * size ** -0.5)

    def gated(pre, F):
        lin(pre + "gate", F, E, 1.5)
        lin(pre + "up", F, E)
        lin(pre + "down", E, F, 1.5)

    E = cfg["width"]
    w = {"embed": r(cfg["vocab"], E), "final.norm": r(E, std=0.2, mean=1.0)}
    lin("head", cfg["vocab"], E)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in "12" if f else "1":
            w[f"{p}norm{n}"] = r(E, std=0.2, mean=1.0)
            w[f"{p}ls{n}"] = r(E, std=0.3, mean=0.8)
        w[p + "shift"] = torch.rand(E, generator=g).bfloat16()
        w[p + "dwa"] = r(i + 2, std=0.4)
        w[p + "dwa"][-1] = 0.9
        q = p + "mix."
        if layer["type"] == "rglru":
            W, B, K = m["width"], m["blocks"], m["conv"]
            for n in "yx":
                lin(q + n, W, E)
                w[q + n + ".b"] = r(W, std=0.5)
            for n in ("ra", "ri"):
                w[q + n] = r(B, W // B, W // B, std=(B / W) ** 0.5)
                w[q + n + ".b"] = r(B, W // B, std=1.0)
            # from channels that forget at once to ones that hold on
            w[q + "lam"] = r(W, std=2.5, mean=-4.0)
            inner = W
        elif layer["type"] == "mamba2":
            H, K = m["heads"], m["conv"]
            inner = H * m["vdim"]
            W = inner + 2 * m["groups"] * m["state"]
            lin(q + "in", inner + W + H, E)
            w[q + "dt_bias"] = r(H, std=1.5, mean=-1.0)
            w[q + "A_log"] = r(H, std=1.5, mean=-1.0)
            w[q + "D"] = r(H)
            w[q + "norm"] = r(inner, std=0.2, mean=1.0)
        else:
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            inner = H * m["vdim"]
            lin(q + "q", 2 * H * D, E)
            w[q + "q.norm"] = r(D, std=0.3, mean=1.3)
            if "kv_from" not in m:
                lin(q + "k", 2 * G * D, E)
                lin(q + "v", G * m["vdim"], E)
                w[q + "k.norm"] = r(D, std=0.3, mean=1.3)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                w[q + n] = r(D, std=0.5 * D ** -0.25)
        if layer["type"] != "attention":
            w[q + "conv"] = r(W, K, std=K ** -0.5)
            w[q + "conv.b"] = r(W, std=0.3)
        lin(q + "o", E, inner)
        if f is None:
            continue
        if f["kind"] == "dense":
            lin(p + "mlp.up", f["ff"], E, 1.5)
            lin(p + "mlp.down", E, f["ff"], 1.5)
            continue
        outputs = f["router"]["experts"] + f["router"]["identity"]
        lin(p + "mlp.router", outputs, E, 2.0)
        w[p + "mlp.correction"] = r(outputs, std=0.3)
        for e in range(f["router"]["experts"]):
            gated(f"{p}mlp.e{e}.", f["expert"]["ff"])
        gated(p + "mlp.shared.", f["shared"]["ff"])
        lin(p + "mlp.shared.sg", 1, E)
    return w
