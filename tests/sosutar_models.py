"""Small random Sosutar models in their on-disk form, for the tests."""

import torch


def dense(ff):
    return None if ff is None else dict(kind="dense", ff=ff)


def mlstm(heads, dim, vdim, cap=9.0, ff=None):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim,
                                         gate_cap=cap), mlp=dense(ff))


def pair(heads, kv_heads, dim, vdim, size, width, ff=None, scale=None,
         coef=0.4, every=30):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                scale=1.3 * dim ** -0.5 if scale is None else scale,
                mask=dict(size=size), q_temp=dict(coef=coef, every=every))
    return dict(type="parallel", mixer=dict(left=left,
                                            right=dict(width=width)),
                mlp=dense(ff))


def again(layers, j):
    """A further layer with the weights of layer ``j``."""
    return dict({k: v for k, v in layers[j].items() if k != "weights_of"},
                weights_of=j)


def config(layers, width=64, vocab=120, eps=1e-5, emb=1.5, logits=0.7,
           positions=700):
    return dict(architecture="Sosutar", vocab=vocab, width=width,
                max_positions=positions, embedding=dict(scale=emb),
                norm=dict(eps=eps), logit_scale=logits, layers=layers)


MIXED = [pair(6, 2, 24, 40, 37, 80, 96), mlstm(3, 28, 20, 6.0, 50),
         mlstm(2, 16, 48), pair(4, 4, 32, 32, 70, 52, None, every=7)]
# the same weights again: next to each other, across others, of a repeat
MIXED += [again(MIXED, 0), again(MIXED, 2), mlstm(5, 8, 8, 15.0, 72)]
MIXED.append(again(MIXED, 5))

MODELS = {
    "mixed": config(MIXED, width=72, vocab=133),
    # sizes that no vector load divides
    "odd": config([mlstm(3, 7, 9, 4.0, 33), pair(3, 1, 10, 9, 12, 21, 19),
                   pair(6, 3, 5, 7, 65, 33, None, coef=0.9, every=3),
                   mlstm(1, 33, 5)], width=27, vocab=61, emb=0.8,
                  logits=3.0),
    # large heads and states
    "wide": config([mlstm(2, 200, 136, 11.0, 64), mlstm(1, 100, 300),
                    pair(4, 2, 120, 160, 100, 300, 64),
                    pair(8, 1, 40, 64, 500, 24, None)], width=48),
    # what can be 1 is 1
    "ones": config([pair(1, 1, 1, 1, 1, 1, 1, scale=0.5, every=1),
                    mlstm(1, 1, 1, 1.0, 8), mlstm(1, 1, 8),
                    pair(2, 1, 2, 1, 2, 3, 1, coef=0.0)], width=40,
                   eps=0.02, emb=1.0, logits=1.0),
    # no attention; no recurrence of matrices
    "memory": config([mlstm(4, 32, 32, 12.0, 80), mlstm(2, 64, 64, 3.0),
                      mlstm(2, 64, 64, 3.0, 40)], emb=0.5),
    "pairs": config([pair(8, 2, 32, 32, 64, 96, 80, every=100),
                     pair(2, 2, 64, 24, 128, 64, 80),
                     pair(12, 4, 16, 48, 33, 128)], width=96),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).bfloat16()

    def lin(key, out, size, std=1.0):
        w[key] = r(out, size, std=std * size ** -0.5)

    E = cfg["width"]
    w = {"embed": r(cfg["vocab"], E), "final.norm": r(E, std=0.2, mean=1.0),
         "pos": r(cfg["max_positions"], E, std=0.4)}
    lin("head", cfg["vocab"], E)
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in "12" if f else "1":
            w[f"{p}norm{n}"] = r(E, std=0.2, mean=1.0)
            w[f"{p}ls{n}"] = r(E, std=0.3, mean=0.8)
        q = p + "mix."
        if layer["type"] == "mlstm":
            H, D, V = m["heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * V),
                            ("g", H * V), ("i", H), ("f", H)):
                lin(q + n, rows, E, 1.5 if n == "k" else 1.0)
            # heads that forget at once and heads that hold on
            w[q + "i.b"] = r(H, std=1.5)
            w[q + "f.b"] = r(H, std=3.0, mean=2.0)
            w[q + "norm"] = r(H * V, std=0.2, mean=1.0)
            lin(q + "o", E, H * V)
        else:
            a, W = m["left"], m["right"]["width"]
            H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            left, right = q + "left.", q + "right."
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * V),
                            ("g", H * V)):
                lin(left + n, rows, E)
            w[left + "q.norm"] = r(H * D, std=0.3, mean=1.3)
            w[left + "k.norm"] = r(G * D, std=0.3, mean=1.3)
            w[left + "sink"] = r(H, std=1.5)
            lin(left + "o", E, H * V)
            for n in "zxg":
                lin(right + n, W, E, 1.5)
            w[right + "z.b"] = r(W, std=3.0, mean=-1.0)
            w[right + "x.b"] = r(W, std=0.5)
            lin(right + "o", E, W)
            w[left + "out"] = r(E, std=0.2, mean=1.0)
            w[right + "out"] = r(E, std=0.2, mean=1.0)
        if f is not None:
            lin(p + "mlp.up", f["ff"], E, 1.5)
            lin(p + "mlp.down", E, f["ff"], 1.5)
    return w
