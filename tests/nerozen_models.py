"""Small random Nerozen models in their on-disk form, for the tests."""

import json
from pathlib import Path

import torch


def h2(heads, dim, vdim, ff=96):
    return dict(type="hgrn2", mixer=dict(heads=heads, dim=dim, vdim=vdim),
                mlp=None if ff is None else dict(kind="dense", ff=ff))


def att(heads, kv_heads, dim, vdim, size, keep, far, scale=0.2, ff=96,
        rows=12):
    """``rows`` (of the bias table) is not configuration: popped on use."""
    return dict(type="attention",
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                           scale=scale, bias_max=far,
                           mask=dict(size=size, keep_first=keep)),
                mlp=None if ff is None else dict(kind="dense", ff=ff),
                rows=rows)


def config(layers, width=64, vocab=120, emb=1.5, eps=1e-5):
    rows = [l.get("rows") for l in layers]
    layers = [{k: v for k, v in l.items() if k != "rows"} for l in layers]
    cfg = dict(architecture="Nerozen", vocab=vocab, width=width,
               embedding=dict(scale=emb), norm=dict(eps=eps), layers=layers)
    return cfg, rows


# name -> (config, table rows per layer)
MODELS = {
    # both mixers, unequal q/k and value sizes, three queries per kv head
    "mixed": config([h2(3, 24, 40), att(6, 2, 48, 20, 37, 3, 90),
                     h2(2, 16, 16), att(3, 3, 32, 64, 70, 0, 30, rows=6)],
                    width=72, vocab=133),
    # one kv head, window of one key plus kept tokens, no feed-forwards
    "narrow": config([att(5, 1, 16, 24, 1, 5, 50, ff=None),
                      h2(1, 1, 3, ff=40), h2(4, 100, 12, ff=None)],
                     width=40, emb=0.3),
    # widths that no vector load divides, table larger than the window
    "odd": config([h2(3, 7, 9, ff=33), att(4, 2, 10, 6, 12, 2, 200, ff=27,
                                            rows=20)],
                  width=27, vocab=61),
    # attention only, head sizes above 128, whole context visible
    "wide": config([att(4, 4, 160, 136, 4096, 1, 64),
                    att(16, 1, 64, 32, 100, 9, 33, rows=16)], width=48),
    # recurrence only
    "recurrent": config([h2(2, 130, 66), h2(5, 32, 20)], width=64),
}


def weights(cfg, rows, seed=0):
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).bfloat16()

    E = cfg["width"]
    w = {"embed": r(cfg["vocab"], E), "final.norm": r(E, std=0.2),
         "head": r(cfg["vocab"], E, std=E ** -0.5)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for n in ("1", "1b") + (("2", "2b") if layer["mlp"] else ()):
            w[f"{p}norm{n}"] = r(E, std=0.2)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        q = p + "mix."
        w[q + "q"] = r(H * D, E, std=E ** -0.5)
        if layer["type"] == "hgrn2":
            w[q + "f"] = r(H * D, E, std=E ** -0.5)
            # from gates that forget at once to gates that hold on
            w[q + "f.b"] = r(H * D, std=3.0, mean=2.0)
            w[q + "lower"] = torch.rand(H * D, generator=g).mul(0.9).bfloat16()
            w[q + "v"] = r(H * V, E, std=E ** -0.5)
            w[q + "norm"] = r(V, std=0.2, mean=1.0)
        else:
            G = m["kv_heads"]
            w[q + "k"] = r(G * D, E, std=E ** -0.5)
            w[q + "v"] = r(G * V, E, std=E ** -0.5)
            w[q + "q.norm"] = r(D, std=0.3, mean=1.4)
            w[q + "k.norm"] = r(D, std=0.3, mean=1.4)
            w[q + "rel"] = r(rows[i], H, std=1.5)
        w[q + "o"] = r(E, H * V, std=(H * V) ** -0.5)
        if layer["mlp"]:
            F = layer["mlp"]["ff"]
            w[p + "mlp.up"] = r(F, E, std=E ** -0.5)
            w[p + "mlp.down"] = r(E, F, std=F ** -0.5)
            w[p + "mlp.act"] = r(2, std=0.5)
    return w


def save(path: Path, cfg, w) -> Path:
    from safetensors.torch import save_file

    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: t.contiguous() for k, t in w.items()},
              str(path / "model.safetensors"))
    return path


def make_runner(cfg, w, device, dtype, n_slots=4, n_tokens=1024,
                max_seq=None):
    """The framework's runner for the model, through its own key layout."""
    from mdi_llm_amd.config import ModelConfig
    from mdi_llm_amd.models.hybrid import native_state_dict
    from mdi_llm_amd.models.stages import StarterStage
    from mdi_llm_amd.parallel.runner import make_runner as make

    config = ModelConfig.from_native(cfg)
    stage = StarterStage(config, config.n_layer)
    stage.load_state_dict(native_state_dict(config, w.__getitem__))
    stage = stage.to(device=device, dtype=dtype).eval()
    stage.max_seq_length = max_seq or n_tokens
    return make(stage, n_slots, torch.device(device), n_tokens=n_tokens)


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def deviation(got, want):
    """rms difference of the mean-free logits of the worst position, over
    the rms of the wanted ones."""
    want = want.double().cpu()
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return float(d.pow(2).mean(-1).sqrt().max() / want.pow(2).mean().sqrt())
