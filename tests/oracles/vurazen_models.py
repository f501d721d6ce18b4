"""Small Vurazen models with random weights, as checkpoint folders.

Weights are drawn so that faults show: attention is sharp, sinks weigh as much
as keys, decays reach from a few tokens to hundreds, norms, gates and
convolutions are far from neutral.

Routers must decide clearly, or rounding alone would choose other experts. So
the first CODE elements of the residual stay what the embedding makes them, a
multiple of one of KINDS patterns (no layer adds to them). Norms leave those
alike but for a common factor, and routers read only those, with rows whose sum
is zero, for choices that hold over a range of factors.
"""

import json
import os

import torch
from safetensors.torch import save_file

from .models import tokens  # noqa: F401  (the same for every design)


CODE, KINDS = 8, 6


def clear_router(codes, experts, top, gen):
    """Of many random routers, (rows, biases) with the clearest decisions."""
    best, best_gap = None, -1.0
    for _ in range(1500):
        w = 0.8 * torch.randn(experts, CODE, generator=gen)
        # multiples of 1/64 that add up to zero also in bfloat16
        w = (w * 64).round() / 64
        w[:, -1] -= w.sum(1)
        b = (0.4 * torch.randn(experts, generator=gen)).bfloat16().float()
        if top == experts:
            return w, b
        z = torch.cat([codes @ w.T / s + b
                       for s in (0.35, 0.6, 0.8, 1, 1.3, 1.7, 2.2, 3, 4)])
        z = z.sort(1, descending=True).values
        gap = float((z[:, top - 1] - z[:, top]).min())
        if gap > best_gap:
            best, best_gap = (w, b), gap
    assert best_gap > 0.03, best_gap
    return best


def mamba(inner, state, rank, taps):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state,
                                        "dt_rank": rank, "conv": taps},
            "mlp": None}


def lightning(heads, dim, vdim, decay):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim,
                                           "vdim": vdim, "decay": decay},
            "mlp": None}


def att(heads, kv_heads, dim, taps, size, keep, dims, base=100.0, cap=8.0,
        scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
            "conv": taps, "mask": {"size": size, "keep_first": keep},
            "rot": {"base": base, "dims": dims}, "softcap": cap,
            "scale": scale or 2.5 * dim ** -0.5}


def delta(heads, kv_heads, dim, vdim, taps):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "conv": taps}


def both(left, right, left_scale, right_scale):
    return {"type": "parallel", "mixer": {
        "left": left, "right": right, "left_scale": left_scale,
        "right_scale": right_scale}, "mlp": None}


def dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def moe(layer, experts, top, ff, limit, shared=None):
    doc = {"kind": "moe", "router": {"experts": experts, "top": top},
           "expert": {"ff": ff, "limit": limit}}
    if shared:
        doc["shared"] = {"ff": shared[0], "limit": shared[1]}
    return dict(layer, mlp=doc)


def config(width, vocab, layers, loop=None, eps=1e-5, scale=1.0, cap=9.0):
    doc = {"architecture": "Vurazen", "width": width, "vocab": vocab,
           "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_softcap": cap, "layers": layers}
    if loop:
        doc["loop"] = dict(zip(("start", "stop", "times"), loop))
    return doc


# name -> (config, inner sizes of the delta rules' decays and gates)
CONFIGS = {
    # every mixer with every feed-forward and without, a loop in the middle
    "mixed": (config(80, 101, [
        moe(lightning(3, 24, 16, [0.5, 0.9, 0.995]), 5, 2, 24, 1.0, (40, 2.0)),
        dense(both(att(4, 2, 24, 3, 24, 3, 12), delta(4, 2, 16, 24, 4),
                   0.7, 1.2), 72),
        mamba(96, 16, 8, 4),
        moe(both(att(4, 4, 32, 2, 40, 0, 32), delta(2, 2, 24, 16, 3),
                 1.1, 0.8), 6, 3, 32, 0.8),
        moe(mamba(64, 24, 5, 3), 3, 1, 16, 3.0, (24, 0.7)),
    ], loop=(1, 4, 2), scale=1.5), (8, 12)),
    # sizes that no vector load divides; the loop reaches the last layer
    "odd": (config(51, 67, [
        dense(mamba(45, 5, 3, 5), 37),
        both(att(3, 1, 9, 4, 17, 19, 6, base=30.0, cap=4.0),
             delta(3, 1, 7, 11, 2), 0.4, 1.3),
        moe(lightning(2, 11, 13, [0.97, 0.3]), 7, 3, 13, 0.6, (19, 1.4)),
    ], loop=(1, 3, 3), eps=1e-2, scale=0.8, cap=9.0), (5, 7)),
    # everything that can be 1 is, or equal; no loop
    "ones": (config(64, 90, [
        moe(both(att(1, 1, 64, 1, 1, 1, 64), delta(1, 1, 64, 64, 1), 1.0, 1.0),
            1, 1, 64, 1.0, (64, 1.0)),
        dense(mamba(64, 1, 1, 1), 64),
        lightning(1, 64, 64, [1.0]),
    ]), (1, 1)),
    # head and state sizes of large models, first layers looped
    "large": (config(192, 90, [
        moe(both(att(3, 3, 128, 4, 48, 4, 64, base=1e4, cap=30.0),
                 delta(2, 2, 128, 128, 4), 0.8, 0.8), 8, 3, 64, 2.0,
            (96, 2.0)),
        dense(mamba(256, 16, 12, 4), 128),
        dense(lightning(2, 128, 128, [0.8, 0.99]), 96),
    ], loop=(0, 2, 2)), (128, 64)),
}


def weights(cfg, ranks, seed):
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def onto(name, inp, gain=1.0):
        mat(name, width, inp, gain)
        w[name][:CODE] = 0.0

    def vec(name, n, mean=0.0, std=0.3):
        w[name] = mean + std * torch.randn(n, generator=g)

    def norm(name):
        vec(name, width, 1.0)
        vec(name + ".b", width)
        w[name][:CODE], w[name + ".b"][:CODE] = 1.0, 0.0

    def glu(pre, ff):
        mat(pre + "gate", ff, width, 1.5)
        mat(pre + "up", ff, width)
        onto(pre + "down", ff)

    codes = torch.randn(KINDS, CODE, generator=g).sign()
    w["embed"] = torch.randn(cfg["vocab"], width, generator=g)
    w["embed"][:, :CODE] = codes[torch.arange(cfg["vocab"]) % KINDS]
    mat("head", cfg["vocab"], width, 3.0)
    norm("final.norm")
    if cfg.get("loop"):
        w["loop.step"] = 0.7 * torch.randn(cfg["loop"]["times"], width,
                                           generator=g)
        w["loop.step"][:, :CODE] = 0.0
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        norm(f"l{i}.norm1")
        if layer["type"] == "mamba1":
            inner, n, rank = m["inner"], m["state"], m["dt_rank"]
            mat(p + "in", 2 * inner, width)
            mat(p + "conv", inner, m["conv"])
            vec(p + "conv.b", inner)
            mat(p + "x", rank + 2 * n, inner, 1.3)
            mat(p + "dt", inner, rank)
            vec(p + "dt.b", inner, -2.0, 1.5)
            w[p + "A_log"] = 2.5 * torch.rand(inner, n, generator=g) - 2
            vec(p + "D", inner, 0.8)
            onto(p + "o", inner)
        elif layer["type"] == "lightning":
            h, d, dv = m["heads"], m["dim"], m["vdim"]
            mat(p + "q", h * d, width)
            mat(p + "k", h * d, width)
            mat(p + "v", h * dv, width)
            mat(p + "g", h * dv, width)
            vec(p + "norm", h * dv, 1.0)
            onto(p + "o", h * dv)
        else:
            a, b = m["left"], m["right"]
            for n, h in (("q", a["heads"]), ("k", a["kv_heads"])):
                mat(f"{p}left.{n}", h * a["dim"], width)
                vec(f"{p}left.{n}.b", h * a["dim"])
                mat(f"{p}left.{n}.conv", h * a["dim"], a["conv"], 1.2)
            vec(p + "left.sink", a["heads"], 0.5, 1.0)
            onto(p + "left.o", a["heads"] * a["dim"])
            h, d, dv = b["heads"], b["dim"], b["vdim"]
            for n, rows in (("q", b["kv_heads"] * d), ("k", b["kv_heads"] * d),
                            ("v", h * dv)):
                mat(f"{p}right.{n}", rows, width)
                mat(f"{p}right.{n}.conv", rows, b["conv"])
            mat(p + "right.b", h, width)
            vec(p + "right.A_log", h, -1.0)
            vec(p + "right.norm", dv, 1.0)
            mat(p + "right.a1", ranks[0], width)
            mat(p + "right.a2", h * d, ranks[0])
            vec(p + "right.dt_bias", h * d, -2.5, 2.0)
            mat(p + "right.g1", ranks[1], width)
            mat(p + "right.g2", h * dv, ranks[1])
            onto(p + "right.o", h * dv)
        p, mlp = f"l{i}.mlp.", layer["mlp"]
        if mlp and mlp["kind"] == "dense":
            glu(p, mlp["ff"])
        elif mlp:
            n = mlp["router"]["experts"]
            w[p + "router"] = torch.zeros(n, width)
            w[p + "router"][:, :CODE], w[p + "router.b"] = clear_router(
                codes, n, mlp["router"]["top"], g)
            for e in range(n):
                glu(f"{p}e{e}.", mlp["expert"]["ff"])
            if mlp.get("shared"):
                glu(p + "shared.", mlp["shared"]["ff"])
    return {k: t.to(torch.bfloat16) for k, t in w.items()}


def write(folder, name, seed=0):
    """(config, weights) of a named model, also written to the folder."""
    cfg, ranks = CONFIGS[name]
    w = weights(cfg, ranks, seed)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(folder, "model.safetensors"))
    return cfg, w
