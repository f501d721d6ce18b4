"""Small Ditalorn models with random weights, as checkpoint folders.

Weights are drawn so that faults show: attention is sharp, weights that are
sigmoids reach from nothing to almost one, falloffs from none to steep, norms,
gates and convolutions are far from neutral.

Routers must decide clearly, or rounding alone would choose other experts. So
the first CODE elements of the residual stay what the embedding makes them, a
multiple of one of KINDS patterns (no layer and no position adds to them).
Norms leave those alike but for a common factor, and routers read only those,
for choices that hold over a range of factors.
"""

import json
import os

import torch
from safetensors.torch import save_file

from .models import tokens  # noqa: F401  (the same for every design)


CODE, KINDS = 8, 6
FACTORS = (0.4, 0.6, 0.8, 1.0, 1.3, 1.7, 2.2, 2.8)


def chosen(s, router, best):
    """Choice scores [n, experts] -> (who is chosen, how clear the closest
    decision is); groups count by their `best` best, 0: no groups."""
    n, top = s.shape[1], router["top"]
    groups = router.get("groups", {"count": 1, "keep": 1})
    size, keep = n // groups["count"], groups["keep"]
    gap = float("inf")
    if best and keep < groups["count"]:
        g = s.view(len(s), -1, size).topk(min(best, size), -1).values.sum(-1)
        order = g.sort(1, descending=True)
        gap = float((order.values[:, keep - 1] - order.values[:, keep]).min())
        out = torch.ones_like(g, dtype=torch.bool).scatter_(
            1, order.indices[:, :keep], False)
        s = s.masked_fill(out.repeat_interleave(size, 1), -1e9)
        n = keep * size
    order = s.sort(1, descending=True)
    if top < n:
        gap = min(gap, float((order.values[:, top - 1] -
                              order.values[:, top]).min()))
    return order.indices[:, :top].sort(1).values, gap


def clear_router(codes, router, gen):
    """Of many random routers, (rows, corrections) with the clearest
    decisions, to which groups and their second best experts matter."""
    n = router["experts"]
    groups = router.get("groups", {"count": 1, "keep": 1})
    matter = (0, 1) if groups["keep"] < groups["count"] < n else ()
    best, best_gap = None, -1.0
    for _ in range(1500):
        w = (0.5 * torch.randn(n, CODE, generator=gen)).bfloat16().float()
        # all below zero, so that choice scores are
        c = (0.4 * torch.randn(n, generator=gen) - 2.5).bfloat16().float()
        s = torch.cat([torch.sigmoid(f * codes @ w.T) for f in FACTORS]) + c
        who, gap = chosen(s, router, 2)
        if gap > best_gap and all(
                int((who != chosen(s, router, b)[0]).any(1).sum()) > KINDS
                for b in matter):
            best, best_gap = (w, c), gap
    assert best_gap > 0.01, best_gap
    return best


def att(heads, kv_heads, dim, vdim, taps, coef=0.4, every=16, scale=None):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "conv": taps, "q_temp": {"coef": coef, "every": every},
        "scale": scale or 1.2 * dim ** -0.5}, "mlp": None}


def latent(heads, dim, vdim, q_rank, kv_rank, size, scale=None):
    return {"type": "latent_attention", "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank,
        "kv_rank": kv_rank, "mask": {"size": size},
        "scale": scale or 1.2 * dim ** -0.5}, "mlp": None}


def moe(layer, experts, top, ff, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return dict(layer, mlp={"kind": "moe", "expert": {"ff": ff}, "router": r})


def config(width, vocab, layers, eps=1e-5, scale=1.0, positions=400):
    return {"architecture": "Ditalorn", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "max_positions": positions, "layers": layers}


CONFIGS = {
    # both mixers with and without experts, grouped heads, several windows
    "mixed": config(80, 101, [
        moe(att(4, 2, 24, 40, 3, 1.5), 9, 3, 40, (3, 2)),
        latent(3, 24, 16, 56, 40, 24),
        moe(latent(5, 16, 24, 32, 72, 50), 4, 1, 56),
        att(6, 1, 16, 24, 4, 0.25, 7),
        moe(att(2, 2, 32, 48, 2, 0.6, 50), 10, 2, 24, (5, 2)),
        moe(latent(2, 40, 32, 24, 64, 17), 6, 3, 32, (2, 1)),
    ], scale=1.5),
    # sizes that no vector load divides; windows of a few keys; one expert in
    # a group
    "odd": config(51, 67, [
        moe(latent(3, 9, 7, 13, 21, 5), 6, 2, 13, (3, 1)),
        att(3, 1, 11, 7, 5, 0.5, 3),
        moe(att(2, 2, 7, 13, 2, 0.3, 1), 5, 2, 7, (5, 4)),
        latent(1, 5, 11, 9, 33, 33),
    ], eps=1e-2, scale=0.7, positions=301),
    # everything that can be 1 is, or equal
    "ones": config(64, 90, [
        moe(att(1, 1, 64, 64, 1, 1.0, 1, 1.0), 1, 1, 64, (1, 1)),
        moe(latent(1, 64, 64, 64, 64, 1, 1.0), 2, 1, 64, (2, 1)),
        moe(latent(1, 64, 64, 64, 64, 64), 2, 2, 64, (1, 1)),
        moe(att(1, 1, 64, 64, 1, 0.0, 1000), 2, 1, 64),
    ]),
    # head and latent sizes of large models, latents alone
    "large": config(192, 90, [
        moe(latent(4, 128, 128, 192, 512, 100), 8, 3, 128, (4, 2)),
        moe(latent(18, 32, 48, 96, 256, 33), 3, 2, 96),
    ], scale=2.0),
    "heads": config(128, 90, [
        moe(att(8, 2, 128, 128, 4, 0.2, 32), 8, 3, 128, (4, 2)),
        moe(att(3, 3, 64, 160, 3, 0.2, 64), 3, 2, 96),
    ], scale=8.0),
}


def weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=0.0, std=0.3):
        w[name] = mean + std * torch.randn(n, generator=g)

    codes = torch.randn(KINDS, CODE, generator=g).sign()
    scale = cfg["embedding"]["scale"]
    w["embed"] = torch.randn(cfg["vocab"], width, generator=g) / scale
    w["embed"][:, :CODE] = \
        codes[torch.arange(cfg["vocab"]) % KINDS] / scale
    w["pos"] = 0.4 * torch.randn(cfg["max_positions"], width, generator=g)
    w["pos"][:, :CODE] = 0.0
    # factors of both signs: a token's own embedding does not win by itself
    vec("final.norm", width, -1.0, 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        h, d, dv = m["heads"], m["dim"], m["vdim"]
        norms = ["norm1", "norm1b"] + (
            ["norm2", "norm2b"] if layer["mlp"] else [])
        for n in norms:
            vec(f"l{i}.{n}", width)
            # what is added leaves the codes alone, what is read has them
            w[f"l{i}.{n}"][:CODE] = -1.0 if n[-1] == "b" else 0.0
        mat(p + "o", width, h * dv)
        if layer["type"] == "attention":
            kv, taps = m["kv_heads"], m["conv"]
            for n, rows in (("q", h * d), ("k", kv * d), ("v", kv * dv)):
                mat(p + n, rows, width)
                vec(f"{p}{n}.b", rows)
                mat(f"{p}{n}.conv", rows, taps, 1.3)
            vec(p + "o.b", width)
            w[p + "r1"] = 2.0 * torch.rand(h, generator=g)
            w[p + "r2"] = 0.1 + 0.9 * torch.rand(h, generator=g)
            vec(p + "pb", h, -1.5, 0.8)
        else:
            mat(p + "dq", m["q_rank"], width)
            vec(p + "dq.norm", m["q_rank"], 1.0)
            mat(p + "uq", h * d, m["q_rank"], 1.3)
            mat(p + "dkv", m["kv_rank"], width)
            vec(p + "dkv.norm", m["kv_rank"], 1.0)
            mat(p + "uk", h * d, m["kv_rank"], 1.3)
            mat(p + "uv", h * dv, m["kv_rank"])
            mat(p + "g", h, width, 2.0)
        if layer["mlp"]:
            p, r = f"l{i}.mlp.", layer["mlp"]["router"]
            w[p + "router"] = torch.zeros(r["experts"], width)
            w[p + "router"][:, :CODE], w[p + "correction"] = clear_router(
                codes, r, g)
            ff = layer["mlp"]["expert"]["ff"]
            for e in range(r["experts"]):
                mat(f"{p}e{e}.gate", ff, width, 1.5)
                mat(f"{p}e{e}.up", ff, width)
                mat(f"{p}e{e}.down", width, ff)
    return {k: t.to(torch.bfloat16) for k, t in w.items()}


def write(folder, name, seed=0):
    """(config, weights) of a named model, also written to the folder."""
    cfg = CONFIGS[name]
    w = weights(cfg, seed)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(folder, "model.safetensors"))
    return cfg, w
