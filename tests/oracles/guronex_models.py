"""Small Guronex models with random weights, as checkpoint folders.

Weights are drawn so that faults show: attention is sharp, the unrotated and
the rotated part of a score weigh alike, norms and gates are far from neutral.

Routers must decide clearly, or rounding alone would choose other experts. So
the first CODE elements of the residual stay what the embedding makes them,
one of KINDS patterns (no layer adds to them), and routers read only those.
"""

import json
import os

import torch
from safetensors.torch import save_file

from .models import tokens  # noqa: F401  (the same for every design)


CODE, KINDS = 8, 16


def clear_router(codes, router, gen):
    """Of many random routers the one whose closest decision is clearest."""
    n, top = router["experts"], router["top"]
    groups = router.get("groups", {"count": 1, "keep": 1})
    size, keep = n // groups["count"], groups["keep"]
    best, best_gap = None, -1.0
    for _ in range(400):
        w = (0.5 * torch.randn(n, CODE, generator=gen)).bfloat16().float()
        z = codes @ w.T
        gap = float("inf")
        g = z.view(KINDS, -1, size).amax(-1)
        if keep < g.shape[1]:
            order = g.sort(1, descending=True)
            gap = float((order.values[:, keep - 1] -
                         order.values[:, keep]).min())
            out = torch.ones_like(g, dtype=torch.bool).scatter_(
                1, order.indices[:, :keep], False)
            z = z.masked_fill(out.repeat_interleave(size, 1), -1e9)
        order = z.sort(1, descending=True).values
        if top < keep * size:
            gap = min(gap, float((order[:, top - 1] - order[:, top]).min()))
        if gap > best_gap:
            best, best_gap = w, gap
    assert best_gap > 0.04, best_gap
    return best


def att(heads, dim, rot_dim, vdim, rank, base=300.0, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": rank, "rot": {"base": base, "dims": rot_dim},
         "scale": scale or 1.0 * (dim + rot_dim) ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None}


def moe(layer, experts, top, ff, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return dict(layer, mlp={"kind": "moe", "expert": {"ff": ff}, "router": r})


def config(width, vocab, layers, eps=1e-5, mult=1.0, side=0):
    doc = {"architecture": "Guronex", "width": width, "vocab": vocab,
           "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    if side:
        doc["token_side"] = {"dim": side}
    return doc


CONFIGS = {
    # layers with and without experts, own and borrowed latents in turn
    "mixed": config(80, 101, [
        moe(att(3, 24, 8, 40, 56), 12, 3, 40, (3, 2)),
        att(5, 16, 8, 24, 56, scale=0.3, kv_from=0),
        moe(att(2, 32, 16, 16, 72, base=2e4), 4, 1, 56),
        moe(att(3, 8, 16, 32, 72, base=2e4, kv_from=2), 10, 2, 24, (5, 1)),
        att(4, 16, 24, 16, 40),
    ], mult=0.7, side=24),
    # sizes that no vector load divides; latents borrowed from afar
    "odd": config(51, 67, [
        moe(att(3, 9, 6, 7, 21), 6, 2, 13, (3, 1)),
        att(1, 5, 2, 11, 33),
        moe(att(2, 11, 6, 9, 21, kv_from=0), 5, 5, 7, (5, 5)),
        moe(att(3, 7, 2, 5, 33, kv_from=1), 7, 3, 17),
    ], eps=1e-2, mult=0.6, side=5),
    # everything that can be 1 is, or equal; no input for the token
    "ones": config(64, 90, [
        moe(att(1, 64, 64, 64, 64), 1, 1, 64, (1, 1)),
        moe(att(1, 64, 64, 64, 64, kv_from=0), 2, 1, 64, (2, 1)),
    ]),
    # head and latent sizes of large models
    "large": config(192, 90, [
        moe(att(4, 128, 64, 128, 512, base=1e4), 8, 3, 128, (4, 2)),
        moe(att(18, 32, 64, 48, 512, base=1e4, kv_from=0), 3, 2, 96),
        att(2, 64, 32, 128, 256),
    ], mult=0.8, side=40),
}


def weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=1.0, std=0.3):
        w[name] = mean + std * torch.randn(n, generator=g)

    codes = 1.5 * torch.randn(KINDS, CODE, generator=g).sign()
    w["embed"] = torch.randn(cfg["vocab"], width, generator=g)
    w["embed"][:, :CODE] = codes[torch.arange(cfg["vocab"]) % KINDS]
    mat("head", cfg["vocab"], width)
    vec("final.norm", width)
    side = cfg.get("token_side", {"dim": 0})["dim"]
    if side:
        w["side.embed"] = torch.randn(cfg["vocab"], side * len(cfg["layers"]),
                                      generator=g)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h, rank = m["heads"], m["kv_rank"]
        vec(p + "norm1", width)
        mat(p + "mix.q", h * (m["dim"] + m["rot_dim"]), width)
        mat(p + "mix.uk", h * m["dim"], rank, 1.4)
        mat(p + "mix.uv", h * m["vdim"], rank)
        mat(p + "mix.g", h * m["vdim"], width, 1.5)
        mat(p + "mix.o", width, h * m["vdim"])
        if "kv_from" not in m:
            mat(p + "mix.dkv", rank + m["rot_dim"], width, 1.4)
            vec(p + "mix.dkv.norm", rank)
        if layer["mlp"]:
            n, ff = layer["mlp"]["router"]["experts"], \
                layer["mlp"]["expert"]["ff"]
            vec(p + "norm2", width)
            w[p + "mlp.router"] = torch.zeros(n, width)
            w[p + "mlp.router"][:, :CODE] = clear_router(
                codes, layer["mlp"]["router"], g)
            for e in range(n):
                mat(f"{p}mlp.e{e}.up", ff, width, 1.5)
                mat(f"{p}mlp.e{e}.down", width, ff)
        if side:
            mat(p + "side.gate", side, width)
            mat(p + "side.proj", width, side)
            vec(p + "side.norm", width)
        for n in ("norm1", "norm2", "side.norm"):
            if p + n in w:
                w[p + n][:CODE] = 0.0
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
