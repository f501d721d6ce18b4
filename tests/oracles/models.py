"""Small Kakovik models with random weights, as checkpoint folders.

Weights are drawn so that faults show: norms and gates are far from neutral,
attention is sharp, distance biases are as large as scores, and recurrent
channels reach from a few tokens to hundreds.
"""

import json
import os

import torch
from safetensors.torch import save_file


def att(heads, kv_heads, dim, vdim, chunk, bias_max, v_mix=True, scale=None):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "mask": {"size": chunk}, "bias_max": bias_max, "v_mix": v_mix,
        "scale": scale or 1.5 * dim ** -0.5}, "mlp": None}


def gla(heads, dim, vdim, tau):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                     "tau": tau}, "mlp": None}


def with_ff(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def config(width, vocab, layers, eps=1e-5, logit_scale=1.0):
    return {"architecture": "Kakovik", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers}


# name -> (config, rows of the distance tables, inner size of the decays)
CONFIGS = {
    # both mixers with and without a feed-forward, grouped heads
    "mixed": (config(80, 101, [
        gla(3, 24, 40, 4.0),
        with_ff(att(4, 2, 32, 24, 40, 130), 112),
        with_ff(gla(2, 16, 16, 1.0), 72),
        with_ff(att(6, 2, 16, 24, 28, 60), 96),
        att(2, 2, 40, 24, 100, 33),
    ], logit_scale=0.7), 12, 8),
    # a layer that does not blend ahead of those that do; one kv head;
    # sizes that no vector load divides
    "odd": (config(51, 67, [
        with_ff(att(3, 1, 20, 12, 17, 20, v_mix=False), 37),
        with_ff(att(3, 3, 9, 7, 24, 50), 45),
        gla(1, 13, 21, 16.0),
        with_ff(att(6, 3, 11, 7, 33, 90), 29),
    ], eps=1e-3), 7, 5),
    # attention only, chunk larger than the prompts; last layer plain
    "attention": (config(64, 90, [
        with_ff(att(4, 4, 64, 64, 512, 300), 64),
        with_ff(att(4, 2, 64, 128, 64, 64), 64),
    ], logit_scale=2.0), 32, 0),
    # recurrent only: nothing is paged
    "recurrent": (config(64, 90, [
        with_ff(gla(4, 32, 64, 16.0), 64), gla(4, 48, 32, 2.0)]), 0, 16),
}


def weights(cfg, rows, rank, seed):
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=0.0, std=0.2):
        w[name] = mean + std * torch.randn(n, generator=g)

    w["embed"] = torch.randn(cfg["vocab"], width, generator=g)
    mat("head", cfg["vocab"], width)
    vec("final.norm", width)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h, d, dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b"):
            vec(p + n, width)
        kv = m.get("kv_heads", h)
        mat(p + "mix.q", h * d, width)
        mat(p + "mix.k", kv * d, width)
        mat(p + "mix.v", kv * dv, width)
        mat(p + "mix.o", width, h * dv)
        if layer["type"] == "attention":
            vec(p + "mix.q.norm", h * d, 1.2)
            vec(p + "mix.k.norm", kv * d, 1.2)
            w[p + "mix.rel"] = 1.5 * torch.randn(rows, h, generator=g)
            if m["v_mix"]:
                w[p + "mix.vmix"] = 0.2 + 0.6 * torch.rand((), generator=g)
            mat(p + "mix.g", h, width, 2.0)
        else:
            mat(p + "mix.g", h * dv, width)
            mat(p + "mix.a1", rank, width)
            mat(p + "mix.a2", h * d, rank, 1.5)
            vec(p + "mix.a2.b", h * d, 2.0, 2.0)
            vec(p + "mix.norm", dv, 1.0)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            for n in ("norm2", "norm2b"):
                vec(p + n, width)
            mat(p + "mlp.gate", ff, width)
            mat(p + "mlp.up", ff, width)
            mat(p + "mlp.down", width, ff)
    return {k: t.to(torch.bfloat16) for k, t in w.items()}


def write(folder, name, seed=0):
    """(config, weights) of a named model, also written to the folder."""
    cfg, rows, rank = CONFIGS[name]
    w = weights(cfg, rows, rank, seed)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(folder, "model.safetensors"))
    return cfg, w


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
