"""Plain, slow Guronex in float64: one function per mechanism, loops where a
loop is clearest, nothing shared with the package under test.

`cfg` is the parsed config.json of a model, `w` maps tensor names to tensors.
A sequence is always processed whole, from position 0.
"""

import math

import torch

F64 = torch.float64


def rms(x, eps):
    """x over its root mean square (last axis), eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def gelu_erf(z):
    return z * 0.5 * (1 + torch.erf(z / math.sqrt(2)))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(
        math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate(x, base, dims):
    """x [n, ..., dims] of positions 0 .. n-1: element i turns with element
    i + dims/2 by the angle position * base^(-2i/dims)."""
    out = x.clone()
    half = dims // 2
    for p in range(x.shape[0]):
        for i in range(half):
            a = p * base ** (-2.0 * i / dims)
            u, v = x[p, ..., i], x[p, ..., i + half]
            out[p, ..., i] = u * math.cos(a) - v * math.sin(a)
            out[p, ..., i + half] = v * math.cos(a) + u * math.sin(a)
    return out


def visible(i, j):
    return j <= i


def attend(qn, qr, kn, kr, v, scale):
    """qn [n, H, d], qr [n, H, r], kn [n, H, d], kr [n, r] (one for all
    heads), v [n, H, dv] -> [n, H, dv]."""
    n, heads, _ = qn.shape
    out = torch.zeros(n, heads, v.shape[2], dtype=qn.dtype)
    for i in range(n):
        js = [j for j in range(n) if visible(i, j)]
        for h in range(heads):
            s = (kn[js, h] @ qn[i, h] + kr[js] @ qr[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[js, h]
    return out


def latents(w, pre, mixer, h, eps):
    """What the cache of a layer holds: normed latent [n, rank] and rotated
    key part [n, rot_dim]."""
    down = h @ w[pre + "dkv"].T
    rank = mixer["kv_rank"]
    c = rms(down[:, :rank], eps) * w[pre + "dkv.norm"]
    return c, rotate(down[:, rank:], mixer["rot"]["base"],
                     mixer["rot"]["dims"])


def latent_attention(w, pre, mixer, h, eps, held):
    """The mixer; `held` is what latents() gives, maybe of another layer."""
    n, heads, d, r = h.shape[0], mixer["heads"], mixer["dim"], mixer["rot_dim"]
    q = (h @ w[pre + "q"].T).view(n, heads, d + r)
    c, kr = held
    qr = rotate(q[:, :, d:], mixer["rot"]["base"], mixer["rot"]["dims"])
    kn = (c @ w[pre + "uk"].T).view(n, heads, d)
    v = (c @ w[pre + "uv"].T).view(n, heads, mixer["vdim"])
    o = attend(q[:, :, :d], qr, kn, kr, v, mixer["scale"]).reshape(n, -1)
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def route(z, router):
    """Scores z of one token -> {expert: weight}."""
    s = torch.exp(z - z.max())
    s = s / s.sum()
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = len(s) // groups["count"]
    best = [max(s[g * size:(g + 1) * size].tolist())
            for g in range(groups["count"])]
    kept = sorted(range(len(best)), key=lambda g: -best[g])[:groups["keep"]]
    open_ = [e for e in range(len(s)) if e // size in kept]
    chosen = sorted(open_, key=lambda e: -float(s[e]))[:router["top"]]
    return {e: s[e] for e in chosen}


def expert(w, pre, x):
    return gelu_erf(x @ w[pre + "up"].T) @ w[pre + "down"].T


def experts(w, pre, router, h):
    out = torch.zeros_like(h)
    z = h @ w[pre + "router"].T
    for t in range(h.shape[0]):
        for e, weight in route(z[t], router).items():
            out[t] += weight * expert(w, f"{pre}e{e}.", h[t])
    return out


def side_input(w, pre, x, e, eps):
    """What a layer adds for the token itself; e [n, dim] is its part of the
    token's side embedding."""
    y = (gelu_tanh(x @ w[pre + "gate"].T) * e) @ w[pre + "proj"].T
    return rms(y, eps) * w[pre + "norm"]


def forward(cfg, weights, tokens, streams=None):
    """Logits [n, vocab]; appends the residual after each layer to `streams`."""
    w = {k: t.to(F64) if t.is_floating_point() else t
         for k, t in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    toks = torch.as_tensor(tokens)
    x = w["embed"][toks]
    side = cfg.get("token_side")
    held = {}
    for i, layer in enumerate(cfg["layers"]):
        p, mixer = f"l{i}.", layer["mixer"]
        if mixer.get("kv_from") is None:
            held[i] = latents(w, p + "mix.", mixer, x, eps)
            src = i
        else:
            src = mixer["kv_from"]
        y = latent_attention(w, p + "mix.", mixer, x, eps, held[src])
        x = x + m * rms(y, eps) * w[p + "norm1"]
        if layer["mlp"] is not None:
            y = experts(w, p + "mlp.", layer["mlp"]["router"], x)
            x = x + m * rms(y, eps) * w[p + "norm2"]
        if side is not None:
            e = w["side.embed"][toks][:, i * side["dim"]:(i + 1) * side["dim"]]
            x = x + m * side_input(w, p + "side.", x, e, eps)
        if streams is not None:
            streams.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
