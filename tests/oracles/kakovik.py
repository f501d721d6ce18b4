"""Plain, slow Kakovik in float64: one function per mechanism, loops where a
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


def stream_norm(x, weight, eps):
    """Norm of the residual stream; the weight is stored around zero."""
    return rms(x, eps) * (1 + weight)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def distance_bucket(n, rows, furthest):
    """Row of the relative-distance table for distance n: one row per distance
    over the first half, then rows at equal steps of ln n up to `furthest`.
    (The small number keeps a distance exactly at a row's start in that row.)
    """
    half = rows // 2
    if n < half:
        return n
    steps = math.log(n / half) / math.log(furthest / half) * (rows - half)
    return min(rows - 1, half + math.floor(steps + 1e-9))


def distance_bias(rel, n_max, furthest):
    """[heads, n_max] additive score bias for distances 0 .. n_max-1."""
    rows = rel.shape[0]
    idx = [distance_bucket(n, rows, furthest) for n in range(n_max)]
    return rel[idx].T


def visible(i, j, chunk):
    return j <= i and i // chunk == j // chunk


def attend(q, k, v, bias, scale, chunk):
    """q [n, H, d], k [n, G, d], v [n, G, dv], bias [H, n] -> [n, H, dv]."""
    n, heads, _ = q.shape
    per = heads // k.shape[1]
    out = torch.zeros(n, heads, v.shape[2], dtype=q.dtype)
    for i in range(n):
        js = [j for j in range(i + 1) if visible(i, j, chunk)]
        dist = torch.tensor([i - j for j in js])
        for h in range(heads):
            g = h // per
            s = k[js, g] @ q[i, h] * scale + bias[h, dist]
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[js, g]
    return out


def mix_values(v, v_first, lam):
    return (1 - lam) * v + lam * v_first


def attention(w, pre, mixer, h, eps, v_first):
    """The attention mixer; returns (output, v_first)."""
    n = h.shape[0]
    heads, groups = mixer["heads"], mixer["kv_heads"]
    q = rms(h @ w[pre + "q"].T, eps) * w[pre + "q.norm"]
    k = rms(h @ w[pre + "k"].T, eps) * w[pre + "k.norm"]
    v = h @ w[pre + "v"].T
    if mixer["v_mix"]:
        if v_first is None:
            v_first = v
        else:
            v = mix_values(v, v_first, w[pre + "vmix"])
    bias = distance_bias(w[pre + "rel"], n, mixer["bias_max"])
    o = attend(q.view(n, heads, -1), k.view(n, groups, -1),
               v.view(n, groups, -1), bias, mixer["scale"],
               mixer["mask"]["size"])
    o = o * sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return o.reshape(n, -1) @ w[pre + "o"].T, v_first


def key_decay(w, pre, h, tau):
    """alpha [n, heads*dim]: the factor of every key channel's state row."""
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    return sigmoid(z) ** (1 / tau)


def recur(q, k, v, alpha, state=None):
    """q, k, alpha [n, H, d], v [n, H, dv]; returns (o [n, H, dv], state)."""
    n, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype) \
        if state is None else state.clone()
    out = []
    for t in range(n):
        s = alpha[t][:, :, None] * s + k[t][:, :, None] * v[t][:, None, :]
        out.append((s * q[t][:, :, None]).sum(1))
    return torch.stack(out), s


def gla(w, pre, mixer, h, eps):
    """The gated-linear-attention mixer."""
    n, heads, d = h.shape[0], mixer["heads"], mixer["dim"]
    q = (h @ w[pre + "q"].T * d ** -0.5).view(n, heads, d)
    k = (h @ w[pre + "k"].T).view(n, heads, d)
    v = (h @ w[pre + "v"].T).view(n, heads, -1)
    alpha = key_decay(w, pre, h, mixer["tau"]).view(n, heads, d)
    o, _ = recur(q, k, v, alpha)
    o = (rms(o, eps) * w[pre + "norm"]).reshape(n, -1)
    return (o * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def feed_forward(w, pre, h):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) \
        @ w[pre + "down"].T


def forward(cfg, weights, tokens, streams=None):
    """Logits [n, vocab]; appends the residual after each layer to `streams`."""
    w = {k: t.to(F64) if t.is_floating_point() else t
         for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = stream_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y, v_first = attention(w, p + "mix.", layer["mixer"], h, eps,
                                   v_first)
        else:
            y = gla(w, p + "mix.", layer["mixer"], h, eps)
        x = x + stream_norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            y = feed_forward(w, p + "mlp.", stream_norm(x, w[p + "norm2"], eps))
            x = x + stream_norm(y, w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return stream_norm(x, w["final.norm"], eps) @ w["head"].T \
        * cfg["logit_scale"]
