"""Plain, slow Vurazen in float64: one function per mechanism, loops where a
loop is clearest, nothing shared with the package under test.

`cfg` is the parsed config.json of a model, `w` maps tensor names to tensors.
A sequence is always processed whole, from position 0.
"""

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def rms(x, eps):
    """x over its root mean square (last axis), eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight + bias


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def short_conv(u, taps):
    """u [n, channels], taps [channels, k]: the last tap is the row's own."""
    k = taps.shape[1]
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(k):
            s = t - (k - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * u[s]
    return out


def rotate(x, base, dims):
    """x [n, heads, d] of positions 0 .. n-1: element 2i turns with element
    2i + 1 by the angle position * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        for p in range(x.shape[0]):
            a = p * base ** (-2.0 * i / dims)
            u, v = x[p, :, 2 * i], x[p, :, 2 * i + 1]
            out[p, :, 2 * i] = u * math.cos(a) - v * math.sin(a)
            out[p, :, 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return out


def visible(i, j, size, keep):
    return j <= i and (i - j < size or j < keep)


def attend(q, k, v, scale, cap, size, keep, sink):
    """q [n, H, d], k and v [n, G, d] -> [n, H, d]."""
    n, heads, _ = q.shape
    per = heads // k.shape[1]
    out = torch.zeros(n, heads, v.shape[2], dtype=q.dtype)
    for i in range(n):
        js = [j for j in range(n) if visible(i, j, size, keep)]
        for h in range(heads):
            s = softcap((k[js, h // per] @ q[i, h]) * scale, cap)
            top = torch.maximum(s.max(), sink[h])
            p = torch.exp(s - top)
            out[i, h] = (p @ v[js, h // per]) / \
                (p.sum() + torch.exp(sink[h] - top))
    return out


def window_attention(w, pre, m, h):
    n, heads, kv, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (short_conv(h @ w[pre + p].T + w[pre + p + ".b"],
                       w[pre + p + ".conv"]) for p in ("q", "k"))
    q, k = q.view(n, heads, d), k.view(n, kv, d)
    v = k
    q, k = (rotate(t, m["rot"]["base"], m["rot"]["dims"]) for t in (q, k))
    o = attend(q, k, v, m["scale"], m["softcap"], m["mask"]["size"],
               m["mask"]["keep_first"], w[pre + "sink"])
    return o.reshape(n, -1) @ w[pre + "o"].T


def delta_recurrence(q, k, v, g, beta):
    """q, k, g [n, H, d], v [n, H, dv], beta [n, H]; q and k as they enter."""
    n, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(n):
        for h in range(heads):
            s[h] = g[t, h][:, None] * s[h]
            u = beta[t, h] * (v[t, h] - s[h].T @ k[t, h])
            s[h] = s[h] + torch.outer(k[t, h], u)
            out[t, h] = s[h].T @ q[t, h]
    return out


def delta_mixer(w, pre, m, h, eps):
    n, heads, kv, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], \
        m["vdim"]
    q, k, v = (silu(short_conv(h @ w[pre + p].T, w[pre + p + ".conv"]))
               for p in ("q", "k", "v"))
    per = heads // kv
    q, k = (unit(t.view(n, kv, d)).repeat_interleave(per, 1) for t in (q, k))
    beta = sigmoid(h @ w[pre + "b"].T)
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "dt_bias"]
    g = torch.exp(-torch.exp(w[pre + "A_log"])[None, :, None] *
                  softplus(z).view(n, heads, d))
    o = delta_recurrence(q * d ** -0.5, k, v.view(n, heads, dv), g, beta)
    gate = sigmoid((h @ w[pre + "g1"].T) @ w[pre + "g2"].T)
    o = rms(o, eps) * w[pre + "norm"]
    return (o.reshape(n, -1) * gate) @ w[pre + "o"].T


def parallel_mixer(w, pre, m, h, eps):
    return m["left_scale"] * window_attention(w, pre + "left.", m["left"], h) \
        + m["right_scale"] * delta_mixer(w, pre + "right.", m["right"], h, eps)


def selective_scan(x, dt, a, b, c, d):
    """x, dt [n, C], a [C, N], b and c [n, N], d [C]."""
    s = torch.zeros_like(a)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        s = torch.exp(dt[t][:, None] * a) * s \
            + (dt[t] * x[t])[:, None] * b[t][None]
        out[t] = s @ c[t] + d * x[t]
    return out


def mamba_mixer(w, pre, m, h):
    inner, rank, n = m["inner"], m["dt_rank"], m["state"]
    p = h @ w[pre + "in"].T
    x, z = p[:, :inner], p[:, inner:]
    x = silu(short_conv(x, w[pre + "conv"]) + w[pre + "conv.b"])
    low = x @ w[pre + "x"].T
    dt = softplus(low[:, :rank] @ w[pre + "dt"].T + w[pre + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[pre + "A_log"]),
                       low[:, rank:rank + n], low[:, rank + n:], w[pre + "D"])
    return (y * silu(z)) @ w[pre + "o"].T


def lightning_recurrence(q, k, v, decay):
    n, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(n):
        for h in range(heads):
            s[h] = decay[h] * s[h] + torch.outer(k[t, h], v[t, h])
            out[t, h] = s[h].T @ q[t, h]
    return out


def lightning_mixer(w, pre, m, h, eps):
    n, heads = h.shape[0], m["heads"]
    q, k, v = (silu(h @ w[pre + p].T).view(n, heads, -1)
               for p in ("q", "k", "v"))
    o = lightning_recurrence(q, k, v, m["decay"]).reshape(n, -1)
    return (rms(o, eps) * w[pre + "norm"] * sigmoid(h @ w[pre + "g"].T)) \
        @ w[pre + "o"].T


def mixer(w, pre, layer, h, eps):
    m = layer["mixer"]
    if layer["type"] == "mamba1":
        return mamba_mixer(w, pre, m, h)
    if layer["type"] == "lightning":
        return lightning_mixer(w, pre, m, h, eps)
    assert layer["type"] == "parallel"
    return parallel_mixer(w, pre, m, h, eps)


def relu_glu(w, pre, h):
    return ((h @ w[pre + "gate"].T).clamp(min=0) * (h @ w[pre + "up"].T)) \
        @ w[pre + "down"].T


def clamped_glu(w, pre, h, limit):
    g = (h @ w[pre + "gate"].T).clamp(max=limit)
    u = (h @ w[pre + "up"].T).clamp(-limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ w[pre + "down"].T


def route(z, top):
    """Scores z of one token -> {expert: weight}."""
    chosen = sorted(range(len(z)), key=lambda e: -float(z[e]))[:top]
    p = torch.exp(z[chosen] - z[chosen].max())
    p = p / p.sum()
    return {e: p[i] for i, e in enumerate(chosen)}


def experts(w, pre, mlp, h):
    out = torch.zeros_like(h)
    z = h @ w[pre + "router"].T + w[pre + "router.b"]
    for t in range(h.shape[0]):
        for e, weight in route(z[t], mlp["router"]["top"]).items():
            out[t] += weight * clamped_glu(w, f"{pre}e{e}.", h[t],
                                           mlp["expert"]["limit"])
    if mlp.get("shared"):
        out = out + clamped_glu(w, pre + "shared.", h, mlp["shared"]["limit"])
    return out


def feed_forward(w, pre, mlp, h):
    if mlp is None:
        return 0
    if mlp["kind"] == "dense":
        return relu_glu(w, pre, h)
    return experts(w, pre, mlp, h)


def passes(cfg):
    """[(layer, number of the pass it begins, or None)] in the order they
    run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": n, "stop": n, "times": 0}
    run = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        for i in range(loop["start"], loop["stop"]):
            run.append((i, t if i == loop["start"] else None))
    return run + [(i, None) for i in range(loop["stop"], n)]


def begin_pass(w, x, embedded, t):
    return x + (embedded if t else 0) + w["loop.step"][t]


def forward(cfg, weights, tokens, streams=None):
    """Logits [n, vocab]; appends the residual after each layer run to
    `streams`."""
    w = {k: t.to(F64) if t.is_floating_point() else t
         for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    embedded = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x = embedded
    for i, t in passes(cfg):
        if t is not None:
            x = begin_pass(w, x, embedded, t)
        p, layer = f"l{i}.", cfg["layers"][i]
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        x = x + mixer(w, p + "mix.", layer, h, eps) \
            + feed_forward(w, p + "mlp.", layer["mlp"], h)
        if streams is not None:
            streams.append(x.clone())
    h = layer_norm(x, w["final.norm"], w["final.norm.b"], eps)
    return softcap(h @ w["head"].T, cfg["logit_softcap"])
