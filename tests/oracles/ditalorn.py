"""Plain, slow Ditalorn in float64: one function per mechanism, loops where a
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


def rms(x, eps):
    """x over its root mean square (last axis), eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, weight, eps):
    """RMS norm; the weight is stored around zero."""
    return rms(x, eps) * (1 + weight)


def embed(w, toks, scale):
    n = len(toks)
    return w["embed"][toks] * scale + w["pos"][:n]


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


def projected(w, name, h):
    """A projection with its bias, then its convolution over time."""
    return short_conv(h @ w[name].T + w[name + ".b"], w[name + ".conv"])


def temperature(p, coef, every):
    return 1 + coef * math.log((p + 1) // every + 1)


def distance_penalty(n, r1, r2):
    return r1 * math.log(1 + r2 * n)


def value_norm(v, eps):
    """Each head's value [..., vdim] over its root mean square."""
    return rms(v, eps)


def causal(i, j):
    return j <= i


def attend_sigmoid(q, k, v, scale, r1, r2, pb):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]; weights do not
    sum to anything in particular."""
    n, heads, _ = q.shape
    per = heads // k.shape[1]
    out = torch.zeros(n, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        fall = torch.tensor([distance_penalty(m, float(r1[h]), float(r2[h]))
                             for m in range(n)], dtype=q.dtype)
        for i in range(n):
            js = [j for j in range(n) if causal(i, j)]
            s = (k[js, h // per] @ q[i, h]) * scale
            s = s - fall[[i - j for j in js]] + pb[h]
            out[i, h] = sigmoid(s) @ v[js, h // per]
    return out


def attention(w, pre, m, h, eps):
    n, heads, kv, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], \
        m["vdim"]
    q, k, v = (projected(w, pre + p, h) for p in ("q", "k", "v"))
    t = torch.tensor([temperature(p, m["q_temp"]["coef"],
                                  m["q_temp"]["every"]) for p in range(n)],
                     dtype=h.dtype)
    q, k = (q * t[:, None]).view(n, heads, d), k.view(n, kv, d)
    v = value_norm(v.view(n, kv, dv), eps)
    o = attend_sigmoid(q, k, v, m["scale"], w[pre + "r1"], w[pre + "r2"],
                       w[pre + "pb"])
    return o.reshape(n, -1) @ w[pre + "o"].T + w[pre + "o.b"]


def windowed(i, j, size):
    return 0 <= i - j < size


def attend(q, k, v, scale, size):
    """q, k [n, H, d], v [n, H, dv] -> [n, H, dv], over a window of keys."""
    n, heads, _ = q.shape
    out = torch.zeros(n, heads, v.shape[2], dtype=q.dtype)
    for i in range(n):
        js = [j for j in range(n) if windowed(i, j, size)]
        for h in range(heads):
            s = (k[js, h] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[js, h]
    return out


def query_latent(w, pre, h, eps):
    return rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]


def latent(w, pre, h, eps):
    """What the cache of a layer holds."""
    return rms(h @ w[pre + "dkv"].T, eps) * w[pre + "dkv.norm"]


def head_gate(w, pre, h):
    """[n, heads]: a factor of each head's output."""
    return sigmoid(h @ w[pre + "g"].T)


def latent_attention(w, pre, m, h, eps):
    n, heads, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (query_latent(w, pre, h, eps) @ w[pre + "uq"].T).view(n, heads, d)
    c = latent(w, pre, h, eps)
    k = (c @ w[pre + "uk"].T).view(n, heads, d)
    v = (c @ w[pre + "uv"].T).view(n, heads, dv)
    o = attend(q, k, v, m["scale"], m["mask"]["size"])
    o = o * head_gate(w, pre, h)[:, :, None]
    return o.reshape(n, -1) @ w[pre + "o"].T


def group_score(choice):
    """Of one group's choice scores, a list."""
    return sum(sorted(choice, reverse=True)[:2])


def route(z, correction, router):
    """Scores z of one token -> {expert: weight}."""
    s = sigmoid(z)
    choice = (s + correction).tolist()
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = len(choice) // groups["count"]
    best = [group_score(choice[g * size:(g + 1) * size])
            for g in range(groups["count"])]
    kept = sorted(range(len(best)), key=lambda g: -best[g])[:groups["keep"]]
    open_ = [e for e in range(len(choice)) if e // size in kept]
    chosen = sorted(open_, key=lambda e: -choice[e])[:router["top"]]
    return {e: s[e] for e in chosen}


def expert(w, pre, x):
    return (silu(x @ w[pre + "gate"].T) * (x @ w[pre + "up"].T)) \
        @ w[pre + "down"].T


def experts(w, pre, router, h):
    out = torch.zeros_like(h)
    z = h @ w[pre + "router"].T
    for t in range(h.shape[0]):
        for e, weight in route(z[t], w[pre + "correction"], router).items():
            out[t] += weight * expert(w, f"{pre}e{e}.", h[t])
    return out


def forward(cfg, weights, tokens, streams=None):
    """Logits [n, vocab]; appends the residual after each layer to `streams`."""
    w = {k: t.to(F64) if t.is_floating_point() else t
         for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = embed(w, torch.as_tensor(tokens), cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixer = {"attention": attention,
                 "latent_attention": latent_attention}[layer["type"]]
        y = mixer(w, p + "mix.", layer["mixer"], norm(x, w[p + "norm1"], eps),
                  eps)
        x = x + norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            y = experts(w, p + "mlp.", layer["mlp"]["router"],
                        norm(x, w[p + "norm2"], eps))
            x = x + norm(y, w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return norm(x, w["final.norm"], eps) @ w["embed"].T
