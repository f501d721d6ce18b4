"""Reference (plain PyTorch, fp32-accumulating) implementations of every op the
HIP kernel library provides.

These are the numerics oracle for the kernel parity tests (a HIP
kernel's test compares it against a plain PyTorch fp32 reference of the same op)
and the CPU execution path for control-plane/system tests on machines without a
GPU. On a ROCm GPU the dispatch layer (substratus_amd/ops/__init__.py) refuses
to fall back to these: the HIP extension is mandatory there.
"""

from __future__ import annotations

import math
from typing import Optional

import torch


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """y = x / rms(x) * weight, accumulating in fp32."""
    xf = x.float()
    var = xf.pow(2).mean(dim=-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps) * weight.float()
    return y.to(x.dtype)


def layer_norm(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor,
               eps: float) -> torch.Tensor:
    return torch.nn.functional.layer_norm(
        x.float(), (x.shape[-1],), weight.float(), bias.float(), eps).to(x.dtype)


def rope_cos_sin(positions: torch.Tensor, head_dim: int, theta: float,
                 dtype: torch.dtype = torch.float32) -> tuple[torch.Tensor, torch.Tensor]:
    """cos/sin tables [N, head_dim/2] for the given positions (fp32)."""
    inv_freq = 1.0 / (theta ** (torch.arange(0, head_dim, 2,
                      dtype=torch.float32, device=positions.device) / head_dim))
    ang = positions.float()[:, None] * inv_freq[None, :]
    return ang.cos(), ang.sin()


def apply_rope(x: torch.Tensor, positions: torch.Tensor, theta: float) -> torch.Tensor:
    """Neox-style rotary embedding. x: [N, H, D]; positions: [N].
    theta <= 0 disables rotation (opt-style models)."""
    if theta <= 0:
        return x
    n, h, d = x.shape
    cos, sin = rope_cos_sin(positions, d, theta)
    xf = x.float()
    x1, x2 = xf[..., : d // 2], xf[..., d // 2:]
    cos = cos[:, None, :]
    sin = sin[:, None, :]
    out = torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1)
    return out.to(x.dtype)


def rope_kv_append(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                   positions: torch.Tensor, k_cache: torch.Tensor,
                   v_cache: torch.Tensor, slots: torch.Tensor,
                   theta: float) -> torch.Tensor:
    """Apply RoPE to q and k (in fp32), then scatter k,v into the paged cache.

    q: [N, Hq, D]; k, v: [N, Hkv, D]; positions: [N] int32 (absolute position,
    drives RoPE); slots: [N] int32/int64 flat slot index = block_id * block_size
    + offset into k_cache/v_cache of shape [num_blocks, Hkv, block_size, D].
    Returns the rotated q. k_cache/v_cache are written in place.
    """
    q_out = apply_rope(q, positions, theta)
    k_rot = apply_rope(k, positions, theta)
    k.copy_(k_rot)  # k is rotated IN PLACE too (prefill consumes it dense)
    num_blocks, hkv, block_size, d = k_cache.shape
    blk = torch.div(slots, block_size, rounding_mode="floor").long()
    off = (slots % block_size).long()
    k_cache[blk, :, off, :] = k_rot.to(k_cache.dtype)
    v_cache[blk, :, off, :] = v.to(v_cache.dtype)
    return q_out


def kv_append(k: torch.Tensor, v: torch.Tensor, k_cache: torch.Tensor,
              v_cache: torch.Tensor, slots: torch.Tensor) -> None:
    """Scatter pre-rotated k,v into the paged cache (no RoPE)."""
    block_size = k_cache.shape[2]
    blk = torch.div(slots, block_size, rounding_mode="floor").long()
    off = (slots % block_size).long()
    k_cache[blk, :, off, :] = k.to(k_cache.dtype)
    v_cache[blk, :, off, :] = v.to(v_cache.dtype)


def paged_attn_decode(q: torch.Tensor, k_cache: torch.Tensor,
                      v_cache: torch.Tensor, block_table: torch.Tensor,
                      seq_lens: torch.Tensor, scale: float) -> torch.Tensor:
    """Single-token decode attention over a block-paged KV cache.

    q: [B, Hq, D]; k_cache/v_cache: [num_blocks, Hkv, block_size, D];
    block_table: [B, max_blocks] int32; seq_lens: [B] int32 (length INCLUDING
    the current token, whose k/v are already in the cache).
    Returns [B, Hq, D] in q.dtype; softmax/accumulation in fp32.
    """
    bsz, hq, d = q.shape
    num_blocks, hkv, block_size, _ = k_cache.shape
    group = hq // hkv
    out = torch.empty_like(q)
    for b in range(bsz):
        n = int(seq_lens[b])
        nblk = (n + block_size - 1) // block_size
        blocks = block_table[b, :nblk].long()
        k = k_cache[blocks].permute(1, 0, 2, 3).reshape(hkv, nblk * block_size, d)[:, :n]
        v = v_cache[blocks].permute(1, 0, 2, 3).reshape(hkv, nblk * block_size, d)[:, :n]
        qb = q[b].float().view(hkv, group, d)
        scores = torch.einsum("hgd,hnd->hgn", qb, k.float()) * scale
        p = torch.softmax(scores, dim=-1)
        ob = torch.einsum("hgn,hnd->hgd", p, v.float())
        out[b] = ob.reshape(hq, d).to(q.dtype)
    return out


def attn_prefill(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                 seq_start: torch.Tensor, scale: float,
                 causal: bool = True) -> torch.Tensor:
    """Varlen causal prefill attention over packed sequences.

    q: [T, Hq, D]; k, v: [T, Hkv, D]; seq_start: [num_seqs+1] int32 cumulative
    token offsets. fp32 softmax/accum.
    """
    t, hq, d = q.shape
    hkv = k.shape[1]
    group = hq // hkv
    out = torch.empty_like(q)
    for s in range(seq_start.numel() - 1):
        a, b = int(seq_start[s]), int(seq_start[s + 1])
        n = b - a
        qs = q[a:b].float().view(n, hkv, group, d)
        ks = k[a:b].float()
        vs = v[a:b].float()
        scores = torch.einsum("ihgd,jhd->hgij", qs, ks) * scale
        if causal:
            mask = torch.full((n, n), float("-inf"), device=q.device).triu(1)
            scores = scores + mask
        p = torch.softmax(scores, dim=-1)
        o = torch.einsum("hgij,jhd->ihgd", p, vs)
        out[a:b] = o.reshape(n, hq, d).to(q.dtype)
    return out


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    """x: [..., 2F] (gate ‖ up) -> silu(gate) * up, fp32 math."""
    gate, up = x.float().chunk(2, dim=-1)
    return (torch.nn.functional.silu(gate) * up).to(x.dtype)


def gelu(x: torch.Tensor) -> torch.Tensor:
    return torch.nn.functional.gelu(x.float(), approximate="tanh").to(x.dtype)


def softmax_sample(logits: torch.Tensor, temperature: torch.Tensor,
                   top_k: torch.Tensor, top_p: torch.Tensor,
                   uniform: torch.Tensor) -> torch.Tensor:
    """Temperature / top-k / top-p sampling of one token per row.

    logits: [B, V] (any float dtype); temperature/top_p: [B] fp32 (temperature
    <= 0 means greedy); top_k: [B] int32 (0 = disabled); uniform: [B] fp32 in
    [0,1) — the random draw, passed in so GPU and reference sample identically.
    Returns [B] int64 token ids.
    """
    bsz, vocab = logits.shape
    out = torch.empty(bsz, dtype=torch.int64, device=logits.device)
    lf = logits.float()
    for b in range(bsz):
        row = lf[b]
        t = float(temperature[b])
        if t <= 0.0:
            out[b] = int(torch.argmax(row))
            continue
        row = row / t
        k = int(top_k[b])
        if 0 < k < vocab:
            kth = torch.topk(row, k).values[-1]
            row = torch.where(row < kth, torch.full_like(row, float("-inf")), row)
        p = torch.softmax(row, dim=-1)
        tp = float(top_p[b])
        if 0.0 < tp < 1.0:
            sp, idx = torch.sort(p, descending=True)
            cum = torch.cumsum(sp, 0)
            keep = cum - sp < tp  # keep tokens until cumulative prob >= top_p
            sp = torch.where(keep, sp, torch.zeros_like(sp))
            sp = sp / sp.sum()
            # inverse-cdf draw on the sorted distribution
            j = int(torch.searchsorted(torch.cumsum(sp, 0), uniform[b], right=False).clamp(max=vocab - 1))
            out[b] = int(idx[j])
        else:
            j = int(torch.searchsorted(torch.cumsum(p, 0), uniform[b], right=False).clamp(max=vocab - 1))
            out[b] = j
    return out


def cross_entropy_fwd_bwd(logits: torch.Tensor, targets: torch.Tensor,
                          ignore_index: int = -100) -> tuple[torch.Tensor, torch.Tensor]:
    """Fused log-softmax + NLL + dlogits (mean over non-ignored targets).

    logits: [N, V] (bf16/fp32); targets: [N] int64. Returns (scalar fp32 loss,
    dlogits in logits.dtype). dlogits = (softmax - onehot)/n_valid.
    """
    lf = logits.float()
    valid = targets != ignore_index
    n_valid = int(valid.sum())
    lse = torch.logsumexp(lf, dim=-1)
    tclamped = targets.clamp(min=0)
    tlogit = lf.gather(1, tclamped[:, None]).squeeze(1)
    losses = (lse - tlogit) * valid
    loss = losses.sum() / max(n_valid, 1)
    p = torch.softmax(lf, dim=-1)
    p.scatter_add_(1, tclamped[:, None],
                   -torch.ones_like(tlogit)[:, None])
    dlogits = p * (valid[:, None] / max(n_valid, 1))
    return loss, dlogits.to(logits.dtype)


def adamw_step(param: torch.Tensor, grad: torch.Tensor, exp_avg: torch.Tensor,
               exp_avg_sq: torch.Tensor, lr: float, beta1: float, beta2: float,
               eps: float, weight_decay: float, step: int,
               grad_scale: float = 1.0) -> None:
    """One fused AdamW update, in place. param may be bf16 (master-less);
    exp_avg/exp_avg_sq are fp32. Decoupled weight decay. grad_scale folds
    gradient clipping into the read of g."""
    g = grad.float() * grad_scale
    exp_avg.mul_(beta1).add_(g, alpha=1 - beta1)
    exp_avg_sq.mul_(beta2).addcmul_(g, g, value=1 - beta2)
    bc1 = 1 - beta1 ** step
    bc2 = 1 - beta2 ** step
    pf = param.float()
    pf.mul_(1 - lr * weight_decay)
    denom = (exp_avg_sq / bc2).sqrt().add_(eps)
    pf.addcdiv_(exp_avg / bc1, denom, value=-lr)
    param.copy_(pf.to(param.dtype))


# ---- hybrid models (ops/hybrid.py) ------------------------------------------

def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def stream_norm(rows, at, weights, x, w_post, w_pre, offset, eps,
                out_scale=1.0, mult=1.0):
    delta = rows.float() if at is None else \
        (rows[at.long()].float() * weights[:, :, None]).sum(1)
    x += mult * _rms(delta, eps) * (offset + w_post)
    y = x if w_pre is None else _rms(x, eps) * ((offset + w_pre) * out_scale)
    return y.to(rows.dtype, copy=True)


def embed_norm(tokens, table, w_pre, offset, eps, scale=1.0, pos=None,
               positions=None):
    x = table[tokens.long()].float() * scale
    if pos is not None:
        x += pos[positions.long()].float()
    y = x if w_pre is None else _rms(x, eps) * (offset + w_pre)
    return x, y.to(table.dtype, copy=True)


def add_norm(x, rows, at, weights, pool, tokens, table, scale, vec, w, b, eps,
             dtype):
    if rows is not None:
        x += rows.float()
    if pool is not None:
        x += (pool[at.long()].float() * weights[:, :, None]).sum(1)
    if table is not None:
        x += table[tokens.long()].float() * scale
    if vec is not None:
        x += vec
    if b is None:
        return (_rms(x, eps) * w).to(dtype)
    d = x - x.mean(-1, keepdim=True)
    return (_rms(d, eps) * w + b).to(dtype)


def softcap(x, cap):
    x.copy_(cap * torch.tanh(x.float() / cap))


def rope_table(positions, turns):
    t = positions.double()[:, None] * turns
    a = ((t - t.round()) * (2 * math.pi)).float()
    return torch.stack([a.cos(), a.sin()], -1)


def short_conv(out, x, in_bias, weight, bias, act, state, state_slots,
               positions, seq_start, max_len):
    taps = weight.shape[1]
    for e, (a, b) in enumerate(_entry_rows(seq_start, x.shape[0])):
        slot = int(state_slots[e])
        u = x[a:b].float() if in_bias is None else x[a:b].float() + in_bias
        old = torch.zeros(taps - 1, x.shape[1], device=x.device)
        if slot >= 0 and int(positions[a]) > 0:
            old = state[slot].float()
            # inputs before the sequence's start are zeros, not biases
            n = min(taps - 1, int(positions[a]))
            if in_bias is not None and n:
                old = old.clone()
                old[taps - 1 - n:] += in_bias
        held = torch.cat([old, u])
        y = sum(held[j:j + b - a] * weight[:, j] for j in range(taps))
        if bias is not None:
            y = y + bias
        if slot >= 0 and taps > 1:
            raw = torch.cat([state[slot] if int(positions[a]) > 0 else
                             torch.zeros_like(state[slot]),
                             x[a:b].to(state.dtype)])
            state[slot] = raw[-(taps - 1):]
        out[a:b] = (torch.nn.functional.silu(y) if act else y).to(out.dtype)


def conv_rope(q, buf, in_bias, weight, state, state_slots, rope, k_cache,
              v_cache, positions, slots, seq_start, max_len):
    rows = weight.shape[0]
    y = torch.empty(buf.shape[0], rows, device=buf.device)
    short_conv(y, buf[:, :rows], in_bias, weight, None, False, state,
               state_slots, positions, seq_start, max_len)
    kv, dim = k_cache.shape[1], k_cache.shape[3]
    y = y.view(buf.shape[0], -1, dim)
    v = y[:, -kv:].clone()
    half = rope.shape[1]
    cos, sin = rope[:, None, :, 0], rope[:, None, :, 1]
    a, b = y[..., 0:2 * half:2].clone(), y[..., 1:2 * half:2].clone()
    y[..., 0:2 * half:2] = a * cos - b * sin
    y[..., 1:2 * half:2] = b * cos + a * sin
    q.copy_(y[:, :-kv].reshape(q.shape).to(q.dtype))
    kv_append(y[:, -kv:], v, k_cache, v_cache, slots)


def conv_qkv(q, buf, in_bias, weight, state, state_slots, k_cache, v_cache,
             positions, slots, seq_start, coef, every, v_eps, max_len):
    rows, kv = weight.shape[0], k_cache.shape[1]
    y = torch.empty(buf.shape[0], rows, device=buf.device)
    short_conv(y, buf[:, :rows], in_bias, weight, None, False, state,
               state_slots, positions, seq_start, max_len)
    yq, k, v = y.split([q.shape[1], kv * k_cache.shape[3],
                        kv * v_cache.shape[3]], dim=1)
    steps = torch.div(positions + 1, every, rounding_mode="floor")
    q.copy_((yq * (1 + coef * torch.log1p(steps.float()))[:, None]).to(
        q.dtype))
    v = v.reshape(-1, kv, v_cache.shape[3])
    kv_append(k.reshape(-1, kv, k_cache.shape[3]),
              v if v_eps < 0 else _rms(v, v_eps), k_cache, v_cache, slots)


def selective_scan(out, u, gate, z, z_bias, low, b_at, a, d, state,
                   state_slots, positions, seq_start, max_len, recurrent):
    n = a.shape[1]
    dt = torch.nn.functional.softplus(z + z_bias)
    x, lowf = u.float(), low[:, b_at:b_at + 2 * n].float()
    for e, (r0, r1) in enumerate(_entry_rows(seq_start, u.shape[0])):
        slot = int(state_slots[e])
        s = torch.zeros_like(a) if slot < 0 or int(positions[r0]) == 0 \
            else state[slot]
        for t in range(r0, r1):
            s = torch.exp(dt[t][:, None] * a) * s \
                + (dt[t] * x[t])[:, None] * lowf[t, :n]
            y = s @ lowf[t, n:] + d * x[t]
            out[t] = (y * torch.nn.functional.silu(gate[t].float())).to(
                out.dtype)
        if slot >= 0:
            state[slot] = s


def lightning(out, x, decay, state, state_slots, positions, seq_start,
              max_len, recurrent):
    _, heads, dim, vdim = state.shape
    f = torch.nn.functional.silu(x[:, :heads * (2 * dim + vdim)].float()).to(
        x.dtype).float()
    q, k, v = f.split([heads * dim] * 2 + [heads * vdim], dim=1)
    q, k = (t.reshape(-1, heads, dim, 1) for t in (q, k))
    v = v.reshape(-1, heads, 1, vdim)
    for e, (a, b) in enumerate(_entry_rows(seq_start, x.shape[0])):
        slot = int(state_slots[e])
        s = torch.zeros(heads, dim, vdim, device=x.device) \
            if slot < 0 or int(positions[a]) == 0 else state[slot]
        for t in range(a, b):
            s = decay[:, None, None] * s + k[t] * v[t]
            out[t] = (s * q[t]).sum(1).reshape(-1).to(out.dtype)
        if slot >= 0:
            state[slot] = s


def joint_gate(out, o, norm, gate, eps):
    y = _rms(o.float(), eps) * norm * torch.sigmoid(gate.float())
    out.copy_(y.to(out.dtype))


def delta(out, qkv, z, z_bias, rate, beta, norm, gate, state, state_slots,
          positions, seq_start, kv_heads, eps, mult, max_len, recurrent):
    _, heads, dim, vdim = state.shape
    f = qkv.float()
    q, k, v = f.split([kv_heads * dim] * 2 + [heads * vdim], dim=1)

    def unit(t):
        t = t.reshape(-1, kv_heads, dim)
        t = t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6)
        return t.repeat_interleave(heads // kv_heads, 1)[..., None]
    q, k = unit(q) * dim ** -0.5, unit(k)
    v = v.reshape(-1, heads, vdim)
    g = torch.exp(-rate[:, None] * torch.nn.functional.softplus(
        z + z_bias).view(-1, heads, dim))[..., None]
    b = torch.sigmoid(beta.float())[..., None]
    for e, (r0, r1) in enumerate(_entry_rows(seq_start, qkv.shape[0])):
        slot = int(state_slots[e])
        s = torch.zeros(heads, dim, vdim, device=f.device) \
            if slot < 0 or int(positions[r0]) == 0 else state[slot]
        for t in range(r0, r1):
            s = g[t] * s
            new = b[t] * (v[t] - (s * k[t]).sum(1))
            s = s + k[t] * new[:, None]
            o = _rms((s * q[t]).sum(1), eps) * norm
            o = o.reshape(-1) * torch.sigmoid(gate[t].float()) * mult
            out[t] = o.to(out.dtype)
        if slot >= 0:
            state[slot] = s


def glu_values(g, u, act, limit):
    if act == "clamped":
        g, u = g.clamp(max=limit), u.clamp(-limit, limit) + 1
        return g * torch.sigmoid(1.702 * g) * u
    return (g.clamp(min=0) if act == "relu"
            else torch.nn.functional.silu(g)) * u


def glu(out, x, act, limit):
    out.copy_(glu_values(*x.float().chunk(2, dim=-1), act, limit).to(
        out.dtype))


def _rotate(x, turns, positions):
    """x [rows, ..., n] float, its first 2 * len(turns) elements turned."""
    half = turns.shape[0]
    t = positions.double()[:, None] * turns
    a = ((t - t.round()) * (2 * math.pi)).float()
    a = a.view(x.shape[0], *[1] * (x.dim() - 2), half)
    u, v = x[..., :half].clone(), x[..., half:2 * half].clone()
    x[..., :half] = u * a.cos() - v * a.sin()
    x[..., half:2 * half] = v * a.cos() + u * a.sin()
    return x


def latent_prepare(buf, heads, dim, rot_dim, c_at, norm, eps, turns,
                   positions, cache, slots, q_norm=None):
    if q_norm is not None:
        n = q_norm.shape[0]
        buf[:, :n] = (_rms(buf[:, :n].float(), eps) * q_norm).to(buf.dtype)
    elif rot_dim:
        n = heads * (dim + rot_dim)
        q = buf[:, :n].to(torch.float32, copy=True).view(-1, heads,
                                                         dim + rot_dim)
        _rotate(q[..., dim:], turns, positions)
        buf[:, :n] = q.view(-1, n).to(buf.dtype)
    if c_at < 0:
        return
    rank = norm.shape[0]
    row = buf[:, c_at:c_at + rank + rot_dim].to(torch.float32, copy=True)
    row = torch.cat([_rms(row[:, :rank], eps) * norm,
                     _rotate(row[:, rank:], turns, positions)], 1)
    bs = cache.shape[2]
    cache[slots.long() // bs, 0, slots.long() % bs] = row.to(cache.dtype)


def head_linear(out, x, w, gate, tail):
    k = w.shape[2]
    o = torch.matmul(x[..., :k].float().transpose(0, 1).contiguous(),
                     w.float().transpose(1, 2).contiguous()).transpose(0, 1)
    if gate is not None:
        o = o * torch.sigmoid(gate.float()).reshape(*o.shape[:2], -1)
    out[..., :w.shape[1]] = o.to(out.dtype)
    if tail:
        out[..., w.shape[1]:] = x[..., k:k + tail]


def moe_select(z, top, groups, keep, over_chosen=False, sigmoid=False,
               correction=None, group_best=1):
    """(ids [rows, top] int32, weights float32), best first, of scores z."""
    s = torch.sigmoid(z) if sigmoid else torch.softmax(z, -1)
    if sigmoid:
        z = s
    if correction is not None:
        z = z + correction
    size = s.shape[1] // groups
    best = z.view(-1, groups, size).topk(min(group_best, size), -1) \
        .values.sum(-1)
    kept = torch.zeros_like(best, dtype=torch.bool).scatter_(
        1, best.topk(keep, 1).indices, True)
    kept = kept.repeat_interleave(size, 1)
    chosen, ids = z.masked_fill(~kept, float("-inf")).topk(top, 1)
    return ids.int(), torch.softmax(chosen, -1) if over_chosen \
        else s.gather(1, ids)


def experts(y, router, bias, up, down, spec, correction=None):
    """(rows, at, weights) of the chosen experts' outputs, token by token.
    Gated experts' matrices have the rows of gate and up in turn."""
    f, top = y.float(), spec.top
    z = f @ router.float().T
    if bias is not None:
        z = z + bias
    ids, weights = moe_select(z, top, spec.groups, spec.keep,
                              spec.over_chosen, spec.sigmoid, correction,
                              spec.group_best)
    out = y.new_zeros(y.shape[0] * top, y.shape[1])
    flat = ids.reshape(-1)
    for e in flat.unique().tolist():
        r = (flat == e).nonzero()[:, 0]
        h = f[r // top] @ up[e].float().T
        h = torch.nn.functional.gelu(h) if spec.glu is None else glu_values(
            h[:, ::2], h[:, 1::2], spec.glu.act, spec.glu.limit)
        out[r] = (h.to(y.dtype).float() @ down[e].float().T).to(y.dtype)
    at = torch.arange(flat.shape[0], dtype=torch.int32).view(-1, top)
    return out, at.to(y.device), weights


def side_gate(out, y, w, tokens, table, at):
    z = torch.nn.functional.gelu(y.float() @ w.float().T, approximate="tanh")
    e = table[tokens.long(), at:at + w.shape[0]].float()
    out.copy_((z * e).to(out.dtype))


def qkv_prepare(buf, nq, q_norm, k_norm, eps, v_first, lam, k_cache, v_cache,
                slots):
    kv, dim, vdim = k_cache.shape[1], k_cache.shape[3], v_cache.shape[3]
    nk, nv = kv * dim, kv * vdim
    q, k, v = (t.float() for t in
               buf[:, :nq + nk + nv].split([nq, nk, nv], dim=1))
    if q_norm is not None:
        q, k = _rms(q, eps) * q_norm, _rms(k, eps) * k_norm
        buf[:, :nq] = q.to(buf.dtype)
    if v_first is not None:
        v = (1 - lam) * v + lam * v_first.float()
    kv_append(k.view(-1, kv, dim), v.view(-1, kv, vdim), k_cache, v_cache,
              slots)


def _entry_rows(seq_start, rows):
    if seq_start is None:
        return [(i, i + 1) for i in range(rows)]
    s = seq_start.tolist()
    return list(zip(s[:-1], s[1:]))


def attn_ctx(out, q, gate, k_cache, v_cache, bias, sink, positions, seq_start,
             block_table, scale, chunk, window, keep, cap, mult, max_len, span,
             any_size, r1=None, r2=None, weight_bias=None):
    kv, bs, dim = k_cache.shape[1:]
    vdim = v_cache.shape[3]
    for e, (a, b) in enumerate(_entry_rows(seq_start, q.shape[0])):
        pos = positions[a:b].long()
        n = int(pos[-1]) + 1
        blocks = block_table[e, :(n + bs - 1) // bs].long()
        k, v = (c[blocks].transpose(1, 2).reshape(-1, kv, c.shape[3])[:n]
                .float() for c in (k_cache, v_cache))
        qe = q[a:b].float().view(b - a, kv, -1, dim)
        s = torch.einsum("ikgd,jkd->kgij", qe, k) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        dist = pos[:, None] - torch.arange(n, device=pos.device)
        if bias is not None:
            s = s + bias[:, dist.clamp(0, bias.shape[1] - 1)].view(
                kv, -1, b - a, n)
        if r1 is not None:
            fall = r1[:, None, None] * torch.log1p(
                r2[:, None, None] * dist.clamp(0))
            s = s - fall.view(kv, -1, b - a, n)
        seen = dist >= 0
        if chunk:
            seen &= (pos // chunk)[:, None] == torch.arange(
                n, device=pos.device) // chunk
        if window:
            seen &= (dist < window) | (torch.arange(
                n, device=pos.device) < keep)
        s = s.masked_fill(~seen, float("-inf"))
        if sink is not None:    # a key without a value
            s = torch.cat([s, sink.view(kv, -1, 1, 1).expand(
                kv, s.shape[1], b - a, 1)], -1)
        p = torch.softmax(s, -1)[..., :n] if weight_bias is None else \
            torch.sigmoid(s + weight_bias.view(kv, -1, 1, 1))
        o = torch.einsum("kgij,jkd->ikgd", p, v).reshape(b - a, -1, vdim)
        if gate is not None:
            o = o * torch.sigmoid(gate[a:b].float())[:, :, None]
        out[a:b] = (o.reshape(b - a, -1) * mult).to(out.dtype)


def gla(out, x, a2, a2_bias, norm, state, state_slots, positions, seq_start,
        inv_tau, eps, max_len, recurrent):
    _, heads, dim, vdim = state.shape
    f = x.float()
    q, k, v, g, a1 = f[:, :2 * heads * (dim + vdim) + a2.shape[1]].split(
        [heads * dim] * 2 + [heads * vdim] * 2 + [a2.shape[1]], dim=1)
    alpha = torch.exp(torch.nn.functional.logsigmoid(a1 @ a2.T + a2_bias)
                      * inv_tau).view(-1, heads, dim, 1)
    q = q.view(-1, heads, dim, 1) * dim ** -0.5
    k = k.view(-1, heads, dim, 1)
    v = v.view(-1, heads, 1, vdim)
    for e, (a, b) in enumerate(_entry_rows(seq_start, x.shape[0])):
        slot = int(state_slots[e])
        s = torch.zeros(heads, dim, vdim, device=x.device) \
            if slot < 0 or int(positions[a]) == 0 else state[slot]
        for t in range(a, b):
            s = alpha[t] * s + k[t] * v[t]
            o = _rms((s * q[t]).sum(1), eps) * norm
            out[t] = (o.reshape(-1) * torch.nn.functional.silu(g[t])).to(
                out.dtype)
        if slot >= 0:
            state[slot] = s
