"""Ops of models whose layers differ from one another (models/hybrid.py):
norms around a 32-bit residual, attention that reads the paged cache for
single tokens and prompt portions alike, attention over a cache of latents,
linear attention, delta-rule and selective-scan recurrences with a state per
request, short convolutions over time, mixtures of experts.

Same policy as the rest of ops: GPU tensors need the HIP extension
(substratus_amd._hybrid), CPU tensors run the plain implementations in ref.py.
Activations are float32 or bfloat16; residual, norm weights, biases, decay
weights and recurrent state are always float32.
"""

from __future__ import annotations

from typing import NamedTuple, Optional, Union

import torch

from . import linear, ref

_EXT = None


def _ext():
    global _EXT
    if _EXT is None:
        try:
            from substratus_amd import _hybrid
        except ImportError as e:
            raise RuntimeError(
                "substratus_amd/_hybrid*.so is not built but a GPU tensor was "
                "passed — no eager fallback on GPU. Build it with `python "
                f"setup.py build_ext --inplace`. Import error: {e}") from e
        _EXT = _hybrid
    return _EXT


class Picked(NamedTuple):
    """Rows of a sum: token t has sum_k weights[t, k] * rows[at[t, k]]."""
    rows: torch.Tensor       # [packed, width]
    at: torch.Tensor         # [tokens, k] int32
    weights: torch.Tensor    # [tokens, k] float32


def stream_norm(delta: Union[torch.Tensor, Picked], x: torch.Tensor,
                w_post: torch.Tensor, w_pre: Optional[torch.Tensor],
                offset: float, eps: float, out_scale: float = 1.0,
                mult: float = 1.0) -> torch.Tensor:
    """x += mult * rms(delta) * (offset + w_post) in place; returns
    rms(x) * (offset + w_pre) * out_scale in delta's dtype, or without w_pre
    x itself."""
    rows, at, weights = delta if isinstance(delta, Picked) \
        else (delta, None, None)
    if not x.is_cuda:
        return ref.stream_norm(rows, at, weights, x, w_post, w_pre, offset,
                               eps, out_scale, mult)
    y = torch.empty(x.shape, dtype=rows.dtype, device=x.device)
    _ext().stream_norm(y, x, rows, at, weights, w_post, w_pre, offset, eps,
                       out_scale, mult)
    return y


def embed_norm(tokens: torch.Tensor, table: torch.Tensor,
               w_pre: Optional[torch.Tensor], offset: float, eps: float,
               scale: float = 1.0, pos: Optional[torch.Tensor] = None,
               positions: Optional[torch.Tensor] = None
               ) -> tuple[torch.Tensor, torch.Tensor]:
    """x = scale * table[tokens] + pos[positions] (float32; without pos, the
    former) and rms(x) * (offset + w_pre), or without w_pre x itself, in the
    table's dtype; tokens and positions int32."""
    if pos is None:
        positions = None
    if not table.is_cuda:
        return ref.embed_norm(tokens, table, w_pre, offset, eps, scale, pos,
                              positions)
    shape = (tokens.shape[0], table.shape[1])
    x = torch.empty(shape, dtype=torch.float32, device=table.device)
    y = torch.empty(shape, dtype=table.dtype, device=table.device)
    _ext().embed_norm(y, x, table, tokens, w_pre, offset, eps, scale, pos,
                      positions)
    return x, y


def qkv_prepare(buf: torch.Tensor, nq: int, q_norm: Optional[torch.Tensor],
                k_norm: Optional[torch.Tensor], eps: float,
                v_first: Optional[torch.Tensor], lam: Optional[torch.Tensor],
                k_cache: torch.Tensor, v_cache: torch.Tensor,
                slots: torch.Tensor) -> None:
    """buf rows are [q (nq) | k | v | ...]. Norms q in place over all its
    heads, writes normed k and (1 - lam) v + lam v_first to the caches."""
    if not buf.is_cuda:
        ref.qkv_prepare(buf, nq, q_norm, k_norm, eps, v_first, lam, k_cache,
                        v_cache, slots)
        return
    _ext().qkv_prepare(buf, nq, q_norm, k_norm, eps, v_first, lam, k_cache,
                       v_cache, slots)


def attn_ctx(q: torch.Tensor, gate: Optional[torch.Tensor],
             k_cache: torch.Tensor, v_cache: torch.Tensor,
             bias: Optional[torch.Tensor], batch, scale: float, chunk: int = 0,
             any_size: bool = False, window: int = 0, keep: int = 0,
             softcap: float = 0.0, sink: Optional[torch.Tensor] = None,
             mult: float = 1.0, out: Optional[torch.Tensor] = None,
             falloff: Optional[tuple[torch.Tensor, torch.Tensor]] = None,
             weight_bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Attention of a batch's rows over the paged cache, which already holds
    their own keys and values.

    q [rows, heads * dim] and gate [rows, heads] may be views of one buffer,
    out [rows, heads * vdim] a view of wider rows. bias [heads, n]: added to
    the score by distance, the last column also for every larger distance.
    chunk > 0: rows see keys of their own chunk of positions only. window > 0:
    rows see that many keys up to their own, and the first `keep`. softcap > 0:
    scores are cap * tanh(score / cap) ahead of the bias. sink [heads]: a score
    in the softmax that has no value. mult multiplies the result. falloff
    (r1, r2), both [heads]: r1 ln(1 + r2 distance) is taken off the score.
    weight_bias [heads]: a key's weight is sigmoid(score + weight_bias), each
    by itself, instead of a softmax. any_size takes the untiled kernel on the
    GPU."""
    heads = q.shape[1] // k_cache.shape[3]
    if out is None:
        out = q.new_empty(q.shape[0], heads * v_cache.shape[3])
    span = batch.max_context
    if chunk:
        span = min(chunk, span)
    if window:
        span = min(window + keep, span)
    fn = _ext().attn_ctx if q.is_cuda else ref.attn_ctx
    r1, r2 = falloff or (None, None)
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], q[rows], None if gate is None else gate[rows], k_cache,
           v_cache, bias, sink, batch.positions[rows], seq_start,
           batch.block_table[ents], scale, chunk, window, keep, softcap, mult,
           max_len, span, any_size, r1, r2, weight_bias)
    return out


def latent_prepare(buf: torch.Tensor, spec, c_at: int,
                   norm: Optional[torch.Tensor], eps: float,
                   turns: torch.Tensor, positions: torch.Tensor,
                   cache: torch.Tensor, slots: torch.Tensor,
                   q_norm: Optional[torch.Tensor] = None) -> None:
    """buf rows begin with queries, head by head [dim, rot_dim], and have
    [latent, rotated key part] from column c_at on (-1: not). Rotates the
    queries in place, writes the normed latent and the rotated key part to
    the cache. q_norm: rows begin with the queries' latent instead, which is
    normed in place."""
    fn = _ext().latent_prepare if buf.is_cuda else ref.latent_prepare
    fn(buf, 0 if q_norm is not None else spec.heads, spec.dim, spec.rot_dim,
       c_at, norm, eps, turns, positions, cache, slots, q_norm)


def head_linear(x: torch.Tensor, w: torch.Tensor,
                gate: Optional[torch.Tensor] = None,
                tail: int = 0,
                out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Per head h: x[:, h, :k] @ w[h].T, times sigmoid(gate) if there is one;
    the `tail` elements that follow in x are appended as they are.

    x [rows, heads, k + tail] may be a view of wider rows; w [heads, n, k];
    gate [rows, heads * n] or [rows, heads]. Returns [rows, heads, n + tail];
    out: contiguous room for it."""
    shape = (x.shape[0], w.shape[0], w.shape[1] + tail)
    out = x.new_empty(shape) if out is None else out.view(shape)
    (_ext() if x.is_cuda else ref).head_linear(out, x, w, gate, tail)
    return out


def _latent_absorbed(out, q, gate, cache, w_uv, uk_t, batch, rows, ents,
                     seq_start, max_len, spec) -> None:
    """Queries are moved into the latent space, where all heads attend to one
    key per token; what they find is expanded to values afterwards."""
    n = q.shape[0]
    qa = head_linear(q.view(n, spec.heads, spec.dim + spec.rot_dim), uk_t,
                     tail=spec.rot_dim)
    o = q.new_empty(n, spec.heads * spec.rank)
    fn = _ext().attn_ctx if q.is_cuda else ref.attn_ctx
    fn(o, qa.view(n, -1), None, cache, cache[..., :spec.rank], None, None,
       batch.positions[rows], seq_start, batch.block_table[ents], spec.scale,
       0, spec.window, 0, 0.0, 1.0, max_len,
       min(spec.window or batch.max_context, batch.max_context), False, None,
       None, None)
    head_linear(o.view(n, spec.heads, spec.rank), w_uv, gate, out=out)


def _latent_expanded(out, q, gate, cache, w_ukv, batch, rows, ents, seq_start,
                     max_len, spec, shared) -> None:
    """Keys and values of all heads are made for all that the batch's portions
    see; layers on the same cache share what is read from it."""
    ctx_start, total, _ = batch.context(spec.window)
    key = cache.data_ptr(), spec.window
    held = shared.get(key)
    if held is None:
        held = shared[key] = tuple(
            q.new_empty(total, n) for n in (spec.rank, spec.rot_dim))
        _ext().latent_gather(*held, cache, batch.block_table[ents], ctx_start,
                             batch.positions[rows], seq_start, spec.window,
                             max_len)
    c, kr = held
    _ext().attn_flat(out, q, gate, linear(c, w_ukv), kr,
                     batch.positions[rows], seq_start, ctx_start, spec.heads,
                     spec.vdim, spec.scale, spec.window, max_len)


EXPAND_BYTES = 4 << 30      # most memory for keys and values of one layer


def _expanding_pays(batch, spec, rows: int) -> bool:
    """Fewer multiplications with keys and values made for every head than
    with queries moved into the latent space."""
    own = spec.rank * (spec.dim + spec.vdim)
    _, total, pairs = batch.context(spec.window)
    if 2 * total * spec.heads * (spec.dim + spec.vdim) > EXPAND_BYTES:
        return False
    return (total - rows) * own < pairs * (
        2 * spec.rank - spec.dim - spec.vdim)


def _flat_takes(q, gate, spec) -> bool:
    """Sizes that attn_flat is made for; any others stay in latent space."""
    return (q.is_cuda and q.dtype == torch.bfloat16
            and not any(n % 8 for n in (spec.dim, spec.rot_dim, spec.vdim,
                                        q.stride(0), q.storage_offset()))
            and (gate is None or spec.head_gate
                 or gate.storage_offset() % 8 == 0)
            and spec.dim + spec.rot_dim <= 256 and spec.vdim <= 256)


def latent_attn(q: torch.Tensor, gate: Optional[torch.Tensor],
                cache: torch.Tensor, w_ukv: torch.Tensor, uk_t: torch.Tensor,
                batch, spec, shared: dict,
                expand: Optional[bool] = None) -> torch.Tensor:
    """Latent attention of a batch's rows over the paged cache, which already
    holds their own latents. q [rows, heads * (dim + rot_dim)] is rotated;
    gate [rows, heads * vdim], or [rows, heads]; w_ukv has the rows that make all heads' keys,
    then those that make their values; uk_t is the former as [heads, rank,
    dim]. `shared` lasts for one batch. expand: how portions are computed,
    None: as pays."""
    out = q.new_empty(q.shape[0], spec.heads * spec.vdim)
    w_uv = w_ukv[spec.heads * spec.dim:].view(spec.heads, spec.vdim, spec.rank)
    for rows, ents, seq_start, max_len in batch.parts():
        args = (out[rows], q[rows], None if gate is None else gate[rows],
                cache)
        where = (batch, rows, ents, seq_start, max_len, spec)
        if seq_start is not None and _flat_takes(q, gate, spec) and (
                _expanding_pays(batch, spec, args[1].shape[0])
                if expand is None else expand):
            _latent_expanded(*args, w_ukv, *where, shared)
        else:
            _latent_absorbed(*args, w_uv, uk_t, *where)
    return out


def experts(y: torch.Tensor, router: torch.Tensor, up: torch.Tensor,
            down: torch.Tensor, spec, bias: Optional[torch.Tensor] = None,
            correction: Optional[torch.Tensor] = None) -> Picked:
    """A mixture of experts: y [rows, width], router [experts, width], bias
    and correction [experts], up [experts, ff, width] (gated experts: twice as
    many rows, of gate and up in turn), down [experts, width, ff]. Scores are
    32-bit; the correction is for the choice only."""
    rows = y.shape[0]
    if not y.is_cuda:
        return Picked(*ref.experts(y, router, bias, up, down, spec,
                                   correction))
    ext = _ext()
    i32 = dict(dtype=torch.int32, device=y.device)
    z = ext.router_scores(y, router)
    ids = torch.empty(rows, spec.top, **i32)
    weights = torch.empty(rows, spec.top, dtype=torch.float32,
                          device=y.device)
    ext.moe_select(ids, weights, z, spec.groups, spec.keep, bias,
                   spec.over_chosen, spec.sigmoid, correction,
                   spec.group_best)
    packed = rows * spec.top
    tile = ext.moe_tile(packed, spec.experts, y.dtype == torch.bfloat16,
                        y.shape[1], spec.ff)
    at = torch.empty(rows, spec.top, **i32)
    src = torch.empty(packed, **i32)
    start = torch.empty(spec.experts + 1, **i32)
    tiles = torch.empty(1 + 2 * ((packed + tile - 1) // tile +
                                 min(spec.experts, packed)), **i32)
    ext.moe_sort(at, src, start, tiles, ids, tile)
    h = y.new_empty(packed, spec.ff)
    act, limit = ("gelu", 0.0) if spec.glu is None else \
        (spec.glu.act, spec.glu.limit)
    ext.expert_linear(h, y, up, src, start, tiles, tile, act, limit)
    out = y.new_empty(packed, y.shape[1])
    ext.expert_linear(out, h, down, None, start, tiles, tile, "none", 0.0)
    return Picked(out, at, weights)


def side_gate(y: torch.Tensor, w: torch.Tensor, tokens: torch.Tensor,
              table: torch.Tensor, at: int) -> torch.Tensor:
    """gelu_tanh(y @ w.T) * table[tokens, at : at + dim]; tokens int32."""
    out = y.new_empty(y.shape[0], w.shape[0])
    (_ext() if y.is_cuda else ref).side_gate(out, y, w, tokens, table, at)
    return out


def gla(x: torch.Tensor, a2: torch.Tensor, a2_bias: torch.Tensor,
        norm: torch.Tensor, state: torch.Tensor, batch, tau: float, eps: float,
        recurrent: bool = False) -> torch.Tensor:
    """Gated linear attention of a batch's rows; updates the state slots.

    x rows are [q | k | v | g | A1 h]; state [slots, heads, dim, vdim].
    recurrent takes the token-by-token kernel for portions, too."""
    out = x.new_empty(x.shape[0], state.shape[1] * state.shape[3])
    fn = _ext().gla if x.is_cuda else ref.gla
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], x[rows], a2, a2_bias, norm, state,
           batch.state_slots[ents], batch.positions[rows], seq_start,
           1.0 / tau, eps, max_len, recurrent)
    return out


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    """silu(first half) * second half, any width, float32 or bfloat16."""
    if not x.is_cuda:
        return ref.silu_mul(x)
    out = x.new_empty(*x.shape[:-1], x.shape[-1] // 2)
    _ext().silu_mul(out, x.contiguous())
    return out


def glu(x: torch.Tensor, spec, out: torch.Tensor) -> None:
    """out = the gated feed-forward's hidden values of x [rows, 2 f], gate
    then up; both may be views of wider rows."""
    (_ext() if x.is_cuda else ref).glu(out, x, spec.act, spec.limit)


def add_norm(x: Optional[torch.Tensor], w: torch.Tensor,
             b: Optional[torch.Tensor], eps: float, dtype: torch.dtype,
             rows: Optional[torch.Tensor] = None,
             picked: Optional[Picked] = None,
             embedded: Optional[tuple] = None,
             vec: Optional[torch.Tensor] = None
             ) -> tuple[torch.Tensor, torch.Tensor]:
    """Adds to the residual x, in place, whatever is given: rows [rows,
    width]; the weighed sum of picked rows; embedded = (tokens, table, scale),
    scale * table[tokens]; vec [width]. x None: the residual begins here.
    Returns x and its layer norm with weight w and bias b, or without b its RMS
    norm, as dtype."""
    if x is None:
        n = embedded[0].shape[0]
        fresh = torch.empty if w.is_cuda else torch.zeros
        x, new = fresh(n, w.shape[0], dtype=torch.float32,
                       device=w.device), True
    else:
        new = False
    pool, at, weights = picked if picked is not None else (None,) * 3
    tokens, table, scale = embedded if embedded is not None else \
        (None, None, 1.0)
    if not x.is_cuda:
        return x, ref.add_norm(x, rows, at, weights, pool, tokens, table,
                               scale, vec, w, b, eps, dtype)
    y = torch.empty(x.shape, dtype=dtype, device=x.device)
    _ext().add_norm(y, x, new, rows, pool, at, weights, tokens, table, scale,
                    vec, w, b, eps)
    return x, y


def softcap(x: torch.Tensor, cap: float) -> torch.Tensor:
    """cap * tanh(x / cap), in place."""
    (_ext() if x.is_cuda else ref).softcap(x, cap)
    return x


def linear32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x @ w.T in float32, unrounded; x may be a view of wider rows."""
    if x.dtype == torch.float32 or not x.is_cuda:
        return torch.nn.functional.linear(x.float(), w.float())
    return _ext().linear32(x, w)


def rope_table(batch, rot, turns: torch.Tensor, shared: dict) -> torch.Tensor:
    """Cosines and sines of a batch's rows, float32 [rows, dims / 2, 2]; made
    once per batch for all layers that rotate alike."""
    held = shared.get(rot)
    if held is None:
        if turns.is_cuda:
            held = torch.empty(batch.positions.shape[0], turns.shape[0], 2,
                               dtype=torch.float32, device=turns.device)
            _ext().rope_table(held, batch.positions, turns)
        else:
            held = ref.rope_table(batch.positions, turns)
        shared[rot] = held
    return held


def short_conv(x: torch.Tensor, weight: torch.Tensor,
               bias: Optional[torch.Tensor], act: bool, state: torch.Tensor,
               batch) -> torch.Tensor:
    """A causal convolution over time per channel, then silu if act: x [rows,
    channels] may be a view of wider rows; weight [channels, taps], the last
    tap is the row's own. state [slots, taps - 1, channels] has each request's
    last inputs and is updated."""
    out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    fn = (_ext() if x.is_cuda else ref).short_conv
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], x[rows], None, weight, bias, act, state,
           batch.state_slots[ents], batch.positions[rows], seq_start, max_len)
    return out


def conv_rope(buf: torch.Tensor, in_bias: Optional[torch.Tensor],
              weight: torch.Tensor, state: torch.Tensor, rope: torch.Tensor,
              k_cache: torch.Tensor, v_cache: torch.Tensor,
              batch) -> torch.Tensor:
    """buf rows are [q | k | ...]. in_bias is added to both, then they pass a
    short convolution (as short_conv); what that makes of k is also the value
    and goes to v_cache; q and k are rotated (rope: rope_table, neighbouring
    elements are pairs) and k goes to k_cache. Returns q."""
    kv, dim = k_cache.shape[1], k_cache.shape[3]
    q = buf.new_empty(buf.shape[0], weight.shape[0] - kv * dim)
    fn = (_ext() if buf.is_cuda else ref).conv_rope
    for rows, ents, seq_start, max_len in batch.parts():
        fn(q[rows], buf[rows], in_bias, weight, state,
           batch.state_slots[ents], rope[rows], k_cache, v_cache,
           batch.positions[rows], batch.slots[rows], seq_start, max_len)
    return q


def conv_qkv(buf: torch.Tensor, in_bias: Optional[torch.Tensor],
             weight: torch.Tensor, state: torch.Tensor, k_cache: torch.Tensor,
             v_cache: torch.Tensor, batch, temp=None,
             v_eps: Optional[float] = None) -> torch.Tensor:
    """buf rows are [q | k | v | ...]. in_bias is added to all, then they pass
    a short convolution (as short_conv). q is multiplied by its position's
    temperature (layers.QueryTemperature); each head's v is divided by its
    root mean square with v_eps under the root (None: not); k and v go to
    their caches. Returns q."""
    kv = k_cache.shape[1]
    q = buf.new_empty(buf.shape[0], weight.shape[0] - kv * (
        k_cache.shape[3] + v_cache.shape[3]))
    coef, every = (temp.coef, temp.every) if temp else (0.0, 1)
    fn = (_ext() if buf.is_cuda else ref).conv_qkv
    for rows, ents, seq_start, max_len in batch.parts():
        fn(q[rows], buf[rows], in_bias, weight, state,
           batch.state_slots[ents], k_cache, v_cache, batch.positions[rows],
           batch.slots[rows], seq_start, coef, every,
           -1.0 if v_eps is None else v_eps, max_len)
    return q


def selective_scan(u: torch.Tensor, gate: torch.Tensor, z: torch.Tensor,
                   z_bias: torch.Tensor, low: torch.Tensor, b_at: int,
                   a: torch.Tensor, d: torch.Tensor, state: torch.Tensor,
                   batch, out: torch.Tensor, recurrent: bool = False) -> None:
    """Per channel c with state S[c, :], updated from token to token:
        dt = softplus(z + z_bias)
        S <- exp(dt a) S + dt u B,   out = (S . C + d u) silu(gate)
    u, gate, out [rows, channels] (gate and out may be views), z float32; low
    rows have B and C from column b_at on; a [channels, n] float32. recurrent
    walks portions without cutting them into segments."""
    fn = (_ext() if u.is_cuda else ref).selective_scan
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], u[rows], gate[rows], z[rows], z_bias, low[rows], b_at,
           a, d, state, batch.state_slots[ents], batch.positions[rows],
           seq_start, max_len, recurrent)


def lightning(x: torch.Tensor, decay: torch.Tensor, state: torch.Tensor,
              batch, recurrent: bool = False) -> torch.Tensor:
    """x rows are [q | k | v | ...], each of which passes silu; per head
    S <- decay S + k v^T and o = S^T q. Returns [rows, heads * vdim]."""
    out = x.new_empty(x.shape[0], state.shape[1] * state.shape[3])
    fn = (_ext() if x.is_cuda else ref).lightning
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], x[rows], decay, state, batch.state_slots[ents],
           batch.positions[rows], seq_start, max_len, recurrent)
    return out


def joint_gate(o: torch.Tensor, norm: torch.Tensor, gate: torch.Tensor,
               eps: float, out: torch.Tensor) -> None:
    """out = rms(o) over whole rows * norm * sigmoid(gate)."""
    (_ext() if o.is_cuda else ref).joint_gate(out, o, norm, gate, eps)


def delta(qkv: torch.Tensor, z: torch.Tensor, z_bias: torch.Tensor,
          rate: torch.Tensor, beta: torch.Tensor, norm: torch.Tensor,
          gate: torch.Tensor, state: torch.Tensor, batch, kv_heads: int,
          eps: float, mult: float, out: torch.Tensor,
          recurrent: bool = False) -> None:
    """Gated delta rule. Per head, with k and q made unit vectors (q also
    times dim^-1/2) and a decay per key channel:
        S <- exp(-rate softplus(z + z_bias)) S,  u = sigmoid(beta) (v - S^T k)
        S <- S + k u^T,   out = rms(S^T q) norm sigmoid(gate) mult
    qkv rows are [q | k | v], q and k with kv_heads heads; z [rows, heads *
    dim] float32; beta [rows, heads], gate and out [rows, heads * vdim], all
    three maybe views of wider rows."""
    fn = (_ext() if qkv.is_cuda else ref).delta
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], qkv[rows], z[rows], z_bias, rate, beta[rows], norm,
           gate[rows], state, batch.state_slots[ents], batch.positions[rows],
           seq_start, kv_heads, eps, mult, max_len, recurrent)
