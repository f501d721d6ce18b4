"""Ops of models whose layers differ from one another (models/hybrid.py):
norms around a 32-bit residual, attention that reads the paged cache for
single tokens and prompt portions alike, gated linear attention with a
recurrent state per request.

Same policy as the rest of ops: GPU tensors need the HIP extension
(substratus_amd._hybrid), CPU tensors run the plain implementations in ref.py.
Activations are float32 or bfloat16; residual, norm weights, biases, decay
weights and recurrent state are always float32.
"""

from __future__ import annotations

from typing import Optional

import torch

from . import ref

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


def stream_norm(delta: torch.Tensor, x: torch.Tensor, w_post: torch.Tensor,
                w_pre: torch.Tensor, offset: float, eps: float,
                out_scale: float = 1.0) -> torch.Tensor:
    """x += rms(delta) * (offset + w_post) in place; returns
    rms(x) * (offset + w_pre) * out_scale in delta's dtype."""
    if not x.is_cuda:
        return ref.stream_norm(delta, x, w_post, w_pre, offset, eps, out_scale)
    y = torch.empty_like(delta)
    _ext().stream_norm(y, x, delta, w_post, w_pre, offset, eps, out_scale)
    return y


def embed_norm(tokens: torch.Tensor, table: torch.Tensor, w_pre: torch.Tensor,
               offset: float, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """x = table[tokens] (float32) and rms(x) * (offset + w_pre) in the
    table's dtype; tokens int32."""
    if not table.is_cuda:
        return ref.embed_norm(tokens, table, w_pre, offset, eps)
    shape = (tokens.shape[0], table.shape[1])
    x = torch.empty(shape, dtype=torch.float32, device=table.device)
    y = torch.empty(shape, dtype=table.dtype, device=table.device)
    _ext().embed_norm(y, x, table, tokens, w_pre, offset, eps)
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
             bias: Optional[torch.Tensor], batch, scale: float, chunk: int,
             any_size: bool = False) -> torch.Tensor:
    """Attention of a batch's rows over the paged cache, which already holds
    their own keys and values.

    q [rows, heads * dim] and gate [rows, heads] may be views of one buffer.
    bias [heads, n]: added to the score by distance, the last column also for
    every larger distance. chunk > 0: rows see keys of their own chunk of
    positions only. any_size takes the untiled kernel on the GPU."""
    heads = q.shape[1] // k_cache.shape[3]
    out = q.new_empty(q.shape[0], heads * v_cache.shape[3])
    span = batch.max_context if chunk == 0 else min(chunk, batch.max_context)
    fn = _ext().attn_ctx if q.is_cuda else ref.attn_ctx
    for rows, ents, seq_start, max_len in batch.parts():
        fn(out[rows], q[rows], None if gate is None else gate[rows], k_cache,
           v_cache, bias, batch.positions[rows], seq_start,
           batch.block_table[ents], scale, chunk, max_len, span, any_size)
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
