"""Decoder-only model whose layers differ: a list of mixers (attention, latent
attention, linear attention, selective scans, ...) and optional feed-forwards
(dense or mixtures of experts) around a 32-bit residual, each sublayer normed
before and after, or after only. A layer may end with an input for the token
itself. Or mixer and feed-forward read one norm and are added together; layers
may run several times in a row.

The engine drives it like the uniform families (models/model.py), with one
difference: a step is a StepBatch (serve/batch.py) of single tokens and prompt
portions, and there is one forward for both. Mixers read and write what the
cache manager keeps for their layer: pages of keys and values, or state slots.

Per layer and step: input projection (one matrix product for everything that
reads the normed input), one fused kernel up to the cache, the mixer, output
projection, one fused kernel for post-norm + residual + next pre-norm. A
parallel layer has one input projection for its mixer and its feed-forward, and
one output projection for both, over their outputs side by side.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from ..ops import hybrid as ops, linear
from ..parallel.comm import state
from ..parallel.tp import Linear
from ..serve.batch import StepBatch
from .config import ModelConfig
from .layers import (AttentionSpec, ConvAttentionSpec, DeltaSpec, GLASpec,
                     LatentAttentionSpec, LayerSpec, LightningSpec, MambaSpec,
                     MixerSpec, MoESpec, SideBySideSpec, distance_bias)


def _f32(*shape: int, device=None) -> nn.Parameter:
    """A small weight that takes part in 32-bit arithmetic."""
    return nn.Parameter(torch.zeros(shape, device=device,
                                    dtype=torch.float32))


def _padded(rows: int) -> int:
    return (rows + 15) // 16 * 16


class AttentionMixer(nn.Module):
    """Attention over the paged cache; what AttentionSpec names is there or
    not: whole-projection q/k norm, distance bias or falloff, chunk mask,
    value blending, output gate, short convolutions with query temperatures
    and value norms, sigmoid weights instead of a softmax."""

    def __init__(self, spec: AttentionSpec, width: int, eps: float,
                 device=None, dtype=None):
        super().__init__()
        self.spec, self.eps = spec, eps
        self.nq = spec.heads * spec.dim
        self.nk = spec.kv_heads * spec.dim
        self.nv = spec.kv_heads * spec.vdim
        self.ng = spec.heads if spec.out_gate else 0
        self.w_in = Linear(width, _padded(self.nq + self.nk + self.nv
                                          + self.ng),
                           device=device, dtype=dtype)
        self.w_out = Linear(spec.heads * spec.vdim, width, spec.out_bias,
                            device=device, dtype=dtype)
        if spec.taps:
            self.in_bias = _f32(spec.conv_rows, device=device)
            self.conv = _f32(spec.conv_rows, spec.taps, device=device)
        if spec.falloff:
            self.r1 = _f32(spec.heads, device=device)
            self.r2 = _f32(spec.heads, device=device)
        if spec.sigmoid:
            self.weight_bias = _f32(spec.heads, device=device)
        if spec.qk_norm:
            self.q_norm = _f32(self.nq, device=device)
            self.k_norm = _f32(self.nk, device=device)
        if spec.bias_rows:
            self.rel = _f32(spec.bias_rows, spec.heads, device=device)
        if spec.v_mix:
            self.vmix = _f32(device=device)
        self._bias: Optional[torch.Tensor] = None

    def finish_weights(self) -> None:
        """The distance table spread out by distance, once per load."""
        if self.spec.bias_rows:
            self._bias = distance_bias(self.rel, self.spec.chunk,
                                       self.spec.bias_max)

    def forward(self, y: torch.Tensor, cache: tuple, batch: StepBatch,
                shared: dict) -> torch.Tensor:
        s = self.spec
        k_cache, v_cache = cache[:2]
        buf = self.w_in(y)
        v_at = self.nq + self.nk
        if s.taps:
            q = ops.conv_qkv(buf, self.in_bias, self.conv, cache[2], k_cache,
                             v_cache, batch, s.temp,
                             self.eps if s.v_norm else None)
        else:
            q = self._prepare(buf, v_at, k_cache, v_cache, batch, shared)
        g_at = v_at + self.nv
        gate = buf[:, g_at:g_at + self.ng] if self.ng else None
        a = ops.attn_ctx(
            q, gate, k_cache, v_cache, self._bias, batch, s.scale, s.chunk,
            falloff=(self.r1, self.r2) if s.falloff else None,
            weight_bias=self.weight_bias if s.sigmoid else None)
        return self.w_out(a)

    def _prepare(self, buf: torch.Tensor, v_at: int, k_cache: torch.Tensor,
                 v_cache: torch.Tensor, batch: StepBatch,
                 shared: dict) -> torch.Tensor:
        """Norms and blends of a projection that is not convolved."""
        s, v_first = self.spec, None
        if s.v_mix:
            v_first = shared.get("v_first")
            if v_first is None:
                # the projection itself, not the cache: it is of these tokens
                shared["v_first"] = buf[:, v_at:v_at + self.nv]
        ops.qkv_prepare(buf, self.nq,
                        self.q_norm if s.qk_norm else None,
                        self.k_norm if s.qk_norm else None, self.eps,
                        v_first, self.vmix if v_first is not None else None,
                        k_cache, v_cache, batch.slots)
        return buf[:, :self.nq]


class GLAMixer(nn.Module):
    """Gated linear attention with a decay per key channel and a 32-bit state
    per request."""

    def __init__(self, spec: GLASpec, width: int, eps: float, device=None,
                 dtype=None):
        super().__init__()
        self.spec, self.eps = spec, eps
        self.w_in = Linear(width, _padded(2 * spec.heads *
                                          (spec.dim + spec.vdim) + spec.rank),
                           device=device, dtype=dtype)
        self.w_out = Linear(spec.heads * spec.vdim, width, device=device,
                            dtype=dtype)
        self.a2 = _f32(spec.heads * spec.dim, spec.rank, device=device)
        self.a2_bias = _f32(spec.heads * spec.dim, device=device)
        self.norm = _f32(spec.vdim, device=device)

    def finish_weights(self) -> None:
        pass

    def forward(self, y: torch.Tensor, cache: tuple, batch: StepBatch,
                shared: dict) -> torch.Tensor:
        o = ops.gla(self.w_in(y), self.a2, self.a2_bias, self.norm, cache[0],
                    batch, self.spec.tau, self.eps)
        return self.w_out(o)


class LatentMixer(nn.Module):
    """Softmax attention over a paged cache of latents, the layer's own or an
    earlier layer's; heads expand keys and values from them, or queries and
    outputs are moved into the latent space (ops.latent_attn). Queries may
    come out of a latent of their own."""

    def __init__(self, spec: LatentAttentionSpec, width: int, eps: float,
                 device=None, dtype=None):
        super().__init__()
        self.spec, self.eps = spec, eps
        self.own = spec.kv_from is None
        nq = spec.heads * (spec.dim + spec.rot_dim)
        self.nq = spec.q_rank or nq
        row = spec.row if self.own else 0
        # gates per head go last: they leave odd numbers of columns
        self.ng = spec.heads * spec.vdim if spec.out_gate else \
            spec.heads if spec.head_gate else 0
        self.g_at, self.c_at = (self.nq + row, self.nq) if spec.head_gate \
            else (self.nq, self.nq + self.ng)
        self.w_in = Linear(width, _padded(self.nq + self.ng + row),
                           device=device, dtype=dtype)
        if spec.q_rank:
            self.q_norm = _f32(spec.q_rank, device=device)
            self.w_uq = Linear(spec.q_rank, nq, device=device, dtype=dtype)
        self.w_out = Linear(spec.heads * spec.vdim, width, device=device,
                            dtype=dtype)
        # keys of all heads, then values of all heads
        self.w_ukv = nn.Parameter(torch.empty(
            spec.heads * (spec.dim + spec.vdim), spec.rank, device=device,
            dtype=dtype))
        if self.own:
            self.c_norm = _f32(spec.rank, device=device)

    def finish_weights(self) -> None:
        s = self.spec
        self._uk_t = self.w_ukv[:s.heads * s.dim].view(
            s.heads, s.dim, s.rank).transpose(1, 2).contiguous()
        self._turns = s.rot.turns(self.w_ukv.device) if s.rot else \
            torch.empty(0, dtype=torch.float64, device=self.w_ukv.device)

    def forward(self, y: torch.Tensor, cache: tuple, batch: StepBatch,
                shared: dict) -> torch.Tensor:
        s, buf = self.spec, self.w_in(y)
        ops.latent_prepare(buf, s, self.c_at if self.own else -1,
                           self.c_norm if self.own else None, self.eps,
                           self._turns, batch.positions, cache[0],
                           batch.slots, self.q_norm if s.q_rank else None)
        gate = buf[:, self.g_at:self.g_at + self.ng] if self.ng else None
        q = buf[:, :self.nq]
        if s.q_rank:
            q = self.w_uq(q)
        o = ops.latent_attn(q, gate, cache[0], self.w_ukv, self._uk_t, batch,
                            s, shared)
        return self.w_out(o)


MIXERS = {AttentionSpec: AttentionMixer, GLASpec: GLAMixer,
          LatentAttentionSpec: LatentMixer}


class Core(nn.Module):
    """A mixer without projections of its own: from rows of its layer's input
    projection (`rows_in` columns) to `cols_out` columns for the output
    projection, which it fills. `mult` is a factor of its result."""
    rows_in: int
    cols_out: int

    def __init__(self, spec: MixerSpec, eps: float, mult: float = 1.0):
        super().__init__()
        self.spec, self.eps, self.mult = spec, eps, mult

    def finish_weights(self) -> None:
        pass

    def forward(self, buf: torch.Tensor, out: torch.Tensor, cache: tuple,
                batch: StepBatch, shared: dict) -> None:
        raise NotImplementedError


class ConvAttention(Core):
    """Softmax attention over the paged cache; queries and keys pass a short
    convolution and are rotated. buf: [q | k]."""

    def __init__(self, spec: ConvAttentionSpec, eps: float, mult: float = 1.0,
                 device=None, dtype=None):
        super().__init__(spec, eps, mult)
        rows = (spec.heads + spec.kv_heads) * spec.dim
        self.rows_in, self.cols_out = rows, spec.heads * spec.dim
        self.bias = _f32(rows, device=device)
        self.conv = _f32(rows, spec.taps, device=device)
        if spec.sink:
            self.sink = _f32(spec.heads, device=device)

    def finish_weights(self) -> None:
        self._turns = self.spec.rot.turns(self.conv.device)

    def forward(self, buf, out, cache, batch, shared):
        s = self.spec
        k_cache, v_cache, conv = cache
        rope = ops.rope_table(batch, s.rot, self._turns, shared)
        q = ops.conv_rope(buf, self.bias, self.conv, conv, rope, k_cache,
                          v_cache, batch)
        ops.attn_ctx(q, None, k_cache, v_cache, None, batch, s.scale,
                     window=s.window, keep=s.keep, softcap=s.softcap,
                     sink=self.sink if s.sink else None, mult=self.mult,
                     out=out)


class DeltaMixer(Core):
    """Gated delta rule, a 32-bit state per request. buf: [q | k | v | decays'
    inner values | output gate's inner values | step sizes]."""

    def __init__(self, spec: DeltaSpec, eps: float, mult: float = 1.0,
                 device=None, dtype=None):
        super().__init__(spec, eps, mult)
        h, hk, hv = spec.heads, spec.heads * spec.dim, spec.heads * spec.vdim
        # inner values begin where 16-byte pieces do
        self.a_at = _padded(spec.conv_rows)
        self.g_at = self.a_at + _padded(spec.decay_rank)
        self.b_at = self.g_at + _padded(spec.gate_rank)
        self.rows_in, self.cols_out = self.b_at + h, hv
        self.conv = _f32(spec.conv_rows, spec.taps, device=device)
        self.a2 = nn.Parameter(torch.empty(hk, spec.decay_rank, device=device,
                                           dtype=dtype))
        self.g2 = nn.Parameter(torch.empty(hv, spec.gate_rank, device=device,
                                           dtype=dtype))
        self.dt_bias = _f32(hk, device=device)
        self.A_log = _f32(h, device=device)
        self.norm = _f32(spec.vdim, device=device)

    def finish_weights(self) -> None:
        self._rate = torch.exp(self.A_log)

    def forward(self, buf, out, cache, batch, shared):
        s = self.spec
        state, conv = cache
        qkv = ops.short_conv(buf[:, :s.conv_rows], self.conv, None, True, conv,
                             batch)
        z = ops.linear32(buf[:, self.a_at:self.a_at + s.decay_rank], self.a2)
        gate = ops.linear(buf[:, self.g_at:self.g_at + s.gate_rank], self.g2)
        ops.delta(qkv, z, self.dt_bias, self._rate,
                  buf[:, self.b_at:self.b_at + s.heads], self.norm, gate,
                  state, batch, s.kv_heads, self.eps, self.mult, out)


class MambaMixer(Core):
    """Selective scan, a 32-bit state per request. buf: [x | gate]."""

    def __init__(self, spec: MambaSpec, eps: float, mult: float = 1.0,
                 device=None, dtype=None):
        super().__init__(spec, eps, mult)
        if mult != 1.0:
            raise NotImplementedError("a selective scan has no factor")
        inner = spec.inner
        self.rows_in, self.cols_out = 2 * inner, inner
        self.conv = _f32(inner, spec.taps, device=device)
        self.conv_bias = _f32(inner, device=device)
        self.w_x = Linear(inner, _padded(spec.rank + 2 * spec.state),
                          device=device, dtype=dtype)
        self.w_dt = nn.Parameter(torch.empty(inner, spec.rank, device=device,
                                             dtype=dtype))
        self.dt_bias = _f32(inner, device=device)
        self.A_log = _f32(inner, spec.state, device=device)
        self.D = _f32(inner, device=device)

    def finish_weights(self) -> None:
        self._a = -torch.exp(self.A_log)

    def forward(self, buf, out, cache, batch, shared):
        s = self.spec
        state, conv = cache
        u = ops.short_conv(buf[:, :s.inner], self.conv, self.conv_bias, True,
                           conv, batch)
        low = self.w_x(u)
        z = ops.linear32(low[:, :s.rank], self.w_dt)
        ops.selective_scan(u, buf[:, s.inner:2 * s.inner], z, self.dt_bias,
                           low, s.rank, self._a, self.D, state, batch, out)


class LightningMixer(Core):
    """Linear attention with constant decays, a 32-bit state per request.
    buf: [q | k | v | gate]."""

    def __init__(self, spec: LightningSpec, eps: float, mult: float = 1.0,
                 device=None, dtype=None):
        super().__init__(spec, eps, mult)
        if mult != 1.0:
            raise NotImplementedError("lightning attention has no factor")
        hv = spec.heads * spec.vdim
        self.g_at = spec.heads * (2 * spec.dim + spec.vdim)
        self.rows_in, self.cols_out = self.g_at + hv, hv
        self.norm = _f32(hv, device=device)

    def finish_weights(self) -> None:
        self._decay = torch.tensor(self.spec.decay, dtype=torch.float32,
                                   device=self.norm.device)

    def forward(self, buf, out, cache, batch, shared):
        o = ops.lightning(buf, self._decay, cache[0], batch)
        ops.joint_gate(o, self.norm, buf[:, self.g_at:self.rows_in], self.eps,
                       out)


class SideBySide(Core):
    """Two mixers on the same input; their scaled outputs lie side by side
    ahead of one output projection, which adds them up. buf: [left's | zeros
    up to a 16-row piece | right's]."""

    def __init__(self, spec: SideBySideSpec, eps: float, mult: float = 1.0,
                 device=None, dtype=None):
        super().__init__(spec, eps, mult)
        self.left, self.right = (
            CORES[type(m)](m, eps, mult * scale, device, dtype)
            for m, scale in ((spec.left, spec.left_scale),
                             (spec.right, spec.right_scale)))
        self.r_at = _padded(self.left.rows_in)
        self.rows_in = self.r_at + self.right.rows_in
        self.cols_out = self.left.cols_out + self.right.cols_out

    def finish_weights(self) -> None:
        self.left.finish_weights()
        self.right.finish_weights()

    def forward(self, buf, out, cache, batch, shared):
        n, c = len(self.spec.left.cache()), self.left.cols_out
        self.left(buf, out[:, :c], cache[:n], batch, shared)
        self.right(buf[:, self.r_at:], out[:, c:], cache[n:], batch, shared)


CORES = {ConvAttentionSpec: ConvAttention, DeltaSpec: DeltaMixer,
         MambaSpec: MambaMixer, LightningSpec: LightningMixer,
         SideBySideSpec: SideBySide}


class Experts(nn.Module):
    """A mixture of experts: what every token adds is left as rows to pick
    and weigh, which the norm that follows does on its way."""

    def __init__(self, spec: MoESpec, width: int, device=None, dtype=None):
        super().__init__()
        self.spec = spec

        def weight(*shape):
            return nn.Parameter(torch.empty(shape, device=device,
                                            dtype=dtype))
        self.router = weight(spec.experts, width)
        if spec.bias:
            self.router_bias = _f32(spec.experts, device=device)
        if spec.correction:
            self.correction = _f32(spec.experts, device=device)
        # gated: rows of gate and up in turn
        self.up = weight(spec.experts, (2 if spec.glu else 1) * spec.ff, width)
        self.down = weight(spec.experts, width, spec.ff)

    def forward(self, y: torch.Tensor) -> ops.Picked:
        return ops.experts(y, self.router, self.up, self.down, self.spec,
                           self.router_bias if self.spec.bias else None,
                           self.correction if self.spec.correction else None)


class SideInput(nn.Module):
    """A layer's input for the token itself: a gate of the stream times the
    token's entry in a table, projected."""

    def __init__(self, dim: int, width: int, device=None, dtype=None):
        super().__init__()
        self.w_gate = nn.Parameter(torch.empty(dim, width, device=device,
                                               dtype=dtype))
        self.w_proj = Linear(dim, width, device=device, dtype=dtype)
        self.norm = _f32(width, device=device)

    def forward(self, y: torch.Tensor, tokens: torch.Tensor,
                table: torch.Tensor, layer: int) -> torch.Tensor:
        return self.w_proj(ops.side_gate(y, self.w_gate, tokens, table,
                                         layer * self.w_gate.shape[0]))


class HybridLayer(nn.Module):
    def __init__(self, spec: LayerSpec, cfg: ModelConfig, device=None,
                 dtype=None):
        super().__init__()
        self.spec = spec
        width = cfg.hidden_size
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, width,
                                              cfg.rms_norm_eps, device, dtype)

        def norm(there):
            return _f32(width, device=device) if there else None
        self.norm1 = norm(cfg.pre_norm)
        self.norm1b = norm(True)
        ff = bool(spec.ff or spec.moe)
        self.norm2 = norm(ff and cfg.pre_norm)
        self.norm2b = norm(ff)
        if spec.ff:
            self.w_gateup = Linear(width, 2 * spec.ff, device=device,
                                   dtype=dtype)
            self.w_down = Linear(spec.ff, width, device=device, dtype=dtype)
        if spec.moe:
            self.experts = Experts(spec.moe, width, device, dtype)
        if cfg.side_dim:
            self.side = SideInput(cfg.side_dim, width, device, dtype)

    def feed_forward(self, y: torch.Tensor):
        if self.spec.moe:
            return self.experts(y)
        return self.w_down(ops.silu_mul(self.w_gateup(y)))


class ParallelLayer(nn.Module):
    """Mixer, dense or shared feed-forward and experts side by side on one
    norm of the residual. One product makes everything that reads the norm
    (but experts' values), one makes what is added to the residual (but
    experts' rows)."""

    def __init__(self, spec: LayerSpec, cfg: ModelConfig, device=None,
                 dtype=None):
        super().__init__()
        self.spec = spec
        width = cfg.hidden_size
        self.norm1 = _f32(width, device=device)
        self.norm1_bias = _f32(width, device=device)
        self.mixer = CORES[type(spec.mixer)](spec.mixer, cfg.layer_norm_eps,
                                             1.0, device, dtype)
        self.ff, self.glu = spec.ff, spec.glu
        if spec.moe:
            self.ff, self.glu = spec.moe.shared_ff, spec.moe.shared_glu
            self.experts = Experts(spec.moe, width, device, dtype)
        self.ff_at = _padded(self.mixer.rows_in)
        self.w_in = Linear(width, _padded(self.ff_at + 2 * self.ff),
                           device=device, dtype=dtype)
        self.w_out = Linear(self.mixer.cols_out + self.ff, width,
                            device=device, dtype=dtype)

    def forward(self, y: torch.Tensor, cache: tuple, batch: StepBatch,
                shared: dict, want: Optional[torch.Tensor]
                ) -> tuple[Optional[torch.Tensor], Optional[ops.Picked]]:
        """What to add to the residual, for all rows or those of `want`."""
        buf = self.w_in(y)
        out = y.new_empty(y.shape[0], self.w_out.weight.shape[1])
        at = self.mixer.cols_out
        self.mixer(buf[:, :self.mixer.rows_in], out[:, :at], cache, batch,
                   shared)
        if want is not None:
            buf, out, y = buf[want], out[want], y[want]
        if not y.shape[0]:
            return None, None
        if self.ff:
            ops.glu(buf[:, self.ff_at:self.ff_at + 2 * self.ff], self.glu,
                    out[:, at:])
        return self.w_out(out), self.experts(y) if self.spec.moe else None


class HybridLM(nn.Module):
    takes_portions = True     # the engine may hand it parts of prompts

    def __init__(self, cfg: ModelConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        if state().tp_size > 1:
            raise NotImplementedError(
                f"{cfg.family} models are served on one GPU: the norms and "
                "the latents of their layers span all heads, which tensor "
                "parallelism divides")
        self.cfg = cfg
        self.eps = cfg.layer_norm_eps if cfg.parallel_block \
            else cfg.rms_norm_eps
        self.n_kv_heads = cfg.num_kv_heads
        self.embed = nn.Embedding(cfg.vocab_size, cfg.hidden_size,
                                  device=device, dtype=dtype)
        self.layers = nn.ModuleList(
            (ParallelLayer if cfg.parallel_block else HybridLayer)(
                s, cfg, device, dtype) for s in cfg.layers)
        if cfg.loop:
            self.loop_step = _f32(cfg.loop.times, cfg.hidden_size,
                                  device=device)
        if cfg.side_dim:
            self.side_embed = nn.Parameter(torch.empty(
                cfg.vocab_size, cfg.side_dim * len(cfg.layers), device=device,
                dtype=dtype))
        if cfg.learned_pos_emb:
            self.pos = nn.Parameter(torch.empty(
                cfg.max_position_embeddings, cfg.hidden_size, device=device,
                dtype=dtype))
        self.final_norm = _f32(cfg.hidden_size, device=device)
        if cfg.parallel_block:
            self.final_norm_bias = _f32(cfg.hidden_size, device=device)
        self.head = None if cfg.tie_word_embeddings else Linear(
            cfg.hidden_size, cfg.vocab_size, device=device, dtype=dtype)

    @torch.no_grad()
    def init_random(self, seed: int = 0) -> None:
        """Fill every parameter (models are built on meta): matrices
        N(0, 0.02), norms neutral, blend factors 1/2, decays near 1, sigmoid
        weights small."""
        g = torch.Generator(device=self.final_norm.device).manual_seed(seed)
        neutral = 1.0 - self.cfg.norm_offset
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm1", "norm1b", "norm2", "norm2b", "final_norm"):
                p.fill_(neutral)
            elif leaf in ("q_norm", "k_norm", "norm", "c_norm", "D"):
                p.fill_(1.0)
            elif leaf == "conv":
                p.normal_(0.0, p.shape[1] ** -0.5, generator=g)
            elif leaf == "dt_bias":
                p.fill_(-4.0)
            elif leaf in ("vmix", "r1", "r2"):
                p.fill_(0.5)
            elif leaf == "weight_bias":
                p.fill_(-4.0)
            elif leaf == "a2_bias":
                p.fill_(2.0)
            else:
                p.normal_(0.0, 0.02, generator=g)
        self.finish_weights()

    def load_state_dict(self, *args, **kwargs):
        out = super().load_state_dict(*args, **kwargs)
        self.finish_weights()
        return out

    @torch.no_grad()
    def finish_weights(self) -> None:
        for layer in self.layers:
            layer.mixer.finish_weights()

    def logits(self, y: torch.Tensor) -> torch.Tensor:
        return linear(y, self.embed.weight) if self.head is None \
            else self.head(y)

    def step_ops(self, batch: StepBatch, caches: list[tuple]):
        """The forward as a generator that yields between op groups (see
        models/model.py decode_ops); returns the logits of batch.want, or of
        every row."""
        if self.cfg.parallel_block:
            return (yield from self._parallel_ops(batch, caches))
        off, eps = self.cfg.norm_offset, self.eps
        mult = self.cfg.residual_mult
        x, y = ops.embed_norm(
            batch.tokens, self.embed.weight, self.layers[0].norm1, off, eps,
            self.cfg.embed_scale, self.pos if self.cfg.learned_pos_emb
            else None, batch.positions)
        tokens = batch.tokens
        shared: dict = {}     # what a layer leaves for later layers' mixers
        for i, layer in enumerate(self.layers):
            last = i + 1 == len(self.layers)
            after = self.final_norm if last else self.layers[i + 1].norm1
            scale = self.cfg.logit_scale if last else 1.0
            delta, post = layer.mixer(y, caches[i], batch, shared), \
                layer.norm1b
            yield
            if last and batch.want is not None:
                # past the last mixer only rows with wanted logits go on
                if batch.want.shape[0] == 0:
                    return y.new_empty(0, self.cfg.vocab_size)
                delta, x, tokens = (t[batch.want] for t in (delta, x, tokens))
            if layer.norm2b is not None:
                y = ops.stream_norm(delta, x, post, layer.norm2, off, eps,
                                    mult=mult)
                delta, post = layer.feed_forward(y), layer.norm2b
                yield
            if self.cfg.side_dim:
                y = ops.stream_norm(delta, x, post, None, off, eps, mult=mult)
                delta, post = layer.side(y, tokens, self.side_embed, i), \
                    layer.side.norm
                yield
            y = ops.stream_norm(delta, x, post, after, off, eps, scale, mult)
        return self.logits(y)

    def _parallel_ops(self, batch: StepBatch, caches: list[tuple]):
        cfg, runs = self.cfg, self.cfg.runs()
        dtype, table = self.embed.weight.dtype, self.embed.weight
        x = rows = picked = None
        shared: dict = {}
        for at, (i, begins) in enumerate(runs):
            layer = self.layers[i]
            embedded = (batch.tokens, table, cfg.embed_scale) \
                if at == 0 or begins else None
            vec = None if begins is None else self.loop_step[begins]
            x, y = ops.add_norm(x, layer.norm1, layer.norm1_bias, self.eps,
                                dtype, rows, picked, embedded, vec)
            # past the last mixer only rows with wanted logits go on
            want = batch.want if at + 1 == len(runs) else None
            rows, picked = layer(y, caches[at], batch, shared, want)
            yield
        if want is not None:
            if rows is None:
                return y.new_empty(0, cfg.vocab_size)
            x = x[want]
        _, y = ops.add_norm(x, self.final_norm, self.final_norm_bias, self.eps,
                            dtype, rows, picked)
        logits = self.logits(y)
        return ops.softcap(logits, cfg.logit_softcap) if cfg.logit_softcap \
            else logits

    def forward_step(self, batch: StepBatch,
                     caches: list[tuple]) -> torch.Tensor:
        gen = self.step_ops(batch, caches)
        while True:
            try:
                next(gen)
            except StopIteration as e:
                return e.value

    def decode_ops(self, tokens: torch.Tensor, positions: torch.Tensor,
                   kv_caches: list[tuple], slots: torch.Tensor,
                   block_table: torch.Tensor, seq_lens: torch.Tensor,
                   state_slots: torch.Tensor, block_size: int):
        """One token per request, device-resident state (graph capture)."""
        n = tokens.shape[0]
        batch = StepBatch(tokens.int(), positions, slots, block_table,
                          state_slots, n, None, 0,
                          block_table.shape[1] * block_size)
        return (yield from self.step_ops(batch, kv_caches))
