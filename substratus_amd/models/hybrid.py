"""Decoder-only model whose layers differ: a list of mixers (attention, gated
linear attention, ...) and optional feed-forwards around a 32-bit residual,
each sublayer normed before and after.

The engine drives it like the uniform families (models/model.py), with one
difference: a step is a StepBatch (serve/batch.py) of single tokens and prompt
portions, and there is one forward for both. Mixers read and write what the
cache manager keeps for their layer: pages of keys and values, or state slots.

Per layer and step: input projection (one matrix product for everything that
reads the normed input), one fused kernel up to the cache, the mixer, output
projection, one fused kernel for post-norm + residual + next pre-norm.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from ..ops import hybrid as ops
from ..parallel.comm import state
from ..parallel.tp import Linear
from ..serve.batch import StepBatch
from .config import ModelConfig
from .layers import AttentionSpec, GLASpec, LayerSpec, distance_bias


def _f32(*shape: int, device=None) -> nn.Parameter:
    """A small weight that takes part in 32-bit arithmetic."""
    return nn.Parameter(torch.zeros(shape, device=device,
                                    dtype=torch.float32))


def _padded(rows: int) -> int:
    return (rows + 15) // 16 * 16


class AttentionMixer(nn.Module):
    """Softmax attention over the paged cache; what AttentionSpec names is
    there or not: whole-projection q/k norm, distance bias, chunk mask, value
    blending, output gate."""

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
        self.w_out = Linear(spec.heads * spec.vdim, width, device=device,
                            dtype=dtype)
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
        k_cache, v_cache = cache
        buf = self.w_in(y)
        v_at = self.nq + self.nk
        v_first = None
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
        g_at = v_at + self.nv
        gate = buf[:, g_at:g_at + self.ng] if self.ng else None
        a = ops.attn_ctx(buf[:, :self.nq], gate, k_cache, v_cache, self._bias,
                         batch, s.scale, s.chunk)
        return self.w_out(a)


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


MIXERS = {AttentionSpec: AttentionMixer, GLASpec: GLAMixer}


class HybridLayer(nn.Module):
    def __init__(self, spec: LayerSpec, width: int, eps: float, device=None,
                 dtype=None):
        super().__init__()
        self.spec = spec
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, width, eps, device,
                                              dtype)
        self.norm1 = _f32(width, device=device)
        self.norm1b = _f32(width, device=device)
        if spec.ff:
            self.norm2 = _f32(width, device=device)
            self.norm2b = _f32(width, device=device)
            self.w_gateup = Linear(width, 2 * spec.ff, device=device,
                                   dtype=dtype)
            self.w_down = Linear(spec.ff, width, device=device, dtype=dtype)

    def feed_forward(self, y: torch.Tensor) -> torch.Tensor:
        if y.shape[0] == 0:
            return y
        return self.w_down(ops.silu_mul(self.w_gateup(y)))


class HybridLM(nn.Module):
    takes_portions = True     # the engine may hand it parts of prompts

    def __init__(self, cfg: ModelConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        if state().tp_size > 1:
            raise NotImplementedError(
                f"{cfg.family} models are served on one GPU: their norms span "
                "all heads of a projection, which tensor parallelism divides")
        self.cfg, self.eps = cfg, cfg.rms_norm_eps
        self.n_kv_heads = cfg.num_kv_heads
        self.embed = nn.Embedding(cfg.vocab_size, cfg.hidden_size,
                                  device=device, dtype=dtype)
        self.layers = nn.ModuleList(
            HybridLayer(s, cfg.hidden_size, self.eps, device, dtype)
            for s in cfg.layers)
        self.final_norm = _f32(cfg.hidden_size, device=device)
        self.head = Linear(cfg.hidden_size, cfg.vocab_size, device=device,
                           dtype=dtype)

    @torch.no_grad()
    def init_random(self, seed: int = 0) -> None:
        """Fill every parameter (models are built on meta): matrices
        N(0, 0.02), norms neutral, blend factors 1/2, decays near 1."""
        g = torch.Generator(device=self.final_norm.device).manual_seed(seed)
        neutral = 1.0 - self.cfg.norm_offset
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm1", "norm1b", "norm2", "norm2b", "final_norm"):
                p.fill_(neutral)
            elif leaf in ("q_norm", "k_norm", "norm"):
                p.fill_(1.0)
            elif leaf == "vmix":
                p.fill_(0.5)
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

    def step_ops(self, batch: StepBatch, caches: list[tuple]):
        """The forward as a generator that yields between op groups (see
        models/model.py decode_ops); returns the logits of batch.want, or of
        every row."""
        off, eps = self.cfg.norm_offset, self.eps
        x, y = ops.embed_norm(batch.tokens, self.embed.weight,
                              self.layers[0].norm1, off, eps)
        shared: dict = {}     # what a layer leaves for later layers' mixers
        for i, layer in enumerate(self.layers):
            last = i + 1 == len(self.layers)
            after = self.final_norm if last else self.layers[i + 1].norm1
            scale = self.cfg.logit_scale if last else 1.0
            delta = layer.mixer(y, caches[i], batch, shared)
            yield
            post = layer.norm1b
            if layer.spec.ff:
                if last:
                    delta, x = self._wanted(delta, x, batch)
                y = ops.stream_norm(delta, x, post, layer.norm2, off, eps)
                delta = layer.feed_forward(y)
                post = layer.norm2b
                yield
            elif last:
                delta, x = self._wanted(delta, x, batch)
            y = ops.stream_norm(delta, x, post, after, off, eps, scale)
        if y.shape[0] == 0:
            return y.new_empty(0, self.cfg.vocab_size)
        return self.head(y)

    @staticmethod
    def _wanted(delta, x, batch: StepBatch):
        """Past the last mixer only rows with wanted logits go on."""
        if batch.want is None:
            return delta, x
        return delta[batch.want], x[batch.want]

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
                   state_slots: torch.Tensor):
        """One token per request, device-resident state (graph capture)."""
        n = tokens.shape[0]
        bs = max((c[0].shape[2] for c in kv_caches if len(c) == 2), default=1)
        batch = StepBatch(tokens.int(), positions, slots, block_table,
                          state_slots, n, None, 0,
                          block_table.shape[1] * bs)
        return (yield from self.step_ops(batch, kv_caches))
