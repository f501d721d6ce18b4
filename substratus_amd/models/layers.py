"""Descriptions of layers for models whose layers are not all alike.

A model is a tuple of LayerSpec; the mixer's spec type selects the mixer
(models/hybrid.py). A mixer's spec also names what the cache manager
(serve/kv_cache.py) keeps for the layer: pages with a row per token, slots
with a state per request.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from functools import lru_cache
from typing import Optional, Union

import torch


@dataclass(frozen=True)
class Pages:
    """Part of a layer's cache with a row of `dim` per token and head."""
    heads: int
    dim: int


@dataclass(frozen=True)
class Slots:
    """Part of a layer's cache with one state per request."""
    shape: tuple[int, ...]
    f32: bool = True         # 32-bit in every serving dtype; else as activations


class MixerSpec:
    """What all mixers' specs have."""

    def cache(self) -> tuple[Union[Pages, Slots], ...]:
        """What the layer keeps, in the order in which its mixer takes it."""
        raise NotImplementedError

    def kv_bytes(self, itemsize: int) -> int:
        """Cache bytes per token."""
        return sum(p.heads * p.dim * itemsize for p in self.cache()
                   if isinstance(p, Pages))

    def state_bytes(self, itemsize: int = 4) -> int:
        """State bytes per request."""
        return sum(math.prod(p.shape) * (4 if p.f32 else itemsize)
                   for p in self.cache() if isinstance(p, Slots))


@dataclass(frozen=True)
class QueryTemperature:
    """Queries at position p are multiplied by
    1 + coef * ln(floor((p + 1) / every) + 1)."""
    coef: float
    every: int


@dataclass(frozen=True)
class AttentionSpec(MixerSpec):
    heads: int
    kv_heads: int
    dim: int                 # query/key size of a head
    vdim: int                # value size of a head
    scale: float
    chunk: int = 0           # > 0: positions see their own chunk only
    qk_norm: bool = False    # RMS norm over the whole q and k projections
    bias_rows: int = 0       # rows of the learned distance table, 0: none
    bias_max: int = 0        # distance from which the last row holds
    v_mix: bool = False      # blend in the first such layer's values
    out_gate: bool = False   # sigmoid gate per head on the output
    taps: int = 0            # > 0: q, k and v have a bias and pass a short
                             #   causal convolution over time
    temp: Optional[QueryTemperature] = None   # after the convolution
    v_norm: bool = False     # values over their root mean square, after it
    out_bias: bool = False   # of the output projection
    falloff: bool = False    # r1 ln(1 + r2 distance) is taken off the score
    sigmoid: bool = False    # weights are sigmoid(score + a bias per head),
                             #   each by itself, not a softmax

    def __post_init__(self) -> None:
        if self.taps and (self.qk_norm or self.v_mix):
            raise ValueError("convolved projections are neither normed as a "
                             "whole nor blended")
        if not self.taps and (self.temp or self.v_norm):
            raise ValueError("query temperatures and value norms follow a "
                             "convolution")

    @property
    def conv_rows(self) -> int:
        return (self.heads + self.kv_heads) * self.dim \
            + self.kv_heads * self.vdim

    def cache(self) -> tuple:
        pages = Pages(self.kv_heads, self.dim), \
            Pages(self.kv_heads, self.vdim)
        return pages if not self.taps else \
            pages + (Slots((self.taps - 1, self.conv_rows), False),)

    def params(self, width: int) -> int:
        rows = self.conv_rows + self.heads * self.out_gate
        return width * (rows + self.heads * self.vdim) \
            + self.conv_rows * self.taps


@dataclass(frozen=True)
class GLASpec(MixerSpec):
    heads: int
    dim: int
    vdim: int
    tau: float               # decays are sigmoid(z) ** (1 / tau)
    rank: int                # inner size of the decay projection

    def cache(self) -> tuple:
        return (Slots((self.heads, self.dim, self.vdim)),)

    def params(self, width: int) -> int:
        rows = 2 * self.heads * (self.dim + self.vdim) + self.rank
        return width * (rows + self.heads * self.vdim) \
            + self.heads * self.dim * self.rank


@dataclass(frozen=True)
class RotarySpec:
    """Rotation of the first `dims` elements of a vector: element i turns with
    element i + dims / 2, or if interleaved 2 i with 2 i + 1, at position p by
    p * base ** (-2 i / dims)."""
    base: float
    dims: int
    interleaved: bool = False

    def turns(self, device=None) -> torch.Tensor:
        """float64 [dims / 2]: full turns per position. Whole turns drop out
        of position * turns before anything is rounded to 32 bits."""
        i = torch.arange(self.dims // 2, dtype=torch.float64)
        return (self.base ** (-2.0 * i / self.dims) / (2 * math.pi)).to(device)


@dataclass(frozen=True)
class LatentAttentionSpec(MixerSpec):
    """Attention whose keys and values are projections of one latent vector
    per token, beside a rotated key part that all heads share."""
    heads: int
    dim: int                 # unrotated query/key size of a head
    rot_dim: int             # rotated query/key size of a head
    vdim: int                # value size of a head
    rank: int                # size of the latent
    scale: float
    rot: Optional[RotarySpec]       # None: rot_dim is 0
    kv_from: Optional[int] = None   # layer whose latents it attends to
    out_gate: bool = False   # sigmoid gate per element on the output
    head_gate: bool = False  # the same per head
    q_rank: int = 0          # > 0: queries are projections of a normed latent
    window: int = 0          # > 0: keys a position sees, its own included

    def __post_init__(self) -> None:
        if self.out_gate and self.head_gate:
            raise ValueError("a gate per element or per head, not both")
        if self.q_rank and self.rot_dim:
            raise ValueError("queries out of a latent are not rotated")

    @property
    def row(self) -> int:
        """Elements the cache holds per token: latent, rotated key part."""
        return self.rank + self.rot_dim

    def cache(self) -> tuple:
        return (Pages(1, self.row),) if self.kv_from is None else ()

    def params(self, width: int) -> int:
        q = self.heads * (self.dim + self.rot_dim)
        rows = self.heads * (self.vdim * (1 + self.out_gate) +
                             self.head_gate) + (self.q_rank or q) \
            + (self.row if self.kv_from is None else 0)
        return width * rows + self.q_rank * q \
            + self.heads * self.rank * (self.dim + self.vdim)


@dataclass(frozen=True)
class ConvAttentionSpec(MixerSpec):
    """Attention whose queries and keys pass a short causal convolution over
    time and are rotated; the values are the keys ahead of their rotation."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    taps: int                # of the convolution
    rot: RotarySpec
    window: int = 0          # > 0: a position sees so many, itself included,
    keep: int = 0            #   and the first `keep` of its sequence
    softcap: float = 0.0     # > 0: scores are cap * tanh(score / cap)
    sink: bool = False       # a learned share of the softmax without a value

    def cache(self) -> tuple:
        rows = (self.heads + self.kv_heads) * self.dim
        return Pages(self.kv_heads, self.dim), \
            Pages(self.kv_heads, self.dim), \
            Slots((self.taps - 1, rows), False)

    def params(self, width: int) -> int:
        rows = (self.heads + self.kv_heads) * self.dim
        return width * (rows + self.heads * self.dim) + rows * self.taps


@dataclass(frozen=True)
class DeltaSpec(MixerSpec):
    """Gated delta rule with a decay per key channel."""
    heads: int
    kv_heads: int            # heads of queries and keys
    dim: int
    vdim: int
    taps: int                # of the convolution of q, k and v
    decay_rank: int          # inner sizes of the decays' and the output
    gate_rank: int           #   gate's projection

    @property
    def conv_rows(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    def cache(self) -> tuple:
        return Slots((self.heads, self.dim, self.vdim)), \
            Slots((self.taps - 1, self.conv_rows), False)

    def params(self, width: int) -> int:
        hv = self.heads * self.vdim
        return width * (self.conv_rows + self.heads + self.decay_rank +
                        self.gate_rank + hv) + self.conv_rows * self.taps \
            + self.heads * self.dim * self.decay_rank + hv * self.gate_rank


@dataclass(frozen=True)
class MambaSpec(MixerSpec):
    """Selective scan: a state of `state` numbers per channel."""
    inner: int               # channels
    state: int
    rank: int                # inner size of the step sizes' projection
    taps: int

    def cache(self) -> tuple:
        return Slots((self.inner, self.state)), \
            Slots((self.taps - 1, self.inner), False)

    def params(self, width: int) -> int:
        return self.inner * (3 * width + 2 * self.rank + 3 * self.state +
                             self.taps)


@dataclass(frozen=True)
class LightningSpec(MixerSpec):
    """Linear attention with a constant decay per head, normed over all heads
    at once."""
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    def __post_init__(self) -> None:
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} "
                             "heads")

    def cache(self) -> tuple:
        return (Slots((self.heads, self.dim, self.vdim)),)

    def params(self, width: int) -> int:
        return width * self.heads * (2 * self.dim + 3 * self.vdim)


@dataclass(frozen=True)
class SideBySideSpec(MixerSpec):
    """Two mixers that read the same input, and the scaled sum of both."""
    left: MixerSpec
    right: MixerSpec
    left_scale: float = 1.0
    right_scale: float = 1.0

    def cache(self) -> tuple:
        return self.left.cache() + self.right.cache()

    def params(self, width: int) -> int:
        return self.left.params(width) + self.right.params(width)


@dataclass(frozen=True)
class GluSpec:
    """How a gated feed-forward forms its hidden values from gate g and u:
    silu      silu(g) * u
    relu      max(g, 0) * u
    clamped   g * sigmoid(1.702 g) * (u + 1), of g up to `limit` and u within
              `limit` of zero"""
    act: str = "silu"
    limit: float = 0.0


@dataclass(frozen=True)
class MoESpec:
    """Experts, of which a token uses the `top` best of the `keep` best
    groups of neighbours. Weights are softmax scores over all experts, or
    over the chosen ones, or the sigmoid of each chosen one's score. What is
    best goes by the scores, for the choice only with a learned correction;
    a group's score is the sum of its `group_best` best ones."""
    experts: int
    top: int
    ff: int                  # inner size of one expert
    groups: int = 1
    keep: int = 1
    glu: Optional[GluSpec] = None   # experts are gated; None: gelu
    over_chosen: bool = False
    bias: bool = False       # of the router's scores
    shared_ff: int = 0       # an expert for every token, 0: none
    shared_glu: Optional[GluSpec] = None
    sigmoid: bool = False
    correction: bool = False
    group_best: int = 1      # 1 or 2

    def __post_init__(self) -> None:
        if self.sigmoid and self.over_chosen:
            raise ValueError("sigmoid scores do not sum to anything")
        if self.experts % self.groups or not 0 < self.keep <= self.groups:
            raise ValueError(f"{self.experts} experts in {self.groups} "
                             f"groups, {self.keep} kept")
        if not 0 < self.top <= self.keep * (self.experts // self.groups):
            raise ValueError(f"top {self.top} of {self.keep} groups of "
                             f"{self.experts // self.groups} experts")

    def params(self, width: int) -> int:
        return width * (self.experts * (1 + (3 if self.glu else 2) * self.ff)
                        + 3 * self.shared_ff)


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: int = 0              # inner size of the gated feed-forward, 0: none
    moe: Optional[MoESpec] = None   # experts instead of it
    glu: GluSpec = GluSpec()

    def params(self, width: int) -> int:
        return self.mixer.params(width) + 3 * width * self.ff \
            + (self.moe.params(width) if self.moe else 0)


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop - 1 run `times` times in a row, with the same
    weights and caches of their own. Every pass begins with a learned vector
    added to the residual; every one but the first, also with the embedding."""
    start: int
    stop: int
    times: int


def distance_bucket(n: int, rows: int, furthest: int) -> int:
    """Row of a distance table for distance n >= 0.

    The first half of the rows stands for one distance each; the rest divide
    [half, furthest) at equal ratios, row half + k starting where
    n / half >= (furthest / half) ** (k / (rows - half)). That comparison is
    made between integers, so a distance exactly at a row's start never falls
    to the row before it by rounding."""
    half = rows // 2
    rest = rows - half
    if n < half or half == 0:
        return min(n, rows - 1)
    if n >= furthest:
        return rows - 1
    reach = n ** rest
    k = 0
    while k + 1 < rest and \
            reach * half ** (k + 1) >= furthest ** (k + 1) * half ** rest:
        k += 1
    return half + k


@lru_cache(maxsize=64)
def _buckets(n: int, rows: int, furthest: int) -> tuple[int, ...]:
    return tuple(distance_bucket(i, rows, furthest) for i in range(n))


def distance_bias(table: torch.Tensor, chunk: int,
                  furthest: int) -> torch.Tensor:
    """[rows, heads] table -> float32 [heads, n], the bias of each distance;
    column n - 1 also stands for every larger distance."""
    n = math.ceil(furthest) + 1
    n = n if chunk == 0 else min(chunk, n)
    rows = torch.tensor(_buckets(max(n, 1), table.shape[0], furthest),
                        device=table.device)
    return table.float()[rows].T.contiguous()
