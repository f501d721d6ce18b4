"""Descriptions of layers for models whose layers are not all alike.

A model is a tuple of LayerSpec; the mixer's spec type selects the mixer
(models/hybrid.py) and what the cache manager keeps for the layer
(serve/kv_cache.py): pages of keys and values, or one state per request.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from functools import lru_cache
from typing import Optional, Union

import torch


@dataclass(frozen=True)
class AttentionSpec:
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

    def kv_bytes(self, itemsize: int) -> int:
        """Cache bytes per token."""
        return self.kv_heads * (self.dim + self.vdim) * itemsize

    def state_bytes(self) -> int:
        return 0

    def params(self, width: int) -> int:
        rows = (self.heads + self.kv_heads) * self.dim \
            + self.kv_heads * self.vdim + self.heads * self.out_gate
        return width * (rows + self.heads * self.vdim)


@dataclass(frozen=True)
class GLASpec:
    heads: int
    dim: int
    vdim: int
    tau: float               # decays are sigmoid(z) ** (1 / tau)
    rank: int                # inner size of the decay projection

    def kv_bytes(self, itemsize: int) -> int:
        return 0

    def state_bytes(self) -> int:
        """State bytes per request; 32-bit in every serving dtype."""
        return self.heads * self.dim * self.vdim * 4

    def params(self, width: int) -> int:
        rows = 2 * self.heads * (self.dim + self.vdim) + self.rank
        return width * (rows + self.heads * self.vdim) \
            + self.heads * self.dim * self.rank


@dataclass(frozen=True)
class RotarySpec:
    """Rotation of the first `dims` elements of a vector: element i turns with
    element i + dims / 2, at position p by p * base ** (-2 i / dims)."""
    base: float
    dims: int

    def turns(self, device=None) -> torch.Tensor:
        """float64 [dims / 2]: full turns per position. Whole turns drop out
        of position * turns before anything is rounded to 32 bits."""
        i = torch.arange(self.dims // 2, dtype=torch.float64)
        return (self.base ** (-2.0 * i / self.dims) / (2 * math.pi)).to(device)


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention whose keys and values are projections of one latent vector
    per token, beside a rotated key part that all heads share."""
    heads: int
    dim: int                 # unrotated query/key size of a head
    rot_dim: int             # rotated query/key size of a head
    vdim: int                # value size of a head
    rank: int                # size of the latent
    scale: float
    rot: RotarySpec
    kv_from: Optional[int] = None   # layer whose latents it attends to
    out_gate: bool = False   # sigmoid gate per element on the output

    @property
    def row(self) -> int:
        """Elements the cache holds per token: latent, rotated key part."""
        return self.rank + self.rot_dim

    def kv_bytes(self, itemsize: int) -> int:
        return self.row * itemsize if self.kv_from is None else 0

    def state_bytes(self) -> int:
        return 0

    def params(self, width: int) -> int:
        rows = self.heads * (self.dim + self.rot_dim +
                             self.vdim * (1 + self.out_gate)) \
            + (self.row if self.kv_from is None else 0)
        return width * rows + self.heads * self.rank * (self.dim + self.vdim)


@dataclass(frozen=True)
class MoESpec:
    """Experts, of which a token uses the `top` best of the `keep` best
    groups of neighbours; weights are softmax scores over all experts."""
    experts: int
    top: int
    ff: int                  # inner size of one expert
    groups: int = 1
    keep: int = 1

    def __post_init__(self) -> None:
        if self.experts % self.groups or not 0 < self.keep <= self.groups:
            raise ValueError(f"{self.experts} experts in {self.groups} "
                             f"groups, {self.keep} kept")
        if not 0 < self.top <= self.keep * (self.experts // self.groups):
            raise ValueError(f"top {self.top} of {self.keep} groups of "
                             f"{self.experts // self.groups} experts")

    def params(self, width: int) -> int:
        return width * self.experts * (1 + 2 * self.ff)


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[AttentionSpec, GLASpec, LatentAttentionSpec]
    ff: int = 0              # inner size of the gated feed-forward, 0: none
    moe: Optional[MoESpec] = None   # experts instead of it

    def params(self, width: int) -> int:
        return self.mixer.params(width) + 3 * width * self.ff \
            + (self.moe.params(width) if self.moe else 0)


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
