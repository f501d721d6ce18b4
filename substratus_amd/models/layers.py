"""Descriptions of layers for models whose layers are not all alike.

A model is a tuple of LayerSpec; the mixer's spec type selects the mixer
(models/hybrid.py) and what the cache manager keeps for the layer
(serve/kv_cache.py): pages of keys and values, or one state per request.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from functools import lru_cache
from typing import Union

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
class LayerSpec:
    mixer: Union[AttentionSpec, GLASpec]
    ff: int = 0              # inner size of the gated feed-forward, 0: none


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
