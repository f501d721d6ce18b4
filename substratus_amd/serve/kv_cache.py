"""Block-paged KV cache sized for 288 GB HBM3E per MI355X GPU.

Layout per layer: k_cache/v_cache of shape [num_blocks, n_kv_heads, block_size,
head_dim] — one block's K rows for one head are a contiguous
block_size × head_dim panel (16×128 bf16 = 4 KiB), the unit the decode
attention kernel streams through LDS/registers with wide coalesced loads.

Models of unlike layers (ModelConfig.layers) keep per layer what its mixer
asks for (MixerSpec.cache): pages with its own head sizes, pages of latents,
a 32-bit recurrent state or a convolution's last inputs for each of
`state_slots` requests. A layer's entry in `layers` has these in the mixer's
order. A layer that attends to another one's latents has that layer's very
entry, and takes no memory of its own. Layers that run more than once have an
entry for every time they run, in the order they run.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import torch

from ..models.config import ModelConfig
from ..models.layers import Pages

DEFAULT_BLOCK_SIZE = 16


class OutOfBlocks(RuntimeError):
    pass


class BlockAllocator:
    def __init__(self, num_blocks: int):
        self.num_blocks = num_blocks
        self._free = list(range(num_blocks - 1, -1, -1))

    @property
    def free_count(self) -> int:
        return len(self._free)

    def alloc(self, n: int = 1) -> list[int]:
        if len(self._free) < n:
            raise OutOfBlocks(f"need {n} KV blocks, {len(self._free)} free")
        return [self._free.pop() for _ in range(n)]

    def free(self, blocks: list[int]) -> None:
        self._free.extend(blocks)


class OutOfSlots(RuntimeError):
    pass


class SlotAllocator:
    """State slots, one per live request. A slot holds whatever its last
    owner left: kernels start from zero at a request's position 0."""

    def __init__(self, num_slots: int):
        self.num_slots = num_slots
        self._free = list(range(num_slots - 1, -1, -1))

    @property
    def free_count(self) -> int:
        return len(self._free)

    def alloc(self) -> int:
        if not self._free:
            raise OutOfSlots(f"all {self.num_slots} state slots are taken")
        return self._free.pop()

    def free(self, slot: int) -> None:
        self._free.append(slot)


class PagedKVCache:
    """Per-rank cache and state manager for every layer of one model."""

    def __init__(self, cfg: ModelConfig, n_kv_heads_local: int, num_blocks: int,
                 block_size: int = DEFAULT_BLOCK_SIZE, device="cpu",
                 dtype=torch.bfloat16, state_slots: int = 0):
        self.cfg = cfg
        self.block_size = block_size
        self.num_blocks = num_blocks
        self.layers: list[tuple[torch.Tensor, ...]] = []
        self.slots = SlotAllocator(
            state_slots if any(s.mixer.state_bytes() for s in cfg.layers)
            else 0)

        def part(p):
            if isinstance(p, Pages):
                return torch.zeros(num_blocks, p.heads, block_size, p.dim,
                                   device=device, dtype=dtype)
            return torch.zeros(state_slots, *p.shape, device=device,
                               dtype=torch.float32 if p.f32 else dtype)
        latest: dict[int, tuple] = {}    # layer -> its last run's entry
        for i, _ in cfg.runs():
            m = cfg.layers[i].mixer
            src = getattr(m, "kv_from", None)
            latest[i] = latest[src] if src is not None else \
                tuple(part(p) for p in m.cache())
            self.layers.append(latest[i])
        for _ in range(0 if cfg.layers else cfg.num_layers):
            k = torch.zeros(num_blocks, n_kv_heads_local, block_size,
                            cfg.head_dim, device=device, dtype=dtype)
            v = torch.zeros_like(k)
            self.layers.append((k, v))
        self.allocator = BlockAllocator(num_blocks)

    def reserve(self, seq: "SequenceState", tokens: int) -> None:
        """Pages for the sequence's first `tokens` tokens and, if the model
        has recurrent layers, a state slot; all of it or OutOfBlocks /
        OutOfSlots and nothing."""
        need = (tokens + self.block_size - 1) // self.block_size
        need -= len(seq.blocks)
        if need > self.allocator.free_count:
            raise OutOfBlocks(f"need {need} KV blocks, "
                              f"{self.allocator.free_count} free")
        if seq.state_slot < 0 and self.slots.num_slots:
            seq.state_slot = self.slots.alloc()
        if need > 0:
            seq.blocks.extend(self.allocator.alloc(need))

    def release(self, seq: "SequenceState") -> None:
        """Give back everything the sequence holds; what it had computed is
        lost with it."""
        if seq.blocks:
            self.allocator.free(seq.blocks)
            seq.blocks = []
        if seq.state_slot >= 0:
            self.slots.free(seq.state_slot)
            seq.state_slot = -1
        seq.num_computed = 0

    @staticmethod
    def state_bytes(cfg: ModelConfig, state_slots: int) -> int:
        return state_slots * sum(cfg.layers[i].mixer.state_bytes()
                                 for i, _ in cfg.runs())

    @staticmethod
    def blocks_for_memory(cfg: ModelConfig, n_kv_heads_local: int,
                          bytes_budget: int,
                          block_size: int = DEFAULT_BLOCK_SIZE,
                          dtype_bytes: int = 2) -> int:
        if cfg.layers:
            per_block = block_size * sum(
                cfg.layers[i].mixer.kv_bytes(dtype_bytes)
                for i, _ in cfg.runs())
        else:
            per_block = (2 * cfg.num_layers * n_kv_heads_local * block_size *
                         cfg.head_dim * dtype_bytes)
        # no attention layer: pages are numbers in a block table only
        return max(bytes_budget // max(per_block, 1), 1)


@dataclass(slots=True)
class SequenceState:
    """Server-side state of one running request."""
    seq_id: int
    tokens: list[int]               # prompt + generated
    num_prompt: int
    max_new_tokens: int
    temperature: float = 0.0
    top_k: int = 0
    top_p: float = 1.0
    blocks: list[int] = field(default_factory=list)
    batch_slot: int = -1            # position in the decode batch
    finished: bool = False
    eos_token: int = -1
    state_slot: int = -1            # recurrent state, -1: holds none
    num_computed: int = 0           # tokens already in the cache and state

    @property
    def length(self) -> int:
        return len(self.tokens)

    @property
    def num_generated(self) -> int:
        return self.length - self.num_prompt

    def needed_blocks(self, block_size: int, extra_tokens: int = 0) -> int:
        total = self.length + extra_tokens
        return (total + block_size - 1) // block_size

    def slot_of(self, pos: int, block_size: int) -> int:
        return self.blocks[pos // block_size] * block_size + pos % block_size
