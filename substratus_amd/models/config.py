"""Model architecture configs for the data plane.

The reference orchestrates external HF images for concrete models named in its
examples (reference: examples/llama2-7b/*, examples/falcon-7b-instruct/*,
examples/facebook-opt-125m/*, examples/llama2-13b-chat-gguf/*,
examples/llama2-70b/server.yaml). We implement those model families natively.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Callable, Optional

from .layers import LayerSpec, LoopSpec


@dataclass
class ModelConfig:
    name: str
    family: str  # "llama" | "falcon" | "opt" | "kakovik" | "guronex" |
                 # "vurazen" | "ditalorn"
    hidden_size: int
    intermediate_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    vocab_size: int
    max_position_embeddings: int
    head_dim: int = 0
    rope_theta: float = 10000.0
    rms_norm_eps: float = 1e-5
    layer_norm_eps: float = 1e-5
    tie_word_embeddings: bool = False
    # falcon-style: attention and MLP in parallel off one layernorm
    parallel_attn: bool = False
    # falcon-40b "new decoder architecture": parallel attn+MLP but with TWO
    # norms of the residual (ln_attn feeds attention, ln_mlp feeds the MLP)
    parallel_norms: bool = False
    # opt-style: learned positional embeddings (+ LayerNorm + gelu)
    learned_pos_emb: bool = False
    activation: str = "silu"  # "silu" (gated) | "gelu"
    # models of unlike layers (models/hybrid.py): one spec per layer; the
    # uniform fields above then only size things for reports
    layers: tuple[LayerSpec, ...] = ()
    norm_offset: float = 0.0  # 1: norm weights are stored around zero
    pre_norm: bool = True     # sublayers read the normed residual, or itself
    residual_mult: float = 1.0  # factor of what sublayers add to the residual
    side_dim: int = 0         # per layer: size of an input for the token itself
    logit_scale: float = 1.0
    # mixer and feed-forward read one norm of the residual and are added to it
    # together, or one after the other
    parallel_block: bool = False
    embed_scale: float = 1.0
    logit_softcap: float = 0.0  # > 0: logits are cap * tanh(logits / cap)
    loop: Optional[LoopSpec] = None

    def __post_init__(self) -> None:
        if self.head_dim == 0 and self.num_heads:
            self.head_dim = self.hidden_size // self.num_heads

    @property
    def kv_dim(self) -> int:
        return self.num_kv_heads * self.head_dim

    def runs(self) -> list[tuple[int, Optional[int]]]:
        """The layers in the order they run, each with the number of the
        loop's pass that begins with it, or None."""
        n = len(self.layers)
        loop = self.loop or LoopSpec(n, n, 0)
        body = [(i, t if i == loop.start else None)
                for t in range(loop.times)
                for i in range(loop.start, loop.stop)]
        return [(i, None) for i in range(loop.start)] + body + \
            [(i, None) for i in range(loop.stop, n)]

    def param_count(self) -> int:
        h, f, L, v = self.hidden_size, self.intermediate_size, self.num_layers, self.vocab_size
        if self.layers:
            side = self.side_dim * len(self.layers)
            tables = v * (1 if self.tie_word_embeddings else 2) \
                + self.learned_pos_emb * self.max_position_embeddings
            return tables * h + side * (v + 2 * h) \
                + sum(s.params(h) for s in self.layers)
        qkv = h * (self.num_heads + 2 * self.num_kv_heads) * self.head_dim
        o = self.num_heads * self.head_dim * h
        if self.activation == "silu":
            mlp = 3 * h * f
        else:
            mlp = 2 * h * f
        emb = v * h * (1 if self.tie_word_embeddings else 2)
        return L * (qkv + o + mlp) + emb


_REGISTRY: dict[str, ModelConfig] = {}


def register(cfg: ModelConfig) -> ModelConfig:
    _REGISTRY[cfg.name] = cfg
    return cfg


# Model folders whose config.json spells out an architecture instead of naming
# a registered model: "architecture" -> parser(document, tensor shapes, name).
_ARCHITECTURES: dict[str, Callable[[dict, dict, str], ModelConfig]] = {}


def register_architecture(name: str):
    def add(parser):
        _ARCHITECTURES[name] = parser
        return parser
    return add


def tensor_shapes(path: str) -> dict[str, tuple[int, ...]]:
    """Names and shapes of a safetensors file, from its header only."""
    with open(path, "rb") as f:
        header = json.loads(f.read(int.from_bytes(f.read(8), "little")))
    return {k: tuple(v["shape"]) for k, v in header.items()
            if k != "__metadata__"}


def load_config(model_dir: str) -> ModelConfig:
    """The config of a model folder (config.json, model.safetensors)."""
    with open(os.path.join(model_dir, "config.json")) as f:
        doc = json.load(f)
    if "architecture" not in doc:
        return get_config(doc["model"])
    if doc["architecture"] not in _ARCHITECTURES:
        raise KeyError(f"unknown architecture {doc['architecture']!r}; known: "
                       f"{sorted(_ARCHITECTURES)}")
    weights = os.path.join(model_dir, "model.safetensors")
    shapes = tensor_shapes(weights) if os.path.exists(weights) else {}
    name = os.path.basename(os.path.abspath(model_dir))
    return _ARCHITECTURES[doc["architecture"]](doc, shapes, name)


def get_config(name: str) -> ModelConfig:
    """A registered model by name, or a model folder by path."""
    if os.path.isfile(os.path.join(name, "config.json")):
        return load_config(name)
    key = name.lower().split("/")[-1]
    if key in _REGISTRY:
        return _REGISTRY[key]
    raise KeyError(f"unknown model config: {name!r}; known: {sorted(_REGISTRY)}")


# Llama-2 family (reference: examples/llama2-7b, examples/llama2-13b-chat-gguf,
# examples/llama2-70b).
register(ModelConfig(
    name="llama2-7b", family="llama", hidden_size=4096, intermediate_size=11008,
    num_layers=32, num_heads=32, num_kv_heads=32, vocab_size=32000,
    max_position_embeddings=4096, rms_norm_eps=1e-5))
register(ModelConfig(
    name="llama2-13b", family="llama", hidden_size=5120, intermediate_size=13824,
    num_layers=40, num_heads=40, num_kv_heads=40, vocab_size=32000,
    max_position_embeddings=4096, rms_norm_eps=1e-5))
register(ModelConfig(
    name="llama2-70b", family="llama", hidden_size=8192, intermediate_size=28672,
    num_layers=80, num_heads=64, num_kv_heads=8, vocab_size=32000,
    max_position_embeddings=4096, rms_norm_eps=1e-5))
# Llama-3 family (beyond reference parity — same llama weight layout, so
# HF checkpoints map via the existing name translation; GQA groups 4 and 8
# ride the MFMA decode kernel, rope theta 500k, 128k vocab).
register(ModelConfig(
    name="llama3-8b", family="llama", hidden_size=4096,
    intermediate_size=14336, num_layers=32, num_heads=32, num_kv_heads=8,
    vocab_size=128256, max_position_embeddings=8192, rope_theta=500000.0,
    rms_norm_eps=1e-5))
register(ModelConfig(
    name="llama3-70b", family="llama", hidden_size=8192,
    intermediate_size=28672, num_layers=80, num_heads=64, num_kv_heads=8,
    vocab_size=128256, max_position_embeddings=8192, rope_theta=500000.0,
    rms_norm_eps=1e-5))

# A small llama-shaped model (random weights), the uniform counterpart of
# kakovik-1b.
register(ModelConfig(
    name="llama-1b", family="llama", hidden_size=2048, intermediate_size=5632,
    num_layers=16, num_heads=16, num_kv_heads=16, vocab_size=32000,
    max_position_embeddings=4096, rms_norm_eps=1e-5))

# A tiny llama for CPU tests and CI.
# Tiny llama for CPU tests/CI and GPU numerics tests (head_dim=64, GQA=2).
register(ModelConfig(
    name="llama-tiny", family="llama", hidden_size=256, intermediate_size=704,
    num_layers=4, num_heads=4, num_kv_heads=2, vocab_size=512,
    max_position_embeddings=2048, rms_norm_eps=1e-5))

# Falcon-7b-instruct (reference: examples/falcon-7b-instruct/finetuned-model.yaml).
# 71 query heads with multi-query attention (1 kv head), parallel attn+mlp.
register(ModelConfig(
    name="falcon-7b-instruct", family="falcon", hidden_size=4544,
    intermediate_size=4 * 4544, num_layers=32, num_heads=71, num_kv_heads=1,
    vocab_size=65024, max_position_embeddings=2048, layer_norm_eps=1e-5,
    parallel_attn=True, activation="gelu", tie_word_embeddings=True))
register(ModelConfig(
    name="falcon-tiny", family="falcon", hidden_size=256,
    intermediate_size=1024, num_layers=2, num_heads=4, num_kv_heads=1,
    vocab_size=512, max_position_embeddings=2048, parallel_attn=True,
    activation="gelu", tie_word_embeddings=True))

# Falcon-40b (reference: examples/falcon-40b/*.yaml). GQA (128 q / 8 kv
# heads) with the "new decoder architecture": two parallel layernorms per
# block (ln_attn -> attention, ln_mlp -> MLP).
register(ModelConfig(
    name="falcon-40b", family="falcon", hidden_size=8192,
    intermediate_size=4 * 8192, num_layers=60, num_heads=128, num_kv_heads=8,
    vocab_size=65024, max_position_embeddings=2048, layer_norm_eps=1e-5,
    parallel_attn=True, parallel_norms=True, activation="gelu",
    tie_word_embeddings=True))
register(ModelConfig(
    name="falcon40-tiny", family="falcon", hidden_size=256,
    intermediate_size=1024, num_layers=2, num_heads=4, num_kv_heads=2,
    vocab_size=512, max_position_embeddings=2048, parallel_attn=True,
    parallel_norms=True, activation="gelu", tie_word_embeddings=True))

# facebook/opt-125m (reference: examples/facebook-opt-125m/base-model.yaml —
# the reference's CPU system-test model, test/system.sh).
register(ModelConfig(
    name="opt-125m", family="opt", hidden_size=768, intermediate_size=3072,
    num_layers=12, num_heads=12, num_kv_heads=12, vocab_size=50272,
    max_position_embeddings=2048, learned_pos_emb=True, activation="gelu",
    tie_word_embeddings=True))
