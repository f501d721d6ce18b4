"""Kakovik: a decoder of attention and gated-linear-attention layers in any
order, normed before and after every sublayer, without rotary positions.

Attention layers see their own chunk of positions, with a learned bias per
distance, norms over whole query and key projections, values blended with the
first such layer's and a gate per head; see models/hybrid.py for the layers
themselves. This module maps config.json and checkpoint names onto them.
"""

from __future__ import annotations

import torch

from .config import ModelConfig, register, register_architecture
from .layers import AttentionSpec, GLASpec, LayerSpec

FAMILY = "kakovik"
ROW_PAD = 16    # input projections are padded to whole 16-row tiles


def _layer(doc: dict, i: int, shapes: dict) -> LayerSpec:
    m = doc["mixer"]
    if doc["type"] == "attention":
        rel = shapes.get(f"l{i}.mix.rel", (32, m["heads"]))
        mixer = AttentionSpec(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], scale=float(m["scale"]), chunk=m["mask"]["size"],
            qk_norm=True, bias_rows=rel[0], bias_max=m["bias_max"],
            v_mix=bool(m["v_mix"]), out_gate=True)
    elif doc["type"] == "gla":
        a1 = shapes.get(f"l{i}.mix.a1", (16, 0))
        mixer = GLASpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                        tau=float(m["tau"]), rank=a1[0])
    else:
        raise ValueError(f"layer {i}: unknown mixer {doc['type']!r}")
    mlp = doc["mlp"]
    if mlp is not None and mlp["kind"] != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    return LayerSpec(mixer, 0 if mlp is None else mlp["ff"])


@register_architecture("Kakovik")
def parse(doc: dict, shapes: dict, name: str) -> ModelConfig:
    return model_config(
        name, doc["width"], doc["vocab"], doc["norm"]["eps"],
        doc["logit_scale"],
        [_layer(d, i, shapes) for i, d in enumerate(doc["layers"])])


def model_config(name: str, width: int, vocab: int, eps: float,
                 logit_scale: float, layers: list[LayerSpec]) -> ModelConfig:
    att = [s.mixer for s in layers if isinstance(s.mixer, AttentionSpec)]
    return ModelConfig(
        name=name, family=FAMILY, hidden_size=width,
        intermediate_size=max((s.ff for s in layers), default=0),
        num_layers=len(layers), num_heads=max((a.heads for a in att), default=0),
        num_kv_heads=max((a.kv_heads for a in att), default=0),
        head_dim=max((a.dim for a in att), default=0), vocab_size=vocab,
        max_position_embeddings=1 << 20, rms_norm_eps=eps,
        layers=tuple(layers), norm_offset=1.0, logit_scale=logit_scale)


def is_kakovik_state_dict(sd: dict) -> bool:
    return "embed" in sd and "l0.norm1b" in sd


def stack_rows(parts: list[torch.Tensor]) -> torch.Tensor:
    """Projections of one input under one another, padded with zero rows."""
    rows = sum(p.shape[0] for p in parts)
    pad = -rows % ROW_PAD
    if pad:
        parts = parts + [parts[0].new_zeros(pad, parts[0].shape[1])]
    return torch.cat(parts)


def kakovik_to_native(sd: dict, cfg: ModelConfig) -> dict:
    """Checkpoint names -> HybridLM names: projections that read the same
    input are stacked, small tensors that take part in 32-bit arithmetic
    become float32."""
    out = {"embed.weight": sd["embed"], "head.weight": sd["head"],
           "final_norm": sd["final.norm"].float()}
    for i, spec in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if spec.ff else ()):
            out[dst + n] = sd[src + n].float()
        if isinstance(spec.mixer, AttentionSpec):
            rows = ("q", "k", "v", "g")
            small = {"q_norm": "q.norm", "k_norm": "k.norm", "rel": "rel"}
            if spec.mixer.v_mix:
                # unused in the first such layer, which may come without it
                out[dst + "mixer.vmix"] = sd.get(
                    src + "mix.vmix", torch.zeros(())).float().reshape(())
        else:
            rows = ("q", "k", "v", "g", "a1")
            small = {"norm": "norm", "a2": "a2", "a2_bias": "a2.b"}
        m = src + "mix."
        out[dst + "mixer.w_in.weight"] = stack_rows([sd[m + r] for r in rows])
        out[dst + "mixer.w_out.weight"] = sd[m + "o"]
        for ours, theirs in small.items():
            out[dst + "mixer." + ours] = sd[m + theirs].float()
        if spec.ff:
            out[dst + "w_gateup.weight"] = torch.cat(
                [sd[src + "mlp.gate"], sd[src + "mlp.up"]])
            out[dst + "w_down.weight"] = sd[src + "mlp.down"]
    return out


def uniform(name: str, width: int, depth: int, heads: int, kv_heads: int,
            dim: int, ff: int, vocab: int, chunk: int, every: int = 4,
            gla_heads: int = 0, gla_vdim: int = 0) -> ModelConfig:
    """A regular model: every `every`-th layer is attention, the others GLA,
    all with a feed-forward."""
    att = AttentionSpec(heads, kv_heads, dim, dim, dim ** -0.5, chunk, True,
                        32, chunk, True, True)
    rec = GLASpec(gla_heads or heads // 2, dim, gla_vdim or 2 * dim, 16.0, 16)
    return model_config(name, width, vocab, 1e-5, 1.0, [
        LayerSpec(att if i % every == 0 else rec, ff) for i in range(depth)])


# Shapes of real layers, random weights only: for benches and tests.
register(uniform("kakovik-tiny", 256, 4, 4, 2, 64, 704, 512, 128, every=2))
register(uniform("kakovik-1b", 2048, 16, 16, 16, 128, 5632, 32000, 4096))
register(uniform("kakovik-7b", 4096, 32, 32, 32, 128, 11008, 32000, 4096))
