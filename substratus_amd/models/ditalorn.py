"""Ditalorn: a decoder of attention layers whose weights are sigmoids and of
windowed latent-attention layers, in any order, normed before and after every
sublayer, with mixtures of experts and learned position vectors.

The attention's queries, keys and values pass a short convolution over time;
scores fall with the logarithm of the distance. See models/hybrid.py for the
layers themselves; this module maps config.json and checkpoint names onto
them.
"""

from __future__ import annotations

import torch

from .config import ModelConfig, register, register_architecture
from .kakovik import stack_rows
from .layers import (AttentionSpec, GluSpec, LatentAttentionSpec, LayerSpec,
                     MixerSpec, MoESpec, QueryTemperature)

FAMILY = "ditalorn"


def _mixer(doc: dict, i: int) -> MixerSpec:
    m = doc["mixer"]
    if doc["type"] == "latent_attention":
        return LatentAttentionSpec(
            heads=m["heads"], dim=m["dim"], rot_dim=0, vdim=m["vdim"],
            rank=m["kv_rank"], scale=float(m["scale"]), rot=None,
            head_gate=True, q_rank=m["q_rank"], window=m["mask"]["size"])
    if doc["type"] == "attention":
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"layer {i}: {m['heads']} heads on "
                             f"{m['kv_heads']}")
        temp = m["q_temp"]
        return AttentionSpec(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], scale=float(m["scale"]), taps=m["conv"],
            temp=QueryTemperature(float(temp["coef"]), temp["every"]),
            v_norm=True, out_bias=True, falloff=True, sigmoid=True)
    raise ValueError(f"layer {i}: unknown mixer {doc['type']!r}")


def _experts(mlp: dict | None, i: int) -> MoESpec | None:
    if mlp is None:
        return None
    if mlp["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    return _moe(r["experts"], r["top"], mlp["expert"]["ff"], groups["count"],
                groups["keep"])


def _moe(experts: int, top: int, ff: int, groups: int, keep: int) -> MoESpec:
    return MoESpec(experts, top, ff, groups, keep, GluSpec("silu"),
                   sigmoid=True, correction=True, group_best=2)


@register_architecture("Ditalorn")
def parse(doc: dict, shapes: dict, name: str) -> ModelConfig:
    positions = shapes.get("pos", (doc["max_positions"],))[0]
    return model_config(
        name, doc["width"], doc["vocab"], doc["norm"]["eps"],
        float(doc["embedding"]["scale"]), positions,
        [LayerSpec(_mixer(d, i), 0, _experts(d["mlp"], i))
         for i, d in enumerate(doc["layers"])])


def model_config(name: str, width: int, vocab: int, eps: float,
                 embed_scale: float, positions: int,
                 layers: list[LayerSpec]) -> ModelConfig:
    att = [s.mixer for s in layers if isinstance(s.mixer, AttentionSpec)]
    return ModelConfig(
        name=name, family=FAMILY, hidden_size=width,
        intermediate_size=max((s.moe.ff * s.moe.top for s in layers if s.moe),
                              default=0),
        num_layers=len(layers), num_heads=max(s.mixer.heads for s in layers),
        num_kv_heads=max((a.kv_heads for a in att), default=1),
        head_dim=max(s.mixer.dim for s in layers), vocab_size=vocab,
        max_position_embeddings=positions, rms_norm_eps=eps,
        layers=tuple(layers), norm_offset=1.0, embed_scale=embed_scale,
        learned_pos_emb=True, tie_word_embeddings=True)


def is_ditalorn_state_dict(sd: dict) -> bool:
    return "pos" in sd and "l0.norm1b" in sd


def ditalorn_to_native(sd: dict, cfg: ModelConfig) -> dict:
    """Checkpoint names -> HybridLM names: projections that read the same
    input are stacked, as are a layer's experts; small tensors that take part
    in 32-bit arithmetic become float32."""
    out = {"embed.weight": sd["embed"], "pos": sd["pos"],
           "final_norm": sd["final.norm"].float()}
    for i, spec in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        m, mixer = src + "mix.", dst + "mixer."
        out[dst + "norm1"] = sd[src + "norm1"].float()
        out[dst + "norm1b"] = sd[src + "norm1b"].float()
        if isinstance(spec.mixer, AttentionSpec):
            rows = ("q", "k", "v")
            for ours, theirs in (("in_bias", ".b"), ("conv", ".conv")):
                out[mixer + ours] = torch.cat(
                    [sd[m + r + theirs] for r in rows]).float()
            for ours, theirs in (("r1", "r1"), ("r2", "r2"),
                                 ("weight_bias", "pb")):
                out[mixer + ours] = sd[m + theirs].float()
            out[mixer + "w_out.bias"] = sd[m + "o.b"]
        else:
            rows = ("dq", "dkv", "g")
            out[mixer + "q_norm"] = sd[m + "dq.norm"].float()
            out[mixer + "c_norm"] = sd[m + "dkv.norm"].float()
            out[mixer + "w_uq.weight"] = sd[m + "uq"]
            out[mixer + "w_ukv"] = torch.cat([sd[m + "uk"], sd[m + "uv"]])
        out[mixer + "w_in.weight"] = stack_rows([sd[m + r] for r in rows])
        out[mixer + "w_out.weight"] = sd[m + "o"]
        if spec.moe:
            ff = src + "mlp."
            out[dst + "norm2"] = sd[src + "norm2"].float()
            out[dst + "norm2b"] = sd[src + "norm2b"].float()
            out[dst + "experts.router"] = sd[ff + "router"]
            out[dst + "experts.correction"] = sd[ff + "correction"].float()
            each = range(spec.moe.experts)
            out[dst + "experts.up"] = torch.stack([
                torch.stack([sd[f"{ff}e{e}.gate"], sd[f"{ff}e{e}.up"]], 1)
                .flatten(0, 1) for e in each])
            out[dst + "experts.down"] = torch.stack(
                [sd[f"{ff}e{e}.down"] for e in each])
    return out


def uniform(name: str, width: int, depth: int, heads: int, kv_heads: int,
            dim: int, q_rank: int, kv_rank: int, window: int, moe: MoESpec,
            vocab: int, positions: int) -> ModelConfig:
    """A regular model: attention and latent attention in turn, every layer
    with experts."""
    att = AttentionSpec(heads, kv_heads, dim, dim, dim ** -0.5, taps=4,
                        temp=QueryTemperature(0.1, 1024), v_norm=True,
                        out_bias=True, falloff=True, sigmoid=True)
    latent = LatentAttentionSpec(heads, dim, 0, dim, kv_rank, dim ** -0.5,
                                 None, head_gate=True, q_rank=q_rank,
                                 window=window)
    return model_config(name, width, vocab, 1e-5, width ** 0.5, positions,
                        [LayerSpec(latent if i % 2 else att, 0, moe)
                         for i in range(depth)])


# Shapes of real layers, random weights only: for benches and tests. A token's
# experts are together as large as the dense feed-forward of the model whose
# size they name, so a token costs about as much.
register(uniform("ditalorn-tiny", 256, 4, 4, 2, 64, 96, 128, 128,
                 _moe(8, 2, 192, 4, 2), 512, 1024))
register(uniform("ditalorn-1b", 2048, 16, 16, 16, 128, 768, 512, 1024,
                 _moe(32, 6, 896, 8, 4), 32000, 8192))
register(uniform("ditalorn-7b", 4096, 32, 32, 32, 128, 1536, 512, 1024,
                 _moe(32, 8, 1344, 8, 4), 32000, 8192))
