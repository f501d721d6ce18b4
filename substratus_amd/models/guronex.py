"""Guronex: a decoder of latent-attention layers with mixtures of experts.

Sublayers read the residual itself and are normed on their output only; every
layer also adds an input of its own for the token at hand. Layers may attend
to the latents of an earlier layer, whose cache they share. See
models/hybrid.py for the layers themselves; this module maps config.json and
checkpoint names onto them.
"""

from __future__ import annotations

import torch

from .config import ModelConfig, register, register_architecture
from .kakovik import stack_rows
from .layers import LatentAttentionSpec, LayerSpec, MoESpec, RotarySpec

FAMILY = "guronex"


def _mixer(doc: dict, i: int) -> LatentAttentionSpec:
    if doc["type"] != "latent_attention":
        raise ValueError(f"layer {i}: unknown mixer {doc['type']!r}")
    m = doc["mixer"]
    rot = RotarySpec(float(m["rot"]["base"]), m["rot"]["dims"])
    if rot.dims % 2 or rot.dims > m["rot_dim"]:
        raise ValueError(f"layer {i}: cannot rotate {rot.dims} of "
                         f"{m['rot_dim']} elements")
    return LatentAttentionSpec(
        heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"],
        rank=m["kv_rank"], scale=float(m["scale"]), rot=rot,
        kv_from=m.get("kv_from"), out_gate=True)


def _experts(mlp: dict | None, i: int) -> MoESpec | None:
    if mlp is None:
        return None
    if mlp["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    return MoESpec(r["experts"], r["top"], mlp["expert"]["ff"],
                   groups["count"], groups["keep"])


@register_architecture("Guronex")
def parse(doc: dict, shapes: dict, name: str) -> ModelConfig:
    return model_config(
        name, doc["width"], doc["vocab"], doc["norm"]["eps"],
        float(doc.get("residual_mult", 1.0)),
        (doc.get("token_side") or {"dim": 0})["dim"],
        [LayerSpec(_mixer(d, i), 0, _experts(d["mlp"], i))
         for i, d in enumerate(doc["layers"])])


def model_config(name: str, width: int, vocab: int, eps: float,
                 residual_mult: float, side_dim: int,
                 layers: list[LayerSpec]) -> ModelConfig:
    for i, spec in enumerate(layers):
        m, j = spec.mixer, spec.mixer.kv_from
        if j is None:
            continue
        src = layers[j].mixer if 0 <= j < i else None
        if src is None or src.kv_from is not None or \
                (src.rank, src.rot_dim, src.rot) != (m.rank, m.rot_dim, m.rot):
            raise ValueError(f"layer {i} cannot use layer {j}'s latents")
    return ModelConfig(
        name=name, family=FAMILY, hidden_size=width,
        intermediate_size=max((s.moe.ff * s.moe.top for s in layers if s.moe),
                              default=0),
        num_layers=len(layers), num_heads=max(s.mixer.heads for s in layers),
        num_kv_heads=1, head_dim=max(s.mixer.dim + s.mixer.rot_dim
                                     for s in layers),
        vocab_size=vocab, max_position_embeddings=1 << 20, rms_norm_eps=eps,
        layers=tuple(layers), pre_norm=False, residual_mult=residual_mult,
        side_dim=side_dim)


def is_guronex_state_dict(sd: dict) -> bool:
    return "embed" in sd and "l0.mix.uk" in sd


def guronex_to_native(sd: dict, cfg: ModelConfig) -> dict:
    """Checkpoint names -> HybridLM names: projections that read the same
    input are stacked, as are a layer's experts; norm weights become
    float32."""
    out = {"embed.weight": sd["embed"], "head.weight": sd["head"],
           "final_norm": sd["final.norm"].float()}
    if cfg.side_dim:
        out["side_embed"] = sd["side.embed"]
    for i, spec in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        m, mixer = src + "mix.", dst + "mixer."
        own = spec.mixer.kv_from is None
        out[mixer + "w_in.weight"] = stack_rows(
            [sd[m + r] for r in ("q", "g") + (("dkv",) if own else ())])
        if own:
            out[mixer + "c_norm"] = sd[m + "dkv.norm"].float()
        out[mixer + "w_ukv"] = torch.cat([sd[m + "uk"], sd[m + "uv"]])
        out[mixer + "w_out.weight"] = sd[m + "o"]
        out[dst + "norm1b"] = sd[src + "norm1"].float()
        if spec.moe:
            out[dst + "norm2b"] = sd[src + "norm2"].float()
            out[dst + "experts.router"] = sd[src + "mlp.router"]
            for part in ("up", "down"):
                out[f"{dst}experts.{part}"] = torch.stack(
                    [sd[f"{src}mlp.e{e}.{part}"]
                     for e in range(spec.moe.experts)])
        if cfg.side_dim:
            out[dst + "side.w_gate"] = sd[src + "side.gate"]
            out[dst + "side.w_proj.weight"] = sd[src + "side.proj"]
            out[dst + "side.norm"] = sd[src + "side.norm"].float()
    return out


def uniform(name: str, width: int, depth: int, heads: int, dim: int,
            rot_dim: int, rank: int, moe: MoESpec, vocab: int, side_dim: int,
            own: int) -> ModelConfig:
    """A regular model: the first `own` layers have latents of their own, the
    others share those of the last of them."""
    rot = RotarySpec(10000.0, rot_dim)

    def mixer(i: int) -> LatentAttentionSpec:
        return LatentAttentionSpec(
            heads, dim, rot_dim, dim, rank, (dim + rot_dim) ** -0.5, rot,
            own - 1 if i >= own else None, True)
    return model_config(name, width, vocab, 1e-5, 1.0, side_dim,
                        [LayerSpec(mixer(i), 0, moe) for i in range(depth)])


# Shapes of real layers, random weights only: for benches and tests. A token's
# experts are together as large as the dense feed-forward of the model whose
# size they name, so a token costs about as much.
register(uniform("guronex-tiny", 256, 4, 4, 64, 32, 128,
                 MoESpec(8, 2, 320, 4, 2), 512, 32, 2))
register(uniform("guronex-1b", 2048, 16, 16, 128, 64, 512,
                 MoESpec(32, 6, 1408, 8, 4), 32000, 128, 8))
register(uniform("guronex-7b", 4096, 32, 32, 128, 64, 512,
                 MoESpec(32, 8, 2048, 8, 4), 32000, 256, 16))
