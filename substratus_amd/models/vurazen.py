"""Vurazen: a decoder whose layers add a mixer and a feed-forward to the
residual together, both reading one layer norm of it.

Mixers are selective scans (Mamba), lightning attention, and windowed
attention beside a gated delta rule; feed-forwards are dense or mixtures of
experts with a shared one. Some layers run several times in a row. See
models/hybrid.py for the layers themselves; this module maps config.json and
checkpoint names onto them.
"""

from __future__ import annotations

import torch

from .config import ModelConfig, register, register_architecture
from .kakovik import stack_rows
from .layers import (ConvAttentionSpec, DeltaSpec, GluSpec, LayerSpec,
                     LightningSpec, LoopSpec, MambaSpec, MixerSpec, MoESpec,
                     RotarySpec, SideBySideSpec)

FAMILY = "vurazen"


def _attention(m: dict, i: int) -> ConvAttentionSpec:
    rot = RotarySpec(float(m["rot"]["base"]), m["rot"]["dims"], True)
    if rot.dims % 2 or rot.dims > m["dim"]:
        raise ValueError(f"layer {i}: cannot rotate {rot.dims} of {m['dim']} "
                         "elements")
    if m.get("vdim", m["dim"]) != m["dim"]:
        raise ValueError(f"layer {i}: values of {m['vdim']} elements cannot "
                         f"be the keys, which have {m['dim']}")
    return ConvAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
        scale=float(m["scale"]), taps=m["conv"], rot=rot,
        window=m["mask"]["size"], keep=m["mask"].get("keep_first", 0),
        softcap=float(m.get("softcap") or 0.0), sink=True)


def _delta(m: dict, i: int, shapes: dict) -> DeltaSpec:
    def rank(name):
        return shapes.get(f"l{i}.mix.right.{name}", (m["dim"],))[0]
    return DeltaSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                     m["conv"], rank("a1"), rank("g1"))


def _mixer(doc: dict, i: int, shapes: dict) -> MixerSpec:
    m = doc["mixer"]
    if doc["type"] == "mamba1":
        return MambaSpec(m["inner"], m["state"], m["dt_rank"], m["conv"])
    if doc["type"] == "lightning":
        return LightningSpec(m["heads"], m["dim"], m["vdim"],
                             tuple(map(float, m["decay"])))
    if doc["type"] == "parallel":
        for side in (m["left"], m["right"]):
            if side["heads"] % side["kv_heads"]:
                raise ValueError(f"layer {i}: {side['heads']} heads on "
                                 f"{side['kv_heads']}")
        return SideBySideSpec(_attention(m["left"], i),
                              _delta(m["right"], i, shapes),
                              float(m["left_scale"]), float(m["right_scale"]))
    raise ValueError(f"layer {i}: unknown mixer {doc['type']!r}")


def _layer(doc: dict, i: int, shapes: dict) -> LayerSpec:
    mixer, mlp = _mixer(doc, i, shapes), doc["mlp"]
    if mlp is None:
        return LayerSpec(mixer)
    if mlp["kind"] == "dense":
        return LayerSpec(mixer, mlp["ff"], glu=GluSpec("relu"))
    if mlp["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")

    def glu(part):
        return GluSpec("clamped", float(part["limit"]))
    shared = mlp.get("shared")
    return LayerSpec(mixer, moe=MoESpec(
        mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"],
        glu=glu(mlp["expert"]), over_chosen=True, bias=True,
        shared_ff=shared["ff"] if shared else 0,
        shared_glu=glu(shared) if shared else None))


@register_architecture("Vurazen")
def parse(doc: dict, shapes: dict, name: str) -> ModelConfig:
    loop = doc.get("loop")
    return model_config(
        name, doc["width"], doc["vocab"], doc["norm"]["eps"],
        float(doc["embedding"]["scale"]), float(doc["logit_softcap"] or 0.0),
        LoopSpec(loop["start"], loop["stop"], loop["times"]) if loop else None,
        [_layer(d, i, shapes) for i, d in enumerate(doc["layers"])])


def model_config(name: str, width: int, vocab: int, eps: float,
                 embed_scale: float, softcap: float, loop: LoopSpec | None,
                 layers: list[LayerSpec]) -> ModelConfig:
    if loop and not 0 <= loop.start <= loop.stop <= len(layers):
        raise ValueError(f"cannot loop over layers {loop.start} to "
                         f"{loop.stop} of {len(layers)}")
    att = [s.mixer.left for s in layers if isinstance(s.mixer, SideBySideSpec)]
    cfg = ModelConfig(
        name=name, family=FAMILY, hidden_size=width,
        intermediate_size=max((s.ff or (s.moe.ff * s.moe.top + s.moe.shared_ff
                                        if s.moe else 0) for s in layers),
                              default=0),
        num_layers=len(layers), num_heads=max((a.heads for a in att),
                                              default=0),
        num_kv_heads=max((a.kv_heads for a in att), default=0),
        head_dim=max((a.dim for a in att), default=0), vocab_size=vocab,
        max_position_embeddings=1 << 20, layer_norm_eps=eps,
        layers=tuple(layers), parallel_block=True, embed_scale=embed_scale,
        logit_softcap=softcap, loop=loop)
    if not cfg.runs():
        raise ValueError("no layer ever runs")
    return cfg


def is_vurazen_state_dict(sd: dict) -> bool:
    return "embed" in sd and "l0.norm1.b" in sd


def _mixer_weights(spec: MixerSpec, sd: dict, m: str
                   ) -> tuple[torch.Tensor, torch.Tensor, dict]:
    """(input projection's rows, output projection, the core's weights)."""
    def f32(**names):
        return {ours: sd[m + theirs].float()
                for ours, theirs in names.items()}

    def stacked(*names):
        return torch.cat([sd[m + n] for n in names])
    if isinstance(spec, SideBySideSpec):
        parts = [_mixer_weights(s, sd, m + side + ".")
                 for side, s in (("left", spec.left), ("right", spec.right))]
        return torch.cat([stack_rows([parts[0][0]]), parts[1][0]]), \
            torch.cat([p[1] for p in parts], 1), \
            {f"{side}.{k}": v for side, p in zip(("left", "right"), parts)
             for k, v in p[2].items()}
    if isinstance(spec, ConvAttentionSpec):
        own = {"bias": stacked("q.b", "k.b").float(),
               "conv": stacked("q.conv", "k.conv").float(), **f32(sink="sink")}
        return stacked("q", "k"), sd[m + "o"], own
    if isinstance(spec, DeltaSpec):
        own = {"conv": stacked("q.conv", "k.conv", "v.conv").float(),
               "a2": sd[m + "a2"], "g2": sd[m + "g2"],
               **f32(dt_bias="dt_bias", A_log="A_log", norm="norm")}
        return torch.cat([stack_rows([stacked("q", "k", "v")]),
                          stack_rows([sd[m + "a1"]]),
                          stack_rows([sd[m + "g1"]]), sd[m + "b"]]), \
            sd[m + "o"], own
    if isinstance(spec, MambaSpec):
        own = {"w_x.weight": stack_rows([sd[m + "x"]]), "w_dt": sd[m + "dt"],
               **f32(conv="conv", conv_bias="conv.b", dt_bias="dt.b",
                     A_log="A_log", D="D")}
        return sd[m + "in"], sd[m + "o"], own
    return stacked("q", "k", "v", "g"), sd[m + "o"], f32(norm="norm")


def vurazen_to_native(sd: dict, cfg: ModelConfig) -> dict:
    """Checkpoint names -> HybridLM names: a layer's projections of its norm
    are stacked, those onto the residual stand side by side, as do its
    experts; small tensors that take part in 32-bit arithmetic become
    float32."""
    out = {"embed.weight": sd["embed"], "head.weight": sd["head"],
           "final_norm": sd["final.norm"].float(),
           "final_norm_bias": sd["final.norm.b"].float()}
    if cfg.loop:
        out["loop_step"] = sd["loop.step"].float()
    for i, spec in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        out[dst + "norm1"] = sd[src + "norm1"].float()
        out[dst + "norm1_bias"] = sd[src + "norm1.b"].float()
        w_in, w_out, own = _mixer_weights(spec.mixer, sd, src + "mix.")
        for k, v in own.items():
            out[f"{dst}mixer.{k}"] = v
        rows, ff = [stack_rows([w_in])], src + "mlp."
        if spec.moe:
            out[dst + "experts.router"] = sd[ff + "router"]
            out[dst + "experts.router_bias"] = sd[ff + "router.b"].float()
            out[dst + "experts.up"] = torch.stack([
                torch.stack([sd[f"{ff}e{e}.gate"], sd[f"{ff}e{e}.up"]], 1)
                .flatten(0, 1) for e in range(spec.moe.experts)])
            out[dst + "experts.down"] = torch.stack(
                [sd[f"{ff}e{e}.down"] for e in range(spec.moe.experts)])
            ff += "shared."
        if spec.ff or spec.moe and spec.moe.shared_ff:
            rows += [sd[ff + "gate"], sd[ff + "up"]]
            w_out = torch.cat([w_out, sd[ff + "down"]], 1)
        out[dst + "w_in.weight"] = stack_rows(rows)
        out[dst + "w_out.weight"] = w_out.contiguous()
    return out


def uniform(name: str, width: int, depth: int, heads: int, dim: int, ff: int,
            vocab: int, window: int, moe: MoESpec, delta_heads: int,
            lightning_heads: int, lightning_dim: int) -> ModelConfig:
    """A regular model: of every four layers two are selective scans with a
    dense feed-forward, one is lightning attention and one windowed attention
    beside a delta rule, both with experts."""
    inner = 2 * width
    scan = LayerSpec(MambaSpec(inner, 16, max(width // 16, 1), 4), ff,
                     glu=GluSpec("relu"))
    att = ConvAttentionSpec(heads, heads, dim, dim ** -0.5, 4,
                            RotarySpec(10000.0, dim, True), window, 4, 30.0,
                            True)
    delta = DeltaSpec(delta_heads, delta_heads, dim, dim, 4, dim, dim)
    both = LayerSpec(SideBySideSpec(att, delta, 0.7, 0.7), moe=moe)
    light = LayerSpec(LightningSpec(
        lightning_heads, lightning_dim, lightning_dim,
        tuple(1 - 2.0 ** (-3 - 5 * h / lightning_heads)
              for h in range(lightning_heads))), moe=moe)
    return model_config(name, width, vocab, 1e-5, 1.0, 30.0, None,
                        [(scan, both, scan, light)[i % 4]
                         for i in range(depth)])


def _moe(experts: int, top: int, ff: int, shared: int) -> MoESpec:
    glu = GluSpec("clamped", 7.0)
    return MoESpec(experts, top, ff, glu=glu, over_chosen=True, bias=True,
                   shared_ff=shared, shared_glu=glu)


# Shapes of real layers, random weights only: for benches and tests. A token's
# experts, the shared one included, are together as large as the dense
# feed-forward of the model whose size they name.
register(uniform("vurazen-tiny", 256, 4, 4, 64, 704, 512, 128,
                 _moe(8, 2, 256, 192), 2, 4, 64))
register(uniform("vurazen-1b", 2048, 16, 16, 128, 5632, 32000, 1024,
                 _moe(32, 6, 768, 1024), 16, 16, 128))
register(uniform("vurazen-7b", 4096, 32, 32, 128, 11008, 32000, 1024,
                 _moe(32, 8, 1024, 2816), 32, 32, 128))
