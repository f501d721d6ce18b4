"""Checkpoint loading: finds a model folder's weights, translates foreign
tensor names, shards for tensor parallelism, fills the model."""

from __future__ import annotations

import os
from typing import Optional

import torch

from .config import ModelConfig


def find_weights(model_dir: str) -> Optional[str]:
    """model.safetensors of the folder, else of its newest checkpoint
    (trainer artifacts layout)."""
    path = os.path.join(model_dir, "model.safetensors")
    if not os.path.exists(path) and os.path.isdir(model_dir):
        ckpts = sorted((d for d in os.listdir(model_dir)
                        if d.startswith("checkpoint-")),
                       key=lambda d: int(d.split("-")[1]))
        if ckpts:
            path = os.path.join(model_dir, ckpts[-1], "model.safetensors")
    return path if os.path.exists(path) else None


def to_native(sd: dict, mcfg: ModelConfig) -> dict:
    """Checkpoint names of any supported layout -> the model's own."""
    from . import hf_compat as hf
    from .ditalorn import ditalorn_to_native, is_ditalorn_state_dict
    from .guronex import guronex_to_native, is_guronex_state_dict
    from .kakovik import is_kakovik_state_dict, kakovik_to_native
    from .vurazen import is_vurazen_state_dict, vurazen_to_native
    for known, convert in (
            (hf.is_hf_llama_state_dict, hf.hf_llama_to_native),
            (hf.is_hf_falcon_state_dict, hf.hf_falcon_to_native),
            (hf.is_hf_opt_state_dict, hf.hf_opt_to_native),
            (is_ditalorn_state_dict, ditalorn_to_native),
            (is_kakovik_state_dict, kakovik_to_native),
            (is_guronex_state_dict, guronex_to_native),
            (is_vurazen_state_dict, vurazen_to_native)):
        if known(sd):
            return convert(sd, mcfg)
    return sd


def load_weights(model, mcfg: ModelConfig, model_dir: str,
                 device: torch.device, dtype: torch.dtype) -> bool:
    """Load the folder's weights into the model; False if it has none."""
    path = find_weights(model_dir)
    if path is None:
        return False
    from safetensors.torch import load_file
    from ..parallel.comm import state
    sd = to_native(load_file(path), mcfg)
    st = state()
    if st.tp_size > 1:
        from .sharding import shard_state_dict
        sd = shard_state_dict(sd, mcfg, st.tp_rank, st.tp_size)
    kept = {k: v.dtype for k, v in model.state_dict().items()}
    model.load_state_dict(
        {k: v.to(device, kept.get(k, dtype)) for k, v in sd.items()})
    return True
