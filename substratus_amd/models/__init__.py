from .config import ModelConfig, get_config, register
from . import ditalorn as _ditalorn  # registers the architecture, its models
from . import guronex as _guronex  # the same
from . import kakovik as _kakovik  # the same
from . import vurazen as _vurazen  # the same
from .hybrid import HybridLM
from .model import CausalLM


def build_model(cfg: ModelConfig, device=None, dtype=None):
    """The model class a config calls for, with uninitialised weights."""
    cls = HybridLM if cfg.layers else CausalLM
    return cls(cfg, device=device, dtype=dtype)
