"""Model classes by configuration: what an engine instantiates for a config."""
from __future__ import annotations


def model_class(cfg):
    """The decoder class that serves ``cfg``."""
    from .config import LlamaConfig, ZegopelConfig
    if isinstance(cfg, ZegopelConfig):
        from .zegopel import ZegopelModel
        return ZegopelModel
    if isinstance(cfg, LlamaConfig):
        from .llama import LlamaModel
        return LlamaModel
    raise ValueError(f"{type(cfg).__name__}: not a generative model")


def build_model(cfg, device, **kw):
    return model_class(cfg)(cfg, device, **kw)
