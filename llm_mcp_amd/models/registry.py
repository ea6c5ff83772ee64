"""Model classes by configuration: what an engine instantiates for a config."""
from __future__ import annotations


def model_class(cfg):
    """The decoder class that serves ``cfg``."""
    from .config import LayerListConfig, LlamaConfig
    if isinstance(cfg, LayerListConfig):
        return layer_list_class(cfg.family)
    if isinstance(cfg, LlamaConfig):
        from .llama import LlamaModel
        return LlamaModel
    raise ValueError(f"{type(cfg).__name__}: not a generative model")


def layer_list_class(family: str):
    """The class of a family whose configuration lists its layers."""
    if family == "zegopel":
        from .zegopel import ZegopelModel
        return ZegopelModel
    if family == "pikesun":
        from .pikesun import PikesunModel
        return PikesunModel
    if family == "refolix":
        from .refolix import RefolixModel
        return RefolixModel
    if family == "zovozen":
        from .zovozen import ZovozenModel
        return ZovozenModel
    raise ValueError(f"{family}: not a layer-list family")


def build_model(cfg, device, **kw):
    return model_class(cfg)(cfg, device, **kw)
