"""Pikesun decoder: gated linear recurrences and windowed latent attention with
dense or mixture-of-experts feed-forwards.  A sublayer reads the residual
stream itself; its output is RMS-normed (plain weight) and added times a
constant.  Layers may share weights.  Everything else is ``models.layerlist``."""
from __future__ import annotations

from .feedforward import GeluMLP, MixtureOfExperts
from .layerlist import LayerListModel
from .mixers import LatentAttentionMixer, RGLRUMixer


class PikesunModel(LayerListModel):
    mixers = {"rglru": RGLRUMixer, "latent_attention": LatentAttentionMixer}
    feedforwards = {"dense": GeluMLP, "moe": MixtureOfExperts}
    tail = ""


tensor_shapes = PikesunModel.tensor_shapes
