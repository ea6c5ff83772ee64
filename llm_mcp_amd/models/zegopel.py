"""Zegopel decoder: linear-attention, state-space and convolved-attention
mixers and ReLU-gated feed-forwards, each between two norms (RMS norms whose
weight w acts as 1 + w).  Everything else is ``models.layerlist``."""
from __future__ import annotations

from .feedforward import ReluGLU
from .layerlist import LayerListModel
from .mixers import ConvAttentionMixer, LightningMixer, Mamba2Mixer


class ZegopelModel(LayerListModel):
    mixers = {"lightning": LightningMixer, "mamba2": Mamba2Mixer, "attention": ConvAttentionMixer}
    feedforwards = {"dense": ReluGLU}
    zero_centred = True


tensor_shapes = ZegopelModel.tensor_shapes
