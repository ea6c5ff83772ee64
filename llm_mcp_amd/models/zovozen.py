"""Zovozen decoder: attention with talking heads in chunks beside a matrix
memory, dense or mixture-of-experts feed-forwards.  A sublayer reads the
residual stream itself; its output is RMS-normed (plain weight) and added.  The
logits use the embedding table.  Everything else is ``models.layerlist``."""
from __future__ import annotations

from .feedforward import ReluSquaredMLP, SoftmaxGroupMoE
from .layerlist import LayerListModel
from .mixers import TalkingMemoryMixer


class ZovozenModel(LayerListModel):
    mixers = {"parallel": TalkingMemoryMixer}
    feedforwards = {"dense": ReluSquaredMLP, "moe": SoftmaxGroupMoE}
    tail = ""
    tied_head = True


tensor_shapes = ZovozenModel.tensor_shapes
