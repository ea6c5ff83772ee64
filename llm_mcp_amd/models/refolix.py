"""Refolix decoder: retention, and windowed attention beside a gated delta rule,
with mixture-of-experts feed-forwards.  A sublayer reads the residual stream
itself; its output, scaled per channel, is added to a multiple of the stream and
the sum is layer-normed.  The logits are scaled and softly capped.  Everything
else is ``models.layerlist``."""
from __future__ import annotations

from .. import ops
from .feedforward import GroupRoutedMoE
from .layerlist import LayerListModel
from .mixers import ParallelMixer, RetentionMixer


class RefolixModel(LayerListModel):
    mixers = {"parallel": ParallelMixer, "retention": RetentionMixer}
    feedforwards = {"moe": GroupRoutedMoE}
    tail = ""
    layer_scale = "ls"

    def _join(self, x, y, post, pre, rows=None):
        w, scale = post or (None, None)
        return ops.sum_norm(x, self.cfg.rms_eps, y, self.cfg.postln_alpha, scale, w, w_pre=pre,
                            rows=rows, dtype=self.dtype)

    def _logits(self, h):
        return ops.soft_cap(ops.linear(h, self.head), self.cfg.logit_scale,
                            self.cfg.logit_softcap)


tensor_shapes = RefolixModel.tensor_shapes
