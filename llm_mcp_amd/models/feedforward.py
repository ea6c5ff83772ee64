"""Feed-forwards of layer-list decoders (``models.layerlist``).

Same protocol as the mixers: ``shapes`` (checkpoint tensors), ``proj`` (served
projections), ``load`` and ``forward(h)`` -> the output rows, or something
``ops.sandwich_norm`` sums itself (``ops.Partials``, ``ops.Mixture``).
"""
from __future__ import annotations

import torch

from .. import ops
from .mixers import _fuse_rows, _up


def _pad_cols(w: torch.Tensor, cols: int) -> torch.Tensor:
    return w if w.shape[-1] == cols else torch.nn.functional.pad(w, (0, cols - w.shape[-1]))


class ReluGLU:
    """W_down (relu(W_gate h) * (W_up h))"""

    def __init__(self, m: dict, width: int):
        self.ff, self.fp = m["ff"], _up(m["ff"], 16)
        self.shapes = {"gate": (self.ff, width), "up": (self.ff, width),
                       "down": (width, self.ff)}
        self.proj = {"gate_up": (2 * self.fp, width), "down": (width, self.fp)}

    def load(self, get, put):
        self.w_gu = put(ops.interleave_gate_up(
            _fuse_rows([get("gate"), get("up")], [self.fp, self.fp]), 16))
        self.w_down = put(_pad_cols(get("down"), self.fp))

    def forward(self, h):
        return ops.linear(ops.linear_relu_glu(h, self.w_gu), self.w_down, defer=True)


class GeluMLP:
    """W_down gelu(W_up h), the tanh form"""

    def __init__(self, m: dict, width: int):
        self.ff, self.fp = m["ff"], _up(m["ff"], 16)
        self.shapes = {"up": (self.ff, width), "down": (width, self.ff)}
        self.proj = {"up": (self.fp, width), "down": (width, self.fp)}

    def load(self, get, put):
        self.w_up = put(_fuse_rows([get("up")], [self.fp]))
        self.w_down = put(_pad_cols(get("down"), self.fp))

    def forward(self, h):
        return ops.linear(ops.linear_gelu(h, self.w_up), self.w_down, defer=True)


class MixtureOfExperts:
    """``top`` of ``experts`` clamped GLUs per token in the proportions of a
    softmax of their router logits, plus an optional one for every token:

        g = min(W_gate h, L), u = clamp(W_up h, -L, L), W_down (g sigmoid(1.702 g) (u + 1))

    The shared expert runs as further experts of the routed ones' width that
    every token uses with weight 1: one grouped product covers all of them."""
    glu = (1.702, 1.0)                     # slope of the gate's sigmoid, added to up
    identity = 0                           # routed experts that return their input

    @staticmethod
    def _limit(m: dict) -> float:
        return float(m["limit"])

    def __init__(self, m: dict, width: int):
        self.width, self.kp, self.np = width, _up(width, 64), _up(width, 16)
        self.E, self.top = m["router"]["experts"], m["router"]["top"]
        self.routed = self.E + self.identity
        if not (self.E > 0 and self.identity >= 0 and 0 < self.top <= self.routed):
            raise ValueError("moe: top experts out of range")
        ex, sh = m["expert"], m.get("shared")
        self.ff, self.sff = ex["ff"], sh["ff"] if sh else 0
        self.fp = max(_up(self.ff, 64), _up(-(-self.sff // 8), 64))   # at most 8 shared ones
        self.shared = -(-self.sff // self.fp)          # experts that hold the shared one
        self.limits = [self._limit(ex)] * self.E + ([self._limit(sh)] * self.shared if sh else [])
        self.shapes = {}
        for e in range(self.E):
            self.shapes.update({f"e{e}.gate": (self.ff, width), f"e{e}.up": (self.ff, width),
                                f"e{e}.down": (width, self.ff)})
        self.shapes["router"] = (self.routed, width)
        if sh:
            self.shapes.update({"shared.gate": (self.sff, width), "shared.up": (self.sff, width),
                                "shared.down": (width, self.sff)})
        self.proj = {}

    def load(self, get, put):
        fp, kp = self.fp, self.kp

        def expert(gate, up, down):
            w1 = ops.interleave_gate_up(_fuse_rows([gate, up], [fp, fp]), 16)
            return put(_pad_cols(w1, kp)), put(_pad_cols(_fuse_rows([down], [self.np]), fp))
        each = [expert(*(get(f"e{e}.{n}") for n in ("gate", "up", "down"))) for e in range(self.E)]
        if self.shared:
            gate, up, down = (get(f"shared.{n}") for n in ("gate", "up", "down"))
            for a in range(0, self.sff, fp):
                each.append(expert(gate[a:a + fp], up[a:a + fp], down[:, a:a + fp]))
        self.w1 = ops.pack_grouped(torch.stack([a for a, _ in each]))
        self.w2 = ops.pack_grouped(torch.stack([b for _, b in each]))
        self.limit = put(torch.tensor(self.limits), fp32=True)
        self.router = put(get("router"))

    def _route(self, h):
        return ops.moe_route(h, self.router, self.top, self.shared)

    def forward(self, h):
        r = self._route(h)
        plan = ops.moe_plan(r, self.E + self.shared, self.w1.packed,
                            ops.wide_tiles(self.w1) and ops.wide_tiles(self.w2))
        y = ops.grouped_linear(_pad_cols(h, self.kp), self.w1, plan, gather=True, glu=self.limit,
                               act=self.glu)
        return ops.Mixture(ops.grouped_linear(y, self.w2, plan), plan.pos, r.weights, r.own)


class GroupRoutedMoE(MixtureOfExperts):
    """SiLU GLUs, routed by sigmoid scores s of the logits: the ``top`` largest
    s + correction among the experts of the best groups (ranked by the sum of
    their two largest), in the proportions of their s; the shared expert is
    weighted by the sigmoid of one more logit."""
    glu = (1.0, 0.0)
    shared_gate = True

    @staticmethod
    def _limit(m: dict) -> float:
        return float("inf")

    def __init__(self, m: dict, width: int):
        super().__init__(m, width)
        g = m["router"].get("groups") or {"count": 1, "keep": 1}
        self.groups, self.keep = g["count"], g["keep"]
        n = self.routed
        if (self.groups < 1 or n % self.groups or not 0 < self.keep <= self.groups
                or self.keep * (n // self.groups) < self.top):
            raise ValueError("moe: groups do not fit the experts")
        self.shapes["correction"] = (n,)
        if self.shared and self.shared_gate:
            self.shapes["shared.sg"] = (1, width)

    def load(self, get, put):
        super().load(get, put)
        self.correction = put(get("correction"), fp32=True)
        if self.shared and self.shared_gate:     # the shared expert's logit: one more row
            self.router = put(torch.cat([get("router"), get("shared.sg")]))

    def _route(self, h):
        return ops.moe_route(h, self.router, self.top, self.shared,
                             ops.GroupScores(self.correction, self.groups, self.keep))


class SoftmaxGroupMoE(GroupRoutedMoE):
    """SiLU GLUs, routed by a softmax over the logits of the experts and of
    ``identity`` experts behind them, whose output is their input: the ``top``
    largest s + correction among the experts of the best groups (ranked by the
    largest), with their s as they are; the shared expert has weight 1.  For
    sublayers that read the stream itself."""
    shared_gate = False

    def __init__(self, m: dict, width: int):
        r = m["router"]
        self.identity = int(r.get("identity") or 0)
        super().__init__(m, width)

    def _route(self, h):
        return ops.moe_route(h, self.router, self.top, self.shared,
                             ops.GroupScores(self.correction, self.groups, self.keep, True,
                                             self.identity))


class ReluSquaredMLP:
    """W_down relu(W_up h + b)^2 + b'"""

    def __init__(self, m: dict, width: int):
        self.ff, self.fp = m["ff"], _up(m["ff"], 16)
        self.shapes = {"up": (self.ff, width), "up.b": (self.ff,), "down": (width, self.ff),
                       "down.b": (width,)}
        self.proj = {"up": (self.fp, width), "down": (width, self.fp)}

    def load(self, get, put):
        self.w_up = put(_fuse_rows([get("up")], [self.fp]))
        self.w_down = put(_pad_cols(get("down"), self.fp))
        b = _pad_cols(get("up.b"), self.fp)
        self.up_bias, self.up_bias_row = put(b, fp32=True), put(b)
        self.down_bias = put(get("down.b"), fp32=True)

    def forward(self, h):
        y = ops.linear_relu2(h, self.w_up, self.up_bias, self.up_bias_row)
        return ops.Biased(ops.linear(y, self.w_down, defer=True), self.down_bias)
