"""Token mixers and feed-forward of layer-list decoders (``models.zegopel``).

A mixer is built for one layer from its ``mixer`` dict; it names its
checkpoint tensors and shapes (``shapes``), fuses them into served weights
(``load``), declares what it keeps per sequence -- ``kv`` (heads, head size) in
the paged cache, ``state`` tensors in the state slots -- and runs on a step's
rows: ``forward(h, inp, cache, state)`` -> the mixer's output rows.

Served layouts:
* every mixer has ONE input projection (its projections fused by rows) and one
  output projection (``proj``: their served shapes); sections start at multiples of 8 rows (zero rows between)
  so row slices stay 16-byte aligned;
* attention heads are padded to D = 64 / 128 / 256 / 512 channels with zero
  rows (and zero output columns), so unequal or odd query / value sizes run on
  the same kernels and cache pages; norms use the true size;
* gains and constants of norms, convolutions and recurrences are fp32.
"""
from __future__ import annotations

import math

import torch

from .. import ops


def _up(n: int, m: int) -> int:
    return -(-n // m) * m


def _fuse_rows(parts: list[torch.Tensor], pads: list[int]) -> torch.Tensor:
    """Concatenate [rows, K] blocks, each padded with zero rows to ``pads``."""
    out = parts[0].new_zeros((sum(pads), parts[0].shape[1]))
    r = 0
    for t, p in zip(parts, pads):
        out[r:r + t.shape[0]] = t
        r += p
    return out


class LightningMixer:
    """Linear attention with a constant decay per head: q, k, v = silu(W h),
    S <- decay S + k v^T, o = S^T q; heads concatenated, RMS-normed, times
    sigmoid(W_g h), projected."""
    kv = None
    q_per_tile = 0

    def __init__(self, m: dict, width: int, eps: float):
        self.H, self.N, self.P, self.eps = m["heads"], m["dim"], m["vdim"], eps
        self.decay = [float(x) for x in m["decay"]]
        if len(self.decay) != self.H:
            raise ValueError("lightning: one decay per head")
        H, N, P = self.H, self.N, self.P
        self.shapes = {"q": (H * N, width), "k": (H * N, width), "v": (H * P, width),
                       "g": (H * P, width), "o": (width, H * P), "norm": (H * P,)}
        self.qk, self.vg = _up(H * N, 8), _up(H * P, 8)
        self.proj = {"in": (2 * (self.qk + self.vg), width), "o": self.shapes["o"]}

    def state_shapes(self, dtype):
        return [((self.H, self.N, self.P), torch.float32)]

    scan_geometry = property(lambda self: (self.H, self.P))

    def load(self, get, put):
        self.w_in = put(_fuse_rows([get("q"), get("k"), get("v"), get("g")],
                                   [self.qk, self.qk, self.vg, self.vg]))
        self.w_o = put(get("o"))
        self.norm = put(get("norm"), fp32=True)
        d = torch.tensor(self.decay, dtype=torch.float64)
        self.decays = (put(d, fp32=True), put(d.log().clamp_min(-1e30), fp32=True))

    def forward(self, h, inp, cache, state):
        qk, vg = self.qk, self.vg
        p = ops.linear(h, self.w_in)
        o = ops.linear_scan(p[:, :qk], p[:, qk:2 * qk], p[:, 2 * qk:2 * qk + vg], state[0],
                            inp.cu_q, inp.context_lens, inp.state_slots, decay=self.decays,
                            silu=True, num_decode=inp.num_decode,
                            segments=inp.aux.get(f"scan{self.scan_geometry}"))
        y = ops.gated_norm(o, p[:, 2 * qk + vg:], self.norm, 1, self.eps, gate_first=False)
        return ops.linear(y, self.w_o, defer=True)


class Mamba2Mixer:
    """State-space mixer (scalar decay per head and token): z | x | B | C | dt
    from one projection, a short convolution with SiLU over x, B and C,
    S <- exp(-exp(A_log) s) S + s B x^T with s = softplus(dt + dt_bias),
    y = S^T C + D x; y silu(z) RMS-normed in parts, projected."""
    kv = None
    q_per_tile = 0

    def __init__(self, m: dict, width: int, eps: float):
        self.H, self.P, self.N, self.G = m["heads"], m["vdim"], m["state"], m["groups"]
        self.taps, self.norm_groups, self.eps = m["conv"], m["norm_groups"], eps
        H, P, N, G = self.H, self.P, self.N, self.G
        if H % G:
            raise ValueError("mamba2: heads must be a multiple of groups")
        self.inner, self.C = H * P, H * P + 2 * G * N
        self.zp, self.cp = _up(self.inner, 8), _up(self.C, 8)
        # a wide projection is rounded up to whole 256-row GEMM tiles
        rows = self.zp + self.cp + _up(H, 8)
        self.dp = (_up(rows, 256) if rows >= 4096 else rows) - self.zp - self.cp
        self.proj = {"in": (self.zp + self.cp + self.dp, width), "o": (width, self.inner)}
        self.shapes = {"in": (2 * self.inner + 2 * G * N + H, width),
                       "conv": (self.C, self.taps), "conv.b": (self.C,), "dt_bias": (H,),
                       "A_log": (H,), "D": (H,), "norm": (self.inner,),
                       "o": (width, self.inner)}

    def state_shapes(self, dtype):
        out = [((self.H, self.N, self.P), torch.float32)]
        if self.taps > 1:
            out.append(((self.taps - 1, self.cp), dtype))
        return out

    scan_geometry = property(lambda self: (self.H, self.P))

    def load(self, get, put):
        w, i, c = get("in"), self.inner, self.C
        self.w_in = put(_fuse_rows([w[:i], w[i:i + c], w[i + c:]], [self.zp, self.cp, self.dp]))
        conv = torch.zeros((self.taps, self.cp))
        conv[:, :c] = get("conv").float().t()
        cb = torch.zeros(self.cp)
        cb[:c] = get("conv.b").float()
        self.conv, self.conv_b = put(conv, fp32=True), put(cb, fp32=True)
        self.dt_bias = put(get("dt_bias"), fp32=True)
        self.neg_a = put(-torch.exp(get("A_log").float()), fp32=True)
        self.D = put(get("D"), fp32=True)
        self.norm = put(get("norm"), fp32=True)
        self.w_o = put(get("o"))

    def forward(self, h, inp, cache, state):
        i, gn = self.inner, self.G * self.N
        p = ops.linear(h, self.w_in)
        z, u, dt = p[:, :i], p[:, self.zp:self.zp + self.cp], p[:, self.zp + self.cp:]
        c = ops.short_conv(u, self.conv, state[1] if self.taps > 1 else None, inp.cu_q,
                           inp.context_lens, inp.state_slots, bias=self.conv_b, silu=True,
                           tiles=inp.aux.get("conv"))
        y = ops.linear_scan(c[:, i + gn:i + 2 * gn], c[:, i:i + gn], c[:, :i], state[0], inp.cu_q,
                            inp.context_lens, inp.state_slots, heads_per_group=self.H // self.G,
                            dt=(dt, self.dt_bias, self.neg_a), skip=self.D,
                            num_decode=inp.num_decode,
                            segments=inp.aux.get(f"scan{self.scan_geometry}"))
        y = ops.gated_norm(y, z, self.norm, self.norm_groups, self.eps, gate_first=True)
        return ops.linear(y, self.w_o, defer=True)


class ConvAttentionMixer:
    """Softmax attention without rotation: biased q, k, v through a short
    convolution, unit-RMS q and k, a position-dependent query temperature, an
    output gate sigmoid(W_g h)."""
    scan_geometry = None

    def __init__(self, m: dict, width: int, eps: float):
        self.Hq, self.Hkv, self.dk, self.dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.taps, self.scale, self.eps = m["conv"], float(m["scale"]), eps
        t = m.get("q_temp") or {"coef": 0.0, "every": 1}
        self.temp = (float(t["coef"]), float(t["every"]))
        if self.Hq % self.Hkv:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        D = 64
        while D < max(self.dk, self.dv):
            D *= 2
        if D > 512:
            raise ValueError("attention: head sizes up to 512")
        self.D = D
        H, G, dk, dv = self.Hq, self.Hkv, self.dk, self.dv
        self.shapes = {"q": (H * dk, width), "k": (G * dk, width), "v": (G * dv, width),
                       "q.b": (H * dk,), "k.b": (G * dk,), "v.b": (G * dv,),
                       "q.conv": (H * dk, self.taps), "k.conv": (G * dk, self.taps),
                       "v.conv": (G * dv, self.taps), "g": (H * dv, width),
                       "o": (width, H * dv)}
        self.kv = (G, D)
        self.qkv = (H + 2 * G) * D
        self.proj = {"in": (self.qkv + H * D, width), "o": (width, H * D)}
        # the MFMA attention kernels: head sizes 64 / 128, up to 16 query heads per kv head
        self.mfma_geometry = D in (64, 128) and H // G <= 16
        # queries per prefill workgroup (4 waves)
        self.q_per_tile = (4 * (4 if D == 64 else ops.PREFILL_GROUPS_PER_WAVE) * (16 // (H // G))
                           if self.mfma_geometry else 0)

    def state_shapes(self, dtype):
        return [((self.taps - 1, self.qkv), dtype)] if self.taps > 1 else []

    def _heads(self, t, n, d):
        """[n * d, ...] rows -> [n * D, ...], each head padded with zeros."""
        out = t.new_zeros((n, self.D) + tuple(t.shape[1:]))
        out[:, :d] = t.reshape((n, d) + tuple(t.shape[1:]))
        return out.reshape((n * self.D,) + tuple(t.shape[1:]))

    def load(self, get, put):
        H, G, dk, dv = self.Hq, self.Hkv, self.dk, self.dv
        geo = (("q", H, dk), ("k", G, dk), ("v", G, dv))
        self.w_in = put(torch.cat([self._heads(get(n), c, d) for n, c, d in geo]
                                  + [self._heads(get("g"), H, dv)]))
        self.in_bias = put(torch.cat([self._heads(get(n + ".b"), c, d) for n, c, d in geo]),
                           fp32=True)
        self.conv = put(torch.cat([self._heads(get(n + ".conv"), c, d) for n, c, d in geo])
                        .float().t(), fp32=True)
        self.w_o = put(self._heads(get("o").t().contiguous(), H, dv).t())

    def forward(self, h, inp, cache, state):
        kc, vc = cache
        p = ops.linear(h, self.w_in)
        gate = p[:, self.qkv:]
        q = ops.conv_qkv_cache(p[:, :self.qkv], self.conv, self.in_bias,
                               state[0] if self.taps > 1 else None, inp.cu_q, inp.context_lens,
                               inp.state_slots, inp.positions, inp.slots, kc, vc, self.Hq,
                               self.dk, self.eps, self.temp, tiles=inp.aux.get("conv"))
        T, nd = inp.num_tokens, inp.num_decode
        if not self.mfma_geometry or q.dtype != torch.bfloat16:
            a = ops.attention_any(q, kc, vc, inp.block_tables, inp.cu_q, inp.context_lens,
                                  inp.positions, self.scale, self.Hq, gate=gate)
            return ops.linear(a, self.w_o, defer=True)
        a = torch.empty((T, self.Hq * self.D), dtype=q.dtype, device=q.device)
        if nd:
            ops.paged_decode_attention(q[:nd], kc, vc, inp.block_tables, inp.context_lens,
                                       self.scale, a[:nd], inp.decode_ws, inp.part_tokens,
                                       Hq=self.Hq, order=inp.decode_order, gate=gate[:nd],
                                       precise=True)
        if T > nd:
            ops.paged_prefill_attention(q, kc, vc, inp.block_tables[nd:], inp.cu_q[nd:],
                                        inp.context_lens[nd:], inp.aux[f"attn{self.q_per_tile}"],
                                        self.scale, a, Hq=self.Hq, q_per_tile=self.q_per_tile,
                                        gate=gate, precise=True)
        return ops.linear(a, self.w_o, defer=True)


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
        down = get("down")
        w = down.new_zeros((down.shape[0], self.fp))
        w[:, :self.ff] = down
        self.w_down = put(w)

    def forward(self, h):
        return ops.linear(ops.linear_relu_glu(h, self.w_gu), self.w_down, defer=True)


MIXERS = {"lightning": LightningMixer, "mamba2": Mamba2Mixer, "attention": ConvAttentionMixer}


def init_std(name: str, shape: tuple, depth: int) -> tuple[float, float]:
    """(mean, std) of a tensor's random initialisation (benchmarks, tests)."""
    leaf = name.rsplit(".", 1)[-1]
    if leaf in ("o", "down"):
        return 0.0, 0.02 / math.sqrt(2 * depth)
    if leaf == "conv":
        return 1.0 / shape[-1], 0.2
    if name.endswith(".mix.norm") or leaf == "D":
        return 1.0, 0.1
    if leaf == "A_log":
        return 0.5, 0.5
    if leaf == "dt_bias":
        return -3.0, 1.0
    if name == "embed":
        return 0.0, 1.0
    return 0.0, 0.02
