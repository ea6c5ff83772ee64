"""Token mixers of layer-list decoders (``models.layerlist``).

A mixer is built for one layer from its ``mixer`` dict; it names its
checkpoint tensors and shapes (``shapes``), fuses them into served weights
(``load``), declares what it keeps per sequence -- ``kv`` (heads, key size,
value size) in the paged cache, ``state`` tensors in the state slots -- and runs
on a step's rows: ``forward(h, inp, cache, state)`` -> the mixer's output rows.
What it needs planned on the host for a step's multi-token sequences comes from
``build_plan`` / ``bind_plan``, one plan for all layers of a ``plan_key``
(``StepInputs.aux[plan_key]``).

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
from ..ops import mixers as mixer_ops


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


def _head_size(d: int) -> int:
    """Channels a head of d is padded to in the cache."""
    D = 64
    while D < d:
        D *= 2
    if D > 512:
        raise ValueError("attention: head sizes up to 512")
    return D


class Mixer:
    kv = None                     # (heads, key size, value size) of its cache pages
    q_per_tile = 0
    plan_key = None
    rot = None                    # its rotary positions: ``ops.rope_freqs`` arguments

    def members(self):
        """The mixers it is made of: those that plan and rotate."""
        return [self]

    def state_shapes(self, dtype):
        return []

    def build_plan(self, qlens, ctx, seq0: int):
        """(items to upload, host value) for the sequences from seq0 on."""
        raise NotImplementedError

    def bind_plan(self, dev: dict, host):
        raise NotImplementedError


class ScanMixer(Mixer):
    """Plan of a segmented scan: ``plan_key`` = ("scan", heads, columns)."""

    def build_plan(self, qlens, ctx, seq0):
        _, H, P = self.plan_key
        segs, first, one = mixer_ops.scan_segments(qlens, seq0, H, P)
        return [(f"segs{H, P}", segs), (f"first{H, P}", first)], (len(segs), one)

    def bind_plan(self, dev, host):
        _, H, P = self.plan_key
        return ops.ScanSegments(dev[f"segs{H, P}"], dev[f"first{H, P}"], *host)


class LightningMixer(ScanMixer):
    """Linear attention with a constant decay per head: q, k, v = silu(W h),
    S <- decay S + k v^T, o = S^T q; heads concatenated, RMS-normed, times
    sigmoid(W_g h), projected."""

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

    plan_key = property(lambda self: ("scan", self.H, self.P))

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
                            segments=inp.aux.get(self.plan_key))
        y = ops.gated_norm(o, p[:, 2 * qk + vg:], self.norm, 1, self.eps, gate_first=False)
        return ops.linear(y, self.w_o, defer=True)


class Mamba2Mixer(ScanMixer):
    """State-space mixer (scalar decay per head and token): z | x | B | C | dt
    from one projection, a short convolution with SiLU over x, B and C,
    S <- exp(-exp(A_log) s) S + s B x^T with s = softplus(dt + dt_bias),
    y = S^T C + D x; y silu(z) RMS-normed in parts, projected."""

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

    plan_key = property(lambda self: ("scan", self.H, self.P))

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
                            segments=inp.aux.get(self.plan_key))
        y = ops.gated_norm(y, z, self.norm, self.norm_groups, self.eps, gate_first=True)
        return ops.linear(y, self.w_o, defer=True)


class ConvAttentionMixer(Mixer):
    """Softmax attention without rotation: biased q, k, v through a short
    convolution, unit-RMS q and k, a position-dependent query temperature, an
    output gate sigmoid(W_g h)."""

    def __init__(self, m: dict, width: int, eps: float):
        self.Hq, self.Hkv, self.dk, self.dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.taps, self.scale, self.eps = m["conv"], float(m["scale"]), eps
        t = m.get("q_temp") or {"coef": 0.0, "every": 1}
        self.temp = (float(t["coef"]), float(t["every"]))
        if self.Hq % self.Hkv:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        D = self.D = _head_size(max(self.dk, self.dv))
        H, G, dk, dv = self.Hq, self.Hkv, self.dk, self.dv
        self.shapes = {"q": (H * dk, width), "k": (G * dk, width), "v": (G * dv, width),
                       "q.b": (H * dk,), "k.b": (G * dk,), "v.b": (G * dv,),
                       "q.conv": (H * dk, self.taps), "k.conv": (G * dk, self.taps),
                       "v.conv": (G * dv, self.taps), "g": (H * dv, width),
                       "o": (width, H * dv)}
        self.kv = (G, D, D)
        self.qkv = (H + 2 * G) * D
        self.proj = {"in": (self.qkv + H * D, width), "o": (width, H * D)}
        # the MFMA attention kernels: head sizes 64 / 128, up to 16 query heads per kv head
        self.mfma_geometry = D in (64, 128) and H // G <= 16
        # queries per prefill workgroup (4 waves)
        self.q_per_tile = (4 * (4 if D == 64 else ops.PREFILL_GROUPS_PER_WAVE) * (16 // (H // G))
                           if self.mfma_geometry else 0)
        if self.q_per_tile:
            self.plan_key = ("attn", self.q_per_tile)

    def build_plan(self, qlens, ctx, seq0):
        q = self.q_per_tile
        return [(f"attn{q}", mixer_ops.row_tiles(qlens, q).reshape(-1))], None

    def bind_plan(self, dev, host):
        return dev[f"attn{self.q_per_tile}"]

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
                                        inp.context_lens[nd:], inp.aux[self.plan_key],
                                        self.scale, a, Hq=self.Hq, q_per_tile=self.q_per_tile,
                                        gate=gate, precise=True)
        return ops.linear(a, self.w_o, defer=True)


class RGLRUMixer(ScanMixer):
    """Gated linear recurrence between two branches: y = gelu(W_y h + b_y) and
    u = conv(W_x h + b_x); gates r, i = sigmoid of block-diagonal maps of u;
    log a = -8 r softplus(lam), S <- a S + sqrt(1 - a^2) i u; W_o (S y).

    Channels are served in blocks padded to powers of two from 32 (zero weights:
    a padded channel stays zero)."""

    def __init__(self, m: dict, width: int, eps: float):
        self.W, self.n, self.taps = m["width"], m["blocks"], m["conv"]
        if self.W % self.n:
            raise ValueError("rglru: width must be a multiple of blocks")
        W, n = self.W, self.n
        self.bs = W // n
        self.bp = 1 << max(5, (self.bs - 1).bit_length())
        self.C = n * self.bp
        self.shapes = {"y": (W, width), "y.b": (W,), "x": (W, width), "x.b": (W,),
                       "conv": (W, self.taps), "conv.b": (W,), "ra": (n, self.bs, self.bs),
                       "ra.b": (n, self.bs), "ri": (n, self.bs, self.bs), "ri.b": (n, self.bs),
                       "lam": (W,), "o": (width, W)}
        self.proj = {"in": (2 * self.C, width), "o": (width, self.C)}
        self.plan_key = ("scan", -(-self.C // ops.RGLRU_TILE), 1)

    def state_shapes(self, dtype):
        out = [((self.C,), torch.float32)]
        if self.taps > 1:
            out.append(((self.taps - 1, self.C), dtype))
        return out

    def _blocks(self, t):
        """[W, ...] channel rows -> [C, ...], each block padded with zeros."""
        out = t.new_zeros((self.n, self.bp) + tuple(t.shape[1:]))
        out[:, :self.bs] = t.reshape((self.n, self.bs) + tuple(t.shape[1:]))
        return out.reshape((self.C,) + tuple(t.shape[1:]))

    def load(self, get, put):
        def vec(name):
            return put(self._blocks(get(name).reshape(-1)), fp32=True)
        self.w_in = put(torch.cat([self._blocks(get("y")), self._blocks(get("x"))]))
        self.y_b, self.x_b, self.conv_b = vec("y.b"), vec("x.b"), vec("conv.b")
        self.conv = put(self._blocks(get("conv")).float().t(), fp32=True)
        gates = torch.stack([get("ra"), get("ri")], 1)              # [n, 2, out, in]
        pad = self.bp - self.bs
        gates = torch.nn.functional.pad(gates, (0, pad, 0, pad)).reshape(self.n, 2 * self.bp, -1)
        self.gates = ops.pack_grouped(put(gates, fp32=self.bp > ops.RGLRU_MAX_BLOCK))
        self.gate_b = put(torch.stack([self._blocks(get(k).reshape(-1).float())
                                       for k in ("ra.b", "ri.b")]), fp32=True)
        lam = get("lam").double()
        self.log_a = put(self._blocks(-8.0 * torch.nn.functional.softplus(lam)), fp32=True)
        self.w_o = put(self._blocks(get("o").t().contiguous()).t())

    def forward(self, h, inp, cache, state):
        C = self.C
        p = ops.linear(h, self.w_in)
        u = ops.short_conv(p[:, C:], self.conv, state[1] if self.taps > 1 else None, inp.cu_q,
                           inp.context_lens, inp.state_slots, bias=self.conv_b,
                           in_bias=self.x_b, tiles=inp.aux.get("conv"))
        y = ops.rglru(u, p[:, :C], self.y_b, self.gates, self.gate_b, self.log_a, state[0],
                      inp.cu_q, inp.context_lens, inp.state_slots, num_decode=inp.num_decode,
                      segments=inp.aux.get(self.plan_key))
        return ops.linear(y, self.w_o, defer=True)


class LatentAttentionMixer(Mixer):
    """Latent attention with a sliding window and an output gate: queries
    W_uq norm(W_dq h); keys and values W_uk c, W_uv c of a normed latent c, plus
    a position-rotated key part common to the heads.  A token's cache page row
    is [c | rotated key].

    Decode rows score latents: q W_uk against c, and W_uv the weighted sum of
    latents.  Prompt rows expand the keys and values of the rows they see."""
    Hkv = 1

    def __init__(self, m: dict, width: int, eps: float):
        self.Hq, self.dn, self.dr, self.dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
        self.R, self.qr, self.scale, self.eps = m["kv_rank"], m["q_rank"], float(m["scale"]), eps
        self.window = int(m["mask"]["size"])
        rot = m["rot"]
        if rot["dims"] != self.dr or self.dr % 2 or self.window < 1:
            raise ValueError("latent_attention: rot.dims = rot_dim, even; a window of at least 1")
        H = self.Hq
        self.rot = (float(rot["base"]), self.dr)
        self.D = self.Rp = next((r for r in (64, 128, 256, 512) if r >= self.R), _up(self.R, 64))
        self.xp = _up(self.dr, 64)
        self.np, self.vp, self.qp = _up(self.dn, 64), _up(self.dv, 64), _up(self.qr, 64)
        self.shapes = {"dq": (self.qr, width), "dq.norm": (self.qr,),
                       "uq": (H * (self.dn + self.dr), self.qr),
                       "dkv": (self.R + self.dr, width), "dkv.norm": (self.R,),
                       "uk": (H * self.dn, self.R), "uv": (H * self.dv, self.R),
                       "g": (H * self.dv, width), "o": (width, H * self.dv)}
        self.kv = (1, self.Rp + self.xp, 0)
        rows = self.qp + self.Rp + self.xp + H * self.vp
        # a wide projection is rounded up to whole 256-row GEMM tiles
        self.tail = (_up(rows, 256) if rows >= 4096 else rows) - rows
        self.proj = {"in": (rows + self.tail, width), "uq": (H * (self.np + self.xp), self.qp),
                     "o": (width, H * self.vp)}
        self.expand = ops.latent_prefill_ok(self.np, self.xp, self.vp)
        if self.expand:            # prompt rows of bf16 engines
            self.plan_key = ("latent", self.window)

    def build_plan(self, qlens, ctx, seq0):
        w = self.window
        rows, tiles, n = mixer_ops.latent_rows(qlens, ctx, w)
        return [(f"lrows{w}", rows), (f"ltiles{w}", tiles)], n

    def bind_plan(self, dev, host):
        return ops.LatentRows(dev[f"lrows{self.window}"], dev[f"ltiles{self.window}"], host)

    def _heads(self, t, d, p):
        """[H * d, ...] rows -> [H, p, ...], padded with zeros."""
        out = t.new_zeros((self.Hq, p) + tuple(t.shape[1:]))
        out[:, :d] = t.reshape((self.Hq, d) + tuple(t.shape[1:]))
        return out

    def load(self, get, put):
        H, dn, dr, dv, R = self.Hq, self.dn, self.dr, self.dv, self.R
        dkv = get("dkv")
        g = self._heads(get("g"), dv, self.vp).reshape(H * self.vp, -1)
        self.w_in = put(_fuse_rows([get("dq"), dkv[:R], dkv[R:], g],
                                   [self.qp, self.Rp, self.xp, H * self.vp + self.tail]))
        pad = torch.nn.functional.pad
        self.q_norm = put(pad(get("dq.norm"), (0, self.qp - self.qr)), fp32=True)
        self.c_norm = put(pad(get("dkv.norm"), (0, self.Rp - R)), fp32=True)
        uq = get("uq").reshape(H, dn + dr, self.qr)
        q = uq.new_zeros((H, self.np + self.xp, self.qp))
        q[:, :dn, :self.qr] = uq[:, :dn]
        q[:, self.np:self.np + dr, :self.qr] = uq[:, dn:]
        self.w_uq = put(q.reshape(-1, self.qp))
        uk = pad(self._heads(get("uk"), dn, self.np), (0, self.Rp - R))      # [H, np, Rp]
        uv = pad(self._heads(get("uv"), dv, self.vp), (0, self.Rp - R))      # [H, vp, Rp]
        self.absorb = ops.pack_grouped(put(uk.transpose(1, 2).contiguous()))
        self.unfold = ops.pack_grouped(put(uv))
        self.w_kv = put(torch.cat([uk, uv], 1).reshape(-1, self.Rp)) if self.expand else None
        self.w_o = put(self._heads(get("o").t().contiguous(), dv, self.vp)
                       .reshape(H * self.vp, -1).t())

    def forward(self, h, inp, cache, state):
        H, T, nd = self.Hq, inp.num_tokens, inp.num_decode
        pages, ang = cache[0], inp.aux["rot", self.rot]
        p = ops.linear(h, self.w_in)
        a0 = self.qp + self.Rp + self.xp
        gate = p[:, a0:a0 + H * self.vp]
        cq = ops.latent_prep(p, self.qr, self.qp, self.q_norm, self.R, self.c_norm, ang,
                             inp.slots, pages, self.Rp, self.eps)
        q = ops.linear(cq, self.w_uq)
        out = torch.empty((T, H * self.vp), dtype=h.dtype, device=h.device)
        fast = self.expand and q.is_cuda and q.dtype == torch.bfloat16
        rows = inp.aux.get(self.plan_key) if fast else None
        n = nd if rows is not None else T              # rows on latents: the first n
        if n:
            ql = ops.latent_query(q[:n], self.absorb, ang, H, self.np, self.xp, self.Rp)
            o = ops.latent_attention(ql, pages, inp.block_tables, inp.cu_q, inp.positions,
                                     self.scale, self.window, H, self.Rp, ws=inp.decode_ws,
                                     part_tokens=inp.part_tokens, num_decode=nd)
            ops.grouped_heads(o, self.unfold, gate=gate[:n], out=out[:n])
        if rows is not None:
            ops.latent_prefill(q, pages, rows, self.w_kv, ang, inp.block_tables[nd:],
                               inp.cu_q[nd:], inp.context_lens[nd:], self.scale, self.window, H,
                               self.np, self.vp, self.Rp, gate, out)
        return ops.linear(out, self.w_o, defer=True)


def rotary(rot: dict | None, dim: int) -> tuple | None:
    """``Mixer.rot`` of a configuration's rotation of the first ``dims`` of
    ``dim`` channels, with its length scaling."""
    if not rot or not rot["dims"]:
        return None
    if rot["dims"] % 2 or not 0 < rot["dims"] <= dim:
        raise ValueError("rotation: an even number of a head's channels")
    s = rot.get("scaling")
    if s and "original" not in s:               # every frequency divided
        s = (float(s["factor"]),)
    elif s:
        s = (float(s["factor"]), float(s["original"]), float(s["fast"]), float(s["slow"]))
    return (float(rot["base"]), int(rot["dims"])) + (s or ())


def _pairs_together(heads: int, dim: int, rot: tuple | None) -> torch.Tensor:
    """Order of [heads * dim] channels that puts each head's rotated pairs (i, i
    + dims/2) next to each other."""
    i = torch.arange(dim)
    if rot is not None:
        d = rot[1]
        i[:d] = torch.stack([i[:d // 2], i[d // 2:d]], 1).reshape(-1)
    return (torch.arange(heads)[:, None] * dim + i).reshape(-1)


class RetentionMixer(ScanMixer):
    """Linear attention with a constant decay per head on rotated queries and
    keys: S <- decay S + k v^T, o = S^T q with k scaled by dim^-1/2; each head
    divided by its root mean square, times silu(W_g h), projected.

    The rotated channels of q and k are served with the pairs (i, i + dims/2)
    next to each other: scores do not depend on the order of the channels."""

    def __init__(self, m: dict, width: int, eps: float):
        self.H, self.N, self.P, self.eps = m["heads"], m["dim"], m["vdim"], eps
        self.decay = [float(x) for x in m["decay"]]
        if len(self.decay) != self.H:
            raise ValueError("retention: one decay per head")
        H, N, P = self.H, self.N, self.P
        self.rot = rotary(m.get("rot"), N)
        self.shapes = {"q": (H * N, width), "k": (H * N, width), "v": (H * P, width),
                       "g": (H * P, width), "o": (width, H * P)}
        self.qk, self.vg = _up(H * N, 8), _up(H * P, 8)
        self.proj = {"in": (2 * (self.qk + self.vg), width), "o": self.shapes["o"]}

    def state_shapes(self, dtype):
        return [((self.H, self.N, self.P), torch.float32)]

    plan_key = property(lambda self: ("scan", self.H, self.P))

    def _paired(self, w):
        """[H * N, ...] rows with each head's rotated pairs next to each other."""
        return w[_pairs_together(self.H, self.N, self.rot).to(w.device)]

    def load(self, get, put):
        self.w_in = put(_fuse_rows([self._paired(get("q")), self._paired(get("k")), get("v"),
                                    get("g")], [self.qk, self.qk, self.vg, self.vg]))
        self.w_o = put(get("o"))
        self.norm = put(torch.ones(self.H * self.P), fp32=True)
        d = torch.tensor(self.decay, dtype=torch.float64)
        self.decays = (put(d, fp32=True), put(d.log().clamp_min(-1e30), fp32=True))

    def forward(self, h, inp, cache, state):
        qk, vg = self.qk, self.vg
        p = ops.linear(h, self.w_in)
        ang = inp.aux["rot", self.rot] if self.rot else None
        o = ops.linear_scan(p[:, :qk], p[:, qk:2 * qk], p[:, 2 * qk:2 * qk + vg], state[0],
                            inp.cu_q, inp.context_lens, inp.state_slots, decay=self.decays,
                            num_decode=inp.num_decode, segments=inp.aux.get(self.plan_key),
                            angles=ang, k_scale=self.N ** -0.5)
        y = ops.gated_norm(o, p[:, 2 * qk + vg:], self.norm, self.H, self.eps, gate_first=False,
                           silu=True)
        return ops.linear(y, self.w_o, defer=True)


class SoftcapAttentionMixer(Mixer):
    """Softmax attention in a sliding window: q and k RMS-normed per head, their
    first channels rotated (neighbours paired), scores softly capped."""

    def __init__(self, m: dict, width: int, eps: float):
        self.Hq, self.Hkv, self.dk, self.dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.scale, self.eps = float(m["scale"]), eps
        self.cap = float(m.get("softcap") or 0.0)
        mask = m.get("mask")
        self.window = int(mask["size"]) if mask else 0
        if mask and self.window < 1:
            raise ValueError("attention: a window of at least 1")
        if self.Hq % self.Hkv:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        self.rot = rotary(m.get("rot"), self.dk)
        H, G, dk, dv = self.Hq, self.Hkv, self.dk, self.dv
        self.D = _head_size(max(dk, dv))
        self.shapes = {"q": (H * dk, width), "k": (G * dk, width), "v": (G * dv, width),
                       "q.norm": (dk,), "k.norm": (dk,), "o": (width, H * dv)}
        self.kv = (G, self.D, self.D)
        self.rows = (H + 2 * G) * self.D
        self.proj = {"in": (self.rows, width), "o": (width, H * self.D)}
        # the MFMA attention kernels: head sizes 64 / 128, up to 16 query heads per kv head
        self.mfma_geometry = self.D in (64, 128) and H // G <= 16
        # queries per prefill workgroup (4 waves)
        self.q_per_tile = (4 * (4 if self.D == 64 else ops.PREFILL_GROUPS_PER_WAVE)
                           * (16 // (H // G)) if self.mfma_geometry else 0)
        self.plan_key = ("rope_attn", self.q_per_tile)

    def build_plan(self, qlens, ctx, seq0):
        q = self.q_per_tile
        items = [("quads", mixer_ops.row_quads(qlens, ctx, seq0))]
        if q:
            items.append((f"attn{q}", mixer_ops.row_tiles(qlens, q).reshape(-1)))
        return items, None

    def bind_plan(self, dev, host):
        return dev["quads"], dev.get(f"attn{self.q_per_tile}")

    def _heads(self, t, n, d):
        """[n * d, ...] rows -> [n * D, ...], each head padded with zeros."""
        out = t.new_zeros((n, self.D) + tuple(t.shape[1:]))
        out[:, :d] = t.reshape((n, d) + tuple(t.shape[1:]))
        return out.reshape((n * self.D,) + tuple(t.shape[1:]))

    def in_rows(self, get):
        return torch.cat([self._heads(get("q"), self.Hq, self.dk),
                          self._heads(get("k"), self.Hkv, self.dk),
                          self._heads(get("v"), self.Hkv, self.dv)])

    def load(self, get, put, own_projection=True):
        if own_projection:
            self.w_in = put(self.in_rows(get))
        self.q_norm = put(self._heads(get("q.norm"), 1, self.dk), fp32=True)
        self.k_norm = put(self._heads(get("k.norm"), 1, self.dk), fp32=True)
        self.w_o = put(self._heads(get("o").t().contiguous(), self.Hq, self.dv).t())

    def forward(self, h, inp, cache, state):
        return self.mix(ops.linear(h, self.w_in), inp, cache, state)

    def mix(self, p, inp, cache, state):
        """Output rows of projection rows p = [q | k | v | ..]."""
        kc, vc = cache
        quads, tiles = inp.aux.get(self.plan_key, (None, None))
        ang = inp.aux["rot", self.rot] if self.rot else None
        q = ops.norm_rope_cache(p, self.q_norm, self.k_norm, ang, inp.slots, kc, vc, self.Hq,
                                self.dk, self.eps, quads)
        T, nd = inp.num_tokens, inp.num_decode
        if not self.mfma_geometry or q.dtype != torch.bfloat16:
            a = ops.attention_any(q, kc, vc, inp.block_tables, inp.cu_q, inp.context_lens,
                                  inp.positions, self.scale, self.Hq, window=self.window,
                                  cap=self.cap)
            return ops.linear(a, self.w_o, defer=True)
        a = torch.empty((T, self.Hq * self.D), dtype=q.dtype, device=q.device)
        if nd:
            ops.paged_decode_attention(q[:nd], kc, vc, inp.block_tables, inp.context_lens,
                                       self.scale, a[:nd], inp.decode_ws, inp.part_tokens,
                                       Hq=self.Hq, order=inp.decode_order, precise=True,
                                       window=self.window, cap=self.cap)
        if T > nd:
            ops.paged_prefill_attention(q, kc, vc, inp.block_tables[nd:], inp.cu_q[nd:],
                                        inp.context_lens[nd:], tiles, self.scale, a, Hq=self.Hq,
                                        q_per_tile=self.q_per_tile, precise=True,
                                        window=self.window, cap=self.cap)
        return ops.linear(a, self.w_o, defer=True)


class GatedDeltaMixer(Mixer):
    """Gated delta rule: q, k, v through a short convolution with SiLU, q and k
    unit vectors per head (shared by heads / kv_heads value heads);

        S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q

    with beta = sigmoid(W_b h) and ln g = -exp(A_log) softplus(W_a h + dt_bias)
    per head; each head of o divided by its root mean square, times a gain and
    silu(W_g h), projected."""

    def __init__(self, m: dict, width: int, eps: float):
        self.H, self.G, self.N, self.P = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.taps, self.eps = m["conv"], eps
        H, G, N, P = self.H, self.G, self.N, self.P
        if H % G:
            raise ValueError("delta rule: heads must be a multiple of kv_heads")
        self.shapes = {"q": (G * N, width), "k": (G * N, width), "v": (H * P, width),
                       "q.conv": (G * N, self.taps), "k.conv": (G * N, self.taps),
                       "v.conv": (H * P, self.taps), "b": (H, width), "A_log": (H,),
                       "norm": (P,), "a": (H, width), "dt_bias": (H,), "g": (H * P, width),
                       "o": (width, H * P)}
        self.qk, self.vp, self.hp = _up(G * N, 8), _up(H * P, 8), _up(H, 8)
        self.C = 2 * self.qk + self.vp             # convolved channels
        self.rows = self.C + self.vp + 2 * self.hp
        self.proj = {"in": (self.rows, width), "o": (width, H * P)}

    plan_key = ("delta",)

    def build_plan(self, qlens, ctx, seq0):
        chunks, first = mixer_ops.delta_chunks(qlens, seq0)
        return [("dchunks", chunks), ("dfirst", first)], len(chunks)

    def bind_plan(self, dev, host):
        return ops.DeltaChunks(dev["dchunks"], dev["dfirst"], host)

    def state_shapes(self, dtype):
        out = [((self.H, self.N, self.P), torch.float32)]
        if self.taps > 1:
            out.append(((self.taps - 1, self.C), dtype))
        return out

    def in_rows(self, get):
        return _fuse_rows([get(n) for n in ("q", "k", "v", "g", "b", "a")],
                          [self.qk, self.qk, self.vp, self.vp, self.hp, self.hp])

    def load(self, get, put, own_projection=True):
        if own_projection:
            self.w_in = put(self.in_rows(get))
        self.conv = put(_fuse_rows([get(n + ".conv").float() for n in "qkv"],
                                   [self.qk, self.qk, self.vp]).t(), fp32=True)
        self.neg_a = put(-torch.exp(get("A_log").float()), fp32=True)
        self.dt_bias = put(get("dt_bias"), fp32=True)
        self.norm = put(get("norm").float().repeat(self.H), fp32=True)
        self.w_o = put(get("o"))

    def forward(self, h, inp, cache, state):
        return self.mix(ops.linear(h, self.w_in), inp, cache, state)

    def mix(self, p, inp, cache, state):
        """Output rows of projection rows p = [q | k | v | g | b | a | ..]."""
        C, qk, vp, hp = self.C, self.qk, self.vp, self.hp
        u = ops.short_conv(p[:, :C], self.conv, state[1] if self.taps > 1 else None, inp.cu_q,
                           inp.context_lens, inp.state_slots, silu=True,
                           tiles=inp.aux.get("conv"))
        b, a = p[:, C + vp:C + vp + hp], p[:, C + vp + hp:C + vp + 2 * hp]
        o = ops.delta_rule(u[:, :qk], u[:, qk:2 * qk], u[:, 2 * qk:], b, a, self.dt_bias,
                           self.neg_a, state[0], inp.cu_q, inp.context_lens, inp.state_slots,
                           self.G, num_decode=inp.num_decode, chunks=inp.aux.get(self.plan_key))
        y = ops.gated_norm(o, p[:, C:C + vp], self.norm, self.H, self.eps, gate_first=False,
                           silu=True)
        return ops.linear(y, self.w_o, defer=True)


class Branches(Mixer):
    """Attention (``left_class``) and a recurrence (``right_class``) side by
    side on the same rows.  One input projection serves both."""
    left_class = right_class = None

    def __init__(self, m: dict, width: int, eps: float):
        self.left = self.left_class(m["left"], width, eps)
        self.right = self.right_class(m["right"], width, eps)
        self.shapes = {f"{name}.{k}": s for name, part in (("left", self.left), ("right", self.right))
                       for k, s in part.shapes.items()}
        self.kv, self.q_per_tile = self.left.kv, self.left.q_per_tile
        self.Hq, self.Hkv, self.D = self.left.Hq, self.left.Hkv, self.left.D
        rows = self.left.rows + self.right.rows
        # a wide projection is rounded up to whole 256-row GEMM tiles
        self.tail = (_up(rows, 256) if rows >= 4096 else rows) - rows
        self.proj = {"in": (rows + self.tail, width)}

    def members(self):
        return [self.left, self.right]

    def state_shapes(self, dtype):
        return self.right.state_shapes(dtype)

    def load(self, get, put):
        left, right = (lambda n, s=s: get(f"{s}.{n}") for s in ("left", "right"))
        parts = [self.left.in_rows(left), self.right.in_rows(right)]
        self.w_in = put(_fuse_rows(parts, [self.left.rows, self.right.rows + self.tail]))
        self.left.load(left, put, own_projection=False)
        self.right.load(right, put, own_projection=False)


class ParallelMixer(Branches):
    """Windowed attention beside a gated delta rule: half the sum of their
    outputs, each RMS-normed over the width."""
    left_class, right_class = SoftcapAttentionMixer, GatedDeltaMixer

    def __init__(self, m: dict, width: int, eps: float):
        super().__init__(m, width, eps)
        self.shapes.update({"left.out": (width,), "right.out": (width,)})
        self.proj.update({"left.o": self.left.proj["o"], "right.o": self.right.proj["o"]})

    def load(self, get, put):
        super().load(get, put)
        self.out_left, self.out_right = (put(0.5 * get(s + ".out").float(), fp32=True)
                                         for s in ("left", "right"))

    def forward(self, h, inp, cache, state):
        p = ops.linear(h, self.w_in)
        n = self.left.rows
        return ops.NormedPair(self.left.mix(p[:, :n], inp, cache, state),
                              self.right.mix(p[:, n:], inp, cache, state),
                              self.out_left, self.out_right)


class TalkingAttentionMixer(Mixer):
    """Softmax attention whose heads' scores are mixed: q and k (biased)
    RMS-normed over the whole projection and partly rotated (pairs i, i +
    dims/2), v divided by its root mean square per head; scores times a number
    per head, mixed over the heads; a row sees its own chunk of positions; a
    sink per head in the softmax; output gate sigmoid(W_g h).

    q is served with the score's scale and the heads' numbers in its gain, and
    with each head's rotated pairs next to each other, as k is."""
    Hkv = 1                       # all heads of a row run in one workgroup

    def __init__(self, m: dict, width: int, eps: float):
        self.Hq, self.G, self.dk, self.dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.scale, self.eps = float(m["scale"]), eps
        mask = m.get("mask")
        self.chunk = int(mask["size"]) if mask else 0
        if mask and self.chunk < 1:
            raise ValueError("attention: a chunk of at least 1")
        if self.Hq % self.G:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        self.rot = rotary(m.get("rot"), self.dk)
        H, G, dk, dv = self.Hq, self.G, self.dk, self.dv
        D = self.D = _head_size(max(dk, dv))
        self.shapes = {"q": (H * dk, width), "k": (G * dk, width), "v": (G * dv, width),
                       "q.b": (H * dk,), "k.b": (G * dk,), "v.b": (G * dv,),
                       "q.norm": (H * dk,), "k.norm": (G * dk,), "talk": (H, H), "temp": (H,),
                       "sink": (H,), "g": (H * dv, width), "o": (width, H * dv), "o.b": (width,)}
        self.kv = (G, D, D)
        self.qkv = (H + 2 * G) * D
        self.rows = self.qkv + H * D
        self.proj = {"in": (self.rows, width), "o": (width, H * D)}
        self.q_per_tile = ops.TALK_QT
        self.plan_key = ("talk", self.chunk)

    def build_plan(self, qlens, ctx, seq0):
        return [("quads", mixer_ops.row_quads(qlens, ctx, seq0)),
                (f"talk{self.chunk}", mixer_ops.talk_tiles(qlens, ctx, self.chunk).reshape(-1))], None

    def bind_plan(self, dev, host):
        return dev["quads"], dev[f"talk{self.chunk}"]

    def _heads(self, t, n, d, pairs=False):
        """[n * d, ...] rows -> [n * D, ...], each head padded with zeros."""
        if pairs:
            t = t[_pairs_together(n, d, self.rot).to(t.device)]
        out = t.new_zeros((n, self.D) + tuple(t.shape[1:]))
        out[:, :d] = t.reshape((n, d) + tuple(t.shape[1:]))
        return out.reshape((n * self.D,) + tuple(t.shape[1:]))

    def _qkv(self, get, suffix=""):
        return [self._heads(get("q" + suffix), self.Hq, self.dk, True),
                self._heads(get("k" + suffix), self.G, self.dk, True),
                self._heads(get("v" + suffix), self.G, self.dv)]

    def in_rows(self, get):
        return torch.cat(self._qkv(get) + [self._heads(get("g"), self.Hq, self.dv)])

    def out_rows(self, get):
        """The output projection, [width, H * D]."""
        return self._heads(get("o").t().contiguous(), self.Hq, self.dv).t()

    def load(self, get, put, own_projection=True):
        if own_projection:
            self.w_in, self.w_o = put(self.in_rows(get)), put(self.out_rows(get))
            self.out_bias = put(get("o.b"), fp32=True)
        self.in_bias = put(torch.cat(self._qkv(get, ".b")), fp32=True)
        w = get("q.norm").float().view(self.Hq, self.dk) * get("temp").float()[:, None] * self.scale
        self.q_norm = put(self._heads(w.reshape(-1), self.Hq, self.dk, True), fp32=True)
        self.k_norm = put(self._heads(get("k.norm"), self.G, self.dk, True), fp32=True)
        self.talk = ops.Talk(put(get("talk")), put(get("sink"), fp32=True))

    def forward(self, h, inp, cache, state):
        p = ops.linear(h, self.w_in)
        a = torch.empty((p.shape[0], self.Hq * self.D), dtype=p.dtype, device=p.device)
        self.attend(p, inp, cache, a)
        return ops.Biased(ops.linear(a, self.w_o, defer=True), self.out_bias)

    def attend(self, p, inp, cache, out, scale=1.0):
        """The gated heads of projection rows p = [q | k | v | g | ..], times
        ``scale``, into ``out`` [T, H * D]."""
        kc, vc = cache
        quads, tiles = inp.aux.get(self.plan_key, (None, None))
        ang = inp.aux["rot", self.rot] if self.rot else None
        q = ops.qkv_norm_rope_cache(p, self.in_bias, self.q_norm, self.k_norm, ang, inp.slots, kc,
                                    vc, self.Hq, self.dk, self.dv, self.eps, quads)
        ops.talking_attention(q, kc, vc, inp.block_tables, inp.cu_q, inp.context_lens,
                              inp.positions, self.talk, self.Hq, p[:, self.qkv:self.rows], out,
                              self.chunk, scale, inp.num_decode, tiles, inp.decode_ws)


class MatrixMemoryMixer(ScanMixer):
    """Matrix memory with exponential gates (``ops.memory_scan``): q, k, v and
    gates projected; each head's output divided by its root mean square, times
    a gain and sigmoid(W_g h), projected."""

    def __init__(self, m: dict, width: int, eps: float):
        self.H, self.N, self.P = m["heads"], m["dim"], m["vdim"]
        self.cap, self.eps = float(m["gate_cap"]), eps
        if not self.cap > 0:
            raise ValueError("matrix memory: a positive gate_cap")
        H, N, P = self.H, self.N, self.P
        self.shapes = {"q": (H * N, width), "k": (H * N, width), "v": (H * P, width),
                       "g": (H * P, width), "o": (width, H * P), "norm": (H * P,),
                       "i": (H, width), "i.b": (H,), "f": (H, width), "f.b": (H,)}
        self.qk, self.vg, self.hp = _up(H * N, 8), _up(H * P, 8), _up(H, 8)
        self.rows = 2 * (self.qk + self.vg + self.hp)
        self.proj = {"in": (self.rows, width), "o": (width, H * P)}

    def state_shapes(self, dtype):
        H, N, P = self.H, self.N, self.P
        return [((H, N, P), torch.float32), ((H, N), torch.float32), ((H,), torch.float32)]

    plan_key = property(lambda self: ("scan", self.H, self.P))

    def in_rows(self, get):
        return _fuse_rows([get(n) for n in ("q", "k", "v", "g", "i", "f")],
                          [self.qk, self.qk, self.vg, self.vg, self.hp, self.hp])

    def out_rows(self, get):
        return get("o")

    def load(self, get, put, own_projection=True):
        if own_projection:
            self.w_in, self.w_o = put(self.in_rows(get)), put(self.out_rows(get))
        self.gate_bias = put(torch.stack([get("i.b").float(), get("f.b").float()]), fp32=True)
        self.norm = put(get("norm"), fp32=True)

    def forward(self, h, inp, cache, state):
        p = ops.linear(h, self.w_in)
        return ops.linear(self.recall(p, inp, state), self.w_o, defer=True)

    def recall(self, p, inp, state, out=None):
        """The gated heads of projection rows p = [q | k | v | g | i | f | ..]."""
        qk, vg, hp = self.qk, self.vg, self.hp
        a = 2 * (qk + vg)
        y = ops.memory_scan(p[:, :qk], p[:, qk:2 * qk], p[:, 2 * qk:2 * qk + vg], p[:, a:a + hp],
                            p[:, a + hp:a + 2 * hp], self.gate_bias, self.cap, state, inp.cu_q,
                            inp.context_lens, inp.state_slots, num_decode=inp.num_decode,
                            segments=inp.aux.get(self.plan_key))
        return ops.gated_norm(y, p[:, 2 * qk + vg:a], self.norm, self.H, self.eps,
                              gate_first=False, out=out)


class TalkingMemoryMixer(Branches):
    """Attention with talking heads beside a matrix memory, left_scale left +
    right_scale right.  The scales act on the branches' rows in fp32 and one
    product projects both."""
    left_class, right_class = TalkingAttentionMixer, MatrixMemoryMixer

    def __init__(self, m: dict, width: int, eps: float):
        super().__init__(m, width, eps)
        self.scales = float(m["left_scale"]), float(m["right_scale"])
        self.split = self.left.Hq * self.left.D
        self.cols = self.split + _up(self.right.H * self.right.P, 8)
        self.proj["o"] = (width, self.cols)

    def load(self, get, put):
        super().load(get, put)
        left, right = (lambda n, s=s: get(f"{s}.{n}") for s in ("left", "right"))
        w = get("left.o").new_zeros(self.proj["o"])
        w[:, :self.split] = self.left.out_rows(left)
        w[:, self.split:self.split + self.right.H * self.right.P] = self.right.out_rows(right)
        self.w_o = put(w)
        self.out_bias = put(self.scales[0] * left("o.b").float(), fp32=True)
        self.right.norm.mul_(self.scales[1])

    def forward(self, h, inp, cache, state):
        p = ops.linear(h, self.w_in)
        T, n, c = p.shape[0], self.split, self.right.H * self.right.P
        y = torch.empty((T, self.cols), dtype=p.dtype, device=p.device)
        if self.cols > n + c:
            y[:, n + c:].zero_()
        self.left.attend(p[:, :self.left.rows], inp, cache, y[:, :n], self.scales[0])
        self.right.recall(p[:, self.left.rows:], inp, state, out=y[:, n:n + c])
        return ops.Biased(ops.linear(y, self.w_o, defer=True), self.out_bias)


def init_std(name: str, shape: tuple, depth: int, zero_centred: bool = True) -> tuple[float, float]:
    """(mean, std) of a tensor's random initialisation (benchmarks, tests)."""
    leaf = name.rsplit(".", 1)[-1]
    if leaf in ("o", "down"):
        return 0.0, 0.02 / math.sqrt(2 * depth)
    if leaf == "conv":
        return 1.0 / shape[-1], 0.2
    if name.endswith((".mix.norm", "dq.norm", "dkv.norm", ".q.norm", ".k.norm", ".right.norm",
                      ".out")) or leaf in ("D", "ls1", "ls2"):
        return 1.0, 0.1
    if leaf == "A_log":
        return 0.5, 0.5
    if leaf == "dt_bias":
        return -3.0, 1.0
    if leaf == "lam":              # decays of 0.9 and slower
        return -4.0, 1.0
    if leaf in ("ra", "ri"):
        return 0.0, shape[-1] ** -0.5
    if leaf == "temp":
        return 1.0, 0.1
    if leaf == "talk":
        return 1.0 / shape[-1], 0.3
    if name.endswith("right.f.b"):     # slow forgetting
        return 4.0, 1.0
    if name == "embed":
        return 0.0, 1.0
    if leaf.startswith("norm"):
        return (0.0 if zero_centred else 1.0), 0.02
    return 0.0, 0.02
