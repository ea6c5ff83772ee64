"""Ops of the token mixers beyond plain attention: linear-attention /
state-space scans, short causal convolutions, sandwich and gated norms, and
paged attention for any head geometry.

Same conventions as the package: GPU tensors run the kernels of
``csrc/kernels`` (bf16 or fp32 rows), CPU tensors the references in
``ops.ref``, and every shape is checked on the host before a launch.

Per-sequence state (recurrent state, convolution inputs) is a tensor
[slots, ...]; a step names each sequence's slot.  Rows that start at position 0
(``ctx == rows of the sequence in this step``) start from the zero state, so
slots are never cleared.
"""
from __future__ import annotations

import importlib
import math
from dataclasses import dataclass

import numpy as np
import torch

from . import Partials, _chk, _ptr, _stream, native, ref
from .grouped import GroupedWeight, Mixture, grouped_heads

CONV_TILE = 64        # tokens per convolution workgroup
SCAN_CHUNK = 64       # SC in csrc/kernels/linscan.hip
SCAN_VT = 128         # v columns per workgroup (64 up to P = 64)
SCAN_FILL = 512       # workgroups wanted before a sequence is cut into segments


def _rows_dtype(t: torch.Tensor, name: str) -> int:
    """1 for bf16 rows, 0 for fp32 rows."""
    _chk(t.dtype in (torch.bfloat16, torch.float32), f"{name}: bf16 or fp32, got {t.dtype}")
    return int(t.dtype == torch.bfloat16)


def _f32(t: torch.Tensor | None, n: int, name: str) -> None:
    _chk(t is None or (t.dtype == torch.float32 and t.numel() == n and t.is_contiguous()),
         f"{name}: fp32 [{n}]")


def _meta(S: int, **ts) -> None:
    for name, t in ts.items():
        _chk(t.dtype == torch.int32 and t.is_cuda and t.is_contiguous()
             and t.numel() >= S + (name == "cu_q"), f"{name}: int32[{S}]")


# -------------------------------------------------------------------- norms --
def sandwich_norm(residual: torch.Tensor, eps: float, y=None, w_post: torch.Tensor | None = None,
                  w_pre: torch.Tensor | None = None, ids: torch.Tensor | None = None,
                  table: torch.Tensor | None = None, rows: torch.Tensor | None = None,
                  dtype: torch.dtype = torch.bfloat16, scale: float = 1.0) -> torch.Tensor:
    """One pass over the fp32 residual stream between two sublayers:

        r = scale table[ids] (if given) else residual
        r += rms(y) * w_post         (y: sublayer output rows, ``Partials``, ``Mixture`` or
                                      one of them ``Biased``)
        residual = r                 (unless ``rows`` is given)
        return rms(r) * w_pre        (``dtype`` rows; r itself without w_pre)

    ``rows`` (int64): only these rows are normed, the residual stays as it is.
    The gains are fp32 vectors."""
    T, d = residual.shape
    bias = own = None
    if isinstance(y, Biased):
        y, bias = y.rows, y.bias
    if isinstance(y, Mixture):
        own = y.own
    if not residual.is_cuda:
        y = y.sum()[:, :d] if isinstance(y, Mixture) else y
        return ref.sandwich_norm(residual, eps, y, w_post, w_pre, ids, table, rows, dtype, scale,
                                 bias, own)
    _chk(residual.dtype == torch.float32 and residual.is_contiguous(), "residual: fp32 rows")
    _f32(w_post, d, "w_post"); _f32(w_pre, d, "w_pre")
    bf = int(dtype == torch.bfloat16)
    yp, y_ld, slabs, sstride, mix = 0, 0, 0, 0, (0, 0, 0)
    if isinstance(y, Partials):
        _chk((y.M, y.N) == (T, d), "sandwich_norm partials shape")
        yp, y_ld, slabs, sstride = _ptr(y.slabs), d, y.S, y.M * y.N
    elif isinstance(y, Mixture):
        _chk(y.rows.shape[1] >= d and y.rows.stride(1) == 1 and y.rows.dtype == dtype
             and y.pos.shape == y.weights.shape and y.pos.shape[0] == T
             and y.pos.dtype == torch.int32 and y.weights.dtype == torch.float32
             and y.pos.is_contiguous() and y.weights.is_contiguous(), "sandwich_norm mixture")
        yp, y_ld, mix = _ptr(y.rows), y.rows.stride(0), (_ptr(y.pos), _ptr(y.weights), y.pos.shape[1])
    elif y is not None:
        _chk(y.shape == (T, d) and y.stride(1) == 1 and y.dtype == dtype, "sandwich_norm y rows")
        yp, y_ld = _ptr(y), y.stride(0)
    _chk((y is None) == (w_post is None), "w_post goes with y")
    _f32(bias, d, "sublayer bias"); _f32(own, T, "the stream's own weights")
    if ids is not None:
        _chk(ids.dtype == torch.int32 and ids.numel() >= T and table.dtype == dtype
             and table.is_contiguous() and table.shape[1] == d, "embedding rows")
    n = T
    if rows is not None:
        _chk(rows.dtype == torch.int64 and rows.is_contiguous(), "rows: int64")
        n = rows.numel()
    out = torch.empty((n, d), dtype=dtype, device=residual.device)
    native().sandwich_norm(_ptr(out), _ptr(residual), yp, y_ld, slabs, sstride, *mix, _ptr(own),
                           _ptr(bias), _ptr(ids),
                           _ptr(table), float(scale), _ptr(w_post), _ptr(w_pre), _ptr(rows), n, d,
                           float(eps), bf, _stream())
    return out


class Biased:
    """Sublayer output rows + bias (fp32 [d]), left to the consuming kernel;
    rows: what ``sandwich_norm`` takes."""
    __slots__ = ("rows", "bias")

    def __init__(self, rows, bias: torch.Tensor):
        self.rows, self.bias = rows, bias


class NormedPair:
    """Sublayer output rows rms(a) * wa + rms(b) * wb of two branches (rows or
    ``Partials``), left to the consuming kernel."""
    __slots__ = ("a", "b", "wa", "wb")

    def __init__(self, a, b, wa: torch.Tensor, wb: torch.Tensor):
        self.a, self.b, self.wa, self.wb = a, b, wa, wb

    def sum(self, eps: float) -> torch.Tensor:
        a, b = (x.float() * torch.rsqrt(x.float().pow(2).mean(-1, keepdim=True) + eps)
                for x in (self.a, self.b))
        return a * self.wa + b * self.wb


def _sublayer_rows(y, T: int, d: int, dtype, name: str) -> tuple:
    """(rows, row stride, slabs, slab stride) of rows or ``Partials``."""
    if isinstance(y, Partials):
        _chk((y.M, y.N) == (T, d), f"{name} partials shape")
        return _ptr(y.slabs), d, y.S, y.M * y.N
    _chk(y.shape == (T, d) and y.stride(1) == 1 and y.dtype == dtype, f"{name} rows")
    return _ptr(y), y.stride(0), 0, 0


def sum_norm(residual: torch.Tensor, eps: float, y, alpha: float, scale: torch.Tensor | None,
             w_post: torch.Tensor | None, w_pre: torch.Tensor | None = None,
             rows: torch.Tensor | None = None,
             dtype: torch.dtype = torch.bfloat16) -> torch.Tensor:
    """The fp32 residual stream of a decoder that layer-norms the sum:

        r = ln(alpha residual + scale y) * w_post    (residual without y)
        residual = r                                  (unless ``rows`` is given)
        return ln(r) * w_pre                          (``dtype`` rows; r itself without w_pre)

    ln(x) = (x - mean) / sqrt(variance + eps).  y: sublayer output rows,
    ``Partials``, ``Mixture`` or ``NormedPair``; ``rows`` (int64) and the fp32
    vectors as in ``sandwich_norm``."""
    T, d = residual.shape
    _chk(not isinstance(y, Biased) and getattr(y, "own", None) is None,
         "sum_norm: no bias, no weight of the stream's own rows")
    if not residual.is_cuda:
        if isinstance(y, Mixture):
            y = y.sum()[:, :d]
        elif isinstance(y, NormedPair):
            y = y.sum(eps)
        return ref.sum_norm(residual, eps, y, alpha, scale, w_post, w_pre, rows, dtype)
    _chk(residual.dtype == torch.float32 and residual.is_contiguous(), "residual: fp32 rows")
    _f32(scale, d, "scale"); _f32(w_post, d, "w_post"); _f32(w_pre, d, "w_pre")
    _chk((y is None) == (w_post is None) == (scale is None) and (y is not None or w_pre is not None),
         "sum_norm: y, its scale and its norm go together")
    a, b, mix, gains = (0, 0, 0, 0), (0, 0, 0, 0), (0, 0, 0), (0, 0)
    if isinstance(y, Mixture):
        _chk(y.rows.shape[1] >= d and y.rows.stride(1) == 1 and y.rows.dtype == dtype
             and y.pos.shape == y.weights.shape and y.pos.shape[0] == T
             and y.pos.dtype == torch.int32 and y.weights.dtype == torch.float32
             and y.pos.is_contiguous() and y.weights.is_contiguous(), "sum_norm mixture")
        a, mix = (_ptr(y.rows), y.rows.stride(0), 0, 0), (_ptr(y.pos), _ptr(y.weights), y.pos.shape[1])
    elif isinstance(y, NormedPair):
        _f32(y.wa, d, "pair gain"); _f32(y.wb, d, "pair gain")
        a, b = (_sublayer_rows(x, T, d, dtype, "sum_norm pair") for x in (y.a, y.b))
        gains = (_ptr(y.wa), _ptr(y.wb))
    elif y is not None:
        a = _sublayer_rows(y, T, d, dtype, "sum_norm y")
    n = T
    if rows is not None:
        _chk(rows.dtype == torch.int64 and rows.is_contiguous(), "rows: int64")
        n = rows.numel()
    out = torch.empty((n, d), dtype=dtype, device=residual.device)
    native().sum_norm(_ptr(out), _ptr(residual), *a, *mix, *b, *gains, float(alpha), _ptr(scale),
                      _ptr(w_post), _ptr(w_pre), _ptr(rows), n, d, float(eps),
                      int(dtype == torch.bfloat16), _stream())
    return out


def soft_cap(x: torch.Tensor, scale: float, cap: float | None) -> torch.Tensor:
    """x <- cap tanh(scale x / cap) in place (cap None: scale x)."""
    if scale == 1.0 and cap is None:
        return x
    if not x.is_cuda:
        y = x.float() * scale
        return x.copy_(y if cap is None else cap * torch.tanh(y / cap))
    bf = _rows_dtype(x, "x")
    _chk(x.is_contiguous(), "soft_cap: contiguous rows")
    native().soft_cap(_ptr(x), x.numel(), float(scale), float(cap or 0.0), bf, _stream())
    return x


def gated_norm(x: torch.Tensor, gate: torch.Tensor, w: torch.Tensor, groups: int, eps: float,
               gate_first: bool, silu: bool = False,
               out: torch.Tensor | None = None) -> torch.Tensor:
    """RMS norm of x in ``groups`` equal parts of a row, gain w (fp32), gated:
    rms(x) * w * sigmoid(gate) (``silu``: silu(gate)), or with ``gate_first``
    rms(x * silu(gate)) * w.  ``out``: rows to write (any row stride)."""
    T, C = x.shape
    _chk(C % groups == 0, "gated_norm groups")
    _chk(out is None or (out.shape == (T, C) and out.dtype == x.dtype and out.stride(1) == 1),
         "gated_norm output rows")
    if not x.is_cuda:
        y = ref.gated_norm(x, gate, w, groups, eps, gate_first, silu)
        return y if out is None else out.copy_(y)
    bf = _rows_dtype(x, "x")
    _f32(w, C, "w")
    _chk(gate.dtype == x.dtype and gate.shape[0] == T and gate.shape[1] >= C
         and gate.stride(1) == 1 and x.stride(1) == 1, "gated_norm rows")
    if out is None:
        out = torch.empty((T, C), dtype=x.dtype, device=x.device)
    native().gated_norm(_ptr(out), out.stride(0), _ptr(x), x.stride(0), _ptr(gate),
                        gate.stride(0), _ptr(w), T, C, groups,
                        1 if gate_first else 2 if silu else 0, float(eps), bf,
                        _stream())
    return out


# -------------------------------------------------------------- convolution --
def row_tiles(qlens, tile: int) -> np.ndarray:
    """int32 [n, 2] (sequence, first row in it): every sequence's rows in tiles."""
    nt = -(-np.asarray(qlens, dtype=np.int64) // tile)
    seq = np.repeat(np.arange(len(nt)), nt)
    base = np.repeat(np.cumsum(nt) - nt, nt)
    start = (np.arange(len(seq)) - base) * tile
    return np.stack([seq, start], 1).astype(np.int32)


def conv_tiles(cu_q) -> np.ndarray:
    """``row_tiles`` of a step's convolutions (all its sequences)."""
    return row_tiles(np.diff(np.asarray(cu_q)), CONV_TILE)


def _conv_meta(u, w, state, tiles, cu_q, ctx, slots):
    taps, C = w.shape
    S = ctx.numel()
    _chk(w.dtype == torch.float32 and w.is_contiguous(), "conv weights: fp32 [taps, C]")
    _chk(u.stride(1) == 1 and u.shape[1] >= C, "conv rows")
    _chk(1 <= taps <= 32, "conv taps 1..32")
    _chk(taps == 1 or (state is not None and state.dtype == u.dtype and state.is_contiguous()
                       and tuple(state.shape[1:]) == (taps - 1, C)),
         "conv state [slots, taps - 1, C]")
    _meta(S, cu_q=cu_q, ctx=ctx, slots=slots)
    if tiles is not None:
        _chk(tiles.dtype == torch.int32 and tiles.is_contiguous(), "conv tiles int32")
    else:
        _chk(u.shape[0] == S, "conv without tiles: one row per sequence")
    return taps, C, (S if tiles is None else tiles.numel() // 2)


def short_conv(u: torch.Tensor, w: torch.Tensor, state: torch.Tensor | None, cu_q, ctx, slots,
               bias: torch.Tensor | None = None, silu: bool = False,
               tiles: torch.Tensor | None = None,
               in_bias: torch.Tensor | None = None) -> torch.Tensor:
    """Causal convolution over time of each channel (w fp32 [taps, C], last
    tap = the current token), optionally SiLU; ``state`` [slots, taps - 1, C]
    carries the last inputs.  ``in_bias``: the projection's own bias (fp32 [C],
    added to u).  ``tiles`` (``conv_tiles``): needed when a sequence has more
    than one row."""
    taps, C = w.shape
    out = torch.empty((u.shape[0], C), dtype=u.dtype, device=u.device)
    if not u.is_cuda:
        ref.short_conv(u, w, bias, state, cu_q, ctx, slots, out, silu, in_bias)
        return out
    bf = _rows_dtype(u, "u")
    taps, C, n = _conv_meta(u, w, state, tiles, cu_q, ctx, slots)
    _f32(bias, C, "conv bias"); _f32(in_bias, C, "projection bias")
    native().short_conv(_ptr(u), u.stride(0), _ptr(w), _ptr(in_bias), _ptr(bias), _ptr(state), _ptr(tiles), n,
                        CONV_TILE, _ptr(cu_q), _ptr(ctx), _ptr(slots), C, taps, _ptr(out),
                        out.stride(0), int(silu), bf, _stream())
    return out


def conv_qkv_cache(u: torch.Tensor, w: torch.Tensor, in_bias: torch.Tensor | None,
                   state: torch.Tensor | None, cu_q, ctx, state_slots, positions, slots,
                   k_cache, v_cache, Hq: int, dk: int, eps: float, temp: tuple[float, float],
                   tiles: torch.Tensor | None = None) -> torch.Tensor:
    """The projection rows' q | k | v heads (each padded to D channels) through
    a short convolution; q and k divided by their root mean square over the
    ``dk`` true channels; q times 1 + temp[0] ln(floor((p + 1) / temp[1]) + 1);
    k and v written to the paged cache at ``slots``.  ``in_bias``: the
    projection's bias (fp32 [C]).  Returns q rows [T, Hq * D]."""
    _, Hkv, BS, D = k_cache.shape
    T = u.shape[0]
    q = torch.empty((T, Hq * D), dtype=u.dtype, device=u.device)
    if not u.is_cuda:
        ref.conv_qkv_cache(u, w, in_bias, state, cu_q, ctx, state_slots, q, k_cache, v_cache,
                           positions, slots, Hq, Hkv, D, dk, eps, temp)
        return q
    bf = _rows_dtype(u, "u")
    taps, C, n = _conv_meta(u, w, state, tiles, cu_q, ctx, state_slots)
    _f32(in_bias, C, "projection bias")
    _chk(C == (Hq + 2 * Hkv) * D and k_cache.dtype == u.dtype and v_cache.dtype == u.dtype
         and k_cache.is_contiguous() and v_cache.is_contiguous(), "q | k | v heads / caches")
    _meta(T, positions=positions, rows=slots)
    native().conv_qkv_cache(_ptr(u), u.stride(0), _ptr(w), _ptr(in_bias), _ptr(state),
                            _ptr(tiles), n, CONV_TILE, _ptr(cu_q), _ptr(ctx), _ptr(state_slots),
                            taps, _ptr(q), q.stride(0), _ptr(k_cache), _ptr(v_cache),
                            _ptr(positions), _ptr(slots), Hq, Hkv, D, dk, BS, float(eps),
                            float(temp[0]), float(temp[1]), bf, _stream())
    return q


# --------------------------------------------------------------------- scan --
@dataclass
class ScanSegments:
    """Row segments of a step's multi-token sequences for the chunked scan."""
    segs: torch.Tensor      # int32 [n, 4]: sequence, first row, end row, last of its sequence
    first: torch.Tensor     # int32 [sequences + 1]: each sequence's first segment
    n: int
    one_pass: bool


def scan_segments(qlens, seq0: int, H: int, P: int) -> tuple[np.ndarray, np.ndarray, bool]:
    """Host plan of ``ScanSegments`` for sequences seq0, seq0 + 1, ... with
    ``qlens`` rows: one segment each when (sequences x heads x column tiles)
    fills the chip, else whole-chunk cuts until it does (at least 4 chunks per
    segment: a segment's start state costs a pass over its k and v)."""
    wgs = max(1, len(qlens) * H * -(-P // SCAN_VT))
    parts = -(-SCAN_FILL // wgs)
    segs, first = [], [0]
    for i, n in enumerate(qlens):
        chunks = -(-int(n) // SCAN_CHUNK)
        p = max(1, min(parts, chunks // 4))
        step = -(-chunks // p) * SCAN_CHUNK
        starts = range(0, int(n), step)
        segs += [(seq0 + i, b, min(b + step, int(n)), int(b + step >= n)) for b in starts]
        first.append(len(segs))
    one_pass = len(segs) == len(qlens)
    return (np.asarray(segs, np.int32).reshape(-1, 4), np.asarray(first, np.int32), one_pass)


def _chunk_ok(N: int, P: int, *rows) -> bool:
    return (N % 8 == 0 and P % 8 == 0 and N <= 256 and
            all(t.dtype == torch.bfloat16 and t.data_ptr() % 16 == 0 and t.stride(0) % 8 == 0
                for t in rows))


def linear_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, state: torch.Tensor, cu_q, ctx,
                slots, heads_per_group: int = 1,
                decay: tuple[torch.Tensor, torch.Tensor] | None = None,
                dt: tuple[torch.Tensor, torch.Tensor, torch.Tensor] | None = None,
                skip: torch.Tensor | None = None, silu: bool = False, num_decode: int = 0,
                segments: ScanSegments | None = None, angles: torch.Tensor | None = None,
                k_scale: float = 1.0) -> torch.Tensor:
    """Per head S <- a S + s k v^T, o = S^T q + skip v over each sequence's rows,
    from and to ``state`` (fp32 [slots, H, N, P]).

    q, k: rows of (H / heads_per_group) x N channels shared by the heads of a
    group; v: rows of H x P channels; ``silu`` applies SiLU to all three first.
    ``decay`` = (a, ln a) fp32 [H]: constant, s = 1.  ``dt`` = (rows [T, H],
    bias fp32 [H], neg_a fp32 [H]): s = softplus(dt + bias), a = exp(neg_a s).
    Sequences before ``num_decode`` (one row each) take the recurrent kernel;
    the others the chunked MFMA kernel when ``segments`` is given and the shape
    allows it, the recurrent one otherwise.  Returns rows [T, H * P].

    ``angles`` (``rope_angles`` [T, n]): the first n channels of q and k are
    turned by them, neighbours paired, and k is multiplied by ``k_scale``; the
    rows of q and k that the chunked kernel reads are rotated in place."""
    _, H, N, P = state.shape
    T, S = q.shape[0], ctx.numel()
    _chk((decay is None) != (dt is None), "linear_scan: decay or dt")
    _chk(H % heads_per_group == 0, "linear_scan: heads per group")
    out = torch.empty((T, H * P), dtype=q.dtype, device=q.device)
    if not q.is_cuda:
        ref.linear_scan(q, k, v, out, state, cu_q, ctx, slots, heads_per_group, decay, dt, skip,
                        silu, range(S), angles, k_scale)
        return out
    bf = _rows_dtype(q, "q")
    gn = H // heads_per_group * N
    for t, c, name in ((q, gn, "q"), (k, gn, "k"), (v, H * P, "v")):
        _chk(t.dtype == q.dtype and t.shape[0] == T and t.shape[1] >= c and t.stride(1) == 1,
             f"linear_scan {name} rows")
    _chk(state.dtype == torch.float32 and state.is_contiguous(), "scan state: fp32")
    _meta(S, cu_q=cu_q, ctx=ctx, slots=slots)
    _f32(skip, H, "skip")
    if dt is not None:
        _chk(dt[0].dtype == q.dtype and dt[0].shape[0] == T and dt[0].shape[1] >= H
             and dt[0].stride(1) == 1, "dt rows")
        _f32(dt[1], H, "dt bias"); _f32(dt[2], H, "neg_a")
        scal = (_ptr(dt[0]), dt[0].stride(0), _ptr(dt[1]), _ptr(dt[2]), 0, 0)
    else:
        _f32(decay[0], H, "decay"); _f32(decay[1], H, "log decay")
        scal = (0, 0, 0, 0, _ptr(decay[0]), _ptr(decay[1]))
    nrot = 0
    if angles is not None:
        nrot = angles.shape[1]
        _f32(angles, T * nrot, "angles")
        _chk(nrot % 2 == 0 and nrot <= N and not silu, "linear_scan: rotated channels")
    turned = angles is not None or k_scale != 1.0
    args = (_ptr(q), q.stride(0), _ptr(k), k.stride(0), _ptr(v), v.stride(0), *scal, _ptr(skip),
            _ptr(out), out.stride(0), _ptr(state), _ptr(cu_q), _ptr(ctx), _ptr(slots), H, N, P,
            heads_per_group, int(silu), bf)
    chunked = segments is not None and S > num_decode and _chunk_ok(N, P, q, k, v)
    n_rec = num_decode if chunked else S
    if n_rec:
        native().linear_scan(*args, _ptr(angles), nrot, float(k_scale), 0, n_rec, 0, 0, 0, 0, 0, 0,
                             _stream())
    if chunked:
        g = segments
        _chk(g.segs.dtype == torch.int32 and g.segs.numel() >= 4 * g.n
             and g.first.dtype == torch.int32 and g.first.numel() == S - num_decode + 1,
             "scan segments")
        ws = wl = None
        if not g.one_pass:
            ws = torch.empty((g.n, H, N, P), dtype=torch.float32, device=q.device)
            wl = torch.empty((g.n, H), dtype=torch.float32, device=q.device)
        if turned:                # decode rows come first, one each
            native().rotate_rows(_ptr(q), q.stride(0), _ptr(k), k.stride(0), _ptr(angles), nrot,
                                 num_decode, T, gn // N, N, float(k_scale), _stream())
        native().linear_scan(*args, 0, 0, 1.0, num_decode, S - num_decode, _ptr(g.segs), g.n,
                             _ptr(g.first), int(g.one_pass), _ptr(ws), _ptr(wl), _stream())
    return out


# ---------------------------------------------------------- gated delta rule --
DELTA_CHUNK = 64           # DC in csrc/kernels/delta.hip


@dataclass
class DeltaChunks:
    """Chunks of a step's multi-token sequences for the chunked delta rule."""
    chunks: torch.Tensor    # int32 [n, 2]: sequence, first row in it
    first: torch.Tensor     # int32 [sequences + 1]: each sequence's first chunk
    n: int


def delta_chunks(qlens, seq0: int) -> tuple[np.ndarray, np.ndarray]:
    """Host plan of ``DeltaChunks`` for sequences seq0, seq0 + 1, ..."""
    t = row_tiles(qlens, DELTA_CHUNK)
    t[:, 0] += seq0
    n = -(-np.asarray(qlens, np.int64) // DELTA_CHUNK)
    return t, np.concatenate([[0], np.cumsum(n)]).astype(np.int32)


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, b: torch.Tensor, a: torch.Tensor,
               dt_bias: torch.Tensor, neg_a: torch.Tensor, state: torch.Tensor, cu_q, ctx, slots,
               G: int, num_decode: int = 0, chunks: DeltaChunks | None = None) -> torch.Tensor:
    """Gated delta rule over each sequence's rows, from and to ``state`` (fp32
    [slots, H, N, P]): with q, k (rows of G x N channels, shared by H / G heads)
    divided by their norms sqrt(sum + 1e-6), q also by sqrt(N), v of H x P,
    beta = sigmoid(b), g = exp(neg_a softplus(a + dt_bias)) per head,

        S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q

    Sequences before ``num_decode`` (one row each) take the recurrent kernel;
    the others the chunked MFMA kernels when ``chunks`` is given and the shape
    allows it, the recurrent one otherwise.  Returns rows [T, H * P]."""
    _, H, N, P = state.shape
    T, S = q.shape[0], ctx.numel()
    _chk(H % G == 0, "delta_rule: heads per group")
    out = torch.empty((T, H * P), dtype=q.dtype, device=q.device)
    if not q.is_cuda:
        ref.delta_rule(q, k, v, b, a, dt_bias, neg_a, out, state, cu_q, ctx, slots, G)
        return out
    bf = _rows_dtype(q, "q")
    for t, c, name in ((q, G * N, "q"), (k, G * N, "k"), (v, H * P, "v"), (b, H, "b"), (a, H, "a")):
        _chk(t.dtype == q.dtype and t.shape[0] == T and t.shape[1] >= c and t.stride(1) == 1,
             f"delta_rule {name} rows")
    _chk(state.dtype == torch.float32 and state.is_contiguous(), "delta_rule state: fp32")
    _meta(S, cu_q=cu_q, ctx=ctx, slots=slots)
    _f32(dt_bias, H, "dt bias"); _f32(neg_a, H, "neg_a")
    args = (_ptr(q), q.stride(0), _ptr(k), k.stride(0), _ptr(v), v.stride(0), _ptr(b), b.stride(0),
            _ptr(a), a.stride(0), _ptr(dt_bias), _ptr(neg_a), _ptr(out), out.stride(0), _ptr(state),
            _ptr(cu_q), _ptr(ctx), _ptr(slots), H, G, N, P)
    chunked = chunks is not None and S > num_decode and _chunk_ok(N, P, q, k, v)
    n_rec = num_decode if chunked else S
    if n_rec:
        native().delta_recurrent(*args, n_rec, bf, _stream())
    if chunked:
        g = chunks
        _chk(g.chunks.dtype == torch.int32 and g.chunks.numel() >= 2 * g.n
             and g.first.dtype == torch.int32 and g.first.numel() == S - num_decode + 1,
             "delta_rule chunks")
        mats = torch.empty((g.n, H, DELTA_MATS), dtype=torch.bfloat16, device=q.device)
        vecs = torch.empty((g.n, H, DELTA_VECS), dtype=torch.float32, device=q.device)
        native().delta_chunks(*args, num_decode, S - num_decode, _ptr(g.chunks), g.n,
                              _ptr(g.first), _ptr(mats), _ptr(vecs), _stream())
    return out


DELTA_MATS = 4 * 6 * 512   # per chunk and head: two triangular matrices as bf16 pairs
DELTA_VECS = 5 * 64        # per chunk and head: per-token factors (delta.hip)


# ---------------------------------------------------------------- attention --
def row_quads(qlens, ctx, seq0: int) -> np.ndarray:
    """int32 [n + 1]: row starts of groups of up to 4 rows that share a key quad
    of the cache (positions 4i .. 4i + 3), then the end; the rows of the seq0
    single-row sequences in front are groups of their own."""
    qlens, ctx = np.asarray(qlens, np.int64), np.asarray(ctx, np.int64)
    p0 = ctx - qlens
    n = (ctx - 1) // 4 - p0 // 4 + 1
    i = np.arange(int(n.sum())) - np.repeat(np.cumsum(n) - n, n)
    row0 = seq0 + np.cumsum(qlens) - qlens
    start = np.maximum((np.repeat(p0 // 4, n) + i) * 4, np.repeat(p0, n))
    rows = np.repeat(row0 - p0, n) + start
    return np.concatenate([np.arange(seq0), rows, [seq0 + qlens.sum()]]).astype(np.int32)


def norm_rope_cache(p: torch.Tensor, q_norm: torch.Tensor, k_norm: torch.Tensor,
                    angles: torch.Tensor | None, slots, k_cache, v_cache, Hq: int, dk: int,
                    eps: float, quads: torch.Tensor | None = None) -> torch.Tensor:
    """The projection rows' q | k | v heads (each padded to D channels): q and k
    RMS-normed over the ``dk`` true channels (gains fp32 [D], zero in the
    padding), their first channels turned by ``angles`` (neighbours paired); k
    and v go to the paged cache at ``slots`` (-1: none).  ``quads``
    (``row_quads``): rows whose values are written together (None: every row
    alone).  Returns q rows [T, Hq * D]."""
    _, Hkv, BS, D = k_cache.shape
    T = p.shape[0]
    if not p.is_cuda:
        return ref.norm_rope_cache(p, q_norm, k_norm, angles, slots, k_cache, v_cache, Hq, dk, eps)
    bf = _rows_dtype(p, "p")
    C = (Hq + 2 * Hkv) * D
    _f32(q_norm, D, "q_norm"); _f32(k_norm, D, "k_norm")
    n = 0
    if angles is not None:
        n = angles.shape[1]
        _f32(angles, T * n, "angles")
    _meta(T, slots=slots)
    _chk(p.shape[1] >= C and p.stride(1) == 1 and p.stride(0) % 8 == 0 and p.data_ptr() % 16 == 0
         and n <= dk <= D and k_cache.dtype == v_cache.dtype == p.dtype
         and k_cache.is_contiguous() and v_cache.is_contiguous(), "norm_rope_cache rows")
    _chk(quads is None or (quads.dtype == torch.int32 and quads.is_contiguous()
                           and quads.numel() >= 2), "row quads")
    q = torch.empty((T, Hq * D), dtype=p.dtype, device=p.device)
    groups = T if quads is None else quads.numel() - 1
    native().norm_rope_cache(_ptr(p), p.stride(0), _ptr(q_norm), _ptr(k_norm), _ptr(angles), n,
                             _ptr(slots), _ptr(quads), groups, _ptr(q), _ptr(k_cache),
                             _ptr(v_cache), Hq, Hkv, D, dk, BS, float(eps), bf, _stream())
    return q


# ------------------------------------------------- attention of mixed heads --
@dataclass
class Talk:
    """What talking heads add to attention: the heads' scores mixed, score_h <-
    sum_g mix[h, g] score_g (scores are already scaled in the queries), and a
    sink per head, exp(sink_h) more in the softmax's denominator."""
    mix: torch.Tensor           # [H, H], the model's dtype
    sink: torch.Tensor          # fp32 [H]


TALK_QT = 8                     # query rows per prefill workgroup (talk.hip)
TALK_MAX_HEADS = 32             # heads of the MFMA kernels (head sizes 64, 128)
TALK_PART = 64                  # least keys of a decode partition


def talk_tiles(qlens, ctx, chunk: int) -> np.ndarray:
    """``row_tiles`` of TALK_QT rows in dispatch order: blocks of 8 neighbours,
    which walk the same pages, keep to one XCD (workgroup b runs on XCD b % 8),
    the longest walks first."""
    t = row_tiles(qlens, TALK_QT)
    n = np.asarray(qlens, np.int64)[t[:, 0]]
    p0 = np.asarray(ctx, np.int64)[t[:, 0]] - n + t[:, 1]
    p1 = p0 + np.minimum(TALK_QT, n - t[:, 1]) - 1
    first = p0 // chunk * chunk if chunk else np.zeros_like(p0)
    walk = p1 // 32 - first // 32 + 1
    blocks = -(-len(t) // 64) * 8
    at = np.full(blocks * 8, -1)
    at[:len(t)] = np.arange(len(t))
    cost = np.zeros(blocks * 8, np.int64)
    cost[:len(t)] = walk
    order = np.argsort(-cost.reshape(blocks, 8).max(1), kind="stable")
    at = at.reshape(blocks, 8)[order].reshape(-1, 8, 8).transpose(0, 2, 1).reshape(-1)
    return t[at[at >= 0]]


def talk_kernel_ok(Hq: int, Hkv: int, D: int) -> bool:
    """Geometries of the MFMA kernels (bf16)."""
    return D in (64, 128) and Hq <= TALK_MAX_HEADS and Hq % Hkv == 0 and Hq // Hkv <= 16


def talking_attention(q: torch.Tensor, k_cache, v_cache, block_tables, cu_q, ctx, positions,
                      talk: Talk, Hq: int, gate: torch.Tensor, out: torch.Tensor,
                      chunk: int = 0, out_scale: float = 1.0, num_decode: int = 0, tiles=None,
                      ws=None) -> torch.Tensor:
    """Causal paged attention of every row with mixed heads (``Talk``), decode
    and prompt rows alike: query rows [T, Hq * D] that carry their scale.
    ``chunk`` (0: none): a row sees the positions up to its own of its chunk of
    that many, counted from position 0.  Output rows times out_scale
    sigmoid(gate) into ``out`` (any row stride).

    Rows before ``num_decode`` are single rows of their sequences; ``tiles``
    (``talk_tiles``) covers the others.  bf16 rows of
    ``talk_kernel_ok`` geometries run on MFMA."""
    _, Hkv, BS, D = k_cache.shape
    T, S, nd = q.shape[0], ctx.numel(), num_decode
    _chk(out.shape == (T, Hq * D) and out.dtype == q.dtype and out.stride(1) == 1
         and gate.dtype == q.dtype and gate.shape[0] == T and gate.shape[1] >= Hq * D
         and gate.stride(1) == 1 and chunk >= 0, "talking_attention rows")
    if not q.is_cuda:
        o = ref.talking_attention(q.reshape(T, Hq, D), k_cache, v_cache, block_tables, cu_q, ctx,
                                  1.0, talk.mix, talk.sink, chunk).reshape(T, Hq * D).float()
        return out.copy_(o * torch.sigmoid(gate[:, :Hq * D].float()) * out_scale)
    bf = _rows_dtype(q, "q")
    _chk(q.shape[1] == Hq * D and q.is_contiguous() and k_cache.dtype == v_cache.dtype == q.dtype
         and BS == 32 and D in (64, 128, 256, 512), "talking_attention")
    _chk(talk.mix.shape == (Hq, Hq) and talk.mix.dtype == q.dtype and talk.mix.is_contiguous(),
         "talking_attention: head mix")
    _f32(talk.sink, Hq, "sink")
    _meta(S, cu_q=cu_q, ctx=ctx)
    _meta(T, positions=positions)
    _chk(block_tables.dtype == torch.int32 and block_tables.shape[0] >= S
         and block_tables.stride(1) == 1, "block tables")
    k = native()
    if not bf or not talk_kernel_ok(Hq, Hkv, D):
        k.talk_any(_ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(block_tables),
                   block_tables.stride(0), _ptr(cu_q), S, _ptr(positions), T, _ptr(talk.mix),
                   _ptr(talk.sink), _ptr(out), out.stride(0), _ptr(gate), gate.stride(0),
                   float(out_scale), Hq, Hkv, D, chunk, bf, _stream())
        return out
    _chk(out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0 and gate.stride(0) % 8 == 0
         and gate.data_ptr() % 16 == 0, "talking_attention: aligned rows")
    args = (_ptr(k_cache), _ptr(v_cache), _ptr(talk.mix), _ptr(talk.sink), float(out_scale), Hq,
            Hkv, D, chunk)
    if nd:
        parts = ws.max_parts if ws is not None else 1
        _chk(parts == 1 or (ws.part_o.numel() >= nd * Hq * parts * D
                            and ws.part_ml.numel() >= nd * Hq * parts * 2),
             "talking_attention workspace")
        k.talk_decode(_ptr(q), *args, _ptr(block_tables), block_tables.stride(0), _ptr(ctx), nd,
                      _ptr(gate), gate.stride(0), _ptr(out), out.stride(0),
                      _ptr(ws.part_o) if ws else 0, _ptr(ws.part_ml) if ws else 0, TALK_PART,
                      parts, _stream())
    if T > nd:
        _chk(tiles is not None and tiles.dtype == torch.int32 and tiles.is_contiguous(),
             "talking_attention tiles")
        k.talk_prefill(_ptr(q), *args, _ptr(block_tables[nd:]), block_tables.stride(0),
                       _ptr(cu_q[nd:]), _ptr(ctx[nd:]), _ptr(tiles), tiles.numel() // 2,
                       _ptr(gate), gate.stride(0), _ptr(out), out.stride(0), _stream())
    return out


def qkv_norm_rope_cache(p: torch.Tensor, bias: torch.Tensor, q_norm: torch.Tensor,
                        k_norm: torch.Tensor, angles: torch.Tensor | None, slots, k_cache, v_cache,
                        Hq: int, dk: int, dv: int, eps: float,
                        quads: torch.Tensor | None = None) -> torch.Tensor:
    """The projection rows' q | k | v heads (each padded to D channels) plus
    ``bias`` (fp32, all heads): q, and k, RMS-normed over the ``dk`` true
    channels of all their heads at once (gains fp32 [heads * D], zero in the
    padding), each head's first channels turned by ``angles`` (neighbours
    paired); v heads divided by their root mean square over ``dv``.  k and v go
    to the paged cache at ``slots`` (-1: none).  ``quads`` as in
    ``norm_rope_cache``.  Returns q rows [T, Hq * D]."""
    _, Hkv, BS, D = k_cache.shape
    T, C = p.shape[0], (Hq + 2 * Hkv) * D
    if not p.is_cuda:
        return ref.qkv_norm_rope_cache(p, bias, q_norm, k_norm, angles, slots, k_cache, v_cache,
                                       Hq, dk, dv, eps)
    bf = _rows_dtype(p, "p")
    _f32(bias, C, "bias"); _f32(q_norm, Hq * D, "q_norm"); _f32(k_norm, Hkv * D, "k_norm")
    n = 0
    if angles is not None:
        n = angles.shape[1]
        _f32(angles, T * n, "angles")
    _meta(T, slots=slots)
    _chk(p.shape[1] >= C and p.stride(1) == 1 and p.stride(0) % 8 == 0 and p.data_ptr() % 16 == 0
         and n <= dk <= D and 0 < dv <= D and k_cache.dtype == v_cache.dtype == p.dtype
         and k_cache.is_contiguous() and v_cache.is_contiguous(), "qkv_norm_rope_cache rows")
    _chk(quads is None or (quads.dtype == torch.int32 and quads.is_contiguous()
                           and quads.numel() >= 2), "row quads")
    q = torch.empty((T, Hq * D), dtype=p.dtype, device=p.device)
    groups = T if quads is None else quads.numel() - 1
    native().qkv_norm_rope_cache(_ptr(p), p.stride(0), _ptr(bias), _ptr(q_norm), _ptr(k_norm),
                                 _ptr(angles), n, _ptr(slots), _ptr(quads), groups, _ptr(q),
                                 _ptr(k_cache), _ptr(v_cache), Hq, Hkv, D, dk, dv, BS, float(eps),
                                 bf, _stream())
    return q


# ------------------------------------------------------------ matrix memory --
def memory_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, ig: torch.Tensor,
                fg: torch.Tensor, bias: torch.Tensor, cap: float, state, cu_q, ctx, slots,
                num_decode: int = 0, segments: ScanSegments | None = None) -> torch.Tensor:
    """Matrix memory with exponential gates over each sequence's rows, from and
    to ``state`` = (S fp32 [slots, H, N, P], n fp32 [slots, H, N], m fp32
    [slots, H]), from S = n = m = 0.  Per head, with i = cap tanh((ig + bias[0])
    / cap), f = ln sigmoid(cap tanh((fg + bias[1]) / cap)) and q scaled by
    N^-1/2,

        m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T, n alike;
        o = S^T q / (max(|n q|, e^-m') + 1e-6)

    q, k: rows of H x N channels, v of H x P, ig and fg of H; bias fp32 [2, H].
    Sequences before ``num_decode`` (one row each) take the recurrent kernel;
    the others the chunked MFMA kernel when ``segments`` is given and the shape
    allows it, the recurrent one otherwise.  Returns rows [T, H * P]."""
    S_, n_, m_ = state
    _, H, N, P = S_.shape
    T, S = q.shape[0], ctx.numel()
    out = torch.empty((T, H * P), dtype=q.dtype, device=q.device)
    if not q.is_cuda:
        ref.memory_scan(q, k, v, ig, fg, bias, cap, out, state, cu_q, ctx, slots)
        return out
    bf = _rows_dtype(q, "q")
    for t, c, name in ((q, H * N, "q"), (k, H * N, "k"), (v, H * P, "v"), (ig, H, "ig"), (fg, H, "fg")):
        _chk(t.dtype == q.dtype and t.shape[0] == T and t.shape[1] >= c and t.stride(1) == 1,
             f"memory_scan {name} rows")
    for t, shape, name in ((S_, (H, N, P), "S"), (n_, (H, N), "n"), (m_, (H,), "m")):
        _chk(t.dtype == torch.float32 and t.is_contiguous() and tuple(t.shape[1:]) == shape
             and t.shape[0] == S_.shape[0], f"memory_scan state {name}")
    _chk(ig.stride(0) == fg.stride(0) and cap > 0, "memory_scan gates")
    _f32(bias, 2 * H, "gate bias")
    _meta(S, cu_q=cu_q, ctx=ctx, slots=slots)
    args = (_ptr(q), q.stride(0), _ptr(k), k.stride(0), _ptr(v), v.stride(0), _ptr(ig), _ptr(fg),
            ig.stride(0), _ptr(bias), float(cap), _ptr(out), out.stride(0), _ptr(S_), _ptr(n_),
            _ptr(m_), _ptr(cu_q), _ptr(ctx), _ptr(slots), H, N, P, bf)
    chunked = segments is not None and S > num_decode and _chunk_ok(N, P, q, k, v)
    n_rec = num_decode if chunked else S
    if n_rec:
        native().memory_scan(*args, 0, n_rec, 0, 0, 0, 0, 0, 0, _stream())
    if chunked:
        g = segments
        _chk(g.segs.dtype == torch.int32 and g.segs.numel() >= 4 * g.n
             and g.first.dtype == torch.int32 and g.first.numel() == S - num_decode + 1,
             "scan segments")
        ws = wn = None
        # a head of several column tiles chains its segments even where each is a
        # whole sequence: the tiles share n and m
        one_pass = g.one_pass and P <= (SCAN_VT if N <= 128 else SCAN_VT // 2)
        if not one_pass:
            ws = torch.empty((g.n, H, N, P), dtype=torch.float32, device=q.device)
            wn = torch.empty((g.n, H, N + 3), dtype=torch.float32, device=q.device)
        native().memory_scan(*args, num_decode, S - num_decode, _ptr(g.segs), g.n, _ptr(g.first),
                             int(one_pass), _ptr(ws), _ptr(wn), _stream())
    return out


def attention_any(q: torch.Tensor, k_cache, v_cache, block_tables, cu_q, ctx, positions,
                  scale: float, Hq: int, gate: torch.Tensor | None = None, window: int = 0,
                  cap: float = 0.0) -> torch.Tensor:
    """Causal paged attention of every row (decode and prompt rows alike), fp32
    arithmetic, for what the MFMA kernels do not cover: fp32 caches, head sizes
    256 / 512, more than 16 query heads per kv head.  Output times
    sigmoid(gate) when given.  ``window`` (0: all): a row sees that many last
    positions; ``cap`` (0: none): scores become cap tanh(score / cap)."""
    _, Hkv, BS, D = k_cache.shape
    T, S = q.shape[0], ctx.numel()
    out = torch.empty((T, Hq * D), dtype=q.dtype, device=q.device)
    if not q.is_cuda:
        o = ref.paged_prefill(q.reshape(T, Hq, D), k_cache, v_cache, block_tables, cu_q, ctx, scale,
                              True, window, cap)
        out.copy_(ref.gate_rows(o.reshape(T, Hq * D), gate))
        return out
    bf = _rows_dtype(q, "q")
    _chk(q.shape[1] == Hq * D and q.stride(1) == 1 and k_cache.dtype == q.dtype
         and v_cache.dtype == q.dtype and BS == 32 and D in (64, 128, 256, 512), "attention_any")
    _meta(S, cu_q=cu_q, ctx=ctx)
    _meta(T, positions=positions)
    _chk(block_tables.dtype == torch.int32 and block_tables.shape[0] >= S
         and block_tables.stride(1) == 1, "block tables")
    _chk(gate is None or (gate.dtype == q.dtype and gate.shape[0] == T
                          and gate.shape[1] >= Hq * D and gate.stride(1) == 1), "gate rows")
    native().attention_any(_ptr(q), q.stride(0), _ptr(k_cache), _ptr(v_cache),
                           _ptr(block_tables), block_tables.stride(0), _ptr(cu_q), S,
                           _ptr(positions), T, _ptr(out), out.stride(0), _ptr(gate),
                           gate.stride(0) if gate is not None else 0, Hq, Hkv, D, BS,
                           float(scale), window, float(cap), bf, _stream())
    return out


# -------------------------------------------------- gated linear recurrence --
RGLRU_TILE = 64            # channels per workgroup (csrc/kernels/rglru.hip)
RGLRU_MAX_BLOCK = 512      # gate blocks the MFMA kernels hold in registers


def rglru(u: torch.Tensor, y: torch.Tensor, y_bias: torch.Tensor, gates: GroupedWeight,
          gate_bias: torch.Tensor, log_a: torch.Tensor, state: torch.Tensor, cu_q, ctx, slots,
          num_decode: int = 0, segments: ScanSegments | None = None) -> torch.Tensor:
    """Per channel, over each sequence's rows and from / to ``state`` (fp32
    [slots, C]):

        r, i = sigmoid(block-diagonal gates of u + gate_bias)      [2, C]
        a = exp(log_a r);  S <- a S + sqrt(1 - a^2) i u
        out = S gelu_tanh(y + y_bias)

    gates: [blocks, 2 * C/blocks, C/blocks], the r rows before the i rows of a
    block.  Sequences before ``num_decode`` (one row each) take the row kernel,
    the others the chunked one (``segments``); fp32 rows and blocks above
    ``RGLRU_MAX_BLOCK`` a plain scan of fp32 gates."""
    T, C = u.shape
    n, bp, S = gates.groups, gates.K, ctx.numel()
    _chk(n * bp == C and gates.N == 2 * bp, "rglru gate blocks")
    out = torch.empty((T, C), dtype=u.dtype, device=u.device)
    if not u.is_cuda:
        ref.rglru(u, y, y_bias, gates.data, gate_bias, log_a, out, state, cu_q, ctx, slots)
        return out
    bf = _rows_dtype(u, "u")
    _chk(u.is_contiguous() and y.dtype == u.dtype and y.shape == (T, C) and y.stride(1) == 1,
         "rglru rows")
    _chk(state.dtype == torch.float32 and state.is_contiguous() and state.shape[1] == C,
         "rglru state")
    _f32(y_bias, C, "y bias"); _f32(gate_bias, 2 * C, "gate bias"); _f32(log_a, C, "log_a")
    _meta(S, cu_q=cu_q, ctx=ctx, slots=slots)
    args = (_ptr(u), _ptr(y), y.stride(0), _ptr(y_bias), _ptr(gate_bias), _ptr(log_a), _ptr(out),
            _ptr(state), _ptr(cu_q), _ptr(ctx), _ptr(slots), C, bp)
    if not gates.packed:
        z = grouped_heads(u.float(), gates)
        native().rglru_scan(*args, _ptr(z), S, bf, _stream())
        return out
    if num_decode:
        native().rglru_rows(*args, _ptr(gates.data), num_decode, _stream())
    if S > num_decode:
        g = segments
        _chk(g is not None and g.segs.dtype == torch.int32 and g.segs.numel() >= 4 * g.n
             and g.first.dtype == torch.int32 and g.first.numel() == S - num_decode + 1,
             "rglru segments")
        ws = None if g.one_pass else torch.empty((3, g.n, C), dtype=torch.float32, device=u.device)
        native().rglru_chunks(*args, _ptr(gates.data), num_decode, _ptr(g.segs), g.n,
                              _ptr(g.first), _ptr(ws), _stream())
    return out


# --------------------------------------------------------- latent attention --
def rope_freqs(base: float, dims: int, factor: float = 1.0, original: float = 0.0,
               fast: float = 0.0, slow: float = 0.0, device="cpu") -> torch.Tensor:
    """base^(-2i / dims) / factor, i < dims / 2 (double).  ``original`` > 0: a context of
    that length stretched by ``factor`` -- components that turn ``fast`` times
    and more within it stay, those that turn ``slow`` times and less are divided
    by the factor, a ramp between them."""
    i = torch.arange(dims // 2, dtype=torch.float64, device=device)
    f = torch.exp(-2.0 * math.log(base) / dims * i)
    if not original:
        return f / factor

    def turning(times):        # the component that turns that often
        return dims * math.log(original / (2 * math.pi * times)) / (2 * math.log(base))
    lo = max(math.floor(turning(fast)), 0)
    hi = min(math.ceil(turning(slow)), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return f / factor * ramp + f * (1 - ramp)


def rope_magnitude(base: float, dims: int, factor: float = 1.0, original: float = 0.0, *_) -> float:
    """What cos and sin of a rotation (``rope_freqs`` arguments) are multiplied by."""
    return 0.1 * math.log(factor) + 1.0 if original else 1.0


def rope_angles(positions: torch.Tensor, freqs: torch.Tensor, scale: float = 1.0) -> torch.Tensor:
    """fp32 [T, dims]: cos | sin of position * frequency, times ``scale``
    (reduced in double, so no table bounds the positions)."""
    if not positions.is_cuda:
        return ref.rope_angles(positions, freqs, scale)
    T, n = positions.numel(), freqs.numel()
    _chk(positions.dtype == torch.int32 and freqs.dtype == torch.float64, "rope_angles")
    out = torch.empty((T, 2 * n), dtype=torch.float32, device=positions.device)
    native().rope_angles(_ptr(positions), _ptr(freqs), T, n, float(scale), _ptr(out), _stream())
    return out


def latent_prep(p: torch.Tensor, qr: int, qp: int, q_norm: torch.Tensor, R: int,
                c_norm: torch.Tensor, angles: torch.Tensor, slots: torch.Tensor,
                pages: torch.Tensor, Rp: int, eps: float) -> torch.Tensor:
    """Projection rows [query latent (qr of qp) | latent c (R of Rp) | rotated
    key part | ..]: returns the RMS-normed query latents [T, qp]; the normed c
    and the key part turned by ``angles`` go to the pages' rows at ``slots``
    (-1: none).  Gains fp32 [qp], [Rp], zero in the padding."""
    T, d = angles.shape
    _, _, BS, D = pages.shape
    if not p.is_cuda:
        return ref.latent_prep(p, qr, qp, q_norm, R, c_norm, angles, slots, pages, Rp, eps)
    bf = _rows_dtype(p, "p")
    _f32(q_norm, qp, "q_norm"); _f32(c_norm, Rp, "c_norm"); _f32(angles, T * d, "angles")
    _meta(T, slots=slots)
    _chk(p.shape[0] == T and p.shape[1] >= qp + D and p.stride(1) == 1 and p.stride(0) % 8 == 0
         and p.data_ptr() % 16 == 0 and qp % 8 == 0 and Rp % 8 == 0 and d <= D - Rp
         and pages.dtype == p.dtype and pages.is_contiguous(), "latent_prep rows")
    cq = torch.empty((T, qp), dtype=p.dtype, device=p.device)
    native().latent_prep(_ptr(p), p.stride(0), T, qr, qp, _ptr(q_norm), R, Rp, _ptr(c_norm),
                         _ptr(angles), d, _ptr(slots), _ptr(pages), BS, D, _ptr(cq), float(eps),
                         bf, _stream())
    return cq


def latent_query(q: torch.Tensor, absorb: GroupedWeight, angles: torch.Tensor, H: int, np_: int,
                 xp: int, Rp: int) -> torch.Tensor:
    """Query rows of H x [np_ unrotated | xp to rotate] -> H x [W_uk^T q (Rp) |
    rotated part (xp)]: queries that score latent rows."""
    T, d = q.shape[0], angles.shape[1]
    if not q.is_cuda:
        return ref.latent_query(q, absorb.data, angles, H, np_, xp, Rp)
    bf = _rows_dtype(q, "q")
    _chk(q.stride(1) == 1 and q.shape[1] == H * (np_ + xp) and absorb.N == Rp
         and absorb.K == np_ and absorb.groups == H and d <= xp and angles.shape[0] >= T,
         "latent_query rows")
    out = torch.empty((T, H * (Rp + xp)), dtype=q.dtype, device=q.device)
    grouped_heads(q, absorb, out=out, in_stride=np_ + xp, out_stride=Rp + xp)
    native().latent_rotate(_ptr(q), q.stride(0), np_, _ptr(angles), d, T, H, xp, _ptr(out),
                           out.stride(0), Rp, bf, _stream())
    return out


def latent_attention(q: torch.Tensor, pages: torch.Tensor, block_tables, cu_q, positions,
                     scale: float, window: int, H: int, Rp: int, ws=None, part_tokens: int = 512,
                     num_decode: int = 0) -> torch.Tensor:
    """Attention of query rows (``latent_query``) over latent pages: row t of a
    sequence sees the ``window`` last positions up to its own; returns the
    weighted sums of latents [T, H * Rp].  Rows before ``num_decode`` are the
    first row of sequence t."""
    T = q.shape[0]
    _, one, BS, D = pages.shape
    S = cu_q.numel() - 1
    if not q.is_cuda:
        return ref.latent_attention(q, pages, block_tables, cu_q, positions, scale, window, H, Rp)
    bf = _rows_dtype(q, "q")
    _chk(one == 1 and BS == 32 and q.shape[1] == H * D and q.is_contiguous()
         and pages.dtype == q.dtype and 0 < Rp < D and window > 0, "latent_attention")
    _meta(S, cu_q=cu_q)
    _meta(T, positions=positions)
    _chk(block_tables.dtype == torch.int32 and block_tables.shape[0] >= S
         and block_tables.stride(1) == 1, "block tables")
    out = torch.empty((T, H * Rp), dtype=q.dtype, device=q.device)
    args = (_ptr(q), _ptr(pages), _ptr(block_tables), block_tables.stride(0), _ptr(cu_q), S,
            _ptr(positions), T)
    tail = (_ptr(out), H, Rp, D, float(scale), window)
    if not bf or D != Rp + 64 or Rp not in LATENT_RANKS:
        native().latent_any(*args, *tail, bf, _stream())
        return out
    # decode steps split a row's keys over workgroups until the chip is filled
    parts = ws.max_parts if ws is not None and T <= num_decode else 1
    if parts > 1:
        _chk(ws.part_o.numel() >= T * H * parts * Rp and ws.part_ml.numel() >= T * H * parts * 2,
             "latent_attention workspace")
    native().latent_rows(*args, num_decode, _ptr(out), _ptr(ws.part_o) if ws else 0,
                         _ptr(ws.part_ml) if ws else 0, *tail[1:], 128, parts, _stream())
    return out


LATENT_RANKS = (64, 128, 256, 512)   # latent widths of the MFMA kernel
LATENT_QT = 128            # query rows per prefill workgroup (latent.hip)


def latent_prefill_ok(np_: int, xp: int, vp: int) -> bool:
    """Head sizes of the expanded prefill kernel (bf16)."""
    return np_ in (64, 128) and xp == 64 and vp in (64, 128)


@dataclass
class LatentRows:
    """Key rows a step's multi-token sequences see, gathered back to back."""
    seqs: torch.Tensor      # int32 [sequences + 1, 2]: first gathered row, first position
    tiles: torch.Tensor     # int32 [n, 2]: sequence, first query row
    n: int                  # gathered rows


def latent_rows(qlens, ctx, window: int) -> tuple[np.ndarray, np.ndarray, int]:
    """Host plan of ``LatentRows``: a sequence with ``qlens`` new rows up to
    position ctx - 1 sees positions from ctx - qlens - window + 1."""
    ctx, qlens = np.asarray(ctx, np.int64), np.asarray(qlens, np.int64)
    k0 = np.maximum(ctx - qlens - (window - 1), 0)
    first = np.concatenate([[0], np.cumsum(ctx - k0)])
    seqs = np.stack([first, np.append(k0, 0)], 1).astype(np.int32)
    return seqs, row_tiles(qlens, LATENT_QT), int(first[-1])


def latent_prefill(q: torch.Tensor, pages: torch.Tensor, rows: LatentRows, w_kv: torch.Tensor,
                   angles: torch.Tensor, block_tables, cu_q, ctx, scale: float, window: int, H: int,
                   np_: int, vp: int, Rp: int, gate: torch.Tensor, out: torch.Tensor) -> None:
    """Prompt rows (bf16, GPU) of the sequences of ``block_tables`` / ``cu_q`` /
    ``ctx``: the cached rows they see are gathered, expanded by ``w_kv`` (H x
    [np_ key | vp value] rows of latents) and attended to; ``q`` as projected
    (H x [np_ | 64 to rotate]).  Output rows times sigmoid(gate), H x vp."""
    linear = importlib.import_module(__package__).linear
    S, D = ctx.numel(), pages.shape[3]
    d = angles.shape[1]
    for t, w in ((q, H * (np_ + 64)), (gate, H * vp), (out, H * vp)):
        _chk(t.dtype == torch.bfloat16 and t.shape[1] >= w and t.stride(1) == 1
             and t.data_ptr() % 16 == 0, "latent_prefill rows")
    _chk(q.shape[0] == gate.shape[0] == out.shape[0] == angles.shape[0]
         and angles.dtype == torch.float32, "latent_prefill rows")
    _chk(pages.dtype == torch.bfloat16 and pages.shape[1:3] == (1, 32) and D == Rp + 64 and d <= 64
         and tuple(w_kv.shape) == (H * (np_ + vp), Rp), "latent_prefill sizes")
    _meta(S, cu_q=cu_q, ctx=ctx)
    _chk(rows.seqs.dtype == rows.tiles.dtype == torch.int32 and rows.seqs.numel() == 2 * (S + 1)
         and rows.seqs.is_contiguous() and rows.tiles.is_contiguous(), "latent_prefill plan")
    _chk(block_tables.dtype == torch.int32 and block_tables.shape[0] == S
         and block_tables.stride(1) == 1, "block tables")
    k = native()
    lat = torch.empty((rows.n, D), dtype=q.dtype, device=q.device)
    k.latent_gather(_ptr(pages), _ptr(block_tables), block_tables.stride(0), _ptr(rows.seqs), S,
                    rows.n, D, _ptr(lat), _stream())
    kv = linear(lat[:, :Rp], w_kv)
    k.latent_prefill(_ptr(q), q.stride(0), _ptr(kv), _ptr(lat), _ptr(angles), _ptr(rows.seqs),
                     _ptr(rows.tiles), rows.tiles.shape[0], _ptr(cu_q), _ptr(ctx), _ptr(gate),
                     gate.stride(0), _ptr(out), out.stride(0), H, np_, vp, D, Rp, d, float(scale),
                     window, _stream())
