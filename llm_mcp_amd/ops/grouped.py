"""Grouped products (per-head maps, mixtures of experts) and what routes rows
to them.  Conventions as in the package: GPU tensors run csrc/kernels/
grouped.hip and moe.hip, CPU tensors the references in ``ops.ref``."""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _chk, _ptr, _stream, native, ref

MOE_MAX_EXPERTS = 256      # experts a router kernel ranks
MOE_MAX_TOP = 32
MOE_MAX_GROUPS = 64


@dataclass
class GroupedWeight:
    """[groups, N, K] weights; bf16 on the GPU: in MFMA fragment order."""
    data: torch.Tensor
    groups: int
    N: int
    K: int
    packed: bool


def pack_grouped(w: torch.Tensor) -> GroupedWeight:
    """[G, N, K] -> ``GroupedWeight``; bf16 on the GPU (N a multiple of 16, K of
    32): [G][N / 16][K / 32][k / 8][n][8]."""
    G, N, K = w.shape
    if not w.is_cuda or w.dtype != torch.bfloat16:
        return GroupedWeight(w.contiguous(), G, N, K, False)
    _chk(N % 16 == 0 and K % 32 == 0, f"packed weights: N {N}, K {K}")
    p = w.view(G, N // 16, 16, K // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).contiguous()
    return GroupedWeight(p, G, N, K, True)


class Mixture:
    """Sublayer output rows as weighted sums of expert rows, left to the
    consuming kernel: row t = sum_j weights[t, j] rows[pos[t, j]] (pos -1: no
    such row), plus ``own``[t] (fp32 [T], optional) times the stream's own row,
    which such a sublayer reads as it is."""
    __slots__ = ("rows", "pos", "weights", "own")

    def __init__(self, rows: torch.Tensor, pos: torch.Tensor, weights: torch.Tensor,
                 own: torch.Tensor | None = None):
        self.rows, self.pos, self.weights, self.own = rows, pos, weights, own

    def sum(self) -> torch.Tensor:
        x = self.rows[self.pos.clamp_min(0).long()].float()
        return (x * (self.weights * (self.pos >= 0))[..., None]).sum(1)


@dataclass
class Route:
    ids: torch.Tensor        # int32 [T, J] expert of each use (-1: an identity expert)
    weights: torch.Tensor    # fp32 [T, J]
    own: torch.Tensor | None = None   # fp32 [T]: weight of a row's identity experts


@dataclass
class GroupScores:
    """Routing by scores s of the logits: experts are chosen by s +
    ``correction`` (fp32 [E]) within the ``keep`` best of ``groups`` groups of
    neighbours.

    ``softmax``: s is the softmax over all E logits, a group ranks by its
    largest corrected score and the weights are the s as they are; otherwise s =
    sigmoid, a group ranks by the sum of its two largest, the weights are in
    proportion to s.  ``identity``: that many of the last experts return their
    input."""
    correction: torch.Tensor
    groups: int = 1
    keep: int = 1
    softmax: bool = False
    identity: int = 0


def moe_route(h: torch.Tensor, w: torch.Tensor, top: int, extra: int = 0,
              scores: GroupScores | None = None) -> Route:
    """The ``top`` largest of the fp32 logits w h per row (lowest index first
    among equals) with the softmax over just those; then experts E, E + 1, ..
    (``extra`` of them) with weight 1.

    With ``scores``: the ``top`` largest s + correction, s = sigmoid(w h), among
    the groups with the largest sums of two such scores, in the proportions of
    their s; a row of w behind the E experts' is the logit whose sigmoid weighs
    the extra ones.  ``GroupScores`` has the other forms; the identity experts a
    row chose are in ``Route.own``, not among the uses."""
    rows, d = w.shape
    E = rows if scores is None else scores.correction.numel()
    T = h.shape[0]
    _chk(0 < top <= E and rows - E in (0, 1), "moe_route: top, router rows")
    if scores is not None:
        _chk(E % scores.groups == 0 and scores.groups <= MOE_MAX_GROUPS
             and 0 < scores.keep <= scores.groups and scores.keep * (E // scores.groups) >= top,
             "moe_route: groups")
        _chk(0 <= scores.identity < E and not (scores.softmax and rows > E),
             "moe_route: identity experts, router rows")
    if not h.is_cuda:
        return Route(*(ref.moe_route(h, w, top, extra) if scores is None else
                       ref.moe_route_groups(h, w, top, extra, scores)))
    _chk(rows <= MOE_MAX_EXPERTS and top + extra <= MOE_MAX_TOP, "moe_route: sizes")
    corr, groups, keep, soft, ident, own = None, 1, 1, 0, 0, None
    if scores is not None:
        corr, groups, keep = scores.correction, scores.groups, scores.keep
        soft, ident = int(scores.softmax), scores.identity
        if ident:
            own = torch.empty(T, dtype=torch.float32, device=h.device)
        _chk(corr.dtype == torch.float32 and corr.is_contiguous() and corr.is_cuda,
             "moe_route: fp32 correction")
    _chk(h.dtype == w.dtype and h.dtype in (torch.bfloat16, torch.float32)
         and h.shape[1] == d and h.stride(1) == 1 and w.is_contiguous(), "moe_route operands")
    ids = torch.empty((T, top + extra), dtype=torch.int32, device=h.device)
    wts = torch.empty((T, top + extra), dtype=torch.float32, device=h.device)
    native().moe_route(_ptr(h), h.stride(0), _ptr(w), T, d, E, rows, top, extra, _ptr(corr), groups,
                       keep, soft, ident, _ptr(ids), _ptr(wts), _ptr(own),
                       int(h.dtype == torch.bfloat16), _stream())
    return Route(ids, wts, own)


@dataclass
class MoePlan:
    """Uses (row, expert) sorted by expert; those with id -1 are left out."""
    src: torch.Tensor        # int32 [n]: row of each sorted use
    pos: torch.Tensor        # int32 [T, J]: sorted place of each use (-1: left out)
    off: torch.Tensor        # int32 [groups + 1]
    tiles: torch.Tensor | None   # int32 [mtiles, 2]: group (-1: none), first sorted row; one
    bm: int                      # more entry: the number of used ones


def _tile_rows(n: int, groups: int, bf16: bool, wide: bool) -> int:
    """Rows per tile of the grouped kernels for n rows over ``groups``; 256: the
    persistent tile of K13, for products of whole 256-column tiles (``wide``)."""
    if not bf16:
        return 32
    mean = n / groups
    return 16 if mean <= 6 else 32 if mean <= 24 else 64 if mean < 96 else 256 if wide and mean >= 192 else 128


def wide_tiles(w: GroupedWeight) -> bool:
    """K13's grouped form takes this weight."""
    return w.packed and w.N % 256 == 0 and w.K % 64 == 0 and w.K >= 192


def moe_plan(r: Route, groups: int, bf16: bool = True, wide: bool = False) -> MoePlan:
    """Sort a route's uses by expert and list the row tiles (``bf16``: of the
    packed kernels; ``wide``: every product of the plan is ``wide_tiles``)."""
    T, J = r.ids.shape
    n = T * J
    ids = r.ids
    if not ids.is_cuda:
        flat = ids.reshape(-1).long()
        order = torch.argsort(torch.where(flat < 0, groups, flat), stable=True)
        pos = torch.empty(n, dtype=torch.int32)
        pos[order] = torch.arange(n, dtype=torch.int32)
        pos[flat < 0] = -1
        cnt = torch.bincount(flat[flat >= 0], minlength=groups)
        off = torch.cat([torch.zeros(1, dtype=torch.int64), cnt.cumsum(0)]).to(torch.int32)
        return MoePlan((order // J).to(torch.int32), pos.view(T, J), off, None, 0)
    _chk(0 < groups <= MOE_MAX_EXPERTS and ids.is_contiguous(), "moe_plan")
    bm = _tile_rows(n, groups, bf16, wide)
    mt = min(n, -(-n // bm) + groups)
    i32 = dict(dtype=torch.int32, device=ids.device)
    src, pos = torch.empty(n, **i32), torch.empty((T, J), **i32)
    off, tiles = torch.empty(groups + 1, **i32), torch.empty((mt + 1, 2), **i32)
    blocks = -(-n // MOE_CHUNK)
    hist = torch.empty((blocks, groups), **i32)
    native().moe_plan(_ptr(ids), n, J, groups, bm, mt, _ptr(hist), _ptr(off), _ptr(src), _ptr(pos),
                      _ptr(tiles), _stream())
    return MoePlan(src, pos, off, tiles, bm)


MOE_CHUNK = 1024           # uses per block of the sort (moe.hip)


def _grouped(a, a_gs, w: GroupedWeight, c, c_gs, M, bm, mtiles, plan=None, src=None, limit=None,
             gate=None, act=(1.702, 1.0)):
    bf = int(w.packed)
    _chk(a.dtype == w.data.dtype == c.dtype and a.stride(1) == 1 and c.stride(1) == 1
         and (w.packed or a.dtype == torch.float32), "grouped operands")
    native().grouped(_ptr(a), a.stride(0), a_gs, _ptr(w.data), _ptr(c), c.stride(0), c_gs,
                     w.groups, w.N, w.K, M, _ptr(plan.tiles) if plan else 0, mtiles,
                     _ptr(plan.off) if plan else 0, _ptr(src), _ptr(limit), *act, _ptr(gate),
                     gate.stride(0) if gate is not None else 0, bm, bf, _stream())


def grouped_linear(x: torch.Tensor, w: GroupedWeight, plan: MoePlan, gather: bool = False,
                   glu: torch.Tensor | None = None,
                   act: tuple[float, float] = (1.702, 1.0)) -> torch.Tensor:
    """Rows in expert order [n, N]: x[src] (``gather``) or x's own rows times
    their expert's w^T.  ``glu`` (fp32 [groups], the clamps; inf: none): w's
    rows are gate / up interleaved per 16, the result is g sigmoid(act[0] g)
    (u + act[1]) of the clamped pair, [n, N / 2]."""
    n = plan.src.numel()
    if not x.is_cuda:
        return ref.grouped_rows(x, w.data, plan.src, plan.off, gather, glu, act)
    _chk(x.shape[1] >= w.K and (gather or x.shape[0] == n), "grouped_linear rows")
    _chk(plan.off.numel() == w.groups + 1 and plan.bm in (16, 32, 64, 128, 256), "grouped_linear plan")
    _chk(glu is None or (glu.dtype == torch.float32 and glu.numel() == w.groups and w.N % 32 == 0),
         "grouped_linear clamps")
    _chk(w.packed or plan.bm == 32, "grouped_linear: plan of another precision")
    out = torch.empty((n, w.N // 2 if glu is not None else w.N), dtype=x.dtype, device=x.device)
    src, mt = plan.src if gather else None, plan.tiles.shape[0] - 1
    if plan.bm == 256:
        _chk(wide_tiles(w) and x.dtype == torch.bfloat16 and x.stride(1) == 1
             and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0, "grouped_linear: K13 operands")
        native().pgemm_grouped(_ptr(out), _ptr(x), _ptr(w.data), n, w.N, w.K, x.stride(0),
                               out.stride(0), x.shape[0], _ptr(plan.tiles), mt, _ptr(plan.off),
                               _ptr(src), _ptr(glu), *act, _stream())
    else:
        _grouped(x, 0, w, out, 0, n, plan.bm, mt, plan, src, glu, act=act)
    return out


def grouped_heads(x: torch.Tensor, w: GroupedWeight, gate: torch.Tensor | None = None,
                  out: torch.Tensor | None = None, in_stride: int | None = None,
                  out_stride: int | None = None) -> torch.Tensor:
    """Each head's columns of x (head h from h * in_stride, K of them) times
    w[h]^T into out's columns from h * out_stride (N of them), times
    sigmoid(gate) at the same columns when given."""
    M, a_gs, c_gs = x.shape[0], in_stride or w.K, out_stride or w.N
    if out is None:
        out = torch.empty((M, w.groups * c_gs), dtype=x.dtype, device=x.device)
    if not x.is_cuda:
        for h in range(w.groups):
            y = x[:, h * a_gs:h * a_gs + w.K].float() @ w.data[h].float().t()
            if gate is not None:
                y = y * torch.sigmoid(gate[:, h * c_gs:h * c_gs + w.N].float())
            out[:, h * c_gs:h * c_gs + w.N] = y.to(out.dtype)
        return out
    last = w.groups - 1
    _chk(x.shape[1] >= last * a_gs + w.K and out.shape[0] == M
         and out.shape[1] >= last * c_gs + w.N, "grouped_heads rows")
    _chk(gate is None or (gate.dtype == x.dtype and gate.stride(1) == 1 and gate.shape[0] == M
                          and gate.shape[1] >= last * c_gs + w.N), "grouped_heads gate")
    bm = 32 if not w.packed else 16 if M <= 16 else 32 if M <= 32 else 64 if M <= 128 else 128
    _grouped(x, a_gs, w, out, c_gs, M, bm, -(-M // bm), gate=gate)
    return out
