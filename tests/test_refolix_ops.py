"""The ops of retention, the gated delta rule, capped window attention, group
routing and the norm of the sum one by one against the plain equations of
``refolix_oracle``, on the CPU references and the GPU kernels."""
import math

import numpy as np
import pytest
import torch

import refolix_oracle as oracle
from llm_mcp_amd import ops
from llm_mcp_amd.ops import mixers
from test_mixer_ops import DEV, OUT_TOL, Batch, close, rnd

GPU = pytest.mark.gpu


@pytest.fixture(autouse=True, scope="module")
def _one_thread():
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def i32(x, dev):
    return torch.tensor(np.asarray(x), dtype=torch.int32, device=dev).contiguous()


# ------------------------------------------------------------- norm of the sum --
@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("d", [64, 100, 4096])
@pytest.mark.parametrize("kind", ["rows", "partials", "mixture", "pair", "pair of partials"])
def test_norm_of_the_sum(dev, dt, d, kind):
    T, eps, alpha = 6, 1e-3, 1.7
    x = rnd(T, d) + 0.5
    s, w, pre = (1 + 0.3 * rnd(d, seed=k) for k in (1, 2, 3))
    ya, yb = rnd(T, d, seed=4, scale=2.0).to(dt), rnd(T, d, seed=5, scale=0.1).to(dt)
    wa, wb = 0.5 + 0.2 * rnd(d, seed=6), 0.5 + 0.2 * rnd(d, seed=7)

    def partials(y):
        a = rnd(T, d, seed=8)
        return ops.Partials(torch.stack([y.float() - a, a]).to(dev).contiguous(), 2, T, d)
    if kind == "mixture":
        g = torch.Generator().manual_seed(9)
        pos = torch.randint(0, T, (T, 3), generator=g).to(torch.int32)
        wt = torch.rand(T, 3, generator=g)
        y = ops.Mixture(ya.to(dev), pos.to(dev), wt.to(dev))
        yr = (ya.double()[pos.long()] * wt.double()[..., None]).sum(1)
    elif kind.startswith("pair"):
        a, b = (partials(ya), partials(yb)) if "partials" in kind else (ya.to(dev), yb.to(dev))
        if dev == "cpu" and "partials" in kind:
            pytest.skip("partials are the GPU products' own")
        y = ops.NormedPair(a, b, wa.to(dev), wb.to(dev))
        yr = oracle.unit_rms(ya.double(), eps) * wa.double() + \
            oracle.unit_rms(yb.double(), eps) * wb.double()
    else:
        if dev == "cpu" and kind == "partials":
            pytest.skip("partials are the GPU products' own")
        y, yr = (partials(ya) if kind == "partials" else ya.to(dev)), ya.double()
    r = oracle.layer_norm(alpha * x.double() + s.double() * yr, w.double(), eps)
    z = oracle.layer_norm(r, pre.double(), eps)
    for w_pre, rows, want in ((None, None, r), (pre, None, z), (pre, [4, 0, 5], z[[4, 0, 5]])):
        res = x.clone().to(dev)
        pick = torch.tensor(rows, device=dev) if rows else None
        h = ops.sum_norm(res, eps, y, alpha, s.to(dev), w.to(dev),
                         None if w_pre is None else w_pre.to(dev), pick, dtype=dt)
        assert h.dtype == dt
        close(h, want, OUT_TOL[dt], kind)
        if rows:
            assert torch.equal(res.cpu(), x)
        else:
            close(res, r, 1e-5, "residual stays fp32")
    res = x.clone().to(dev)
    h = ops.sum_norm(res, eps, None, alpha, None, None, pre.to(dev), torch.tensor([2], device=dev),
                     dtype=dt)
    close(h, oracle.layer_norm(x.double(), pre.double(), eps)[[2]], OUT_TOL[dt], "norm alone")


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("n", [37, 4096])
def test_soft_cap(dev, dt, n):
    x = rnd(3, n, scale=20.0).to(dt)
    close(ops.soft_cap(x.clone().to(dev), 0.7, 9.0), oracle.soft_cap(x.double() * 0.7, 9.0),
          OUT_TOL[dt])
    close(ops.soft_cap(x.clone().to(dev), 0.7, None), x.double() * 0.7, OUT_TOL[dt])


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("part", [8, 12, 64, 128, 200, 512, 1024])
def test_gated_norm_with_silu(dev, dt, part):
    """Parts of a lane group, of a workgroup, and of neither."""
    T, H, eps = 5, 3, 1e-4
    x, g = rnd(T, H * part).to(dt), rnd(T, H * part + 16, seed=1).to(dt)
    w = 1 + 0.3 * rnd(H * part, seed=2)
    want = oracle.unit_rms(x.double().view(T, H, part), eps).view(T, -1) * w.double() * \
        oracle.silu(g.double()[:, :H * part])
    close(ops.gated_norm(x.to(dev), g.to(dev), w.to(dev), H, eps, gate_first=False, silu=True),
          want, OUT_TOL[dt])


# ------------------------------------------------------------------ rotation --
ROTS = [dict(base=1e4, dims=8), dict(base=300.0, dims=12, scaling=dict(factor=3.0, original=48, fast=6.0, slow=0.5)),
        dict(base=1e6, dims=64, scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0)),
        # both ends of the ramp outside the components, and a ramp of no width
        dict(base=10.0, dims=6, scaling=dict(factor=2.0, original=8, fast=900.0, slow=1e-6)),
        dict(base=1e4, dims=16, scaling=dict(factor=2.0, original=64, fast=1e9, slow=1e8))]


def rot_args(rot):
    s = rot.get("scaling") or {}
    return (rot["base"], rot["dims"], *(s[k] for k in ("factor", "original", "fast", "slow") if s))


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda", marks=GPU)])
@pytest.mark.parametrize("rot", ROTS, ids=range(len(ROTS)))
def test_angles(dev, rot):
    pos = torch.tensor([0, 1, 7, 100, 65537, 1000003])
    args = rot_args(rot)
    f = ops.rope_freqs(*args, device=dev)
    ang = ops.rope_angles(i32(pos, dev), f, ops.rope_magnitude(*args))
    a = pos.double()[:, None] * oracle.frequencies(rot)
    close(ang, oracle.magnitude(rot) * torch.cat([a.cos(), a.sin()], 1), 2e-6)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("Hq,Hkv,D,dk,rot", [(4, 2, 64, 64, ROTS[2]), (6, 2, 128, 90, ROTS[1]),
                                             (3, 3, 64, 7, ROTS[3]), (2, 1, 512, 300, ROTS[0]),
                                             (2, 2, 64, 20, None)])
def test_head_norm_rotation_and_cache(dev, dt, Hq, Hkv, D, dk, rot):
    """Norm, rotation and cache write of portions that start and end inside key
    quads and pages, single rows beside them, rows without a slot."""
    eps, qlens, starts = 1e-4, [1, 1, 9, 2, 34], [5, 0, 3, 6, 29]
    T = sum(qlens)
    pos = np.concatenate([np.arange(s, s + n) for n, s in zip(qlens, starts)])
    perm = np.random.default_rng(0).permutation(12)
    pages = [perm[2 * i:2 * i + 2] for i in range(5)]
    slots = np.concatenate([[pages[i][p // 32] * 32 + p % 32 for p in range(s, s + n)]
                            for i, (n, s) in enumerate(zip(qlens, starts))])
    slots[1] = -1
    x = rnd(T, Hq + 2 * Hkv, D)
    x[:, :Hq + Hkv, dk:] = 0
    p = torch.cat([x.view(T, -1), torch.zeros(T, 8)], 1).to(dt)
    wq, wk = torch.zeros(D), torch.zeros(D)
    wq[:dk], wk[:dk] = 1 + 0.3 * rnd(dk, seed=1), 1 + 0.3 * rnd(dk, seed=2)
    ang = None
    if rot:
        args = rot_args(rot)
        ang = ops.rope_angles(i32(pos, dev), ops.rope_freqs(*args, device=dev),
                              ops.rope_magnitude(*args))
    kc = torch.full((12, Hkv, 32, D), 9.0, dtype=dt, device=dev)
    vc = torch.full((12, Hkv, 8, D, 4), 9.0, dtype=dt, device=dev)
    quads = mixers.row_quads(qlens[2:], np.add(qlens, starts)[2:], 2)
    assert quads[-1] == T and all(0 < b - a <= 4 for a, b in zip(quads, quads[1:]))
    q = ops.norm_rope_cache(p.to(dev), wq.to(dev), wk.to(dev), ang, i32(slots, dev), kc, vc, Hq, dk,
                            eps, i32(quads, dev))
    xd = p.double()[:, :(Hq + 2 * Hkv) * D].view(T, -1, D)
    y = xd[:, :Hq + Hkv, :dk]
    y = torch.cat([oracle.unit_rms(y[:, :Hq], eps) * wq[:dk].double(),
                   oracle.unit_rms(y[:, Hq:], eps) * wk[:dk].double()], 1)
    if rot:
        y = oracle.rotate_interleaved(y, torch.tensor(pos), rot)
    close(q.view(T, Hq, D)[..., :dk], y[:, :Hq], OUT_TOL[dt], "q")
    on = slots >= 0
    close(kc[slots[on] // 32, :, slots[on] % 32][..., :dk], y[on, Hq:], OUT_TOL[dt], "k")
    close(vc[slots[on] // 32, :, slots[on] % 32 // 4, :, slots[on] % 4], xd[on, Hq + Hkv:], 1e-9, "v")
    assert int((kc[:, 0, :, 0] != 9).sum()) == on.sum() == int((vc[:, 0, :, 0] != 9).sum())
    # every row alone (decode steps)
    kc2, vc2 = torch.full_like(kc, 9.0), torch.full_like(vc, 9.0)
    q2 = ops.norm_rope_cache(p.to(dev), wq.to(dev), wk.to(dev), ang, i32(slots, dev), kc2, vc2, Hq,
                             dk, eps)
    assert torch.equal(q, q2) and torch.equal(kc, kc2) and torch.equal(vc, vc2)


# ----------------------------------------------------------------- attention --
def run_attention(dev, dt, q, kc, vc, bt, qlens, ctx, scale, Hq, window, cap, parts):
    """Decode rows and portions through the kernels a mixer would take."""
    D, T = kc.shape[3], q.shape[0]
    b = Batch(dev, qlens, np.subtract(ctx, qlens), range(len(qlens)))
    pos = i32(np.concatenate([np.arange(c - n, c) for c, n in zip(ctx, qlens)]), dev)
    if dt == torch.float32 or D not in (64, 128) or Hq // kc.shape[1] > 16:
        return ops.attention_any(q, kc, vc, bt, b.cu, b.ctx, pos, scale, Hq, window=window, cap=cap)
    out = torch.full((T, Hq * D), 7.0, dtype=dt, device=dev)
    nd = b.nd
    if nd:
        ws = ops.DecodeWorkspace(nd, Hq, D, parts, dev) if dev != "cpu" else None
        ops.paged_decode_attention(q[:nd], kc, vc, bt[:nd], b.ctx[:nd], scale, out[:nd], ws, 128,
                                   Hq=Hq, precise=True, window=window, cap=cap)
    if T > nd:
        per = 4 * (4 if D == 64 else ops.PREFILL_GROUPS_PER_WAVE) * (16 // (Hq // kc.shape[1]))
        tiles = i32(mixers.row_tiles(qlens[nd:], per).reshape(-1), dev)
        ops.paged_prefill_attention(q, kc, vc, bt[nd:], b.cu[nd:], b.ctx[nd:], tiles, scale, out,
                                    Hq=Hq, q_per_tile=per, precise=True, window=window, cap=cap)
    return out


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("parts", [1, 4])
@pytest.mark.parametrize("Hq,Hkv,D", [(4, 2, 64), (8, 2, 128), (6, 6, 128), (20, 1, 64), (2, 1, 256)])
@pytest.mark.parametrize("window,cap", [(33, 4.0), (64, 0.0), (1, 2.0), (0, 3.0), (200, 5.0), (95, 20.0)])
def test_window_and_cap(dev, dt, parts, Hq, Hkv, D, window, cap):
    """Decode rows (one and several partitions) and portions around the window's
    edges; at each row the oldest visible key or the first hidden one stands
    out."""
    if parts > 1 and dev == "cpu":
        pytest.skip("partitions are the kernel's own")
    scale = D ** -0.5
    qlens, ctx = [1, 1, 1, 70, 2, 33], [300, 31, 97, 230, 64, 33]
    npg = [-(-c // 32) for c in ctx]
    perm = np.random.default_rng(1).permutation(sum(npg) + 3)
    bt = np.zeros((6, max(npg)), np.int32)
    keys = [rnd(c, Hkv, D, seed=10 + i).to(dt) for i, c in enumerate(ctx)]
    vals = [rnd(c, Hkv, D, seed=20 + i).to(dt) for i, c in enumerate(ctx)]
    qs = [rnd(n, Hq, D, seed=30 + i) for i, n in enumerate(qlens)]
    for i, (n, c) in enumerate(zip(qlens, ctx)):
        for t in range(n):
            edge = c - n + t - window + (t % 2)          # hidden / oldest visible in turn
            if window and edge >= 0:
                qs[i][t] = 4.0 * keys[i][edge].float().repeat_interleave(Hq // Hkv, 0) * 8 / D ** 0.5
    qs = [q.to(dt) for q in qs]
    kc = torch.zeros((sum(npg) + 3, Hkv, 32, D), dtype=dt)
    vc = torch.zeros((sum(npg) + 3, Hkv, 8, D, 4), dtype=dt)
    at = 0
    for i, c in enumerate(ctx):
        bt[i, :npg[i]] = perm[at:at + npg[i]]
        at += npg[i]
        j = np.arange(c)
        blk, off = bt[i, j // 32], j % 32
        kc[blk, :, off] = keys[i]
        vc[blk, :, off // 4, :, off % 4] = vals[i]
    got = run_attention(dev, dt, torch.cat(qs).view(-1, Hq * D).to(dev), kc.to(dev), vc.to(dev),
                        i32(bt, dev), qlens, ctx, scale, Hq, window, cap, parts).cpu()
    at = 0
    for i, (n, c) in enumerate(zip(qlens, ctx)):
        q = torch.cat([torch.zeros(c - n, Hq, D).to(dt), qs[i]])
        want = oracle.window_attention(q.double(), keys[i].double(), vals[i].double(), scale,
                                       window or None, cap or None)[c - n:]
        close(got[at:at + n].view(n, Hq, D), want, OUT_TOL[dt], f"sequence {i}")
        at += n


# ----------------------------------------------------------------- retention --
@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("H,N,P,n", [(2, 32, 48, 16), (3, 10, 7, 6), (2, 128, 128, 128), (1, 264, 24, 8),
                                     (2, 64, 72, 0)])
def test_retention(dev, dt, H, N, P, n):
    """Portions of several sizes carried through a reused slot; rotation and key
    scale in both forms of the scan."""
    T, scale = 200, N ** -0.5
    rot = dict(base=200.0, dims=n)
    qkv = [rnd(T, H * c, seed=k).to(dt) for k, c in enumerate((N, N, P))]
    decay = torch.linspace(0.7, 0.999, H, dtype=torch.float64)
    pos = torch.arange(T)
    q, k = (x.double().view(T, H, N) for x in qkv[:2])
    if n:
        q, k = (oracle.rotate_interleaved(x, pos, rot) for x in (q, k))
    want = oracle.retention(q, k * scale, qkv[2].double().view(T, H, P), decay.tolist()).reshape(T, -1)
    dec = (decay.float().to(dev), decay.log().float().to(dev))
    ang = ops.rope_angles(i32(pos, dev), ops.rope_freqs(200.0, n, device=dev)) if n else None
    for cuts in ([200], [2, 1, 64, 65, 1, 67], [130, 1, 1, 68]):
        st = torch.full((3, H, N, P), 9.0, device=dev)
        got, at = [], 0
        for m in cuts:
            b = Batch(dev, [m], [at], [1])
            x = [t[at:at + m].clone().to(dev) for t in qkv]
            segs = b.segments(H, P) if b.nd < 1 else None
            got.append(ops.linear_scan(*x, st, b.cu, b.ctx, b.slots, decay=dec, num_decode=b.nd,
                                       segments=segs, k_scale=scale,
                                       angles=None if ang is None else ang[at:at + m].contiguous()))
            at += m
        close(torch.cat(got), want, 3 * OUT_TOL[dt], f"cuts {cuts}")


@pytest.mark.parametrize("dev,dt", DEV)
def test_retention_of_a_mixed_batch(dev, dt):
    """Decode rows beside portions: each sequence as if alone."""
    H, N, P, n = 2, 64, 64, 64
    qlens, starts, slots = [1, 1, 66, 7], [4, 0, 3, 0], [2, 0, 3, 1]
    T = sum(qlens)
    qkv = [rnd(T, H * c, seed=k).to(dt) for k, c in enumerate((N, N, P))]
    pos = np.concatenate([np.arange(s, s + m) for m, s in zip(qlens, starts)])
    dec = (torch.tensor([0.9, 0.99], device=dev), torch.tensor([0.9, 0.99], device=dev).log())
    f = ops.rope_freqs(100.0, n, device=dev)
    st0 = rnd(4, H, N, P, seed=9).to(dev)

    def run(rows, b, state):
        return ops.linear_scan(*(t[rows].clone().to(dev) for t in qkv), state, b.cu, b.ctx, b.slots,
                               decay=dec, num_decode=b.nd, k_scale=0.125,
                               segments=b.segments(H, P) if b.nd < len(b.q) else None,
                               angles=ops.rope_angles(i32(pos[rows], dev), f))
    b, st = Batch(dev, qlens, starts, slots), st0.clone()
    got = run(slice(0, T), b, st)
    for s in range(4):
        one = st0.clone()
        y = run(b.rows(s), Batch(dev, qlens[s:s + 1], starts[s:s + 1], slots[s:s + 1]), one)
        close(got[b.rows(s)], y.cpu(), OUT_TOL[dt], f"sequence {s}")
        close(st[slots[s]], one[slots[s]].cpu(), OUT_TOL[dt], f"state {s}")


# ---------------------------------------------------------------- delta rule --
class Delta:
    def __init__(self, H, G, N, P, T, dt, seed=0, slow=3.0, alike=0.0):
        self.geo = (H, G, N, P)
        q, k = rnd(T, G * N, seed=seed), rnd(T, G * N, seed=seed + 1)
        if alike:                    # keys that nearly repeat: T of the chunk far from 1
            k = alike * rnd(1, G * N, seed=seed + 7) + k
        self.q, self.k = q.to(dt), k.to(dt)
        self.v = rnd(T, H * P, seed=seed + 2).to(dt)
        self.b, self.a = (rnd(T, H, seed=seed + j).to(dt) for j in (3, 4))
        self.dt_bias, self.A = rnd(H, seed=seed + 5) - slow, 0.5 * rnd(H, seed=seed + 6)

    def want(self, at=0, end=None):
        """Outputs of rows at.. as a sequence of their own."""
        H, G, N, P = self.geo
        s = slice(at, end)
        q, k = (oracle.unit(x.double()[s].view(-1, G, N)).repeat_interleave(H // G, 1)
                for x in (self.q, self.k))
        g = torch.exp(-torch.exp(self.A.double()) *
                      oracle.softplus(self.a.double()[s] + self.dt_bias.double()))
        o = oracle.gated_delta_rule(q * N ** -0.5, k, self.v.double()[s].view(-1, H, P), g,
                                    oracle.sigmoid(self.b.double()[s]))
        return o.reshape(o.shape[0], -1)

    def run(self, rows, b, state, dev, chunked=True):
        H, G, N, P = self.geo

        def put(x):                  # rows of a wider, aligned buffer
            x = x[rows]
            w = -(-x.shape[1] // 8) * 8 + 8
            y = torch.zeros(x.shape[0], w, dtype=x.dtype)
            y[:, :x.shape[1]] = x
            return y.to(dev)[:, :w - 8]
        chunks = None
        if chunked and b.nd < len(b.q):
            c, first = mixers.delta_chunks(b.q[b.nd:], b.nd)
            chunks = ops.DeltaChunks(i32(c, dev), i32(first, dev), len(c))
        return ops.delta_rule(put(self.q), put(self.k), put(self.v), put(self.b), put(self.a),
                              self.dt_bias.to(dev), (-torch.exp(self.A)).to(dev), state, b.cu, b.ctx,
                              b.slots, G, num_decode=b.nd, chunks=chunks)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("H,G,N,P", [(4, 2, 24, 40), (3, 1, 7, 9), (2, 2, 64, 64), (4, 2, 128, 128),
                                     (2, 1, 256, 136), (2, 1, 264, 24), (1, 1, 8, 200), (2, 2, 96, 16)])
def test_delta_rule(dev, dt, H, G, N, P):
    """Portions of several sizes carried through a reused slot, chunked and
    token by token."""
    T = 200
    x = Delta(H, G, N, P, T, dt)
    want = x.want()
    for cuts, chunked in (([200], True), ([2, 1, 64, 65, 1, 67], True), ([130, 1, 1, 68], True),
                          ([128, 63, 9], True), ([150, 50], False)):
        st = torch.full((3, H, N, P), 9.0, device=dev)
        got, at = [], 0
        for m in cuts:
            got.append(x.run(slice(at, at + m), Batch(dev, [m], [at], [1]), st, dev, chunked))
            at += m
        close(torch.cat(got), want, 2 * OUT_TOL[dt], f"cuts {cuts}")
        assert bool((st[0] == 9).all() and (st[2] == 9).all())


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("slow,alike", [(9.0, 0.0), (9.0, 4.0), (-3.0, 0.0), (3.0, 4.0)])
def test_delta_rule_of_long_memories_and_repeating_keys(dev, dt, slow, alike):
    """Hardly any decay, decay within a few tokens, and keys close to each
    other, whose writes correct one another."""
    H, G, N, P, T = 2, 1, 64, 64, 260
    x = Delta(H, G, N, P, T, dt, seed=40, slow=slow, alike=alike)
    st = torch.zeros(1, H, N, P, device=dev)
    got = x.run(slice(0, T), Batch(dev, [T], [0], [0]), st, dev)
    close(got, x.want(), 2 * OUT_TOL[dt])
    # token by token from there on, against the chunked state
    y = Delta(H, G, N, P, T + 6, dt, seed=40, slow=slow, alike=alike)
    st = torch.zeros(1, H, N, P, device=dev)
    y.run(slice(0, T), Batch(dev, [T], [0], [0]), st, dev)
    tail = [y.run(slice(t, t + 1), Batch(dev, [1], [t], [0]), st, dev) for t in range(T, T + 6)]
    close(torch.cat(tail), y.want()[T:], 2 * OUT_TOL[dt], "decoded")


@pytest.mark.parametrize("dev,dt", DEV)
def test_delta_rule_of_a_mixed_batch(dev, dt):
    """Decode rows, fresh and continued portions in one step: each sequence as
    if alone; a padding row is skipped."""
    H, G, N, P = 4, 2, 64, 72
    qlens, starts, slots = [1, 1, 1, 66, 7, 130], [4, 0, 3, 3, 0, 0], [2, 0, -1, 3, 1, 4]
    x = Delta(H, G, N, P, sum(qlens), dt, seed=60)
    st0 = rnd(5, H, N, P, seed=9).to(dev)
    b, st = Batch(dev, qlens, starts, slots), st0.clone()
    got = x.run(slice(0, b.T), b, st, dev)
    for s in (0, 1, 3, 4, 5):
        one = st0.clone()
        y = x.run(b.rows(s), Batch(dev, qlens[s:s + 1], starts[s:s + 1], slots[s:s + 1]), one, dev)
        close(got[b.rows(s)], y.cpu(), OUT_TOL[dt], f"sequence {s}")
        close(st[slots[s]], one[slots[s]].cpu(), OUT_TOL[dt], f"state {s}")
        if starts[s] == 0:
            r = b.rows(s)
            close(got[r], x.want(r.start, r.stop), 2 * OUT_TOL[dt], f"fresh {s}")


# ------------------------------------------------------------------- routing --
@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("E,top,groups,keep,extra,d", [(8, 2, 2, 1, 2, 64), (16, 4, 4, 2, 1, 200),
                                                       (9, 3, 9, 3, 0, 44), (128, 6, 8, 4, 2, 64),
                                                       (200, 8, 8, 3, 1, 72), (5, 5, 1, 1, 1, 21),
                                                       (128, 8, 64, 16, 0, 128)])
def test_group_routing(dev, dt, E, top, groups, keep, extra, d):
    T = 21
    h, w = rnd(T, d).to(dt), rnd(E + (extra > 0), d, seed=1, scale=2 / math.sqrt(d)).to(dt)
    corr = 0.5 * rnd(E, seed=2) - 0.6                      # negative choice scores among them
    r = ops.moe_route(h.to(dev), w.to(dev), top, extra, ops.GroupScores(corr.to(dev), groups, keep))
    ids, wts = oracle.route(h.double(), w[:E].double(), corr.double(),
                            dict(top=top, groups=dict(count=groups, keep=keep)))
    assert torch.equal(r.ids[:, :top].cpu().long(), ids)
    close(r.weights[:, :top], wts, 1e-5)
    if extra:
        assert r.ids[:, top:].cpu().tolist() == [list(range(E, E + extra))] * T
        close(r.weights[:, top:], oracle.sigmoid(h.double() @ w[E].double())[:, None].expand(T, extra),
              1e-5)


@pytest.mark.parametrize("dev,dt", DEV)
def test_routing_ties_take_the_lowest_index(dev, dt):
    h, w = torch.zeros(3, 32, dtype=dt), torch.ones(12, 32, dtype=dt)
    r = ops.moe_route(h.to(dev), w.to(dev), 3, 0, ops.GroupScores(torch.zeros(12, device=dev), 4, 2))
    assert r.ids.cpu().tolist() == [[0, 1, 2]] * 3
    close(r.weights, torch.full((3, 3), 1 / 3), 1e-6)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("T", [3, 40, 300, 2500])
def test_experts_with_silu(dev, dt, T):
    """The routed product with its GLU at every tile size."""
    E, K, F = 4, 256, 256 if T > 1000 else 64
    if dev == "cpu" and T > 300:
        pytest.skip("tile sizes are the kernel's own")
    x, w1 = rnd(T, K).to(dt), rnd(E, 2 * F, K, seed=1, scale=K ** -0.5).to(dt)
    g = torch.Generator().manual_seed(2)
    ids = torch.stack([torch.randperm(E, generator=g)[:2] for _ in range(T)]).to(torch.int32)
    r = ops.Route(ids.to(dev), torch.ones(T, 2, device=dev))
    wp = ops.pack_grouped(torch.stack([ops.interleave_gate_up(w, 16) for w in w1]).to(dev))
    plan = ops.moe_plan(r, E, wp.packed, ops.wide_tiles(wp))
    y = ops.grouped_linear(x.to(dev), wp, plan, gather=True, act=(1.0, 0.0),
                           glu=torch.full((E,), math.inf, device=dev)).cpu()
    pos = plan.pos.cpu().long()
    for j in range(2):
        w = w1.double()[ids[:, j].long()]
        z = torch.einsum("tk,tnk->tn", x.double(), w) if T <= 300 else \
            torch.stack([w1.double()[int(ids[t, j])] @ x.double()[t] for t in range(T)])
        close(y[pos[:, j]], oracle.silu(z[:, :F]) * z[:, F:], 2 * OUT_TOL[dt])
