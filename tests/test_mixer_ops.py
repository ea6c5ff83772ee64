"""The token-mixer ops one by one against the plain equations of
``zegopel_oracle``, on the CPU references and the GPU kernels."""
import math

import numpy as np
import pytest
import torch

import zegopel_oracle as oracle
from llm_mcp_amd import ops
from llm_mcp_amd.ops import mixers

GPU = pytest.mark.gpu
DEV = [pytest.param("cpu", torch.float32, id="cpu-fp32"),
       pytest.param("cpu", torch.bfloat16, id="cpu-bf16"),
       pytest.param("cuda", torch.float32, id="gpu-fp32", marks=GPU),
       pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=GPU)]
OUT_TOL = {torch.float32: 1e-5, torch.bfloat16: 8e-3}     # of the output's largest value


def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(shape, generator=g) * scale


def close(got, want, tol, what=""):
    got, want = got.double().cpu(), want.double()
    e = float((got - want).abs().max() / want.abs().max().clamp_min(1e-6))
    assert e < tol, f"{what}: {e:.2e}"


class Batch:
    """Index tensors of a step: decode sequences (one row) first."""

    def __init__(self, dev, qlens, starts, slots):
        i32 = dict(dtype=torch.int32, device=dev)
        self.q, self.starts, self.dev = list(qlens), list(starts), dev
        self.nd = 0
        while self.nd < len(qlens) and qlens[self.nd] == 1:
            self.nd += 1
        cu = np.concatenate([[0], np.cumsum(qlens)]).astype(np.int32)
        self.cu_np = cu
        self.cu = torch.tensor(cu, **i32)
        self.ctx = torch.tensor([a + b for a, b in zip(qlens, starts)], **i32)
        self.slots = torch.tensor(slots, **i32)
        self.tiles = torch.tensor(mixers.conv_tiles(cu), **i32).contiguous()
        self.T = int(cu[-1])

    def segments(self, H, P):
        segs, first, one = mixers.scan_segments(self.q[self.nd:], self.nd, H, P)
        dev = dict(dtype=torch.int32, device=self.dev)
        return ops.ScanSegments(torch.tensor(segs, **dev), torch.tensor(first, **dev), len(segs),
                                one)

    def rows(self, s):
        return slice(int(self.cu_np[s]), int(self.cu_np[s + 1]))


@pytest.fixture(autouse=True, scope="module")
def _one_thread():
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


# -------------------------------------------------------------------- norms --
@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("d", [64, 100, 4096])
def test_sandwich_norm(dev, dt, d):
    T, eps = 5, 1e-3
    x, y = rnd(T, d), rnd(T, d, seed=1, scale=3.0).to(dt)
    wp, wq = 0.3 * rnd(d, seed=2), 0.3 * rnd(d, seed=3)
    res = x.clone().to(dev)
    h = ops.sandwich_norm(res, eps, y=y.to(dev), w_post=(1 + wp).to(dev), w_pre=(1 + wq).to(dev),
                          dtype=dt)
    r = x.double() + oracle.norm_zero_centred(y.double(), wp.double(), eps)
    close(res, r, 2e-6, "residual stays fp32")
    close(h, oracle.norm_zero_centred(r, wq.double(), eps), OUT_TOL[dt])
    # final norm of picked rows: the residual is left alone
    keep = res.clone()
    rows = torch.tensor([4, 1], device=dev)
    f = ops.sandwich_norm(res, eps, y=y.to(dev), w_post=(1 + wp).to(dev), w_pre=(1 + wq).to(dev),
                          rows=rows, dtype=dt)
    r2 = keep.double().cpu() + oracle.norm_zero_centred(y.double(), wp.double(), eps)
    close(f, oracle.norm_zero_centred(r2, wq.double(), eps)[[4, 1]], OUT_TOL[dt])
    assert torch.equal(res, keep)
    # the embedding as the residual's first value
    table = rnd(7, d, seed=4).to(dt)
    ids = torch.tensor([6, 0, 3, 3, 1], dtype=torch.int32)
    h = ops.sandwich_norm(res, eps, w_pre=(1 + wq).to(dev), ids=ids.to(dev), table=table.to(dev),
                          dtype=dt)
    assert torch.equal(res.cpu(), table[ids.long()].float())
    close(h, oracle.norm_zero_centred(table[ids.long()].double(), wq.double(), eps), OUT_TOL[dt])


@pytest.mark.gpu
def test_sandwich_norm_sums_split_k_slabs():
    d, T, eps = 256, 3, 1e-5
    slabs = rnd(3, T, d).cuda()
    w = torch.ones(d, device="cuda")
    a, b = rnd(T, d, seed=1).cuda(), rnd(T, d, seed=1).cuda()
    ha = ops.sandwich_norm(a, eps, y=ops.Partials(slabs, 3, T, d), w_post=w, w_pre=w)
    hb = ops.sandwich_norm(b, eps, y=slabs.sum(0).to(torch.float32), w_post=w, w_pre=w,
                           dtype=torch.float32)
    close(a, b.double().cpu(), 1e-6)
    close(ha, hb.double().cpu(), 8e-3)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("C,groups", [(96, 1), (96, 3), (42, 2), (4096, 8)])
def test_gated_norm(dev, dt, C, groups):
    T, eps = 4, 1e-4
    x, w = rnd(T, C, seed=1).to(dt), 1 + 0.3 * rnd(C, seed=2)
    x[1, :C // groups] *= 20          # parts of unequal size: a shared norm would show
    g = rnd(T, C + 8, seed=3).to(dt)[:, :C]
    xd, gd, wd = x.double(), g.double(), w.double()
    gg = rnd(T, C + 8, seed=3).to(dt).to(dev)[:, :C]
    got = ops.gated_norm(x.to(dev), gg, w.to(dev), groups, eps, gate_first=False)
    close(got, oracle.grouped_norm(xd, wd, groups, eps) * oracle.sigmoid(gd), OUT_TOL[dt])
    got = ops.gated_norm(x.to(dev), gg, w.to(dev), groups, eps, gate_first=True)
    close(got, oracle.grouped_norm(xd * oracle.silu(gd), wd, groups, eps), OUT_TOL[dt])


@pytest.mark.parametrize("dev,dt", DEV)
def test_relu_glu(dev, dt):
    x = rnd(3, 48).to(dt)
    got = ops.relu_mul(x.to(dev))
    close(got, torch.relu(x[:, :24].double()) * x[:, 24:].double(), OUT_TOL[dt])


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("M,I,K", [(3, 48, 40), (64, 14336, 4096), (600, 256, 384)])
def test_relu_glu_projection(dev, dt, M, I, K):
    """Plain product + GLU kernel, the decode GEMM's pair epilogue (a measured
    shape) and the prefill GEMM's."""
    if dev == "cpu" and I > 1000:
        pytest.skip("GPU GEMM shape")
    x, w = rnd(M, K).to(dt), rnd(2 * I, K, seed=1, scale=K ** -0.5).to(dt)
    got = ops.linear_relu_glu(x.to(dev), ops.interleave_gate_up(w, 16).to(dev))
    y = x.to(dev).float() @ w.to(dev).float().t()
    close(got, (torch.relu(y[:, :I]) * y[:, I:]).cpu(), 2e-2 if dt == torch.bfloat16 else 1e-4)


# -------------------------------------------------------------- convolution --
@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("C,taps", [(64, 4), (16, 3), (40, 2), (24, 1), (24, 7), (13, 3)])
def test_short_conv_over_portions_and_slots(dev, dt, C, taps):
    """Sequences whose rows arrive in portions (shorter and longer than the
    window), in slots that held something else before."""
    n = [150, 6, 5]
    u = [rnd(k, C, seed=i).to(dt) for i, k in enumerate(n)]
    w, b = rnd(taps, C, seed=8), rnd(C, seed=9)
    want = [oracle.silu(oracle.causal_conv(x.double(), w.double().t(), b.double())) for x in u]
    state = torch.full((4, max(1, taps - 1), C), 7.0).to(dt).to(dev)
    state = state if taps > 1 else None
    # steps of (sequence, rows): decode rows first
    at = [0, 0, 0]
    for step in ([(1, 1), (0, 80)], [(1, 1), (2, 1), (0, 2)], [(1, 2), (2, 3), (0, 67)],
                 [(2, 1), (1, 2)], [(0, 1)]):
        bt = Batch(dev, [k for _, k in step], [at[s] for s, _ in step], [2 - s for s, _ in step])
        rows = torch.cat([u[s][at[s]:at[s] + k] for s, k in step]).to(dev)
        # rows of a wider projection: the stride is not the width
        wide = torch.zeros(bt.T, C + 24, dtype=dt, device=dev)
        wide[:, 8:8 + C] = rows
        y = ops.short_conv(wide[:, 8:8 + C], w.to(dev), state, bt.cu, bt.ctx, bt.slots,
                           bias=b.to(dev), silu=True,
                           tiles=bt.tiles if bt.nd < len(step) else None)
        for i, (s, k) in enumerate(step):
            close(y[bt.rows(i)], want[s][at[s]:at[s] + k], OUT_TOL[dt], f"{s} at {at[s]}")
            at[s] += k
    assert at == [150, 6, 5]


# --------------------------------------------------------------------- scan --
def _scan_inputs(T, H, N, P, hpg, dt, seed):
    G = H // hpg
    q, k = rnd(T, G * N, seed=seed, scale=0.5), rnd(T, G * N, seed=seed + 1, scale=0.5)
    v, d = rnd(T, H * P, seed=seed + 2), rnd(T, H, seed=seed + 3)
    return [x.to(dt) for x in (q, k, v, d)]


def _scan_want(x, form, H, N, P, hpg, par):
    q, k, v, d = (t.double() for t in x)
    T, G = q.shape[0], H // hpg
    grp = torch.arange(H) // hpg
    v = v.view(T, H, P)
    if form == "decay":
        q, k, v = oracle.silu(q), oracle.silu(k), oracle.silu(v)
        s, dec = torch.ones(T, H).double(), par["decay"].double().expand(T, H)
    else:
        s = oracle.softplus(d + par["bias"].double())
        dec = torch.exp(par["neg_a"].double() * s)
    q, k = q.view(T, G, N)[:, grp], k.view(T, G, N)[:, grp]
    o = oracle.linear_attention(q, k * s[:, :, None], v, dec)
    return (o + par["skip"].double()[:, None] * v if form == "dt" else o).reshape(T, H * P)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("form", ["decay", "dt"])
@pytest.mark.parametrize("H,N,P,hpg", [(4, 64, 64, 1), (6, 40, 24, 3), (2, 128, 136, 2),
                                       (3, 9, 7, 3), (2, 200, 16, 1), (1, 96, 80, 1)])
def test_linear_scan(dev, dt, form, H, N, P, hpg):
    """Both forms over portions around the 64-token chunk, decode rows beside
    them, slots that held another sequence's state."""
    n = [200, 70, 3]
    par = {"decay": torch.linspace(0.3, 0.999, H), "bias": rnd(H, seed=70) - 1,
           "neg_a": -torch.exp(0.5 * rnd(H, seed=71)), "skip": rnd(H, seed=72)}
    if form == "dt":
        par["neg_a"][0] = -0.01      # one head that hardly forgets
    x = [_scan_inputs(k, H, N, P, hpg, dt, 10 * i) for i, k in enumerate(n)]
    want = [_scan_want(xi, form, H, N, P, hpg, par) for xi in x]
    state = torch.full((4, H, N, P), 5.0, device=dev)
    dpar = {k: t.to(dev) for k, t in par.items()}
    at = [0, 0, 0]
    tol = OUT_TOL[dt] * (1 if form == "dt" else 1.5)      # SiLU is rounded to bf16 rows
    for step in ([(1, 1), (0, 64)], [(2, 1), (1, 65), (0, 63)], [(0, 1)], [(0, 2), (1, 4)],
                 [(2, 1), (0, 70)], [(2, 1)]):
        b = Batch(dev, [k for _, k in step], [at[s] for s, _ in step], [3 - s for s, _ in step])
        q, k, v, d = (torch.cat([x[s][j][at[s]:at[s] + c] for s, c in step]).to(dev)
                      for j in range(4))
        kw = dict(decay=(dpar["decay"], dpar["decay"].log()), silu=True) if form == "decay" else \
            dict(dt=(d, dpar["bias"], dpar["neg_a"]), skip=dpar["skip"])
        y = ops.linear_scan(q, k, v, state, b.cu, b.ctx, b.slots, heads_per_group=hpg,
                            num_decode=b.nd, segments=b.segments(H, P) if b.nd < len(step)
                            else None, **kw)
        for i, (s, c) in enumerate(step):
            close(y[b.rows(i)], want[s][at[s]:at[s] + c], tol, f"{s} at {at[s]}")
            at[s] += c


@pytest.mark.gpu
@pytest.mark.parametrize("form", ["decay", "dt"])
def test_scan_segments_chain_and_keep_fp32_state(form):
    """One long sequence is cut into segments; the chunked result (bf16 rows,
    fp32 state) matches the recurrent kernel's state far below bf16 rounding."""
    H, N, P, T = 2, 128, 64, 2000
    par = {"decay": torch.tensor([0.9, 0.9999]), "bias": torch.tensor([-4.0, -1.0]),
           "neg_a": torch.tensor([-0.05, -1.5]), "skip": torch.tensor([0.5, 2.0])}
    x = _scan_inputs(T, H, N, P, 1, torch.bfloat16, 5)
    d = {k: t.cuda() for k, t in par.items()}
    kw = dict(decay=(d["decay"], d["decay"].log())) if form == "decay" else \
        dict(dt=(x[3].cuda(), d["bias"], d["neg_a"]), skip=d["skip"])
    outs = []
    for chunked in (True, False):
        state = torch.zeros(2, H, N, P, device="cuda")
        b = Batch("cuda", [T], [0], [1])
        seg = b.segments(H, P)
        assert seg.n > 4 and not seg.one_pass
        y = ops.linear_scan(*[t.cuda() for t in x[:3]], state, b.cu, b.ctx, b.slots,
                            segments=seg if chunked else None, **kw)
        # a second portion continues from the chained state
        b2 = Batch("cuda", [T], [T], [1])
        y2 = ops.linear_scan(*[t.cuda() for t in x[:3]], state, b2.cu, b2.ctx, b2.slots,
                             segments=b2.segments(H, P) if chunked else None, **kw)
        outs.append((y, y2, state[1].cpu()))
    close(outs[0][2], outs[1][2].double(), 1e-4, "state")
    for i in (0, 1):
        close(outs[0][i], outs[1][i].double().cpu(), 8e-3)


def test_scan_segment_plan_covers_every_row_once():
    rng = np.random.default_rng(0)
    for _ in range(50):
        ql = rng.integers(2, 3000, rng.integers(1, 6)).tolist()
        H, P = int(rng.integers(1, 40)), int(rng.choice([16, 64, 128]))
        segs, first, one = mixers.scan_segments(ql, 3, H, P)
        for i, n in enumerate(ql):
            mine = segs[first[i]:first[i + 1]]
            assert (mine[:, 0] == 3 + i).all() and mine[0, 1] == 0 and mine[-1, 2] == n
            assert (mine[1:, 1] == mine[:-1, 2]).all() and (mine[:, 1] % 64 == 0).all()
            assert mine[:, 3].tolist() == [0] * (len(mine) - 1) + [1]
        assert one == (len(segs) == len(ql))
    t = mixers.row_tiles([1, 64, 65, 130], 64)
    assert t.tolist() == [[0, 0], [1, 0], [2, 0], [2, 64], [3, 0], [3, 64], [3, 128]]


# ---------------------------------------------------------------- attention --
ATT = [dict(Hq=4, Hkv=2, D=64, dk=64, dv=64), dict(Hq=6, Hkv=1, D=128, dk=96, dv=112),
       dict(Hq=2, Hkv=2, D=256, dk=150, dv=200), dict(Hq=18, Hkv=1, D=64, dk=32, dv=16)]


class AttnRig:
    """Padded q | k | v rows of sequences through conv_qkv_cache and attention."""

    def __init__(self, dev, dt, g, taps, seed=0, every=8.0, coef=0.7, scale=0.25, pages=24):
        self.dev, self.dt, self.g, self.taps = dev, dt, g, taps
        self.temp, self.scale, self.eps = (coef, every), scale, 1e-4
        Hq, Hkv, D = g["Hq"], g["Hkv"], g["D"]
        self.heads = [(g["dk"], Hq), (g["dk"], Hkv), (g["dv"], Hkv)]
        self.C = (Hq + 2 * Hkv) * D
        self.w = self.pad(rnd(taps, self.true, seed=seed + 1, scale=0.5) + 0.3)
        self.b = self.pad(rnd(1, self.true, seed=seed + 2, scale=0.5))[0]
        z = dict(dtype=dt, device=dev)
        self.kc = torch.zeros((pages, Hkv, 32, D), **z)
        self.vc = torch.zeros((pages, Hkv, 8, D, 4), **z)
        self.state = torch.full((3, max(1, taps - 1), self.C), 3.0).to(**z)
        self.state = self.state if taps > 1 else None
        self.ws = ops.DecodeWorkspace(4, Hq, D, 4, dev) if dev == "cuda" else None

    true = property(lambda self: sum(d * h for d, h in self.heads))

    def pad(self, x):
        """[n, true channels] -> [n, padded channels]"""
        out, at, D = [], 0, self.g["D"]
        for d, h in self.heads:
            blk = x[:, at:at + d * h].reshape(-1, h, d)
            out.append(torch.nn.functional.pad(blk, (0, D - d)).reshape(-1, h * D))
            at += d * h
        return torch.cat(out, 1)

    def unpad(self, x, d, h):
        return x.reshape(x.shape[0], h, self.g["D"])[..., :d]

    def want(self, u, gate):
        """Oracle over a whole sequence's padded projection rows (no bias in u)."""
        g, T = self.g, u.shape[0]
        y = oracle.causal_conv(u.double() + self.b.double(), self.w.double().t())
        Hq, Hkv, D = g["Hq"], g["Hkv"], g["D"]
        q = oracle.unit_rms(self.unpad(y[:, :Hq * D], g["dk"], Hq), self.eps)
        k = oracle.unit_rms(self.unpad(y[:, Hq * D:(Hq + Hkv) * D], g["dk"], Hkv), self.eps)
        v = self.unpad(y[:, (Hq + Hkv) * D:], g["dv"], Hkv)
        t = oracle.query_temperature(torch.arange(T).double(), *self.temp)
        o = oracle.softmax_attention(q * t[:, None, None], k, v, self.scale)
        return o * oracle.sigmoid(self.unpad(gate.double(), g["dv"], Hq))

    def step(self, batch, u, gate, tables):
        """u, gate: rows of the step; tables: page ids per sequence of the step."""
        g, dev = self.g, self.dev
        Hq, Hkv, D = g["Hq"], g["Hkv"], g["D"]
        pos, slots = [], []
        for n, s0, tab in zip(batch.q, batch.starts, tables):
            pos += range(s0, s0 + n)
            slots += [tab[p // 32] * 32 + p % 32 for p in range(s0, s0 + n)]
        i32 = dict(dtype=torch.int32, device=dev)
        pos, slots = torch.tensor(pos, **i32), torch.tensor(slots, **i32)
        width = max(len(t) for t in tables)
        bt = torch.tensor([t + [0] * (width - len(t)) for t in tables], **i32)
        rows = torch.cat([u, gate], 1).to(self.dt).to(dev)
        gate = rows[:, self.C:]
        nd, S = batch.nd, len(batch.q)
        q = ops.conv_qkv_cache(rows[:, :self.C], self.w.contiguous().to(dev), self.b.to(dev),
                               self.state, batch.cu, batch.ctx, batch.slots, pos, slots, self.kc,
                               self.vc, Hq, g["dk"], self.eps, self.temp,
                               tiles=batch.tiles if nd < S else None)
        if D > 128 or Hq // Hkv > 16 or self.dt != torch.bfloat16:
            a = ops.attention_any(q, self.kc, self.vc, bt, batch.cu, batch.ctx, pos, self.scale,
                                  Hq, gate=gate)
        else:
            a = torch.empty((batch.T, Hq * D), dtype=self.dt, device=dev)
            if nd:
                ops.paged_decode_attention(q[:nd], self.kc, self.vc, bt, batch.ctx, self.scale,
                                           a[:nd], self.ws, 128, Hq=Hq, gate=gate[:nd],
                                           precise=True)
            if nd < S:
                qt = 4 * (4 if D == 64 else 2) * (16 // (Hq // Hkv))
                tiles = mixers.row_tiles(batch.q[nd:], qt).reshape(-1)
                ops.paged_prefill_attention(q, self.kc, self.vc, bt[nd:], batch.cu[nd:],
                                            batch.ctx[nd:], torch.tensor(tiles, **i32),
                                            self.scale, a, Hq=Hq, q_per_tile=qt, gate=gate,
                                            precise=True)
        return self.unpad(a.float().cpu(), g["dv"], Hq)


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("g", ATT, ids=lambda g: f"D{g['D']}G{g['Hq'] // g['Hkv']}")
@pytest.mark.parametrize("taps", [4, 1])
def test_convolved_attention(dev, dt, g, taps):
    """Portions and decode rows of two sequences with scattered pages."""
    r = AttnRig(dev, dt, g, taps)
    n = [100, 40]
    u = [r.pad(rnd(k, r.true, seed=20 + i)).to(dt).float() for i, k in enumerate(n)]
    gate = [torch.nn.functional.pad(rnd(k, g["Hq"], g["dv"], seed=30 + i),
                                    (0, g["D"] - g["dv"])).reshape(k, -1).to(dt).float()
            for i, k in enumerate(n)]
    want = [r.want(a, b) for a, b in zip(u, gate)]
    tabs = [[9, 2, 17, 4], [11, 5]]
    at = [0, 0]
    tol = 1e-5 if dt == torch.float32 else 2e-2
    for step in ([(1, 1), (0, 33)], [(1, 2), (0, 30)], [(0, 1), (1, 36)], [(1, 1), (0, 2)],
                 [(0, 34)]):
        b = Batch(dev, [k for _, k in step], [at[s] for s, _ in step], [s for s, _ in step])
        y = r.step(b, torch.cat([u[s][at[s]:at[s] + k] for s, k in step]),
                   torch.cat([gate[s][at[s]:at[s] + k] for s, k in step]),
                   [tabs[s] for s, _ in step])
        for i, (s, k) in enumerate(step):
            close(y[b.rows(i)], want[s][at[s]:at[s] + k], tol, f"{s} at {at[s]}")
            at[s] += k
    assert at == n


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("g", ATT[:2] + ATT[3:], ids=lambda g: f"D{g['D']}G{g['Hq'] // g['Hkv']}")
def test_one_far_key_stands_out(dev, dt, g):
    """A query that matches one key far back (first token, both sides of a page
    border, itself) must read that key's value, in a prompt and in decoding."""
    n, targets = 330, [0, 1, 31, 32, 63, 64, 159, 160, 256, 329]
    r = AttnRig(dev, dt, g, 1, coef=0.0, scale=1.0)
    r.b = torch.zeros_like(r.b)
    r.w = r.pad(torch.ones(1, r.true))
    base = rnd(n, r.true, seed=40)
    qn = g["Hq"] * g["dk"]
    k = base[:, qn:qn + g["Hkv"] * g["dk"]].view(n, g["Hkv"], g["dk"])
    tab = [list(range(3, 3 + 11))]
    gate = torch.full((n, g["Hq"] * g["D"]), 20.0)       # sigmoid 1
    for decode in (False, True):
        for t in targets:
            x = base.clone()
            x[n - 1, :qn] = k[t].repeat_interleave(g["Hq"] // g["Hkv"], 0).reshape(-1)
            u = r.pad(x)
            if decode:
                r.step(Batch(dev, [n - 1], [0], [0]), u[:-1], gate[:-1], tab)
                y = r.step(Batch(dev, [1], [n - 1], [0]), u[-1:], gate[-1:], tab)[0]
            else:
                y = r.step(Batch(dev, [n], [0], [0]), u, gate, tab)[-1]
            v = x[t, qn + g["Hkv"] * g["dk"]:].view(g["Hkv"], g["dv"])
            v = v.repeat_interleave(g["Hq"] // g["Hkv"], 0)
            # exp(score gap) leaves the others far below: an off-by-one key would show
            assert float((y - v).abs().max()) < 0.05, (t, decode)


def test_temperature_steps_at_its_interval():
    p = torch.arange(0, 40).double()
    t = oracle.query_temperature(p, 0.5, 8)
    assert t[6] == 1.0 and t[7] == pytest.approx(1 + 0.5 * math.log(2)) and t[15] == pytest.approx(
        1 + 0.5 * math.log(3))


@pytest.mark.parametrize("dev,dt", DEV)
@pytest.mark.parametrize("every", [1.0, 8.0, 255.0])
def test_query_temperature_of_the_kernel(dev, dt, every):
    """q rows leave the convolution kernel scaled by the temperature: positions
    around its steps, far out as well."""
    g = dict(Hq=2, Hkv=1, D=64, dk=64, dv=64)
    pos = [0, 6, 7, 8, 254, 255, 256, 510, 511, 99999, 1048574]
    T, C = len(pos), 256
    u = rnd(T, C).to(dt).to(dev)
    i32 = dict(dtype=torch.int32, device=dev)
    z = torch.zeros(T, **i32)
    kc, vc = torch.zeros(T, 1, 32, 64, dtype=dt, device=dev), \
        torch.zeros(T, 1, 8, 64, 4, dtype=dt, device=dev)
    q = ops.conv_qkv_cache(u, torch.ones(1, C, device=dev), None, None,
                           torch.arange(T + 1, **i32), z + 1, torch.arange(T, **i32),
                           torch.tensor(pos, **i32), torch.arange(T, **i32) * 32, kc, vc, 2, 64,
                           1e-5, (0.6, every))
    want = oracle.unit_rms(u.double().cpu()[:, :128].view(T, 2, 64), 1e-5) * \
        oracle.query_temperature(torch.tensor(pos).double(), 0.6, every)[:, None, None]
    got = q.double().cpu().view(T, 2, 64)
    assert float(((got - want).abs() / want.abs().clamp_min(1e-2)).max()) < \
        (2e-6 if dt == torch.float32 else 5e-3)
