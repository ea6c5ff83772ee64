"""Plain PyTorch (fp32-accumulating) reference implementations of every HIP
kernel in ``csrc/kernels``.

They serve two purposes:
* numerics oracle for the kernel parity tests (``tests/test_kernels_gpu.py``);
* the CPU execution path of the ops (tests, CPU-only plumbing configs).  A
  CUDA/HIP tensor never takes this path: ``ops.kernels`` dispatches device
  tensors to the native kernels and raises if the extension is missing.

Cache layouts match the kernels: k_cache [NB, Hkv, BS, D], v_cache [NB, Hkv, BS/4, D, 4]
(key-quad: v_cache[blk, h, key // 4, d, key % 4]).
"""
from __future__ import annotations

import math

import torch


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float,
             residual: torch.Tensor | None = None) -> torch.Tensor:
    if residual is not None:
        h = (x.float() + residual.float()).to(x.dtype)
        residual.copy_(h)
        x = h
    xf = x.float()
    y = xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return (y * w.float()).to(x.dtype)


def layer_norm(x, w, b, eps, residual=None):
    if residual is not None:
        x = (x.float() + residual.float()).to(x.dtype)
    return torch.nn.functional.layer_norm(x.float(), (x.shape[-1],), w.float(), b.float(),
                                          eps).to(x.dtype)


def rope_cos_sin(max_pos: int, dim: int, theta: float, device=None,
                 scaling: dict | None = None) -> torch.Tensor:
    """[max_pos, dim] fp32 table: cos in [:, :dim/2], sin in [:, dim/2:]."""
    inv = 1.0 / (theta ** (torch.arange(0, dim, 2, dtype=torch.float64) / dim))
    if scaling and scaling.get("rope_type") == "llama3":
        # Llama-3.1 frequency-dependent scaling
        factor = scaling.get("factor", 8.0)
        lo = scaling.get("low_freq_factor", 1.0)
        hi = scaling.get("high_freq_factor", 4.0)
        old = scaling.get("original_max_position_embeddings", 8192)
        wavelen = 2 * math.pi / inv
        lo_wl, hi_wl = old / lo, old / hi
        smooth = (old / wavelen - lo) / (hi - lo)
        scaled = torch.where(wavelen > lo_wl, inv / factor, inv)
        mid = (wavelen <= lo_wl) & (wavelen >= hi_wl)
        inv = torch.where(mid, (1 - smooth) * inv / factor + smooth * inv, scaled)
    t = torch.arange(max_pos, dtype=torch.float64)
    f = torch.outer(t, inv)
    return torch.cat([f.cos(), f.sin()], dim=-1).float().to(device)


def apply_rope(x: torch.Tensor, positions: torch.Tensor, cos_sin: torch.Tensor) -> torch.Tensor:
    """x [T, H, D] -> rotated (rotate-half form)."""
    D = x.shape[-1]
    cs = cos_sin[positions.long()]
    cos, sin = cs[:, None, : D // 2], cs[:, None, D // 2:]
    x1, x2 = x[..., : D // 2].float(), x[..., D // 2:].float()
    return torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1).to(x.dtype)


def head_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """Per-head RMSNorm over the last dim, kept in fp32 (Qwen3 q_norm/k_norm)."""
    xf = x.float()
    return xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps) * w.float()


def rope_cache(qkv, positions, cos_sin, Hq, Hkv, D, slots, k_cache, v_cache, rotate_k_inplace,
               q_norm=None, k_norm=None, eps=1e-6):
    T = qkv.shape[0]
    v3 = qkv.view(T, -1, D)
    qh, kh = v3[:, :Hq], v3[:, Hq:Hq + Hkv]
    if q_norm is not None:
        qh, kh = head_norm(qh, q_norm, eps), head_norm(kh, k_norm, eps)
    q = apply_rope(qh, positions, cos_sin).to(qkv.dtype)
    k = apply_rope(kh, positions, cos_sin).to(qkv.dtype)
    v = v3[:, Hq + Hkv:Hq + 2 * Hkv]
    v3[:, :Hq] = q
    if rotate_k_inplace or k_cache is None:
        v3[:, Hq:Hq + Hkv] = k
    if k_cache is not None and slots is not None:
        write_cache(k, v, slots, k_cache, v_cache)


def write_cache(k, v, slots, k_cache, v_cache):
    BS = k_cache.shape[2]
    s = slots.long()
    keep = s >= 0
    s, k, v = s[keep], k[keep], v[keep]
    blk, off = s // BS, s % BS
    k_cache[blk, :, off, :] = k.to(k_cache.dtype)
    v_cache[blk, :, off // 4, :, off % 4] = v.to(v_cache.dtype)


def gather_kv(k_cache, v_cache, block_table, n):
    """Dense K, V [n, Hkv, D] of one sequence from the paged cache."""
    BS = k_cache.shape[2]
    idx = torch.arange(n, device=k_cache.device)
    blk = block_table.long()[idx // BS]
    off = idx % BS
    k = k_cache[blk, :, off, :]           # [n, Hkv, D]
    v = v_cache[blk, :, off // 4, :, off % 4]   # [n, Hkv, D]
    return k, v


def attention_dense(q, k, v, scale, causal_offset: int | None, window: int = 0, cap: float = 0.0):
    """q [Tq, Hq, D], k/v [Tk, Hkv, D]; query i sees keys <= causal_offset + i
    (the last ``window`` of them), scores softly capped."""
    Hq, Hkv = q.shape[1], k.shape[1]
    G = Hq // Hkv
    kf = k.float().repeat_interleave(G, dim=1)
    vf = v.float().repeat_interleave(G, dim=1)
    s = torch.einsum("qhd,khd->hqk", q.float(), kf) * scale
    if cap:
        s = cap * torch.tanh(s / cap)
    if causal_offset is not None:
        Tq, Tk = q.shape[0], k.shape[0]
        qi = torch.arange(Tq, device=q.device)[:, None] + causal_offset
        ki = torch.arange(Tk, device=q.device)[None, :]
        hidden = (ki > qi) | (ki <= qi - window) if window else ki > qi
        s = s.masked_fill(hidden[None], float("-inf"))
    p = torch.softmax(s, dim=-1)
    return torch.einsum("hqk,khd->qhd", p, vf)


def paged_decode(q, k_cache, v_cache, block_tables, context_lens, scale, window=0, cap=0.0):
    """q [B, Hq, D] -> [B, Hq, D] (one query per sequence at position ctx-1)."""
    out = torch.empty_like(q)
    for b in range(q.shape[0]):
        n = int(context_lens[b])
        k, v = gather_kv(k_cache, v_cache, block_tables[b], n)
        out[b] = attention_dense(q[b:b + 1], k, v, scale, n - 1, window, cap)[0].to(q.dtype)
    return out


def paged_prefill(q, k_cache, v_cache, block_tables, cu_q, context_lens, scale, causal=True,
                  window=0, cap=0.0):
    """q [T, Hq, D] for a varlen batch; keys come from the paged cache."""
    out = torch.empty_like(q)
    for s in range(len(context_lens)):
        a, b = int(cu_q[s]), int(cu_q[s + 1])
        n = int(context_lens[s])
        k, v = gather_kv(k_cache, v_cache, block_tables[s], n)
        off = (n - (b - a)) if causal else None
        out[a:b] = attention_dense(q[a:b], k, v, scale, off, window, cap).to(q.dtype)
    return out


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    I = x.shape[-1] // 2
    g, u = x[..., :I].float(), x[..., I:].float()
    return (torch.nn.functional.silu(g) * u).to(x.dtype)


def gelu_mul(x: torch.Tensor) -> torch.Tensor:
    I = x.shape[-1] // 2
    g, u = x[..., :I].float(), x[..., I:].float()
    return (torch.nn.functional.gelu(g, approximate="tanh") * u).to(x.dtype)


def mean_pool_l2(h, cu, dims, normalize=True):
    outs = []
    for s in range(len(cu) - 1):
        a, b = int(cu[s]), int(cu[s + 1])
        m = h[a:b].float().mean(0)[:dims] if b > a else \
            torch.zeros(dims, dtype=torch.float32, device=h.device)
        if normalize:
            m = m / m.norm().clamp_min(1e-12)
        outs.append(m)
    return torch.stack(outs)


def gemm_nt(a, w, bias=None, act=0, residual=None):
    y = a.float() @ w.float().t()
    if bias is not None:
        y = y + bias.float()
    if act == 1:
        y = torch.nn.functional.gelu(y, approximate="tanh")
    elif act == 2:
        y = torch.nn.functional.silu(y)
    elif act == 4:
        y = torch.nn.functional.gelu(y)
    elif act == 7:
        y = torch.relu(y) ** 2
    if residual is not None:
        y = y + residual.float()
    return y.to(a.dtype)


def _uniform(seed: int, off: int, idx: torch.Tensor) -> torch.Tensor:
    # host-side mirror of the kernel's counter-based hash is not needed for the
    # CPU path; a seeded torch generator gives the same *distribution*.
    g = torch.Generator().manual_seed((seed * 1000003 + off) & 0x7FFFFFFFFFFFFFFF)
    return torch.rand(idx.shape, generator=g)


def sample(logits, temperature, top_k, top_p, seeds, offsets):
    """Greedy when temperature <= 0, else softmax(logits / T) truncated by
    top-k / top-p.  Returns (tokens int32 [B], logprobs fp32 [B])."""
    B, V = logits.shape
    toks = torch.empty(B, dtype=torch.int32)
    lps = torch.empty(B, dtype=torch.float32)
    for b in range(B):
        x = logits[b].float().cpu()
        t = float(temperature[b])
        k = int(top_k[b]) if top_k is not None else 0
        if t <= 0 or k == 1:
            j = int(torch.argmax(x))
            toks[b] = j
            lps[b] = float(torch.log_softmax(x, -1)[j])
            continue
        z = x / t
        logp = torch.log_softmax(z, -1)
        p = logp.exp()
        keep = torch.ones(V, dtype=torch.bool)
        if k > 0 and k < V:
            kth = torch.topk(z, k).values[-1]
            keep &= z >= kth
        tp = float(top_p[b]) if top_p is not None else 1.0
        if tp < 1.0:
            sp, si = torch.sort(p, descending=True)
            above = torch.cumsum(sp, 0) - sp
            nucleus = torch.zeros(V, dtype=torch.bool)
            nucleus[si[above < tp]] = True
            keep &= nucleus
        pk = torch.where(keep, p, torch.zeros_like(p))
        u = _uniform(int(seeds[b]) if seeds is not None else 0,
                     int(offsets[b]) if offsets is not None else 0, torch.zeros(1))
        c = torch.cumsum(pk / pk.sum(), 0)
        j = int(torch.searchsorted(c, u.clamp(max=float(c[-1]) - 1e-7)))
        toks[b] = j
        lps[b] = float(logp[j])
    return toks, lps


_M32 = 0xFFFFFFFF


def _lowbias32(x: torch.Tensor) -> torch.Tensor:
    x = x ^ (x >> 16)
    x = (x * 0x7FEB352D) & _M32
    x = x ^ (x >> 15)
    x = (x * 0x846CA68B) & _M32
    return x ^ (x >> 16)


def _mix64(z: int) -> int:
    m = (1 << 64) - 1
    z = ((z ^ (z >> 30)) * 0xBF58476D1CE4E5B9) & m
    z = ((z ^ (z >> 27)) * 0x94D049BB133111EB) & m
    return z ^ (z >> 31)


def _row_key(seed: int, off: int, rnd: int) -> tuple[int, int]:
    m = (1 << 64) - 1
    h = _mix64((seed & m) ^ _mix64((off * 0x9E3779B97F4A7C15 + rnd) & m))
    return h & _M32, h >> 32


def race_gumbel(seed: int, off: int, rnd: int, idx: torch.Tensor) -> torch.Tensor:
    """The race kernel's per-element noise G_i = -log(-log U_i), U_i a hash of
    (seed, offset, round, global index i)."""
    k0, k1 = _row_key(seed, off, rnd)
    h = _lowbias32((_lowbias32(idx.to(torch.int64) ^ k0) + k1) & _M32)
    u = ((h >> 8).to(torch.float32) + 0.5) * (1.0 / 16777216.0)
    return -torch.log(-torch.log(u))


def sample_race(logits, temperature, top_k, top_p, seeds, offsets, exchange, v0, V,
                max_rounds):
    """CPU mirror of ops.sample_race (race_kernel's phases, same records and
    exchanges -- one per round, the next round raced speculatively with each
    mass pass): exact race winners, so every rank -- and a one-shard run
    over the whole row -- picks the same tokens."""
    B, Vs = logits.shape
    x = logits.float()
    idx = torch.arange(v0, v0 + Vs, dtype=torch.int64)
    temp = [float(t) for t in temperature[:B]]
    kk = [int(k) for k in top_k[:B]] if top_k is not None else [0] * B
    tp = [float(p) for p in top_p[:B]] if top_p is not None else [1.0] * B
    sd = [int(s) for s in seeds[:B]] if seeds is not None else [0x1234] * B
    of = [int(o) for o in offsets[:B]] if offsets is not None else [0] * B
    greedy = [not (t > 0) or k == 1 for t, k in zip(temp, kk)]
    inv_t = [1.0 if g else 1.0 / t for g, t in zip(greedy, temp)]
    trunc = [not g and (p < 1.0 or 0 < k < V) for g, p, k in zip(greedy, tp, kk)]
    NONE = (-math.inf, 0x7FFFFFFF, -math.inf)

    def race(b, rnd, pivot):
        keep = x[b] > pivot
        if not bool(keep.any()):
            return NONE
        key = x[b] * inv_t[b] + race_gumbel(sd[b], of[b], rnd, idx)
        key = torch.where(keep, key, torch.full_like(key, -math.inf))
        j = int(torch.argmax(key))          # first maximum: the lowest index
        return float(key[j]), v0 + j, float(x[b, j])

    rec = torch.zeros(B, 8)
    for b in range(B):                       # phase 0
        m = float(x[b].max())
        s_ = float(torch.exp((x[b] - m) * inv_t[b]).sum())
        j = int(torch.argmax(x[b]))
        c = race(b, 0, -math.inf) if not greedy[b] else NONE
        # indices travel as floats here (exact below 2^24)
        rec[b] = torch.tensor([m, s_, float(x[b, j]), float(v0 + j), c[0], float(c[1]), c[2], 0])
    g = exchange(rec)
    W = g.shape[0]
    xmax, S = [0.0] * B, [0.0] * B
    am = [(0.0, 0)] * B
    done = [False] * B
    tok, lp = [0] * B, [0.0] * B
    cand = [(0, 0.0)] * B

    def finish(b, t, x_):
        done[b], tok[b], lp[b] = True, t, (x_ - xmax[b]) * inv_t[b] - math.log(S[b])

    for rnd in range(max_rounds + 1):        # phase 1 rounds, then phase 2
        last = rnd == max_rounds
        rec = torch.zeros(B, 8)
        rec[:, 4] = -math.inf
        for b in range(B):
            if rnd == 0:
                xmax[b] = max(float(g[q, b, 0]) for q in range(W))
                S[b] = sum(float(g[q, b, 1]) * math.exp((float(g[q, b, 0]) - xmax[b]) * inv_t[b])
                           for q in range(W) if float(g[q, b, 0]) != -math.inf)
                best = (-math.inf, 0x7FFFFFFF)
                for q in range(W):
                    v, j = float(g[q, b, 2]), int(g[q, b, 3])
                    if v > best[0] or (v == best[0] and j < best[1]):
                        best = (v, j)
                am[b] = best
                if greedy[b]:
                    done[b], tok[b] = True, best[1]
                    lp[b] = best[0] - xmax[b] - math.log(S[b])
            elif not done[b]:
                mass = sum(float(g[q, b, 0]) for q in range(W)) / S[b]
                cnt = sum(float(g[q, b, 1]) for q in range(W))
                if mass < tp[b] and (kk[b] <= 0 or cnt < kk[b]):
                    finish(b, cand[b][0], cand[b][1])
                elif last:
                    finish(b, am[b][1], am[b][0])
            if last or done[b]:
                continue
            best = NONE
            for q in range(W):
                k_, j_, x_ = float(g[q, b, 4]), int(g[q, b, 5]), float(g[q, b, 6])
                if k_ > best[0] or (k_ == best[0] and j_ < best[1]):
                    best = (k_, j_, x_)
            if best[0] == -math.inf:
                finish(b, am[b][1], am[b][0])
                continue
            if not trunc[b]:
                finish(b, best[1], best[2])
                continue
            cand[b] = (best[1], best[2])
            above = x[b] > best[2]
            rec[b, 0] = float(torch.exp((x[b][above] - xmax[b]) * inv_t[b]).sum())
            rec[b, 1] = float(above.sum())
            if rnd + 1 < max_rounds:
                k_, j_, x_ = race(b, rnd + 1, best[2])
                rec[b, 4], rec[b, 5], rec[b, 6] = k_, float(j_), x_
        if not last:
            g = exchange(rec)
    return torch.tensor(tok, dtype=torch.int32), torch.tensor(lp, dtype=torch.float32)


def apply_penalties(logits, window, ngen, pen, v0: int = 0):
    """In place: repetition (every window token), presence / frequency (counts
    over the generated tail of the right-aligned window)."""
    B, W = window.shape
    for b in range(B):
        ids = window[b].tolist()
        g0 = W - int(ngen[b])
        rep, pres, freq = (float(v) for v in pen[b])
        seen = set()
        for i, t in enumerate(ids):
            if t < 0 or t in seen:
                continue
            seen.add(t)
            if not v0 <= t < v0 + logits.shape[1]:     # another rank's vocabulary shard
                continue
            cnt = sum(1 for j in range(max(i, g0), W) if ids[j] == t)
            x = float(logits[b, t - v0])
            if rep != 1.0:
                x = x / rep if x > 0 else x * rep
            x -= freq * cnt + (pres if cnt > 0 else 0.0)
            logits[b, t - v0] = x
    return logits


# ------------------------------------- gated / recurrent token mixers ------
def relu_mul(x):
    I = x.shape[-1] // 2
    return (torch.relu(x[..., :I].float()) * x[..., I:].float()).to(x.dtype)


def gate_rows(o, gate):
    """o * sigmoid(gate) (gate None: o)."""
    if gate is None:
        return o
    return (o.float() * torch.sigmoid(gate[:, :o.shape[1]].float())).to(o.dtype)


def _unit(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def sandwich_norm(residual, eps, y=None, w_post=None, w_pre=None, ids=None, table=None,
                  rows=None, dtype=torch.bfloat16, scale=1.0, bias=None, own=None):
    r = table[ids.long()].float() * scale if ids is not None else residual
    if y is not None:
        y = y.float()
        if bias is not None:
            y = y + bias
        if own is not None:
            y = y + own[:, None] * residual
    if rows is not None:
        r, y = r[rows], None if y is None else y[rows]
    if y is not None:
        r = r + _unit(y, eps) * w_post
    if rows is None:
        residual.copy_(r)
    return (r if w_pre is None else _unit(r, eps) * w_pre).to(dtype)


def sum_norm(residual, eps, y, alpha, scale, w_post, w_pre=None, rows=None, dtype=torch.bfloat16):
    def norm(z, w):
        z = z - z.mean(-1, keepdim=True)
        return _unit(z, eps) * w
    r = residual if rows is None else residual[rows]
    if y is not None:
        y = y if rows is None else y[rows]
        r = norm(alpha * r + scale * y.float(), w_post)
    if rows is None:
        residual.copy_(r)
    return (r if w_pre is None else norm(r, w_pre)).to(dtype)


def gated_norm(x, gate, w, groups, eps, gate_first, silu=False):
    T, C = x.shape
    v, g = x.float(), gate[:, :C].float()
    if gate_first:
        v = v * torch.nn.functional.silu(g)
    v = _unit(v.reshape(T, groups, C // groups), eps).reshape(T, C) * w
    if not gate_first:
        v = v * (torch.nn.functional.silu(g) if silu else torch.sigmoid(g))
    return v.to(x.dtype)


def _conv_rows(u, w, bias, in_bias, state, cu_q, ctx, slots):
    """fp32 conv output of every row; advances ``state`` in place."""
    taps, C = w.shape
    y = torch.zeros((u.shape[0], C), dtype=torch.float32, device=u.device)
    for s in range(len(ctx)):
        a, b, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
        if slot < 0:
            continue
        x = u[a:b, :C].float()
        if in_bias is not None:
            x = x + in_bias
        old = torch.zeros((taps - 1, C)) if taps == 1 or int(ctx[s]) == b - a \
            else state[slot].float()
        full = torch.cat([old.to(x.device), x])
        for j in range(taps):
            y[a:b] += full[j:j + b - a] * w[j]
        if taps > 1:
            state[slot] = full[b - a:].to(state.dtype)
    return y if bias is None else y + bias


def short_conv(u, w, bias, state, cu_q, ctx, slots, out, silu, in_bias=None):
    y = _conv_rows(u, w, bias, in_bias, state, cu_q, ctx, slots)
    out.copy_(torch.nn.functional.silu(y) if silu else y)


def conv_qkv_cache(u, w, in_bias, state, cu_q, ctx, state_slots, q_out, k_cache, v_cache,
                   positions, slots, Hq, Hkv, D, dk, eps, temp):
    T = u.shape[0]
    y = _conv_rows(u, w, None, in_bias, state, cu_q, ctx, state_slots).view(T, -1, D)
    inv = torch.rsqrt(y.pow(2).sum(-1, keepdim=True) / dk + eps)
    coef, every = temp
    t = 1.0 + coef * torch.log(torch.floor((positions.float() + 1.0) / every) + 1.0)
    q_out.copy_((y[:, :Hq] * inv[:, :Hq] * t[:, None, None]).reshape(T, Hq * D))
    write_cache((y * inv)[:, Hq:Hq + Hkv], y[:, Hq + Hkv:Hq + 2 * Hkv], slots, k_cache, v_cache)


def norm_rope_cache(p, q_norm, k_norm, ang, slots, k_cache, v_cache, Hq, dk, eps):
    _, Hkv, _, D = k_cache.shape
    T = p.shape[0]
    x = p[:, :(Hq + 2 * Hkv) * D].float().view(T, -1, D)
    qk = x[:, :Hq + Hkv]
    qk = qk * torch.rsqrt(qk.pow(2).sum(-1, keepdim=True) / dk + eps)
    qk = rotate_pairs(torch.cat([qk[:, :Hq] * q_norm, qk[:, Hq:] * k_norm], 1), ang)
    write_cache(qk[:, Hq:], x[:, Hq + Hkv:], slots, k_cache, v_cache)
    return qk[:, :Hq].reshape(T, Hq * D).to(p.dtype)


def rotate_pairs(x, ang):
    """x [T, H, d] fp32: components (2i, 2i + 1) turned by the angles [T, n] of
    ``rope_angles``, the first n of d (None: none)."""
    if ang is None:
        return x
    n = ang.shape[1]
    c, s = ang[:, None, :n // 2], ang[:, None, n // 2:]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([y, x[..., n:]], -1)


def delta_rule(q, k, v, b, a, dt_bias, neg_a, out, state, cu_q, ctx, slots, G):
    """See ops.delta_rule; one token after the other, fp32."""
    _, H, N, P = state.shape
    T = q.shape[0]

    def heads(x):
        x = x[:, :G * N].float().view(T, G, N)
        x = x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)
        return x.repeat_interleave(H // G, 1)
    qs, ks, vs = heads(q) * N ** -0.5, heads(k), v[:, :H * P].float().view(T, H, P)
    beta = torch.sigmoid(b[:, :H].float())
    g = torch.exp(neg_a * torch.nn.functional.softplus(a[:, :H].float() + dt_bias))
    for s in range(len(ctx)):
        t0, t1, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
        if slot < 0:
            continue
        S = torch.zeros(H, N, P) if int(ctx[s]) == t1 - t0 else state[slot].clone()
        for t in range(t0, t1):
            S = g[t][:, None, None] * S
            u = beta[t][:, None] * (vs[t] - torch.einsum("hnp,hn->hp", S, ks[t]))
            S = S + ks[t][:, :, None] * u[:, None, :]
            out[t, :H * P] = torch.einsum("hnp,hn->hp", S, qs[t]).reshape(-1).to(out.dtype)
        state[slot] = S


def linear_scan(q, k, v, out, state, cu_q, ctx, slots, hpg, decay, dt, skip, silu, seqs,
                angles=None, k_scale=1.0):
    """See ops.linear_scan; one token after the other, fp32."""
    _, H, N, P = state.shape
    G = H // hpg
    if angles is not None or k_scale != 1.0:
        T = q.shape[0]
        q = rotate_pairs(q[:, :G * N].float().view(T, G, N), angles).to(q.dtype).view(T, -1)
        k = (rotate_pairs(k[:, :G * N].float().view(T, G, N), angles) * k_scale).to(k.dtype) \
            .view(T, -1)
    act = (lambda x: torch.nn.functional.silu(x.float()).to(q.dtype).float()) if silu \
        else (lambda x: x.float())
    for s in seqs:
        a, b, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
        if slot < 0:
            continue
        n = b - a
        qs = act(q[a:b, :G * N]).view(n, G, N).repeat_interleave(hpg, 1)
        ks = act(k[a:b, :G * N]).view(n, G, N).repeat_interleave(hpg, 1)
        vs = act(v[a:b, :H * P]).view(n, H, P)
        if dt is not None:
            rows, bias, neg_a = dt
            st = torch.nn.functional.softplus(rows[a:b, :H].float() + bias)
            dec = torch.exp(neg_a * st)
        else:
            st, dec = torch.ones(n, H), decay[0].expand(n, H)
        S = torch.zeros(H, N, P) if int(ctx[s]) == n else state[slot].clone()
        for t in range(n):
            S = dec[t][:, None, None] * S + ks[t][:, :, None] * (vs[t] * st[t][:, None])[:, None, :]
            o = torch.einsum("hn,hnp->hp", qs[t], S)
            if skip is not None:
                o = o + skip[:, None] * vs[t]
            out[a + t, :H * P] = o.reshape(-1).to(out.dtype)
        state[slot] = S


def rglru(u, y, y_bias, gates, gate_bias, log_a, out, state, cu_q, ctx, slots):
    """See ops.rglru; one token after the other, fp32.  gates [n, 2 bp, bp]."""
    T, C = u.shape
    n, _, bp = gates.shape
    x = u.float()
    z = torch.einsum("tnk,nzok->tzno", x.view(T, n, bp),
                     gates.float().view(n, 2, bp, bp)).reshape(T, 2, C)
    r, i = torch.sigmoid(z + gate_bias).unbind(1)
    la = log_a * r
    b = torch.sqrt(-torch.expm1(2.0 * la)) * i * x
    a = torch.exp(la)
    g = torch.nn.functional.gelu(y.float() + y_bias, approximate="tanh")
    for s in range(len(ctx)):
        t0, t1, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
        if slot < 0:
            continue
        S = torch.zeros(C) if int(ctx[s]) == t1 - t0 else state[slot].clone()
        for t in range(t0, t1):
            S = a[t] * S + b[t]
            out[t] = (S * g[t]).to(out.dtype)
        state[slot] = S


# ------------------------------------------------------- latent attention ---
def rope_angles(positions, freqs, scale=1.0):
    a = positions.double()[:, None] * freqs
    return (torch.cat([a.cos(), a.sin()], 1) * scale).float()


def rotate(x, ang):
    """x [T, ..., d] (halves paired) by the angles of ``rope_angles`` [T, d]."""
    h = x.shape[-1] // 2
    cs = ang.reshape((x.shape[0],) + (1,) * (x.dim() - 2) + (2 * h,))
    c, s = cs[..., :h], cs[..., h:]
    a, b = x[..., :h].float(), x[..., h:].float()
    return torch.cat([a * c - b * s, b * c + a * s], -1)


def latent_prep(p, qr, qp, q_norm, R, c_norm, ang, slots, pages, Rp, eps):
    T, d = ang.shape
    cq = torch.zeros((T, qp), dtype=p.dtype)
    cq[:, :qr] = (_unit(p[:, :qr].float(), eps) * q_norm[:qr]).to(p.dtype)
    row = torch.zeros((T, pages.shape[3]))
    row[:, :R] = _unit(p[:, qp:qp + R].float(), eps) * c_norm[:R]
    row[:, Rp:Rp + d] = rotate(p[:, qp + Rp:qp + Rp + d], ang)
    BS = pages.shape[2]
    for t in range(T):
        s = int(slots[t])
        if s >= 0:
            pages[s // BS, 0, s % BS] = row[t].to(pages.dtype)
    return cq


def latent_query(q, absorb, ang, H, np_, xp, Rp):
    T, d = q.shape[0], ang.shape[1]
    q3 = q.view(T, H, np_ + xp)
    out = torch.zeros((T, H, Rp + xp), dtype=q.dtype)
    out[..., :Rp] = torch.einsum("thk,hrk->thr", q3[..., :np_].float(), absorb.float()).to(q.dtype)
    out[..., Rp:Rp + d] = rotate(q3[..., np_:np_ + d], ang[:T]).to(q.dtype)
    return out.view(T, -1)


def latent_attention(ql, pages, block_tables, cu_q, positions, scale, window, H, Rp):
    T = ql.shape[0]
    BS = pages.shape[2]
    q = ql.view(T, H, -1).float()
    out = torch.zeros((T, H, Rp), dtype=ql.dtype)
    cu = [int(x) for x in cu_q]
    for s in range(len(cu) - 1):
        for t in range(cu[s], min(cu[s + 1], T)):
            p = int(positions[t])
            j = torch.arange(max(0, p - window + 1), p + 1)
            k = pages[block_tables[s, j // BS].long(), 0, j % BS].float()
            w = torch.softmax((q[t] @ k.T) * scale, -1)
            out[t] = (w @ k[:, :Rp]).to(out.dtype)
    return out.view(T, -1)


# ----------------------------------------------------- grouped products -----
def clamped_glu(g, u, limit, act=(1.702, 1.0)):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(act[0] * g) * (u + act[1])


def moe_route_groups(h, w, top, extra, scores):
    E, n = scores.correction.numel(), scores.groups
    z = h.float() @ w.float().t()
    z = torch.softmax(z, -1) if scores.softmax else torch.sigmoid(z)
    s, T = z[:, :E], h.shape[0]
    c = s + scores.correction
    best = 1 if scores.softmax else min(2, E // n)
    rank = c.view(T, n, E // n).topk(best, -1).values.sum(-1)
    g = torch.sort(rank, dim=-1, descending=True, stable=True).indices[:, :scores.keep]
    kept = torch.zeros(T, n, dtype=torch.bool).scatter_(1, g, True)
    c = c.masked_fill(~kept.repeat_interleave(E // n, 1), float("-inf"))
    ids = torch.sort(c, dim=-1, descending=True, stable=True).indices[:, :top]
    wts = s.gather(1, ids)
    if not scores.softmax:
        wts = wts / (wts.sum(-1, keepdim=True) + 1e-20)
    own = None
    if scores.identity:
        E -= scores.identity
        own = (wts * (ids >= E)).sum(-1)
        wts = wts * (ids < E)
        ids = torch.where(ids < E, ids, -1)
    ids = torch.cat([ids, torch.arange(E, E + extra).expand(T, extra)], 1)
    shared = z[:, E:].expand(T, extra) if z.shape[1] > scores.correction.numel() \
        else torch.ones(T, extra)
    return ids.to(torch.int32), torch.cat([wts, shared], 1), own


def moe_route(h, w, top, extra):
    z = h.float() @ w.float().t()
    v, e = torch.sort(z, dim=-1, descending=True, stable=True)
    T, E = z.shape
    ids = torch.cat([e[:, :top], torch.arange(E, E + extra).expand(T, extra)], 1)
    wts = torch.cat([torch.softmax(v[:, :top], -1), torch.ones(T, extra)], 1)
    return ids.to(torch.int32), wts


def grouped_rows(x, w, src, off, gather, limit, act=(1.702, 1.0)):
    """Rows off[e]..off[e+1] of the expert order times w[e]^T."""
    K = w.shape[2]
    out = torch.zeros((src.numel(), w.shape[1] // (2 if limit is not None else 1)), dtype=x.dtype)
    for e in range(w.shape[0]):
        a, b = int(off[e]), int(off[e + 1])
        rows = x[src[a:b].long()] if gather else x[a:b]
        y = rows[:, :K].float() @ w[e].float().t()
        if limit is not None:
            y = y.view(b - a, w.shape[1] // 32, 2, 16)
            y = clamped_glu(y[:, :, 0], y[:, :, 1], float(limit[e]), act).reshape(b - a, out.shape[1])
        out[a:b] = y.to(x.dtype)
    return out


# ------------------------------- talking heads, matrix memory, projections --
def qkv_norm_rope_cache(p, bias, q_norm, k_norm, ang, slots, k_cache, v_cache, Hq, dk, dv, eps):
    """See ops.qkv_norm_rope_cache."""
    _, Hkv, _, D = k_cache.shape
    T = p.shape[0]
    x = (p[:, :(Hq + 2 * Hkv) * D].float() + bias).view(T, -1, D)

    def whole(y, w):
        inv = torch.rsqrt(y.pow(2).sum((1, 2)) / (y.shape[1] * dk) + eps)
        return rotate_pairs(y * inv[:, None, None] * w.view(1, -1, D), ang)
    v = x[:, Hq + Hkv:]
    v = v * torch.rsqrt(v.pow(2).sum(-1, keepdim=True) / dv + eps)
    write_cache(whole(x[:, Hq:Hq + Hkv], k_norm), v, slots, k_cache, v_cache)
    return whole(x[:, :Hq], q_norm).reshape(T, Hq * D).to(p.dtype)


def talking_attention(q, k_cache, v_cache, block_tables, cu_q, ctx, scale, talk, sink, chunk):
    """q [T, Hq, D], every row of the sequences; see ops.talking_attention."""
    T, H, D = q.shape
    out = torch.zeros_like(q)
    for s in range(len(ctx)):
        a, b, n = int(cu_q[s]), int(cu_q[s + 1]), int(ctx[s])
        k, v = gather_kv(k_cache, v_cache, block_tables[s], n)
        per = H // k.shape[1]
        k, v = (x.float().repeat_interleave(per, 1) for x in (k, v))
        raw = torch.einsum("thd,nhd->htn", q[a:b].float(), k) * scale
        if talk is not None:
            raw = torch.einsum("hg,gtn->htn", talk.float(), raw)
        p = torch.arange(n - (b - a), n)[:, None]
        j = torch.arange(n)[None]
        seen = j <= p
        if chunk:
            seen = seen & (j >= p // chunk * chunk)
        x = raw.masked_fill(~seen, float("-inf"))
        if sink is not None:
            x = torch.cat([x, sink.float()[:, None, None].expand(H, b - a, 1)], -1)
        w = torch.softmax(x, -1)[..., :n]
        out[a:b] = torch.einsum("htn,nhd->thd", w, v).to(q.dtype)
    return out


def memory_scan(q, k, v, ig, fg, bias, cap, out, state, cu_q, ctx, slots):
    """See ops.memory_scan; one token after the other, fp32."""
    S_, n_, m_ = state
    _, H, N, P = S_.shape
    T = q.shape[0]
    qs, ks = (x[:, :H * N].float().view(T, H, N) for x in (q, k))
    qs, vs = qs * N ** -0.5, v[:, :H * P].float().view(T, H, P)
    i, f = (cap * torch.tanh((x[:, :H].float() + b) / cap) for x, b in zip((ig, fg), bias))
    f = torch.nn.functional.logsigmoid(f)
    for s in range(len(ctx)):
        a, b, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
        if slot < 0:
            continue
        if int(ctx[s]) == b - a:
            S, n, m = torch.zeros(H, N, P), torch.zeros(H, N), torch.zeros(H)
        else:
            S, n, m = S_[slot].clone(), n_[slot].clone(), m_[slot].clone()
        for t in range(a, b):
            new = torch.maximum(f[t] + m, i[t])
            keep, add = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
            S = keep[:, None, None] * S + (add[:, None] * ks[t])[:, :, None] * vs[t][:, None, :]
            n = keep[:, None] * n + add[:, None] * ks[t]
            m = new
            den = torch.maximum((n * qs[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
            o = torch.einsum("hnp,hn->hp", S, qs[t]) / den[:, None]
            out[t, :H * P] = o.reshape(-1).to(out.dtype)
        S_[slot], n_[slot], m_[slot] = S, n, m


def bias_relu2(x, bias):
    y = torch.relu(x.float() + bias)
    return (y * y).to(x.dtype)
