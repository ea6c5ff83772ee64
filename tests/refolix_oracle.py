"""Plain, slow reference of the Refolix decoder: one sequence, one token after
the other where the mechanism is a recurrence, float64 throughout.

One function per mechanism, written from the equations in the docstrings; it
shares no code with ``llm_mcp_amd``.  Weights are a flat dict of tensor name ->
tensor, the configuration is the parsed ``config.json``.
"""
import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    """ln(1 + e^z)"""
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    """w (x - mean) / sqrt(mean((x - mean)^2) + eps)"""
    c = x - x.mean(-1, keepdim=True)
    return w * c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps)


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


# ------------------------------------------------------------- rotation -----
def frequencies(rot):
    """base^(-2i/dims); with ``scaling``, slow components are divided by the
    factor: component i blends from its own frequency (up to lo) to the divided
    one (from hi on), lo and hi being where a component turns ``fast`` and
    ``slow`` times within the original length."""
    base, dims = rot["base"], rot["dims"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if s:
        def component(turns):
            return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
        lo = max(math.floor(component(s["fast"])), 0)
        hi = min(math.ceil(component(s["slow"])), dims - 1)
        for i in range(len(f)):
            r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f[i] = f[i] / s["factor"] * r + f[i] * (1.0 - r)
    return torch.tensor(f, dtype=F64)


def magnitude(rot):
    """What cos and sin are multiplied by."""
    s = rot.get("scaling")
    return 0.1 * math.log(s["factor"]) + 1.0 if s else 1.0


def turn(u, v, pos, rot):
    """Pairs (u, v) [T, H, dims/2] turned by position x frequency."""
    a = (pos.to(F64)[:, None] * frequencies(rot))[:, None]
    c, s = magnitude(rot) * torch.cos(a), magnitude(rot) * torch.sin(a)
    return u * c - v * s, v * c + u * s


def rotate_interleaved(x, pos, rot):
    """Components (2i, 2i + 1) of the first dims are a pair."""
    d = rot["dims"]
    u, v = turn(x[..., 0:d:2], x[..., 1:d:2], pos, rot)
    out = x.clone()
    out[..., 0:d:2], out[..., 1:d:2] = u, v
    return out


def rotate_half(x, pos, rot):
    """Components (i, i + dims/2) of the first dims are a pair."""
    d = rot["dims"]
    u, v = turn(x[..., :d // 2], x[..., d // 2:d], pos, rot)
    return torch.cat([u, v, x[..., d:]], -1)


# --------------------------------------------------------------- mixers -----
def window_attention(q, k, v, scale, window, cap):
    """q [T, H, d], k [T, G, d], v [T, G, e], query head h with key head
    h // (H/G): position i sees 0 <= i - j < window; scores softly capped."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    i = torch.arange(T)
    seen = i[:, None] >= i[None]
    if window is not None:
        seen &= i[:, None] - i[None] < window
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if cap is not None:
            s = soft_cap(s, cap)
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, h // per]
    return out


def attention_branch(h, W, p, m, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    pos = torch.arange(T)
    q = (h @ W[p + "q"].T).reshape(T, H, m["dim"])
    k = (h @ W[p + "k"].T).reshape(T, G, m["dim"])
    v = (h @ W[p + "v"].T).reshape(T, G, m["vdim"])
    q = rotate_interleaved(unit_rms(q, eps) * W[p + "q.norm"], pos, m["rot"])
    k = rotate_interleaved(unit_rms(k, eps) * W[p + "k.norm"], pos, m["rot"])
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"], m["softcap"])
    return o.reshape(T, -1) @ W[p + "o"].T


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_{t - taps + 1 + j}, zeros
    before the first token."""
    T, C = u.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u])
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * w[:, j]
    return y


def unit(x):
    """x / sqrt(sum(x^2) + 1e-6)"""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def gated_delta_rule(q, k, v, g, beta):
    """Per head S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, from
    S = 0.  q, k [T, H, n], v [T, H, p], g, beta [T, H] -> [T, H, p]."""
    T, H, n = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(n, v.shape[2], dtype=v.dtype)
        for t in range(T):
            S = g[t, h] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, h])
            S = S + torch.outer(k[t, h], u)
            out[t, h] = S.T @ q[t, h]
    return out


def delta_branch(h, W, p, m, eps):
    T, H, G, n, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + c].T, W[p + c + ".conv"])) for c in "qkv")
    q = (unit(q.reshape(T, G, n)) * n ** -0.5).repeat_interleave(H // G, 1)
    k = unit(k.reshape(T, G, n)).repeat_interleave(H // G, 1)
    beta = sigmoid(h @ W[p + "b"].T)
    g = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = gated_delta_rule(q, k, v.reshape(T, H, e), g, beta)
    o = unit_rms(o, eps) * W[p + "norm"]
    o = o * silu(h @ W[p + "g"].T).reshape(T, H, e)
    return o.reshape(T, -1) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    """Half the sum of both branches, each RMS-normed over the width."""
    a = unit_rms(attention_branch(h, W, p + "left.", m["left"], eps), eps) * W[p + "left.out"]
    b = unit_rms(delta_branch(h, W, p + "right.", m["right"], eps), eps) * W[p + "right.out"]
    return 0.5 * (a + b)


def retention(q, k, v, decay):
    """Per head S_t = decay S_{t-1} + k_t v_t^T, o_t = S_t^T q_t."""
    T, H, n = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(n, v.shape[2], dtype=v.dtype)
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def retention_mixer(h, W, p, m, eps):
    T, H, n = h.shape[0], m["heads"], m["dim"]
    pos = torch.arange(T)
    q = rotate_half((h @ W[p + "q"].T).reshape(T, H, n), pos, m["rot"])
    k = rotate_half((h @ W[p + "k"].T).reshape(T, H, n), pos, m["rot"]) * n ** -0.5
    o = retention(q, k, (h @ W[p + "v"].T).reshape(T, H, m["vdim"]), m["decay"])
    o = unit_rms(o, eps).reshape(T, -1)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# --------------------------------------------------------- feed-forward -----
def glu(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, w, correction, router):
    """Experts [T, top] and their weights.  Groups of neighbours are ranked by
    the sum of their two largest corrected scores; the best experts of the kept
    groups by corrected score; the weights are the plain scores in proportion."""
    s = sigmoid(h @ w.T)
    T, E = s.shape
    top, groups = router["top"], router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    ids, wts = torch.zeros(T, top, dtype=torch.long), torch.zeros(T, top, dtype=s.dtype)
    for t in range(T):
        c = (s[t] + correction).tolist()
        rank = [sum(sorted(c[i:i + size])[-2:]) for i in range(0, E, size)]
        kept = sorted(range(len(rank)), key=lambda i: (-rank[i], i))[:groups["keep"]]
        best = sorted((e for e in range(E) if e // size in kept), key=lambda e: (-c[e], e))[:top]
        w_ = s[t, best]
        ids[t], wts[t] = torch.tensor(best), w_ / (w_.sum() + 1e-20)
    return ids, wts


def moe_ff(h, W, p, m):
    e, wt = route(h, W[p + "router"], W[p + "correction"], m["router"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(e.shape[1]):
            y[t] += wt[t, j] * glu(h[t:t + 1], W, f"{p}e{int(e[t, j])}.")[0]
    return y + sigmoid(h @ W[p + "shared.sg"].T) * glu(h, W, p + "shared.")


MIXERS = {"parallel": parallel_mixer, "retention": retention_mixer}


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence; the residual after every layer is
    appended to ``layers_out``."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[L["type"]](x, W, p + "mix.", L["mixer"], eps) * W[p + "ls1"]
        x = layer_norm(alpha * x + y, W[p + "norm1"], eps)
        if L["mlp"] is not None:
            y = moe_ff(x, W, p + "mlp.", L["mlp"]) * W[p + "ls2"]
            x = layer_norm(alpha * x + y, W[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    z = layer_norm(x, W["final.norm"], eps) @ W["head"].T * cfg["logit_scale"]
    return soft_cap(z, cfg["logit_softcap"])
