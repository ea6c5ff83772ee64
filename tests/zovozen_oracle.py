"""Plain, slow reference of the Zovozen decoder: one sequence, one token after
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


def log_sigmoid(z):
    """ln sigmoid(z) = min(z, 0) - ln(1 + e^-|z|)"""
    return torch.clamp(z, max=0) - torch.log1p(torch.exp(-z.abs()))


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def affine(h, W, name):
    """W h + b"""
    return h @ W[name].T + W[name + ".b"]


# ------------------------------------------------------------ attention -----
def frequencies(rot):
    """base^(-2i/dims), all divided by the scaling factor where there is one."""
    f = torch.tensor([rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)],
                     dtype=F64)
    s = rot.get("scaling")
    return f / s["factor"] if s else f


def rotate_half(x, pos, rot):
    """x [T, H, d]: components (i, i + dims/2) of the first dims are a pair,
    turned by position x frequency."""
    d = rot["dims"]
    a = (pos.to(F64)[:, None] * frequencies(rot))[:, None]
    u, v = x[..., :d // 2], x[..., d // 2:d]
    return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., d:]], -1)


def talking_attention(q, k, v, scale, chunk, temp, talk, sink):
    """q [T, H, d], k [T, G, d], v [T, G, e], query head h with key head
    h // (H/G): raw scores scale temp[h] (q k), mixed over the heads by talk
    [H, H]; position i sees the positions up to its own of its chunk; the
    softmax's denominator also has exp(sink[h])."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    i = torch.arange(T)
    seen = (i[:, None] >= i[None]) & (i[:, None] // chunk == i[None] // chunk)
    raw = torch.stack([scale * temp[h] * (q[:, h] @ k[:, h // per].T) for h in range(H)])
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = sum(talk[h, g] * raw[g] for g in range(H)).masked_fill(~seen, -math.inf)
        m = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        w = torch.exp(s - m)
        out[:, h] = (w @ v[:, h // per]) / (w.sum(-1, keepdim=True) + torch.exp(sink[h] - m))
    return out


def attention_branch(h, W, p, m, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    pos = torch.arange(T)
    q = unit_rms(affine(h, W, p + "q"), eps) * W[p + "q.norm"]
    k = unit_rms(affine(h, W, p + "k"), eps) * W[p + "k.norm"]
    q = rotate_half(q.reshape(T, H, m["dim"]), pos, m["rot"])
    k = rotate_half(k.reshape(T, G, m["dim"]), pos, m["rot"])
    v = unit_rms(affine(h, W, p + "v").reshape(T, G, m["vdim"]), eps)
    o = talking_attention(q, k, v, m["scale"], m["mask"]["size"], W[p + "temp"], W[p + "talk"],
                          W[p + "sink"])
    return affine(o.reshape(T, -1) * sigmoid(h @ W[p + "g"].T), W, p + "o")


# -------------------------------------------------------- matrix memory -----
def matrix_memory(q, k, v, i, f):
    """q, k [T, H, n], v [T, H, e], log gates i, f [T, H].  Per head, from S =
    0, n = 0, m = 0:

        m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T, n alike;
        o = S^T q / (max(|n q|, e^-m') + 1e-6)"""
    T, H, N = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S, n, m = torch.zeros(N, v.shape[2], dtype=v.dtype), torch.zeros(N, dtype=v.dtype), 0.0
        for t in range(T):
            new = max(float(f[t, h]) + m, float(i[t, h]))
            keep, add = torch.exp(f[t, h] + m - new), torch.exp(i[t, h] - new)
            S = keep * S + add * torch.outer(k[t, h], v[t, h])
            n = keep * n + add * k[t, h]
            m = new
            out[t, h] = (S.T @ q[t, h]) / (max(abs(float(n @ q[t, h])), math.exp(-m)) + 1e-6)
    return out


def memory_gates(h, W, p, cap):
    """(ln of the input gate, ln of the forget gate) [T, H]"""
    def capped(name):
        return cap * torch.tanh(affine(h, W, p + name) / cap)
    return capped("i"), log_sigmoid(capped("f"))


def memory_branch(h, W, p, m, eps):
    T, H, n, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).reshape(T, H, n) * n ** -0.5
    k = (h @ W[p + "k"].T).reshape(T, H, n)
    v = (h @ W[p + "v"].T).reshape(T, H, e)
    o = unit_rms(matrix_memory(q, k, v, *memory_gates(h, W, p, m["gate_cap"])), eps)
    return (o.reshape(T, -1) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    return m["left_scale"] * attention_branch(h, W, p + "left.", m["left"], eps) + \
        m["right_scale"] * memory_branch(h, W, p + "right.", m["right"], eps)


# --------------------------------------------------------- feed-forward -----
def dense_ff(h, W, p, m):
    return affine(torch.clamp(affine(h, W, p + "up"), min=0) ** 2, W, p + "down")


def glu(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, w, correction, router):
    """Experts [T, top] and their weights.  Scores are a softmax over all
    outputs of the router, identity experts included; groups of neighbours are
    ranked by their largest corrected score, the best of the kept groups are
    chosen by corrected score; the weights are the plain scores."""
    s = torch.softmax(h @ w.T, -1)
    T, E = s.shape
    top, groups = router["top"], router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    ids, wts = torch.zeros(T, top, dtype=torch.long), torch.zeros(T, top, dtype=s.dtype)
    for t in range(T):
        c = (s[t] + correction).tolist()
        rank = [max(c[a:a + size]) for a in range(0, E, size)]
        kept = sorted(range(len(rank)), key=lambda a: (-rank[a], a))[:groups["keep"]]
        best = sorted((e for e in range(E) if e // size in kept), key=lambda e: (-c[e], e))[:top]
        ids[t], wts[t] = torch.tensor(best), s[t, best]
    return ids, wts


def moe_ff(h, W, p, m):
    e, wt = route(h, W[p + "router"], W[p + "correction"], m["router"])
    E = m["router"]["experts"]
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(e.shape[1]):
            i = int(e[t, j])
            y[t] += wt[t, j] * (glu(h[t:t + 1], W, f"{p}e{i}.")[0] if i < E else h[t])
    return y + glu(h, W, p + "shared.") if m.get("shared") else y


FEEDFORWARDS = {"dense": dense_ff, "moe": moe_ff}


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence; the residual after every layer is
    appended to ``layers_out``."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + unit_rms(parallel_mixer(x, W, p + "mix.", L["mixer"], eps), eps) * W[p + "norm1"]
        if L["mlp"] is not None:
            y = FEEDFORWARDS[L["mlp"]["kind"]](x, W, p + "mlp.", L["mlp"])
            x = x + unit_rms(y, eps) * W[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return (unit_rms(x, eps) * W["final.norm"]) @ W["embed"].T
