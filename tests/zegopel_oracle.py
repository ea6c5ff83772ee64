"""Plain, slow reference of the Zegopel decoder: one sequence, one token after
the other where the mechanism is a recurrence, float64 throughout.

One function per mechanism, written from the equations in the docstrings; it
shares no code with ``llm_mcp_amd``.  Weights are a flat dict of tensor name ->
tensor, the configuration is the parsed ``config.json``.
"""
import math

import torch
import torch.nn.functional as F

F64 = torch.float64


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_zero_centred(x, w, eps):
    """RMS norm whose stored weight w acts as 1 + w."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(x):
    return x / (1.0 + torch.exp(-x))


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def causal_conv(u, w, bias=None):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_{t - taps + 1 + j} + bias,
    zeros before the first token (the last column weighs the current token)."""
    T, C = u.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u])
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * w[:, j]
    return y if bias is None else y + bias


def linear_attention(q, k, v, decay):
    """q, k [T, H, N], v [T, H, P], decay [T, H]: per head S <- decay S + k v^T,
    o = S^T q, S zero at the start."""
    T, H, N = q.shape
    S = torch.zeros(H, N, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = decay[t][:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def query_temperature(pos, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1)"""
    return 1.0 + coef * torch.log(torch.floor((pos + 1.0) / every) + 1.0)


def softmax_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, e]; query head h reads head h // (H / G);
    position i sees j <= i."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    mask = torch.ones(T, T).tril().bool()
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(~mask, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def grouped_norm(y, w, groups, eps):
    """RMS norm of each of ``groups`` equal parts, times w."""
    T, C = y.shape
    return unit_rms(y.reshape(T, groups, C // groups), eps).reshape(T, C) * w


def lightning_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, N, P = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ W[p + "q"].T).reshape(T, H, N)
    k = silu(h @ W[p + "k"].T).reshape(T, H, N)
    v = silu(h @ W[p + "v"].T).reshape(T, H, P)
    decay = torch.tensor(m["decay"], dtype=h.dtype).expand(T, H)
    o = linear_attention(q, k, v, decay).reshape(T, H * P)
    o = grouped_norm(o, W[p + "norm"], 1, eps) * sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def mamba2_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    u = h @ W[p + "in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + W[p + "dt_bias"])
    decay = torch.exp(-torch.exp(W[p + "A_log"]) * dt)
    grp = torch.arange(H) // (H // G)
    y = linear_attention(C[:, grp], B[:, grp] * dt[:, :, None], x, decay)
    y = y + W[p + "D"][:, None] * x
    y = y.reshape(T, inner) * silu(z)
    return grouped_norm(y, W[p + "norm"], m["norm_groups"], eps) @ W[p + "o"].T


def attention_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    r = {}
    for n in ("q", "k", "v"):
        r[n] = causal_conv(h @ W[p + n].T + W[p + n + ".b"], W[p + n + ".conv"])
    q = unit_rms(r["q"].reshape(T, H, d), eps)
    k = unit_rms(r["k"].reshape(T, G, d), eps)
    pos = torch.arange(T, dtype=h.dtype)
    q = q * query_temperature(pos, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    o = softmax_attention(q, k, r["v"].reshape(T, G, e), m["scale"]).reshape(T, H * e)
    return (o * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def relu_glu(h, W, p):
    return (torch.relu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"lightning": lightning_mixer, "mamba2": mamba2_mixer, "attention": attention_mixer}


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence; the residual after every layer is
    appended to ``layers_out``."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm_zero_centred(x, W[p + "norm1"], eps)
        y = MIXERS[L["type"]](h, W, p + "mix.", L["mixer"], eps)
        x = x + norm_zero_centred(y, W[p + "norm1b"], eps)
        if L["mlp"] is not None:
            h = norm_zero_centred(x, W[p + "norm2"], eps)
            x = x + norm_zero_centred(relu_glu(h, W, p + "mlp."), W[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_zero_centred(x, W["final.norm"], eps) @ W["head"].T
