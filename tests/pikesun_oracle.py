"""Plain, slow reference of the Pikesun decoder: one sequence, one token after
the other where the mechanism is a recurrence, float64 throughout.

One function per mechanism, written from the equations in the docstrings; it
shares no code with ``llm_mcp_amd``.  Weights are a flat dict of tensor name ->
tensor, the configuration is the parsed ``config.json``.
"""
import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    """w x / sqrt(mean(x^2) + eps) over the last axis."""
    return w * x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    """ln(1 + e^z)"""
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    """z/2 (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))"""
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, w, bias):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_{t - taps + 1 + j} + bias,
    zeros before the first token (the last column weighs the current token)."""
    T, C = u.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u])
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * w[:, j]
    return y + bias


def block_gate(u, w, b):
    """sigmoid of a block-diagonal affine map: u [T, C], w [n, C/n, C/n] as
    [out, in], b [n, C/n]."""
    T, C = u.shape
    n = w.shape[0]
    part = u.reshape(T, n, C // n)
    z = torch.stack([part[:, i] @ w[i].T + b[i] for i in range(n)], 1)
    return sigmoid(z).reshape(T, C)


def gated_linear_recurrence(u, r, i, lam):
    """Per channel log a = -8 r softplus(lam), S <- a S + sqrt(1 - a^2) i u from
    S = 0; returns every S [T, C]."""
    S = torch.zeros(u.shape[1], dtype=u.dtype)
    out = []
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = torch.exp(log_a) * S + torch.sqrt(1.0 - torch.exp(2.0 * log_a)) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru_mixer(h, W, p, m, eps):
    y = gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"])
    u = causal_conv(h @ W[p + "x"].T + W[p + "x.b"], W[p + "conv"], W[p + "conv.b"])
    r = block_gate(u, W[p + "ra"], W[p + "ra.b"])
    i = block_gate(u, W[p + "ri"], W[p + "ri.b"])
    return (gated_linear_recurrence(u, r, i, W[p + "lam"]) * y) @ W[p + "o"].T


def rotate_half(x, pos, base):
    """x [T, ..., d]: components (i, i + d/2) turned by pos base^(-2i/d)."""
    d = x.shape[-1]
    f = torch.tensor([base ** (-2.0 * i / d) for i in range(d // 2)], dtype=x.dtype)
    a = pos.to(x.dtype)[:, None] * f
    a = a.reshape((x.shape[0],) + (1,) * (x.dim() - 2) + (d // 2,))
    u, v = x[..., :d // 2], x[..., d // 2:]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)], -1)


def window_attention(q, k, v, scale, window):
    """q, k [T, H, d], v [T, H, e]: position i sees 0 <= i - j < window."""
    T, H, _ = q.shape
    i = torch.arange(T)
    seen = (i[:, None] >= i[None]) & (i[:, None] - i[None] < window)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = ((q[:, h] @ k[:, h].T) * scale).masked_fill(~seen, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h]
    return out


def latent_attention_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, pos = m["rot"]["base"], torch.arange(T)
    cq = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps)
    q = (cq @ W[p + "uq"].T).reshape(T, H, dn + dr)
    q = torch.cat([q[..., :dn], rotate_half(q[..., dn:], pos, base)], -1)
    z = h @ W[p + "dkv"].T
    c = rms_norm(z[:, :R], W[p + "dkv.norm"], eps)
    kr = rotate_half(z[:, R:], pos, base)
    k = torch.cat([(c @ W[p + "uk"].T).reshape(T, H, dn), kr[:, None].expand(T, H, dr)], -1)
    v = (c @ W[p + "uv"].T).reshape(T, H, dv)
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"]).reshape(T, H * dv)
    return (o * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def dense_ff(h, W, p):
    return gelu_tanh(h @ W[p + "up"].T) @ W[p + "down"].T


def clamped_glu(h, W, p, limit):
    """g = min(W_gate h, L), u = clamp(W_up h, -L, L); W_down (g sigmoid(1.702 g) (u + 1))"""
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def route(h, w, top):
    """The ``top`` largest of w h per token and the softmax over just those."""
    z, e = torch.sort(h @ w.T, dim=-1, descending=True, stable=True)
    return e[:, :top], torch.softmax(z[:, :top], -1)


def moe_ff(h, W, p, m):
    e, wt = route(h, W[p + "router"], m["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(e.shape[1]):
            y[t] += wt[t, j] * clamped_glu(h[t:t + 1], W, f"{p}e{int(e[t, j])}.",
                                           m["expert"]["limit"])[0]
    if m.get("shared"):
        y = y + clamped_glu(h, W, p + "shared.", m["shared"]["limit"])
    return y


MIXERS = {"rglru": rglru_mixer, "latent_attention": latent_attention_mixer}


def source_layer(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence; the residual after every layer is
    appended to ``layers_out``."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{source_layer(cfg['layers'], i)}."
        y = MIXERS[L["type"]](x, W, p + "mix.", L["mixer"], eps)
        x = x + mult * rms_norm(y, W[p + "norm1"], eps)
        if L["mlp"] is not None:
            y = dense_ff(x, W, p + "mlp.") if L["mlp"]["kind"] == "dense" else \
                moe_ff(x, W, p + "mlp.", L["mlp"])
            x = x + mult * rms_norm(y, W[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T
