"""Small Zegopel configurations and random weights of the tests."""
import math

import torch

LIGHT = dict(heads=2, dim=32, vdim=32, decay=[0.7, 0.99])
MAMBA = dict(heads=4, vdim=16, state=24, groups=2, conv=4, norm_groups=2)
ATTN = dict(heads=4, kv_heads=2, dim=64, vdim=64, conv=3, scale=0.2,
            q_temp=dict(coef=0.4, every=16))
MLP = dict(kind="dense", ff=96)


def layer(kind, mixer, mlp=None, **over):
    return {"type": kind, "mixer": {**mixer, **over}, "mlp": mlp}


def config(layers, width=64, vocab=61, eps=1e-5):
    return {"architecture": "Zegopel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": layers}


CASES = {
    # the three mixers, feed-forward on the attention layer only
    "mixed": config([layer("lightning", LIGHT), layer("mamba2", MAMBA),
                     layer("attention", ATTN, MLP)]),
    # attention first and last with different geometries, feed-forwards elsewhere
    "reordered": config([layer("attention", ATTN, None, heads=6, kv_heads=1, dim=48, vdim=80,
                               conv=2, scale=0.1, q_temp=dict(coef=1.5, every=5)),
                         layer("mamba2", MAMBA, MLP, heads=6, vdim=24, groups=3, conv=2,
                               norm_groups=1, state=40),
                         layer("lightning", LIGHT, dict(kind="dense", ff=40), heads=3, dim=64,
                               vdim=72, decay=[0.2, 0.9, 0.9995]),
                         layer("attention", ATTN, None, heads=2, kv_heads=2, dim=32, vdim=16,
                               conv=5)], width=96, vocab=83, eps=1e-4),
    # sizes no vector path covers
    "odd": config([layer("lightning", LIGHT, dict(kind="dense", ff=21), heads=3, dim=20, vdim=10,
                         decay=[0.5, 0.95, 0.999]),
                   layer("mamba2", MAMBA, None, heads=3, vdim=7, state=9, groups=1, conv=6,
                         norm_groups=3),
                   layer("attention", ATTN, dict(kind="dense", ff=33), heads=3, kv_heads=3, dim=18,
                         vdim=34, conv=7)], width=44, vocab=37),
    # head size above 128, a group of more than 16 query heads, single-tap convolutions
    "wide": config([layer("attention", ATTN, None, heads=2, kv_heads=1, dim=160, vdim=136, conv=1),
                    layer("mamba2", MAMBA, None, heads=2, vdim=80, state=136, groups=2, conv=1),
                    layer("attention", ATTN, MLP, heads=20, kv_heads=1, dim=16, vdim=16),
                    layer("lightning", LIGHT, None, heads=1, dim=144, vdim=128, decay=[0.98])],
                   width=128),
    # the sizes of the fast kernels: 128-channel heads and states
    "fast": config([layer("mamba2", MAMBA, None, heads=4, vdim=64, state=128, groups=1),
                    layer("attention", ATTN, MLP, heads=8, kv_heads=2, dim=128, vdim=128, conv=4,
                          scale=0.09),
                    layer("lightning", LIGHT, None, heads=2, dim=128, vdim=128,
                          decay=[0.9, 0.999])], width=128),
}


def shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        out[p + "norm1"] = out[p + "norm1b"] = (d,)
        x = p + "mix."
        if L["type"] == "lightning":
            qk, vg = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({x + "q": (qk, d), x + "k": (qk, d), x + "v": (vg, d), x + "g": (vg, d),
                        x + "o": (d, vg), x + "norm": (vg,)})
        elif L["type"] == "mamba2":
            inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            c = inner + 2 * gn
            out.update({x + "in": (inner + c + m["heads"], d), x + "conv": (c, m["conv"]),
                        x + "conv.b": (c,), x + "dt_bias": (m["heads"],),
                        x + "A_log": (m["heads"],), x + "D": (m["heads"],), x + "norm": (inner,),
                        x + "o": (d, inner)})
        else:
            for n, h, s in (("q", "heads", "dim"), ("k", "kv_heads", "dim"),
                            ("v", "kv_heads", "vdim")):
                r = m[h] * m[s]
                out.update({x + n: (r, d), x + n + ".b": (r,), x + n + ".conv": (r, m["conv"])})
            out.update({x + "g": (m["heads"] * m["vdim"], d), x + "o": (d, m["heads"] * m["vdim"])})
        if L["mlp"]:
            f = L["mlp"]["ff"]
            out[p + "norm2"] = out[p + "norm2b"] = (d,)
            out.update({p + "mlp.gate": (f, d), p + "mlp.up": (f, d), p + "mlp.down": (d, f)})
    out.update({"final.norm": (d,), "head": (cfg["vocab"], d)})
    return out


def weights(cfg, seed=0):
    """bf16 weights under which every mechanism moves the logits: gains away
    from 1, biases and convolutions of order one, decays that neither vanish
    nor hold."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(s, generator=g)
        if leaf == "conv":
            t = t * 0.6 / math.sqrt(s[-1]) + 0.4 / s[-1]
        elif leaf == "norm" and ".mix." in name or leaf == "D":
            t = 1.0 + 0.3 * t
        elif leaf in ("norm1", "norm1b", "norm2", "norm2b", "norm"):
            t = 0.3 * t
        elif leaf == "dt_bias":
            t = t - 1.0
        elif leaf in ("A_log", "b"):
            t = 0.5 * t
        elif name != "embed":
            t = t / math.sqrt(s[-1])
        out[name] = t.to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
