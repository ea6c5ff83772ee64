"""Small Refolix configurations and random weights of the tests."""
import math

import torch


def scaling(factor=3.0, original=48, fast=6.0, slow=0.5):
    return dict(factor=factor, original=original, fast=fast, slow=slow)


def attention(heads=4, kv_heads=2, dim=24, vdim=40, window=37, dims=12, base=500.0, scale=0.4,
              cap=3.0, scale_by=scaling()):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window),
                rot=dict(base=base, dims=dims, scaling=scale_by), scale=scale, softcap=cap)


def delta(heads=4, kv_heads=2, dim=24, vdim=40, conv=4):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def moe(experts=6, top=2, ff=40, shared=56, groups=3, keep=2):
    return dict(kind="moe", router=dict(experts=experts, top=top,
                                        groups=dict(count=groups, keep=keep)),
                expert=dict(ff=ff), shared=dict(ff=shared))


def ret(mlp=None, heads=3, dim=32, vdim=24, dims=16, base=300.0, decay=None):
    decay = decay or [1.0 - 2.0 ** (-1.0 - 1.7 * h) for h in range(heads)]
    return {"type": "retention", "mlp": mlp, "mixer": dict(
        heads=heads, dim=dim, vdim=vdim, decay=decay, rot=dict(base=base, dims=dims))}


def par(mlp=None, left=None, right=None):
    return {"type": "parallel", "mlp": mlp,
            "mixer": dict(left=left or attention(), right=right or delta())}


def config(layers, width=64, vocab=61, eps=1e-5, scale=3.0, alpha=1.7, logit_scale=0.7, cap=6.0):
    return {"architecture": "Refolix", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "postln_alpha": alpha, "logit_scale": logit_scale,
            "logit_softcap": cap, "layers": layers}


CASES = {
    "mixed": config([ret(moe()), par(moe(experts=8, top=3, groups=2, keep=1)),
                     ret(None, dims=32), par(None, attention(window=5, heads=2))]),
    # sizes no vector path covers; a single tap, a long convolution; every group
    # kept; a window of one; query heads with a key head each
    "odd": config([ret(moe(experts=5, top=5, ff=21, shared=13, groups=1, keep=1), heads=1, dim=10,
                       vdim=7, dims=6),
                   par(None, attention(3, 3, 18, 10, 9, 6),
                       delta(heads=3, kv_heads=1, dim=7, vdim=9, conv=1)),
                   par(moe(experts=9, top=2, ff=33, shared=40, groups=9, keep=3),
                       attention(1, 1, 7, 5, 1, 2, scale_by=None),
                       delta(heads=2, kv_heads=2, dim=13, vdim=6, conv=6))],
                  width=44, vocab=37, eps=1e-3),
    # more than 16 query heads per key head, head sizes above 128, a window
    # longer than the prompts, states beyond the chunked kernels
    "beyond": config([par(moe(experts=40, top=6, groups=8, keep=3, shared=200),
                          attention(20, 1, 100, 72, 300, 64, base=1e4, scale_by=scaling(1.0)),
                          delta(heads=2, kv_heads=1, dim=264, vdim=40, conv=2)),
                      ret(None, heads=2, dim=264, vdim=24, dims=264),
                      par(None, attention(4, 2, 136, 140, 50, 136, base=1e4),
                          delta(heads=2, kv_heads=2, dim=40, vdim=140, conv=3))], width=128,
                     eps=1e-6, scale=0.5),
    # the sizes of the fast kernels
    "fast": config([ret(moe(experts=8, top=2, ff=64, shared=128, groups=4, keep=2), heads=2,
                        dim=128, vdim=128, dims=128),
                    par(moe(experts=8, top=2, ff=128, shared=64, groups=2, keep=1),
                        attention(8, 2, 128, 128, 70, 64, base=1e4, scale=0.09, cap=5.0),
                        delta(heads=4, kv_heads=2, dim=128, vdim=128)),
                    par(None, attention(8, 8, 64, 64, 130, 32, base=1e4, scale=0.125),
                        delta(heads=2, kv_heads=1, dim=64, vdim=64))], width=128),
}


def shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        out.update({p + "norm1": (d,), p + "ls1": (d,)})
        x = p + "mix."
        if L["type"] == "retention":
            H, n, e = m["heads"], m["dim"], m["vdim"]
            out.update({x + "q": (H * n, d), x + "k": (H * n, d), x + "v": (H * e, d),
                        x + "g": (H * e, d), x + "o": (d, H * e)})
        else:
            a, y = m["left"], x + "left."
            H, G, n, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            out.update({y + "q": (H * n, d), y + "k": (G * n, d), y + "v": (G * e, d),
                        y + "q.norm": (n,), y + "k.norm": (n,), y + "o": (d, H * e),
                        y + "out": (d,)})
            a, y = m["right"], x + "right."
            H, G, n, e, taps = a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"]
            for k, c in (("q", G * n), ("k", G * n), ("v", H * e)):
                out.update({y + k: (c, d), y + k + ".conv": (c, taps)})
            out.update({y + "b": (H, d), y + "a": (H, d), y + "A_log": (H,), y + "dt_bias": (H,),
                        y + "norm": (e,), y + "g": (H * e, d), y + "o": (d, H * e),
                        y + "out": (d,)})
        f = L["mlp"]
        if not f:
            continue
        out.update({p + "norm2": (d,), p + "ls2": (d,)})
        x = p + "mlp."
        ffs = {f"e{e}": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        ffs["shared"] = f["shared"]["ff"]
        for e, n in ffs.items():
            out.update({f"{x}{e}.gate": (n, d), f"{x}{e}.up": (n, d), f"{x}{e}.down": (d, n)})
        E = f["router"]["experts"]
        out.update({x + "router": (E, d), x + "correction": (E,), x + "shared.sg": (1, d)})
    out.update({"final.norm": (d,), "head": (cfg["vocab"], d)})
    return out


def weights(cfg, seed=0, calm=False):
    """bf16 weights under which every mechanism moves the logits: gains away
    from 1, corrections that outweigh scores, decays that neither vanish nor
    hold.  ``calm``: routers whose choices stay clear of ties (a choice that
    falls the other way in bf16 moves every later token)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(s, generator=g)
        if leaf == "conv":
            t = t * 0.6 / math.sqrt(s[-1]) + 0.4 / s[-1]
        elif leaf.startswith("norm") or leaf in ("out", "ls1", "ls2"):
            t = 1.0 + 0.3 * t
        elif leaf == "correction":
            t = 0.4 * t - 0.3
        elif leaf == "router" and calm:
            t = 0.03 * t / math.sqrt(s[-1])
        elif leaf == "A_log":
            t = 0.5 * t
        elif leaf == "dt_bias":
            t = t - 3.0
        elif name != "embed":
            t = 1.5 * t / math.sqrt(s[-1])
        out[name] = t.to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
