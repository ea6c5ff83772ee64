"""Small Zovozen configurations and random weights of the tests."""
import math

import torch


def attention(heads=4, kv_heads=2, dim=24, vdim=40, chunk=37, dims=12, base=500.0, scale=0.3,
              factor=3.0):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=chunk),
                rot=dict(base=base, dims=dims, scaling=dict(factor=factor)), scale=scale)


def memory(heads=3, dim=24, vdim=40, cap=7.0):
    return dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap)


def dense(ff=72):
    return dict(kind="dense", ff=ff)


def moe(experts=7, identity=2, top=3, ff=40, shared=56, groups=3, keep=2):
    return dict(kind="moe", router=dict(experts=experts, identity=identity, top=top,
                                        groups=dict(count=groups, keep=keep)),
                expert=dict(ff=ff), shared=dict(ff=shared))


def par(mlp=None, left=None, right=None, scales=(0.7, 1.3)):
    return {"type": "parallel", "mlp": mlp,
            "mixer": dict(left=left or attention(), right=right or memory(),
                          left_scale=scales[0], right_scale=scales[1])}


def config(layers, width=64, vocab=61, eps=1e-5):
    return {"architecture": "Zovozen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": layers}


CASES = {
    "mixed": config([par(dense()), par(moe()), par(None), par(moe(6, 3, 2, groups=1, keep=1))]),
    # sizes no vector path covers; a chunk of one, one longer than the prompts; query
    # heads with a key head each; every group kept, no identity expert
    "odd": config([par(moe(5, 0, 5, 21, 13, 1, 1), attention(3, 3, 18, 10, 1, 6), memory(1, 7, 9)),
                   par(dense(33), attention(1, 1, 7, 5, 400, 2, factor=1.0), memory(3, 13, 6, 2.0)),
                   par(moe(8, 1, 2, 33, 40, 9, 3), attention(6, 2, 10, 70, 9, 10), memory(2, 5, 3))],
                  width=44, vocab=37, eps=1e-3),
    # more heads than one mixing step, head sizes above 128, memories beyond the
    # chunked kernels or of several column tiles
    "beyond": config([par(moe(40, 8, 6, groups=8, keep=3, shared=200),
                          attention(34, 2, 20, 72, 50, 8), memory(2, 264, 40)),
                      par(dense(200), attention(4, 2, 136, 140, 300, 136, base=1e4),
                          memory(2, 40, 200)),
                      par(None, attention(18, 1, 24, 24, 33, 24), memory(1, 136, 72))], width=128,
                     eps=1e-6),
    # the sizes of the fast kernels
    "fast": config([par(moe(6, 2, 2, 64, 128, 4, 2), attention(32, 8, 128, 128, 70, 64, 1e4, 0.08),
                        memory(4, 128, 128)),
                    par(dense(256), attention(8, 8, 64, 64, 130, 32, 1e4, 0.12), memory(2, 64, 64)),
                    par(None, attention(12, 2, 128, 64, 64, 128, 1e4, 0.09), memory(1, 128, 64)),
                    par(None, attention(16, 8, 64, 32, 95, 64, 1e4, 0.12), memory(2, 32, 128))],
                   width=128),
}


def shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"] = (d,)
        a, y = L["mixer"]["left"], p + "mix.left."
        H, G, n, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        for k, r in (("q", H * n), ("k", G * n), ("v", G * e)):
            out.update({y + k: (r, d), y + k + ".b": (r,)})
        out.update({y + "q.norm": (H * n,), y + "k.norm": (G * n,), y + "talk": (H, H),
                    y + "temp": (H,), y + "sink": (H,), y + "g": (H * e, d), y + "o": (d, H * e),
                    y + "o.b": (d,)})
        a, y = L["mixer"]["right"], p + "mix.right."
        H, n, e = a["heads"], a["dim"], a["vdim"]
        out.update({y + "q": (H * n, d), y + "k": (H * n, d), y + "v": (H * e, d),
                    y + "g": (H * e, d), y + "o": (d, H * e), y + "norm": (H * e,)})
        for k in "if":
            out.update({y + k: (H, d), y + k + ".b": (H,)})
        f, x = L["mlp"], p + "mlp."
        if not f:
            continue
        out[p + "norm2"] = (d,)
        if f["kind"] == "dense":
            out.update({x + "up": (f["ff"], d), x + "up.b": (f["ff"],), x + "down": (d, f["ff"]),
                        x + "down.b": (d,)})
            continue
        r = f["router"]
        ffs = {f"e{e}": f["expert"]["ff"] for e in range(r["experts"])}
        if f.get("shared"):
            ffs["shared"] = f["shared"]["ff"]
        for e, n in ffs.items():
            out.update({f"{x}{e}.gate": (n, d), f"{x}{e}.up": (n, d), f"{x}{e}.down": (d, n)})
        E = r["experts"] + r.get("identity", 0)
        out.update({x + "router": (E, d), x + "correction": (E,)})
    out["final.norm"] = (d,)
    return out


def weights(cfg, seed=0, calm=False):
    """bf16 weights under which every mechanism moves the logits: gains away
    from 1, mixed heads, sinks that weigh, corrections that outweigh scores,
    memories that neither vanish nor hold.  ``calm``: routers whose choices stay
    clear of ties (a choice that falls the other way in bf16 moves every later
    token), memories whose queries resemble the keys (the divisor n q of others
    nearly cancels now and then)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(s, generator=g)
        if leaf.startswith("norm"):
            t = 1.0 + 0.3 * t
        elif leaf == "temp":
            t = 1.2 + 0.4 * t
        elif leaf == "talk":
            t = torch.eye(s[0]) + 0.7 * t / math.sqrt(s[0])
        elif leaf == "sink":
            t = 1.0 + t
        elif leaf == "correction":
            t = 0.4 * t - 0.3
        elif leaf == "router" and calm:
            t = 0.03 * t / math.sqrt(s[-1])
        elif name.endswith("right.f.b"):
            t = 2.0 + t
        elif name.endswith("right.i.b"):
            t = 1.5 * t - 0.5
        elif leaf == "b":
            t = 0.5 * t
        elif name != "embed":
            t = 1.5 * t / math.sqrt(s[-1])
        out[name] = t.to(torch.bfloat16)
        if calm and name.endswith("right.k"):
            q = name[:-1] + "q"
            out[q] = (0.5 * out[q].float() + t).to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
