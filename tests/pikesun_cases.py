"""Small Pikesun configurations and random weights of the tests."""
import math

import torch

RG = dict(width=96, blocks=3, conv=4)
LA = dict(heads=4, dim=24, rot_dim=16, vdim=40, kv_rank=48, q_rank=56, scale=0.3,
          mask=dict(size=37), rot=dict(base=500.0, dims=16))
DENSE = dict(kind="dense", ff=72)


def latent(**over):
    m = {**LA, **over}
    m["rot"] = dict(base=m.pop("base", 500.0), dims=m["rot_dim"])
    m["mask"] = dict(size=m.pop("window", 37))
    return m


def moe(experts=6, top=2, ff=40, limit=1.5, shared=(56, 0.8)):
    return dict(kind="moe", router=dict(experts=experts, top=top),
                expert=dict(ff=ff, limit=limit),
                shared=dict(ff=shared[0], limit=shared[1]) if shared else None)


def rec(mlp=None, **over):
    return {"type": "rglru", "mixer": {**RG, **over}, "mlp": mlp}


def att(mlp=None, **over):
    return {"type": "latent_attention", "mixer": latent(**over), "mlp": mlp}


def config(layers, width=64, vocab=61, eps=1e-5, scale=3.0, mult=0.7):
    return {"architecture": "Pikesun", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "residual_mult": mult, "layers": layers}


def again(layers, i):
    """A layer that runs with layer i's weights."""
    return {**layers[i], "weights_of": i}


_MIXED = [rec(moe()), att(DENSE)]
_MIXED += [again(_MIXED, 0), att(moe(top=3)), again(_MIXED, 1)]
_WIDE = [att(moe(experts=40, top=6, shared=(200, 3.0)), heads=20, dim=100, rot_dim=64, vdim=72,
             kv_rank=200, q_rank=96, window=300, base=1e4),
         rec(None, width=100, blocks=1, conv=1),
         rec(moe(experts=3, top=3, ff=130, shared=(16, 0.5)), width=256, blocks=8, conv=2)]

CASES = {
    # both mixers and feed-forwards, shared weights, attention in two windows
    "mixed": config(_MIXED + [att(None, window=5, heads=2)]),
    # sizes no vector path covers; every expert used; no shared expert; a window of one
    "odd": config([rec(moe(experts=5, top=5, ff=21, shared=None), width=42, blocks=3, conv=6),
                   att(None, heads=3, dim=18, rot_dim=6, vdim=10, kv_rank=36, q_rank=20, window=9),
                   att(dict(kind="dense", ff=33), heads=1, dim=7, rot_dim=2, vdim=5, kv_rank=9,
                       q_rank=11, window=1),
                   rec(dict(kind="dense", ff=33), width=42, blocks=2, conv=3)],
                  width=44, vocab=37, eps=1e-3, mult=1.0),
    # more than 16 heads, a window longer than the prompts, single-tap convolution
    "wide": config(_WIDE, width=128, eps=1e-6, scale=0.5),
    # beyond the MFMA kernels: wide rotated parts, latents, heads and gate blocks
    "beyond": config([att(DENSE, heads=2, dim=136, rot_dim=66, vdim=140, kv_rank=520, q_rank=40,
                          window=20),
                      rec(None, width=520, blocks=1),
                      att(None, heads=2, dim=30, rot_dim=70, vdim=30, kv_rank=64, window=33)]),
    # the sizes of the fast kernels
    "fast": config([rec(moe(experts=8, top=2, ff=64, shared=(128, 2.0)), width=512, blocks=2),
                    att(moe(experts=8, top=2, ff=128, shared=(64, 2.0)), heads=16, dim=128,
                        rot_dim=64, vdim=128, kv_rank=512, q_rank=192, window=130, scale=0.1,
                        base=1e4)], width=128),
}


def shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        m, p = L["mixer"], f"l{i}."
        out[p + "norm1"] = (d,)
        x = p + "mix."
        if L["type"] == "rglru":
            w, n = m["width"], m["blocks"]
            for k in ("y", "x"):
                out.update({x + k: (w, d), x + k + ".b": (w,)})
            out.update({x + "conv": (w, m["conv"]), x + "conv.b": (w,), x + "lam": (w,),
                        x + "o": (d, w)})
            for k in ("ra", "ri"):
                out.update({x + k: (n, w // n, w // n), x + k + ".b": (n, w // n)})
        else:
            H, R = m["heads"], m["kv_rank"]
            out.update({x + "dq": (m["q_rank"], d), x + "dq.norm": (m["q_rank"],),
                        x + "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                        x + "dkv": (R + m["rot_dim"], d), x + "dkv.norm": (R,),
                        x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R),
                        x + "g": (H * m["vdim"], d), x + "o": (d, H * m["vdim"])})
        f = L["mlp"]
        if not f:
            continue
        out[p + "norm2"] = (d,)
        x = p + "mlp."
        if f["kind"] == "dense":
            out.update({x + "up": (f["ff"], d), x + "down": (d, f["ff"])})
            continue
        ffs = {f"e{e}": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        if f["shared"]:
            ffs["shared"] = f["shared"]["ff"]
        for e, n in ffs.items():
            out.update({f"{x}{e}.gate": (n, d), f"{x}{e}.up": (n, d), f"{x}{e}.down": (d, n)})
        out[x + "router"] = (f["router"]["experts"], d)
    out.update({"final.norm": (d,), "head": (cfg["vocab"], d)})
    return out


def weights(cfg, seed=0):
    """bf16 weights under which every mechanism moves the logits: gains away
    from 1, biases of order one, decays that neither vanish nor hold."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(s, generator=g)
        if leaf == "conv":
            t = t * 0.6 / math.sqrt(s[-1]) + 0.4 / s[-1]
        elif leaf.startswith("norm"):
            t = 1.0 + 0.3 * t
        elif leaf == "lam":
            t = 1.5 * t - 3.5
        elif leaf == "b":
            t = 0.5 * t
        elif leaf in ("ra", "ri"):
            t = 2.0 * t / math.sqrt(s[-1])
        elif name != "embed":
            t = t / math.sqrt(s[-1])
        out[name] = t.to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
