"""Zegopel decoder for the in-process serving engine.

A layer is a token mixer and, where the layer has one, a ReLU-gated
feed-forward, each between two norms around an fp32 residual stream:

    x += norm1b(mixer(norm1(x)));   x += norm2b(ff(norm2(x)))

(RMS norms whose weight w acts as 1 + w).  The norm after a sublayer, the
residual add and the norm before the next sublayer are one kernel
(``ops.sandwich_norm``), so a step is

  embedding + first norm -> per sublayer: input projection -> mixer kernels
  -> output projection -> sandwich norm -> ... -> LM head on the sampled rows

The mixers (``models.mixers``) differ in what a sequence keeps between steps:
attention layers use the paged KV cache, every recurrent state and convolution
tail lives in the sequence's state slot.  Both come from the engine.
"""
from __future__ import annotations

import torch

from .. import ops
from ..ops import mixers as mixer_ops
from .config import ZegopelConfig
from .llama import StepInputs, TPContext
from .mixers import MIXERS, ReluGLU, init_std


def _layer_parts(cfg: ZegopelConfig) -> list:
    """[(mixer, feed-forward or None)] of every layer, unloaded."""
    return [(MIXERS[L["type"]](L["mixer"], cfg.hidden_size, cfg.rms_eps),
             ReluGLU(L["mlp"], cfg.hidden_size) if L.get("mlp") else None) for L in cfg.layers]


def tensor_shapes(cfg: ZegopelConfig) -> dict[str, tuple]:
    """Checkpoint tensor names and shapes."""
    d = cfg.hidden_size
    out = {"embed": (cfg.vocab_size, d)}
    for i, (mix, ff) in enumerate(_layer_parts(cfg)):
        out.update({f"l{i}.norm1": (d,), f"l{i}.norm1b": (d,)})
        out.update({f"l{i}.mix.{k}": s for k, s in mix.shapes.items()})
        if ff is not None:
            out.update({f"l{i}.norm2": (d,), f"l{i}.norm2b": (d,)})
            out.update({f"l{i}.mlp.{k}": s for k, s in ff.shapes.items()})
    out.update({"final.norm": (d,), "head": (cfg.vocab_size, d)})
    return out


class ZegopelModel:
    layer_parts = staticmethod(_layer_parts)
    prefix_cache_ok = False       # a cached page does not bring the state behind it

    def __init__(self, cfg: ZegopelConfig, device: torch.device | str = "cuda",
                 dtype=torch.bfloat16, tp: TPContext | None = None, seed: int = 0,
                 weights: dict | None = None):
        """``weights``: checkpoint tensors by name (``weights.load_weights``);
        None: random."""
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp = tp or TPContext()
        if self.tp.size > 1:
            raise ValueError("zegopel: no tensor-parallel form")
        if not cfg.layers:
            raise ValueError("zegopel: no layers")
        self.vocab_shard = cfg.vocab_size
        self.parts = _layer_parts(cfg)
        kv = [m for m, _ in self.parts if m.kv is not None]
        # the engine's decode workspace covers the largest attention layer
        self.Hq = max((m.Hq for m in kv), default=1)
        self.Hkv = min((m.Hkv for m in kv), default=1)
        self.D = max((m.D for m in kv), default=64)
        self.q_per_tile = next((m.q_per_tile for m in kv if m.q_per_tile), 16)
        self._attn_tiles = sorted({m.q_per_tile for m in kv if m.q_per_tile})
        self._scans = sorted({m.scan_geometry for m, _ in self.parts if m.scan_geometry})
        self._load(weights, seed)

    # ----------------------------------------------------------- weights ----
    def _load(self, weights: dict | None, seed: int) -> None:
        shapes = tensor_shapes(self.cfg)
        rnd = None
        if weights is None:
            rnd = torch.Generator(device=self.device)
            rnd.manual_seed(seed)

        def get(name: str) -> torch.Tensor:
            if weights is not None:
                return weights[name]
            mean, std = init_std(name, shapes[name], len(self.cfg.layers))
            t = torch.empty(shapes[name], dtype=torch.bfloat16, device=self.device)
            return t.normal_(mean, std, generator=rnd)

        def put(t: torch.Tensor, fp32: bool = False) -> torch.Tensor:
            return t.to(device=self.device, dtype=torch.float32 if fp32 else self.dtype) \
                .contiguous()

        def gain(name: str) -> torch.Tensor:      # stored around zero
            return put(1.0 + get(name).float(), fp32=True)

        self.embed = put(get("embed"))
        self.norms = []                           # per layer: norm1, norm1b[, norm2, norm2b]
        for i, (mix, ff) in enumerate(self.parts):
            mix.load(lambda n, p=f"l{i}.mix.": get(p + n), put)
            names = ["norm1", "norm1b"]
            if ff is not None:
                ff.load(lambda n, p=f"l{i}.mlp.": get(p + n), put)
                names += ["norm2", "norm2b"]
            self.norms.append([gain(f"l{i}.{n}") for n in names])
        self.final_norm = gain("final.norm")
        self.head = put(get("head"))

    def weight_bytes(self, copies: bool = False) -> int:
        """Bytes of the served weights (padding included)."""
        ts = [self.embed, self.head, self.final_norm] + [n for ns in self.norms for n in ns]
        for mix, ff in self.parts:
            for o in (mix, ff):
                ts += [t for t in vars(o).values() if isinstance(t, torch.Tensor)] if o else []
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------- caches, host plan ----
    @property
    def kv_layers(self) -> list:
        return [m.kv for m, _ in self.parts if m.kv is not None]

    def state_shapes(self) -> list:
        return [s for m, _ in self.parts for s in m.state_shapes(self.dtype)]

    def host_plan(self, plan: dict) -> tuple[list, dict]:
        """Index arrays of an eager step: convolution tiles over every
        sequence, scan segments and per-geometry attention tiles over the
        multi-token ones."""
        nd = plan["num_decode"]
        cu = plan["cu_q"]
        S = len(cu) - 1
        if nd == S:
            return [], {}
        qlens = (cu[1:] - cu[:-1])[nd:]
        items = [("conv", mixer_ops.conv_tiles(cu))]
        host = {}
        for H, P in self._scans:
            segs, first, one = mixer_ops.scan_segments(qlens, nd, H, P)
            items += [(f"segs{H, P}", segs), (f"first{H, P}", first)]
            host[f"scan{H, P}"] = (len(segs), one)
        for q in self._attn_tiles:
            items.append((f"attn{q}", mixer_ops.row_tiles(qlens, q).reshape(-1)))
        return items, host

    def bind_plan(self, dev: dict, host: dict) -> dict:
        """``StepInputs.aux`` from the uploaded ``host_plan`` arrays."""
        aux = {k: dev[k] for k in dev if k == "conv" or k.startswith("attn")}
        for H, P in self._scans:
            if f"scan{H, P}" in host:
                n, one = host[f"scan{H, P}"]
                aux[f"scan{H, P}"] = ops.ScanSegments(dev[f"segs{H, P}"], dev[f"first{H, P}"], n,
                                                      one)
        return aux

    # ----------------------------------------------------------- forward ----
    def forward(self, inp: StepInputs, k_caches: list, v_caches: list, decode_ws=None,
                part_tokens: int = 512, layers_out: list | None = None) -> torch.Tensor:
        """Logits [len(sample_rows), vocab].  ``layers_out``: receives a copy of
        the residual after every layer (debugging)."""
        eps, dt = self.cfg.rms_eps, self.dtype
        inp.decode_ws, inp.part_tokens = decode_ws, part_tokens
        if inp.aux is None:
            inp.aux = {}
        T = inp.num_tokens
        x = torch.empty((T, self.cfg.hidden_size), dtype=torch.float32, device=self.device)
        h = ops.sandwich_norm(x, eps, w_pre=self.norms[0][0], ids=inp.input_ids,
                              table=self.embed, dtype=dt)
        kv = iter(zip(k_caches, v_caches))
        states = iter(inp.states or [])
        all_rows = inp.sample_rows.numel() == T
        for i, ((mix, ff), n) in enumerate(zip(self.parts, self.norms)):
            state = [next(states) for _ in mix.state_shapes(dt)]
            y = mix.forward(h, inp, next(kv) if mix.kv is not None else None, state)
            last = i + 1 == len(self.parts)
            if ff is not None:
                h = ops.sandwich_norm(x, eps, y=y, w_post=n[1], w_pre=n[2], dtype=dt)
                y = ff.forward(h)
            post = n[3] if ff is not None else n[1]
            if not last:
                h = ops.sandwich_norm(x, eps, y=y, w_post=post, w_pre=self.norms[i + 1][0],
                                      dtype=dt)
            elif layers_out is None:
                # the final norm on the sampled rows only
                h = ops.sandwich_norm(x, eps, y=y, w_post=post, w_pre=self.final_norm,
                                      rows=None if all_rows else inp.sample_rows, dtype=dt)
            else:
                ops.sandwich_norm(x, eps, y=y, w_post=post, dtype=dt)
                h = ops.sandwich_norm(x, eps, w_pre=self.final_norm, rows=inp.sample_rows,
                                      dtype=dt)
            if layers_out is not None:
                layers_out.append(x.clone())
        return ops.linear(h, self.head)
