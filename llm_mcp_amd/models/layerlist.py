"""Decoders whose configuration lists their layers one by one (Zegopel,
Pikesun, Refolix, Zovozen), in the in-process serving engine.

A layer is a token mixer (``models.mixers``) and, where it has one, a
feed-forward (``models.feedforward``), each between an optional norm before and
a norm after it around an fp32 residual stream:

    x += post1(mixer(pre1(x)));   x += post2(ff(pre2(x)))

The norm after a sublayer, the residual add and the norm before the next
sublayer (or the plain copy of the stream where there is none) are one kernel
(``ops.sandwich_norm``; a family that norms the sum itself has its own form,
``_join``), so a step is

  embedding + first norm -> per sublayer: input projection -> mixer kernels
  -> output projection -> sandwich norm -> ... -> LM head on the sampled rows

A family is a subclass: its mixers and feed-forwards by name, which norms a
sublayer has and what their stored weights mean; the configuration adds a scale
of the embedding and of what a sublayer adds.  A layer may run with another
layer's tensors (``weights_of``); what it keeps between steps is its own.

The mixers differ in what a sequence keeps between steps: attention layers use
the paged cache, every recurrent state and convolution tail lives in the
sequence's state slot.  Both come from the engine.
"""
from __future__ import annotations

import torch

from .. import ops
from ..ops import mixers as mixer_ops
from .llama import StepInputs, TPContext
from .mixers import init_std


def weight_source(layers: list, i: int) -> int:
    """The layer whose tensors layer i uses."""
    seen = set()
    while layers[i].get("weights_of") is not None:
        if i in seen or not 0 <= layers[i]["weights_of"] < len(layers):
            raise ValueError(f"layer {i}: bad weights_of")
        seen.add(i)
        i = layers[i]["weights_of"]
    return i


class LayerListModel:
    prefix_cache_ok = False       # a cached page does not bring the state behind it
    needs_plan = True             # the step's index arrays (``host_plan``)
    mixers: dict = {}             # layer "type" -> mixer class
    feedforwards: dict = {}       # mlp "kind" -> feed-forward class
    zero_centred = False          # stored gains act as 1 + w
    tail = "b"                    # suffix of the norm after a sublayer ("": no norm before it)
    tied_head = False             # the logits use the embedding table
    layer_scale = ""              # name of the per-channel scale of a sublayer's output, if any

    # ------------------------------------------------------------ layout ----
    @classmethod
    def layer_parts(cls, cfg) -> list:
        """[(mixer, feed-forward or None)] of every layer, unloaded; a layer
        that shares another's tensors shares its parts."""
        made: dict = {}
        for i, L in enumerate(cfg.layers):
            j = weight_source(cfg.layers, i)
            if j != i and any(L.get(k) != cfg.layers[j].get(k) for k in ("type", "mixer", "mlp")):
                raise ValueError(f"layer {i} does not match layer {j}, whose weights it uses")
            if j not in made:
                S, ff = cfg.layers[j], cfg.layers[j].get("mlp")
                made[j] = (cls.mixers[S["type"]](S["mixer"], cfg.hidden_size, cfg.rms_eps),
                           cls.feedforwards[ff["kind"]](ff, cfg.hidden_size) if ff else None)
        return [made[weight_source(cfg.layers, i)] for i in range(len(cfg.layers))]

    @classmethod
    def check_layers(cls, layers: list) -> None:
        for i, L in enumerate(layers):
            if L["type"] not in cls.mixers:
                raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
            if L.get("mlp") is not None and L["mlp"].get("kind") not in cls.feedforwards:
                raise ValueError(f"layer {i}: unknown feed-forward {L['mlp'].get('kind')!r}")

    @classmethod
    def sublayer_norms(cls, i: int, n: int) -> list:
        """Tensor names (before, after) of layer i's n sublayers; before is
        None where a sublayer reads the stream itself."""
        pre = bool(cls.tail)
        return [(f"l{i}.norm{k}" if pre else None, f"l{i}.norm{k}{cls.tail}")
                for k in range(1, n + 1)]

    @classmethod
    def tensor_shapes(cls, cfg) -> dict[str, tuple]:
        """Checkpoint tensor names and shapes."""
        d = cfg.hidden_size
        out = {"embed": (cfg.vocab_size, d)}
        for i, (mix, ff) in enumerate(cls.layer_parts(cfg)):
            if weight_source(cfg.layers, i) != i:
                continue
            for names in cls.sublayer_norms(i, 1 if ff is None else 2):
                out.update({n: (d,) for n in names if n})
            if cls.layer_scale:
                out.update({f"l{i}.{cls.layer_scale}{k}": (d,)
                            for k in range(1, 2 if ff is None else 3)})
            out.update({f"l{i}.mix.{k}": s for k, s in mix.shapes.items()})
            if ff is not None:
                out.update({f"l{i}.mlp.{k}": s for k, s in ff.shapes.items()})
        out["final.norm"] = (d,)
        if not cls.tied_head:
            out["head"] = (cfg.vocab_size, d)
        return out

    def __init__(self, cfg, device: torch.device | str = "cuda", dtype=torch.bfloat16,
                 tp: TPContext | None = None, seed: int = 0, weights: dict | None = None):
        """``weights``: checkpoint tensors by name (``weights.load_weights``);
        None: random."""
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp = tp or TPContext()
        if self.tp.size > 1:
            raise ValueError(f"{cfg.family}: no tensor-parallel form")
        if not cfg.layers:
            raise ValueError(f"{cfg.family}: no layers")
        self.vocab_shard = cfg.vocab_size
        self.parts = self.layer_parts(cfg)
        kv = [m for m, _ in self.parts if m.kv is not None]
        # the engine's decode workspace covers the largest attention layer
        self.Hq = max((m.Hq for m in kv), default=1)
        self.Hkv = min((m.Hkv for m in kv), default=1)
        self.D = max((m.D for m in kv), default=64)
        self.q_per_tile = next((m.q_per_tile for m in kv if m.q_per_tile), 16)
        self._plans = {}                       # key -> the part that builds that plan
        mixing = [p for m, _ in self.parts for p in m.members()]
        for m in mixing:
            if m.plan_key is not None:
                self._plans.setdefault(m.plan_key, m)
        self._angles = sorted({m.rot for m in mixing if m.rot is not None})
        self._load(weights, seed)

    # ----------------------------------------------------------- weights ----
    def _load(self, weights: dict | None, seed: int) -> None:
        cfg = self.cfg
        shapes = self.tensor_shapes(cfg)
        rnd = None
        if weights is None:
            rnd = torch.Generator(device=self.device)
            rnd.manual_seed(seed)

        def get(name: str) -> torch.Tensor:
            if weights is not None:
                return weights[name]
            mean, std = init_std(name, shapes[name], len(cfg.layers), self.zero_centred)
            t = torch.empty(shapes[name], dtype=torch.bfloat16, device=self.device)
            return t.normal_(mean, std, generator=rnd)

        def put(t: torch.Tensor, fp32: bool = False) -> torch.Tensor:
            return t.to(device=self.device, dtype=torch.float32 if fp32 else self.dtype) \
                .contiguous()

        def gain(name: str | None, scale: float = 1.0) -> torch.Tensor | None:
            if name is None:
                return None
            w = get(name).float()
            return put(scale * (1.0 + w if self.zero_centred else w), fp32=True)

        self.embed = put(get("embed"))
        source = [weight_source(cfg.layers, i) for i in range(len(cfg.layers))]
        norms = {}                             # (before, after) of each sublayer
        for i in sorted(set(source)):
            mix, ff = self.parts[i]
            mix.load(lambda n, p=f"l{i}.mix.": get(p + n), put)
            if ff is not None:
                ff.load(lambda n, p=f"l{i}.mlp.": get(p + n), put)
            norms[i] = [(gain(a), gain(b, cfg.residual_mult))
                        for a, b in self.sublayer_norms(i, 1 if ff is None else 2)]
            if self.layer_scale:       # after: (norm, scale)
                norms[i] = [(a, (b, put(get(f"l{i}.{self.layer_scale}{k + 1}"), fp32=True)))
                            for k, (a, b) in enumerate(norms[i])]
        self.norms = [norms[j] for j in source]
        self.final_norm = gain("final.norm")
        self.head = self.embed if self.tied_head else put(get("head"))
        self._freqs = {r: ops.rope_freqs(*r, device=self.device) for r in self._angles}

    def weight_bytes(self, copies: bool = False) -> int:
        """Bytes of the served weights (padding included)."""
        ts = [self.embed, self.head, self.final_norm]
        ts += [t for ns in self.norms for pair in ns for p in pair
               for t in (p if isinstance(p, tuple) else (p,)) if t is not None]
        for o in (o for m, ff in self.parts for o in (m, *m.members(), ff) if o is not None):
            vals = [v.data if isinstance(v, ops.GroupedWeight) else
                    v.mix if isinstance(v, ops.Talk) else v for v in vars(o).values()]
            ts += [t for t in vals if isinstance(t, torch.Tensor)]
        return sum({t.data_ptr(): t.numel() * t.element_size() for t in ts}.values())

    # ------------------------------------------------- caches, host plan ----
    @property
    def kv_layers(self) -> list:
        return [m.kv for m, _ in self.parts if m.kv is not None]

    def state_shapes(self) -> list:
        return [s for m, _ in self.parts for s in m.state_shapes(self.dtype)]

    def host_plan(self, plan: dict) -> tuple[list, dict]:
        """Index arrays of an eager step: convolution tiles over every
        sequence, and what the mixers plan for the multi-token ones (scan
        segments, attention tiles, key rows)."""
        nd = plan["num_decode"]
        cu = plan["cu_q"]
        S = len(cu) - 1
        if nd == S:
            return [], {}
        qlens = (cu[1:] - cu[:-1])[nd:]
        ctx = plan["context_lens"][nd:]
        items = [("conv", mixer_ops.conv_tiles(cu))]
        host = {}
        for key, m in self._plans.items():
            more, host[key] = m.build_plan(qlens, ctx, nd)
            items += [x for x in more if x[0] not in {name for name, _ in items}]
        return items, host

    def bind_plan(self, dev: dict, host: dict) -> dict:
        """``StepInputs.aux`` from the uploaded ``host_plan`` arrays."""
        aux = {"conv": dev["conv"]} if "conv" in dev else {}
        for key, h in host.items():
            aux[key] = self._plans[key].bind_plan(dev, h)
        return aux

    # ----------------------------------------------------------- forward ----
    def _join(self, x, y, post, pre, rows=None):
        """Take a sublayer's output y into the residual x (``post``: what
        belongs to the norm after it) and return the rows the next one reads."""
        return ops.sandwich_norm(x, self.cfg.rms_eps, y=y, w_post=post, w_pre=pre, rows=rows,
                                 dtype=self.dtype)

    def _logits(self, h):
        return ops.linear(h, self.head)

    def forward(self, inp: StepInputs, k_caches: list, v_caches: list, decode_ws=None,
                part_tokens: int = 512, layers_out: list | None = None) -> torch.Tensor:
        """Logits [len(sample_rows), vocab].  ``layers_out``: receives a copy of
        the residual after every layer (debugging)."""
        eps, dt = self.cfg.rms_eps, self.dtype
        inp.decode_ws, inp.part_tokens = decode_ws, part_tokens
        inp.aux = dict(inp.aux or {})
        for r in self._angles:
            inp.aux["rot", r] = ops.rope_angles(inp.positions, self._freqs[r],
                                                ops.rope_magnitude(*r))
        T = inp.num_tokens
        x = torch.empty((T, self.cfg.hidden_size), dtype=torch.float32, device=self.device)
        h = ops.sandwich_norm(x, eps, w_pre=self.norms[0][0][0], ids=inp.input_ids,
                              table=self.embed, scale=self.cfg.embed_scale, dtype=dt)
        kv = iter(zip(k_caches, v_caches))
        states = iter(inp.states or [])
        all_rows = inp.sample_rows.numel() == T
        for i, ((mix, ff), n) in enumerate(zip(self.parts, self.norms)):
            state = [next(states) for _ in mix.state_shapes(dt)]
            y = mix.forward(h, inp, next(kv) if mix.kv is not None else None, state)
            last = i + 1 == len(self.parts)
            if ff is not None:
                h = self._join(x, y, n[0][1], n[1][0])
                y = ff.forward(h)
            post = n[-1][1]
            if not last:
                h = self._join(x, y, post, self.norms[i + 1][0][0])
            elif layers_out is None:
                # the final norm on the sampled rows only
                h = self._join(x, y, post, self.final_norm,
                               None if all_rows else inp.sample_rows)
            else:
                self._join(x, y, post, None)
                h = self._join(x, None, None, self.final_norm, inp.sample_rows)
            if layers_out is not None:
                layers_out.append(x.clone())
        return self._logits(h)
