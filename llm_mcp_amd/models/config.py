"""Model architecture configs (public HF config.json values) and the local
model registry entries derived from them.

The reference infers tier / thinking / context / kind from model *names*
(core/internal/discovery/discovery.go:482-649).  Here they are derived from the
architecture itself (`params_b`, `context_k`, `kind`), and the name heuristics
are kept only for foreign names (policy/inference.py)."""
from __future__ import annotations

import json
import math
from dataclasses import asdict, dataclass, field
from pathlib import Path


@dataclass
class LlamaConfig:
    name: str = "llama-3-8b"
    vocab_size: int = 128256
    hidden_size: int = 4096
    intermediate_size: int = 14336
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    rope_theta: float = 500000.0
    rope_scaling: dict | None = None
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    bos_token_id: int = 128000
    eos_token_ids: tuple = (128001, 128009)
    family: str = "llama"
    kind: str = "chat"
    qkv_bias: bool = False          # Qwen2 / Qwen2.5: biased q/k/v projections
    qk_norm: bool = False           # Qwen3: per-head RMSNorm of q and k before RoPE
    # > 1: a one-GPU stand-in for ONE rank of a TP group of this size (the
    # preset's shapes are already the per-rank shard): the O / down GEMMs
    # produce bf16 as a TP rank does before its all-reduce (no split-K
    # partials handed to the norm, no residual epilogue), so the proxy runs
    # exactly the rank's kernels; the all-reduces themselves are not run
    proxy_tp: int = 0

    @property
    def params(self) -> int:
        d, I, L, V = self.hidden_size, self.intermediate_size, self.num_layers, self.vocab_size
        qkv = d * (self.num_heads + 2 * self.num_kv_heads) * self.head_dim
        if self.qkv_bias:
            qkv += (self.num_heads + 2 * self.num_kv_heads) * self.head_dim
        o = self.num_heads * self.head_dim * d
        mlp = 3 * d * I
        emb = V * d * (1 if self.tie_embeddings else 2)
        qkn = 2 * self.head_dim if self.qk_norm else 0
        return L * (qkv + o + mlp + 2 * d + qkn) + emb + d

    @property
    def params_b(self) -> float:
        return round(self.params / 1e9, 2)

    @property
    def context_k(self) -> int:
        return self.max_position // 1024

    def kv_bytes_per_token(self, tp: int = 1, dtype_bytes: int = 2) -> int:
        kvh = max(1, self.num_kv_heads // tp)
        return self.num_layers * 2 * kvh * self.head_dim * dtype_bytes

    def to_dict(self) -> dict:
        return asdict(self)


@dataclass
class NomicBertConfig:
    """nomic-embed-text(-v1.5): post-norm BERT with rotary, SwiGLU, mean pool."""
    name: str = "nomic-embed-text"
    vocab_size: int = 30528
    hidden_size: int = 768
    intermediate_size: int = 3072
    num_layers: int = 12
    num_heads: int = 12
    head_dim: int = 64
    rope_theta: float = 1000.0
    ln_eps: float = 1e-12
    max_position: int = 8192
    type_vocab_size: int = 2
    qkv_bias: bool = False
    mlp_bias: bool = False
    family: str = "nomic-bert"
    kind: str = "embed"
    embed_dim: int = 768

    @property
    def params(self) -> int:
        d, I, L = self.hidden_size, self.intermediate_size, self.num_layers
        return L * (4 * d * d + 3 * d * I + 4 * d) + (self.vocab_size + self.type_vocab_size) * d

    @property
    def params_b(self) -> float:
        return round(self.params / 1e9, 3)

    @property
    def context_k(self) -> int:
        return self.max_position // 1024

    def to_dict(self) -> dict:
        return asdict(self)


@dataclass
class BertConfig:
    """Classic BERT encoder (absolute positions, post-norm, exact-GELU FFN with
    biases); ``pooling`` = "cls" (mxbai / bge / arctic) or "mean"."""
    name: str = "mxbai-embed-large"
    vocab_size: int = 30522
    hidden_size: int = 1024
    intermediate_size: int = 4096
    num_layers: int = 24
    num_heads: int = 16
    head_dim: int = 64
    ln_eps: float = 1e-12
    max_position: int = 512
    type_vocab_size: int = 2
    pooling: str = "cls"
    family: str = "bert"
    kind: str = "embed"
    embed_dim: int = 1024

    @property
    def params(self) -> int:
        d, I, L = self.hidden_size, self.intermediate_size, self.num_layers
        return (L * (4 * d * d + 2 * d * I + 9 * d + I)
                + (self.vocab_size + self.max_position + self.type_vocab_size + 2) * d)

    @property
    def params_b(self) -> float:
        return round(self.params / 1e9, 3)

    @property
    def context_k(self) -> int:
        return max(1, self.max_position // 1024)

    def to_dict(self) -> dict:
        return asdict(self)


@dataclass
class LayerListConfig:
    """A decoder whose layers each name their own token mixer and feed-forward,
    with their own sizes.  ``layers`` holds one dict per layer, as in the
    checkpoint's config.json: ``{"type": ..., "mixer": {sizes and constants},
    "mlp": {"kind", ...} | None, "weights_of": layer (optional)}``."""
    name: str = ""
    vocab_size: int = 512
    hidden_size: int = 256
    layers: list = field(default_factory=list)
    rms_eps: float = 1e-5
    # no table bounds the positions
    max_position: int = 1 << 20
    bos_token_id: int | None = None
    eos_token_ids: tuple = ()
    family: str = ""
    kind: str = "chat"
    architecture: str = ""          # config.json's name of the family
    embed_scale: float = 1.0        # the embedding's rows are multiplied by it
    residual_mult: float = 1.0      # and so is what a sublayer adds

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def params(self) -> int:
        from .registry import model_class
        return sum(math.prod(s) for s in model_class(self).tensor_shapes(self).values())

    @property
    def params_b(self) -> float:
        return round(self.params / 1e9, 3)

    @property
    def context_k(self) -> int:
        return self.max_position // 1024

    def to_dict(self) -> dict:
        return asdict(self)

    def to_json(self) -> dict:
        """The checkpoint's config.json."""
        js = {"architecture": self.architecture, "layers": self.layers,
              "norm": {"eps": self.rms_eps}, "vocab": self.vocab_size, "width": self.hidden_size}
        if self.eos_token_ids:
            js["eos_token_id"] = list(self.eos_token_ids)
        if self.bos_token_id is not None:
            js["bos_token_id"] = self.bos_token_id
        return js

    @classmethod
    def from_json(cls, js: dict, name: str):
        from .registry import layer_list_class
        layer_list_class(cls.family).check_layers(js["layers"])
        eos = js.get("eos_token_id", ())
        return cls(name=name, vocab_size=js["vocab"], hidden_size=js["width"],
                   layers=js["layers"], rms_eps=js["norm"]["eps"],
                   bos_token_id=js.get("bos_token_id"),
                   eos_token_ids=tuple(eos) if isinstance(eos, (list, tuple)) else (eos,))


@dataclass
class ZegopelConfig(LayerListConfig):
    """``lightning`` linear attention, ``mamba2`` state-space and ``attention``
    with short convolutions."""
    name: str = "zegopel"
    family: str = "zegopel"
    architecture: str = "Zegopel"


@dataclass
class PikesunConfig(LayerListConfig):
    """``rglru`` gated linear recurrences and ``latent_attention``, dense and
    ``moe`` feed-forwards."""
    name: str = "pikesun"
    family: str = "pikesun"
    architecture: str = "Pikesun"

    def to_json(self) -> dict:
        return {**super().to_json(), "embedding": {"scale": self.embed_scale},
                "residual_mult": self.residual_mult}

    @classmethod
    def from_json(cls, js: dict, name: str):
        cfg = super().from_json(js, name)
        cfg.embed_scale = float(js.get("embedding", {}).get("scale", 1.0))
        cfg.residual_mult = float(js.get("residual_mult", 1.0))
        return cfg


@dataclass
class RefolixConfig(LayerListConfig):
    """``retention`` and ``parallel`` (windowed attention beside a gated delta
    rule) mixers, ``moe`` feed-forwards, the norm after the sum."""
    name: str = "refolix"
    family: str = "refolix"
    architecture: str = "Refolix"
    postln_alpha: float = 1.0       # the residual's weight in the sum that is normed
    logit_scale: float = 1.0
    logit_softcap: float | None = None

    def to_json(self) -> dict:
        return {**super().to_json(), "embedding": {"scale": self.embed_scale},
                "postln_alpha": self.postln_alpha, "logit_scale": self.logit_scale,
                "logit_softcap": self.logit_softcap}

    @classmethod
    def from_json(cls, js: dict, name: str):
        cfg = super().from_json(js, name)
        cfg.embed_scale = float(js.get("embedding", {}).get("scale", 1.0))
        cfg.postln_alpha = float(js.get("postln_alpha", 1.0))
        cfg.logit_scale = float(js.get("logit_scale", 1.0))
        cap = js.get("logit_softcap")
        cfg.logit_softcap = float(cap) if cap is not None else None
        return cfg


@dataclass
class ZovozenConfig(LayerListConfig):
    """``parallel`` mixers (attention with talking heads in chunks beside a
    matrix memory), ``dense`` and ``moe`` feed-forwards, the head tied to the
    embedding."""
    name: str = "zovozen"
    family: str = "zovozen"
    architecture: str = "Zovozen"


LAYER_LISTS = {c.architecture: c for c in (ZegopelConfig, PikesunConfig, RefolixConfig,
                                           ZovozenConfig)}


def zegopel_stack(pattern: str, ff: int, lightning: dict, mamba2: dict,
                  attention: dict) -> list:
    """Layer list from a pattern of L (lightning), M (mamba2), A (attention):
    attention layers carry the feed-forward."""
    kinds = {"L": ("lightning", lightning), "M": ("mamba2", mamba2), "A": ("attention", attention)}
    return [{"type": kinds[c][0], "mixer": dict(kinds[c][1]),
             "mlp": {"kind": "dense", "ff": ff} if c == "A" else None} for c in pattern]


def _slopes(heads: int) -> list:
    """Per-head decays exp(-2^(-8 (h + 1) / heads)): from fast to slow."""
    return [math.exp(-2.0 ** (-8.0 * (h + 1) / heads)) for h in range(heads)]


def _zegopel_tiny() -> ZegopelConfig:
    return ZegopelConfig(
        name="tiny-zegopel", vocab_size=512, hidden_size=192, bos_token_id=506,
        eos_token_ids=(510,), layers=zegopel_stack(
            "LMALA", 256,
            dict(heads=3, dim=32, vdim=48, decay=[0.5, 0.9, 0.995]),
            dict(heads=6, vdim=32, state=40, groups=3, conv=4, norm_groups=2),
            dict(heads=4, kv_heads=2, dim=64, vdim=64, conv=3, scale=0.125,
                 q_temp=dict(coef=0.3, every=64))))


def _zegopel_8b() -> ZegopelConfig:
    """Llama-3-8B's width, head layout and size (random weights: benchmarks)."""
    return ZegopelConfig(
        name="zegopel-8b", vocab_size=128256, hidden_size=4096, bos_token_id=128000,
        eos_token_ids=(128001, 128009), layers=zegopel_stack(
            "LMA" * 16, 14336,
            dict(heads=32, dim=128, vdim=128, decay=_slopes(32)),
            dict(heads=64, vdim=128, state=128, groups=8, conv=4, norm_groups=8),
            dict(heads=32, kv_heads=8, dim=128, vdim=128, conv=4, scale=128 ** -0.5,
                 q_temp=dict(coef=0.1, every=8192))))


def pikesun_stack(pattern: str, rglru: dict, latent: dict, dense: dict, moe: dict) -> list:
    """Layer list from a pattern of R (rglru), A (latent attention): the first
    layer's feed-forward is dense, the others' mixtures of experts."""
    kinds = {"R": ("rglru", rglru), "A": ("latent_attention", latent)}
    return [{"type": kinds[c][0], "mixer": dict(kinds[c][1]),
             "mlp": dict(moe if i else dense)} for i, c in enumerate(pattern)]


def _latent(heads: int, dim: int, rot: int, vdim: int, rank: int, q_rank: int, window: int,
            base: float = 10000.0) -> dict:
    return dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank, q_rank=q_rank,
                scale=(dim + rot) ** -0.5, mask=dict(size=window), rot=dict(base=base, dims=rot))


def _moe(experts: int, top: int, ff: int, shared: int, limit: float = 7.0) -> dict:
    return dict(kind="moe", router=dict(experts=experts, top=top),
                expert=dict(ff=ff, limit=limit), shared=dict(ff=shared, limit=limit))


def _pikesun_tiny() -> PikesunConfig:
    layers = pikesun_stack("RARA", dict(width=192, blocks=3, conv=4),
                           _latent(4, 48, 32, 40, 96, 64, 70), dict(kind="dense", ff=256),
                           _moe(8, 2, 64, 96))
    return PikesunConfig(name="tiny-pikesun", vocab_size=512, hidden_size=192, bos_token_id=506,
                         eos_token_ids=(510,), layers=layers, embed_scale=192 ** 0.5,
                         residual_mult=0.5)


def _pikesun_8b() -> PikesunConfig:
    """Llama-3-8B's width and size, all experts counted (random weights:
    benchmarks)."""
    layers = pikesun_stack("RRA" * 8, dict(width=4096, blocks=16, conv=4),
                           _latent(32, 128, 64, 128, 512, 1536, 2048),
                           dict(kind="dense", ff=14336), _moe(16, 4, 1024, 2048))
    return PikesunConfig(name="pikesun-8b", vocab_size=128256, hidden_size=4096,
                         bos_token_id=128000, eos_token_ids=(128001, 128009), layers=layers,
                         embed_scale=64.0, residual_mult=0.5)


def refolix_stack(pattern: str, retention: dict, parallel: dict, moe: dict) -> list:
    """Layer list from a pattern of R (retention), P (parallel)."""
    kinds = {"R": ("retention", retention), "P": ("parallel", parallel)}
    return [{"type": kinds[c][0], "mixer": dict(kinds[c][1]), "mlp": dict(moe)} for c in pattern]


def _grouped_moe(experts: int, top: int, ff: int, shared: int, groups: int, keep: int) -> dict:
    return dict(kind="moe", router=dict(experts=experts, top=top,
                                        groups=dict(count=groups, keep=keep)),
                expert=dict(ff=ff), shared=dict(ff=shared))


def _refolix_tiny() -> RefolixConfig:
    left = dict(heads=4, kv_heads=2, dim=64, vdim=48, scale=0.125, softcap=30.0,
                mask=dict(size=70), rot=dict(base=10000.0, dims=32, scaling=dict(
                    factor=4.0, original=256, fast=32.0, slow=1.0)))
    layers = refolix_stack(
        "RPR", dict(heads=3, dim=32, vdim=56, decay=_retention_decays(3),
                    rot=dict(base=10000.0, dims=32)),
        dict(left=left, right=dict(heads=4, kv_heads=2, dim=48, vdim=40, conv=4)),
        _grouped_moe(8, 2, 64, 96, 4, 2))
    return RefolixConfig(name="tiny-refolix", vocab_size=512, hidden_size=192, bos_token_id=506,
                         eos_token_ids=(510,), layers=layers, embed_scale=192 ** 0.5,
                         postln_alpha=2.0, logit_scale=0.5, logit_softcap=30.0)


def _retention_decays(heads: int) -> list:
    """Per-head decays 1 - 2^(-5 - 7 h / heads): from fast to slow."""
    return [1.0 - 2.0 ** (-5.0 - 7.0 * h / heads) for h in range(heads)]


def _refolix_8b() -> RefolixConfig:
    """Llama-3-8B's width and size, all experts counted (random weights:
    benchmarks)."""
    left = dict(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5, softcap=50.0,
                mask=dict(size=2048), rot=dict(base=500000.0, dims=64, scaling=dict(
                    factor=4.0, original=8192, fast=32.0, slow=1.0)))
    layers = refolix_stack(
        "RRP" * 7, dict(heads=32, dim=128, vdim=128, decay=_retention_decays(32),
                        rot=dict(base=10000.0, dims=128)),
        dict(left=left, right=dict(heads=32, kv_heads=16, dim=128, vdim=128, conv=4)),
        _grouped_moe(16, 4, 1024, 2048, 4, 2))
    return RefolixConfig(name="refolix-8b", vocab_size=128256, hidden_size=4096,
                         bos_token_id=128000, eos_token_ids=(128001, 128009), layers=layers,
                         embed_scale=64.0, postln_alpha=3.0, logit_scale=0.25,
                         logit_softcap=30.0)


def zovozen_stack(pattern: str, parallel: dict, dense: dict, moe: dict) -> list:
    """Layer list from a pattern of D (dense), M (mixture of experts): every
    layer has both mixers."""
    return [{"type": "parallel", "mixer": dict(parallel),
             "mlp": dict(dense if c == "D" else moe)} for c in pattern]


def _identity_moe(experts: int, identity: int, top: int, ff: int, shared: int, groups: int,
                  keep: int) -> dict:
    return dict(kind="moe", router=dict(experts=experts, identity=identity, top=top,
                                        groups=dict(count=groups, keep=keep)),
                expert=dict(ff=ff), shared=dict(ff=shared))


def _zovozen_tiny() -> ZovozenConfig:
    left = dict(heads=6, kv_heads=3, dim=40, vdim=64, scale=40 ** -0.5, mask=dict(size=72),
                rot=dict(base=10000.0, dims=24, scaling=dict(factor=4.0)))
    layers = zovozen_stack(
        "DMM", dict(left=left, right=dict(heads=3, dim=32, vdim=40, gate_cap=15.0),
                    left_scale=0.8, right_scale=1.1), dict(kind="dense", ff=320),
        _identity_moe(9, 3, 3, 64, 96, 3, 2))
    return ZovozenConfig(name="tiny-zovozen", vocab_size=512, hidden_size=192, bos_token_id=506,
                         eos_token_ids=(510,), layers=layers)


def _zovozen_8b() -> ZovozenConfig:
    """Llama-3-8B's width and size, all experts counted (random weights:
    benchmarks)."""
    left = dict(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5, mask=dict(size=2048),
                rot=dict(base=500000.0, dims=64, scaling=dict(factor=4.0)))
    layers = zovozen_stack(
        "DMM" * 7, dict(left=left, right=dict(heads=32, dim=128, vdim=128, gate_cap=15.0),
                        left_scale=0.8, right_scale=0.6), dict(kind="dense", ff=14336),
        _identity_moe(14, 2, 4, 1024, 2048, 4, 2))
    return ZovozenConfig(name="zovozen-8b", vocab_size=128256, hidden_size=4096,
                         bos_token_id=128000, eos_token_ids=(128001, 128009), layers=layers)


_LLAMA32_ROPE = {"rope_type": "llama3", "factor": 32.0, "low_freq_factor": 1.0,
                 "high_freq_factor": 4.0, "original_max_position_embeddings": 8192}


def _qwen3(name, **kw):
    base = dict(name=name, vocab_size=151936, head_dim=128, rope_theta=1000000.0, rms_eps=1e-6,
                max_position=40960, bos_token_id=151643, eos_token_ids=(151645, 151643),
                family="qwen3", qk_norm=True)
    base.update(kw)
    return LlamaConfig(**base)


PRESETS: dict[str, object] = {
    "llama-3-8b": LlamaConfig(),
    "llama-3-70b": LlamaConfig(name="llama-3-70b", hidden_size=8192, intermediate_size=28672,
                               num_layers=80, num_heads=64, num_kv_heads=8),
    "llama-3.1-8b": LlamaConfig(name="llama-3.1-8b", max_position=131072,
                                rope_scaling={"rope_type": "llama3", "factor": 8.0,
                                              "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                                              "original_max_position_embeddings": 8192}),
    "llama-3.2-1b": LlamaConfig(name="llama-3.2-1b", hidden_size=2048, intermediate_size=8192,
                                num_layers=16, num_heads=32, num_kv_heads=8, head_dim=64,
                                tie_embeddings=True, max_position=131072,
                                rope_scaling=_LLAMA32_ROPE),
    # the reference's default OLLAMA_MODEL (llama3.2:3b); GQA group 3
    "llama-3.2-3b": LlamaConfig(name="llama-3.2-3b", hidden_size=3072, intermediate_size=8192,
                                num_layers=28, num_heads=24, num_kv_heads=8, head_dim=128,
                                tie_embeddings=True, max_position=131072,
                                rope_scaling=_LLAMA32_ROPE),
    # tiny configs for tests / smoke (same code paths, D = 128 heads)
    "tiny-llama": LlamaConfig(name="tiny-llama", vocab_size=512, hidden_size=256,
                              intermediate_size=512, num_layers=2, num_heads=4, num_kv_heads=2,
                              head_dim=128, max_position=2048, bos_token_id=506,
                              eos_token_ids=(510,)),
    # the Llama-3-70B head layout shrunk (64 q / 8 kv heads -> 16 / 8): splits
    # over TP = 8 like 70B does (per rank 2 q heads and 1 kv head, I / 8 = 128)
    "tiny-llama-tp8": LlamaConfig(name="tiny-llama-tp8", vocab_size=1024, hidden_size=512,
                                  intermediate_size=1024, num_layers=2, num_heads=16,
                                  num_kv_heads=8, head_dim=128, max_position=2048,
                                  bos_token_id=1018, eos_token_ids=(1022,)),
    # one rank of Llama-3-70B at TP = 8 (config 4) as a TP = 1 model: 8 q / 1 kv
    # heads, FFN 28672 / 8, the vocab shard 16128 (128256 / 8 padded to 256-row
    # tiles), 80 layers -- QKV 1280 x 8192, O 8192 x 1024, gate/up 7168 x 8192,
    # down 8192 x 3584, LM head 16128 x 8192 per decode step, measured on one GPU
    "llama-3-70b-tp8-rank": LlamaConfig(name="llama-3-70b-tp8-rank", vocab_size=16128,
                                        hidden_size=8192, intermediate_size=3584,
                                        num_layers=80, num_heads=8, num_kv_heads=1,
                                        bos_token_id=16122, eos_token_ids=(16123,),
                                        proxy_tp=8),
    # Qwen2.5 (biased QKV, GQA group 7 / 7 -- not a divisor of 16)
    "qwen2.5-7b": LlamaConfig(name="qwen2.5-7b", vocab_size=152064, hidden_size=3584,
                              intermediate_size=18944, num_layers=28, num_heads=28,
                              num_kv_heads=4, head_dim=128, rope_theta=1000000.0, rms_eps=1e-6,
                              max_position=32768, bos_token_id=151643,
                              eos_token_ids=(151643, 151645), family="qwen2", qkv_bias=True),
    "qwen2.5-0.5b": LlamaConfig(name="qwen2.5-0.5b", vocab_size=151936, hidden_size=896,
                                intermediate_size=4864, num_layers=24, num_heads=14,
                                num_kv_heads=2, head_dim=64, rope_theta=1000000.0, rms_eps=1e-6,
                                max_position=32768, tie_embeddings=True, bos_token_id=151643,
                                eos_token_ids=(151643, 151645), family="qwen2", qkv_bias=True),
    "tiny-qwen": LlamaConfig(name="tiny-qwen", vocab_size=512, hidden_size=448,
                             intermediate_size=512, num_layers=2, num_heads=7, num_kv_heads=1,
                             head_dim=64, rope_theta=1000000.0, rms_eps=1e-6, max_position=2048,
                             bos_token_id=506, eos_token_ids=(510,), family="qwen2",
                             qkv_bias=True),
    # Qwen3 (per-head q/k RMSNorm; num_heads x head_dim may differ from hidden)
    "qwen3-8b": _qwen3("qwen3-8b", hidden_size=4096, intermediate_size=12288, num_layers=36,
                       num_heads=32, num_kv_heads=8),
    "qwen3-32b": _qwen3("qwen3-32b", hidden_size=5120, intermediate_size=25600, num_layers=64,
                        num_heads=64, num_kv_heads=8),
    "qwen3-0.6b": _qwen3("qwen3-0.6b", hidden_size=1024, intermediate_size=3072, num_layers=28,
                         num_heads=16, num_kv_heads=8, tie_embeddings=True),
    "tiny-qwen3": _qwen3("tiny-qwen3", vocab_size=512, hidden_size=256, intermediate_size=512,
                         num_layers=2, num_heads=4, num_kv_heads=2, max_position=2048,
                         bos_token_id=506, eos_token_ids=(510,)),
    "nomic-embed-text": NomicBertConfig(),
    # BERT-architecture embedders (Ollama: mxbai-embed-large, bge-large, snowflake-arctic-embed)
    "mxbai-embed-large": BertConfig(),
    "bge-large-en-v1.5": BertConfig(name="bge-large-en-v1.5"),
    "bge-base-en-v1.5": BertConfig(name="bge-base-en-v1.5", hidden_size=768,
                                   intermediate_size=3072, num_layers=12, num_heads=12,
                                   embed_dim=768),
    "snowflake-arctic-embed-m": BertConfig(name="snowflake-arctic-embed-m", hidden_size=768,
                                           intermediate_size=3072, num_layers=12, num_heads=12,
                                           embed_dim=768),
    "tiny-bert": BertConfig(name="tiny-bert", vocab_size=512, hidden_size=256,
                            intermediate_size=512, num_layers=2, num_heads=4, head_dim=64,
                            embed_dim=256, max_position=256),
    "tiny-bert-mean": BertConfig(name="tiny-bert-mean", vocab_size=512, hidden_size=256,
                                 intermediate_size=512, num_layers=2, num_heads=2, head_dim=128,
                                 embed_dim=256, max_position=256, pooling="mean"),
    "tiny-zegopel": _zegopel_tiny(),
    "zegopel-8b": _zegopel_8b(),
    "tiny-pikesun": _pikesun_tiny(),
    "pikesun-8b": _pikesun_8b(),
    "tiny-refolix": _refolix_tiny(),
    "refolix-8b": _refolix_8b(),
    "tiny-zovozen": _zovozen_tiny(),
    "zovozen-8b": _zovozen_8b(),
    "tiny-nomic": NomicBertConfig(name="tiny-nomic", vocab_size=512, hidden_size=256,
                                  intermediate_size=512, num_layers=2, num_heads=2, head_dim=128,
                                  embed_dim=256, max_position=2048),
}

# OpenAI-style aliases (Ollama tags used by the reference's defaults)
ALIASES = {
    "llama3": "llama-3-8b", "llama3:8b": "llama-3-8b", "llama-3-8b-instruct": "llama-3-8b",
    "meta-llama-3-8b": "llama-3-8b", "llama3:70b": "llama-3-70b",
    "llama3.2:1b": "llama-3.2-1b", "llama3.2:3b": "llama-3.2-3b", "llama3.2": "llama-3.2-3b",
    "nomic-embed-text:latest": "nomic-embed-text",
    "qwen3:8b": "qwen3-8b", "qwen3:32b": "qwen3-32b", "qwen3:0.6b": "qwen3-0.6b",
    "qwen3": "qwen3-8b",
    "nomic-embed-text-v1.5": "nomic-embed-text",
    "qwen2.5:7b": "qwen2.5-7b", "qwen2.5:0.5b": "qwen2.5-0.5b",
    "qwen2.5-7b-instruct": "qwen2.5-7b",
    "mxbai-embed-large:latest": "mxbai-embed-large", "mxbai-embed-large:335m": "mxbai-embed-large",
    "mixedbread-ai/mxbai-embed-large-v1": "mxbai-embed-large",
    "bge-large": "bge-large-en-v1.5", "bge-large:335m": "bge-large-en-v1.5",
    "snowflake-arctic-embed:110m": "snowflake-arctic-embed-m",
}


def resolve(name: str):
    """Preset by name or alias.  ``<name>@L<n>`` keeps the preset's shapes
    with only n layers (e.g. ``llama-3-70b@L8``: one-GPU rehearsals of the
    70B TP layout; never a number for the full model).  A directory with a
    config.json is a checkpoint: its own configuration."""
    if is_checkpoint_dir(name):
        return from_hf_config(Path(name) / "config.json")
    base, _, layers = name.partition("@L")
    key = ALIASES.get(base, base)
    if key not in PRESETS:
        raise KeyError(f"unknown model {name!r}; known: {sorted(PRESETS)}")
    cfg = PRESETS[key]
    if layers:
        import dataclasses
        n = int(layers)
        if n < 1 or n > cfg.num_layers:
            raise KeyError(f"{name!r}: layer count must be 1..{cfg.num_layers}")
        if isinstance(cfg, LayerListConfig):
            return dataclasses.replace(cfg, name=name, layers=cfg.layers[:n])
        cfg = dataclasses.replace(cfg, name=name, num_layers=n)
    return cfg


def is_checkpoint_dir(name: str) -> bool:
    return (Path(name) / "config.json").is_file()


def from_hf_config(path: str | Path):
    """Build a config from a HF config.json (local file; no network)."""
    cfg = json.loads(Path(path).read_text())
    family = LAYER_LISTS.get(cfg.get("architecture"))
    if family is not None:
        return family.from_json(cfg, Path(path).resolve().parent.name)
    arch = (cfg.get("architectures") or [""])[0]
    if "Llama" in arch or "Qwen2" in arch or "Qwen3" in arch or "Mistral" in arch:
        qwen = "Qwen2" in arch
        qwen3 = "Qwen3" in arch
        return LlamaConfig(
            name=cfg.get("_name_or_path", "llama"), vocab_size=cfg["vocab_size"],
            hidden_size=cfg["hidden_size"], intermediate_size=cfg["intermediate_size"],
            num_layers=cfg["num_hidden_layers"], num_heads=cfg["num_attention_heads"],
            num_kv_heads=cfg.get("num_key_value_heads", cfg["num_attention_heads"]),
            head_dim=cfg.get("head_dim", cfg["hidden_size"] // cfg["num_attention_heads"]),
            rope_theta=cfg.get("rope_theta", 10000.0), rope_scaling=cfg.get("rope_scaling"),
            rms_eps=cfg.get("rms_norm_eps", 1e-5),
            max_position=cfg.get("max_position_embeddings", 8192),
            tie_embeddings=cfg.get("tie_word_embeddings", False),
            bos_token_id=cfg.get("bos_token_id", 128000),
            eos_token_ids=tuple(cfg["eos_token_id"]) if isinstance(cfg.get("eos_token_id"), list)
            else (cfg.get("eos_token_id", 128001),),
            family="qwen2" if qwen else ("qwen3" if qwen3 else
                                         ("mistral" if "Mistral" in arch else "llama")),
            qkv_bias=qwen or bool(cfg.get("attention_bias", False)), qk_norm=qwen3)
    if "NomicBert" in arch or cfg.get("model_type") == "nomic_bert":
        return NomicBertConfig(
            vocab_size=cfg["vocab_size"], hidden_size=cfg["n_embd"],
            intermediate_size=cfg["n_inner"], num_layers=cfg["n_layer"],
            num_heads=cfg["n_head"], head_dim=cfg["n_embd"] // cfg["n_head"],
            rope_theta=cfg.get("rotary_emb_base", 1000.0),
            ln_eps=cfg.get("layer_norm_epsilon", 1e-12),
            max_position=cfg.get("n_positions", 8192),
            qkv_bias=cfg.get("qkv_proj_bias", False), mlp_bias=cfg.get("mlp_fc1_bias", False),
            embed_dim=cfg["n_embd"])
    if arch in ("BertModel", "BertForMaskedLM") or cfg.get("model_type") == "bert":
        d, H = cfg["hidden_size"], cfg["num_attention_heads"]
        return BertConfig(
            name=cfg.get("_name_or_path", "bert"), vocab_size=cfg["vocab_size"], hidden_size=d,
            intermediate_size=cfg["intermediate_size"], num_layers=cfg["num_hidden_layers"],
            num_heads=H, head_dim=d // H, ln_eps=cfg.get("layer_norm_eps", 1e-12),
            max_position=cfg.get("max_position_embeddings", 512),
            type_vocab_size=cfg.get("type_vocab_size", 2), embed_dim=d,
            pooling=cfg.get("pooling", "cls"))
    raise ValueError(f"unsupported architecture {arch!r}")
