"""Prefill and decode throughput of two models side by side, engine only
(``bench.py --compare MODEL``): random weights, synthetic prompts, the two
engines timed in turn at each size so that clock drift hits both."""
from __future__ import annotations

import time

PREFILL = ((1, 2048), (1, 7680), (16, 2048))          # (prompts, tokens each)
DECODE = ((1, 1024), (16, 1024), (64, 1024), (256, 512))   # (streams, context)
NEW_TOKENS = 48


def make_engine(model: str, batch: int, device, max_len: int = 8320, dtype: str = "bfloat16"):
    from ..engine.engine import EngineConfig, LLMEngine
    return LLMEngine(EngineConfig(model=model, max_num_seqs=batch, max_batched_tokens=36864,
                                  mixed_prefill_tokens=0, max_model_len=max_len,
                                  prefix_cache=False, kv_cache_gb=32, dtype=dtype),
                     device=device)


def _prompts(e, n: int, length: int, seed: int):
    import torch
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, e.cfg.vocab_size, (n, length), generator=g).tolist()


def prefill_once(e, n: int, length: int, seed: int = 0) -> float:
    """Seconds from submitting n prompts to all first tokens."""
    import torch

    from ..engine.engine import SamplingParams
    p = _prompts(e, n, length, seed)
    torch.cuda.synchronize()
    t = time.perf_counter()
    e.generate(p, SamplingParams(temperature=0, max_tokens=1, ignore_eos=True))
    torch.cuda.synchronize()
    return time.perf_counter() - t


def decode_once(e, n: int, ctx: int, new: int = NEW_TOKENS, seed: int = 0) -> float:
    """Seconds per decode step of n streams around context ctx (graph steps)."""
    from ..engine.engine import SamplingParams
    p = _prompts(e, n, ctx, seed)
    s0, g0 = e.stats["decode_step_s"], e.stats["graph_steps"]
    e.generate(p, SamplingParams(temperature=0, max_tokens=new, ignore_eos=True))
    return (e.stats["decode_step_s"] - s0) / max(1, e.stats["graph_steps"] - g0)


def compare(models: list[str], device="cuda", repeats: int = 3, say=lambda s: None) -> dict:
    """{"prefill": [...], "decode": [...]}: tokens/s of each model per size,
    the median of ``repeats`` alternating measurements."""
    batch = max(n for n, _ in DECODE)
    engines = {}
    for m in models:
        engines[m] = make_engine(m, batch, device)
        say(f"{m}: {engines[m].cfg.params_b} B parameters, engine ready")
    out: dict = {"models": {m: {"params_b": e.cfg.params_b} for m, e in engines.items()},
                 "prefill": [], "decode": []}

    def row(kind, size, fn, tokens):
        ts = {m: [] for m in models}
        for r in range(repeats + 1):             # the first round warms up
            for m in models:
                ts[m].append(fn(engines[m], r))
        med = {m: sorted(t[1:])[len(t[1:]) // 2] for m, t in ts.items()}
        rec = {**size, "tok_s": {m: round(tokens / med[m], 1) for m in models},
               "ms": {m: round(med[m] * 1e3, 3) for m in models}}
        if len(models) == 2:
            rec["time_ratio"] = round(med[models[0]] / med[models[1]], 3)
        out[kind].append(rec)
        say(f"{kind} {size}: {rec['ms']} ms")

    for n, length in PREFILL:
        row("prefill", {"prompts": n, "tokens": length},
            lambda e, r: prefill_once(e, n, length, r), n * length)
    for n, ctx in DECODE:
        row("decode", {"streams": n, "context": ctx},
            lambda e, r: decode_once(e, n, ctx, seed=r), n)
    return out


def profile(model: str, what: str, n: int, length: int, device="cuda") -> None:
    """One workload for a kernel trace: ``rocprofv3 --kernel-trace --stats --
    python3 -m llm_mcp_amd.bench.model_compare MODEL prefill|decode N LENGTH``."""
    e = make_engine(model, n, device)
    for seed in range(3):
        if what == "prefill":
            print(f"{prefill_once(e, n, length, seed) * 1e3:.2f} ms", flush=True)
        else:
            print(f"{decode_once(e, n, length, seed=seed) * 1e3:.3f} ms/step", flush=True)


if __name__ == "__main__":
    import sys
    profile(sys.argv[1], sys.argv[2], int(sys.argv[3]), int(sys.argv[4]))
