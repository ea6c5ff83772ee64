"""Trace replay: given token ids through a model, step by step, logits out.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Reads one JSON object a line from standard input,

    {"step": n, "entries": [{"id": name, "tokens": [ids], "want": [places]}, ...], "end": [names]}

and runs each line as one step of the serving engine (``LLMEngine.feed``: its
scheduler, paged cache, state slots and kernels; nothing is sampled).  A step
with wanted places writes DIR/<step>.f32, the logits at those places as
little-endian fp32 [wanted, vocab]; every step ends with a line ``done <step>``
on standard output.  ``end`` names the requests that are finished after the
step.

The KV pool holds ``--max-tokens`` tokens (in 32-token pages) and there are
state slots for ``--max-seqs`` live requests.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def parser() -> argparse.ArgumentParser:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace")
    ap.add_argument("--model", required=True, help="checkpoint directory")
    ap.add_argument("--dtype", default="bfloat16", choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="directory of the logits files")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens held by live requests at any time (the KV pool)")
    ap.add_argument("--max-seqs", type=int, default=4, help="live requests at any time")
    ap.add_argument("--gpu", type=int, default=0)
    return ap


def build_engine(model: str, dtype: str, max_tokens: int, max_seqs: int, device):
    """A serving engine over a checkpoint directory, its KV pool sized in tokens."""
    from ..models import config as mc
    from ..models.weights import load_weights
    from .engine import EngineConfig, LLMEngine
    cfg = mc.resolve(model)
    # page tables as wide as the pool; a whole pool's tokens fit one step
    pool = max(max_tokens, 64)
    ecfg = EngineConfig(model=model, max_num_seqs=max_seqs, max_batched_tokens=pool,
                        mixed_prefill_tokens=0, max_model_len=pool, kv_cache_tokens=pool,
                        prefix_cache=False, use_graphs=False, dtype=dtype)
    return LLMEngine(ecfg, device=device, model_cfg=cfg,
                     weights=load_weights(model, cfg, device))


def replay(engine, lines, out_dir: str, say) -> None:
    """Run every line's step; ``say(text)`` reports each finished one."""
    ids: dict[str, int] = {}
    nxt = 1
    for line in lines:
        if not line.strip():
            continue
        st = json.loads(line)
        entries = []
        for e in st["entries"]:
            if e["id"] not in ids:
                ids[e["id"]], nxt = nxt, nxt + 1
            if e["tokens"]:
                entries.append((ids[e["id"]], e["tokens"], e.get("want", [])))
        logits = engine.feed(entries, [ids.pop(r) for r in st.get("end", []) if r in ids])
        if logits.shape[0]:
            part = os.path.join(out_dir, f".{st['step']}.part")
            with open(part, "wb") as f:
                f.write(logits.numpy().astype("<f4").tobytes())
            os.replace(part, os.path.join(out_dir, f"{st['step']}.f32"))
        say(f"done {st['step']}")


def main(argv=None) -> int:
    a = parser().parse_args(argv)
    import torch

    from .. import native
    if not torch.cuda.is_available():
        print("trace_run: no GPU", file=sys.stderr)
        return 2
    native.kernels()
    torch.cuda.set_device(a.gpu)
    torch.backends.cuda.matmul.allow_tf32 = False
    os.makedirs(a.out, exist_ok=True)
    engine = build_engine(a.model, a.dtype, a.max_tokens, a.max_seqs,
                          torch.device("cuda", a.gpu))
    with torch.inference_mode():
        replay(engine, sys.stdin, a.out, lambda t: print(t, flush=True))
    return 0
