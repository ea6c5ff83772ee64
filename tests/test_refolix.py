"""Refolix in the serving engine against the plain reference of
``refolix_oracle``: whole prompts, token-by-token decoding, portions, batches,
slots and pages that are used again, windows' edges, generation -- on the CPU
references and on the GPU kernels, in bf16 and fp32."""
import json

import numpy as np
import pytest
import torch

import refolix_oracle as oracle
from llm_mcp_amd.engine.engine import EngineConfig, LLMEngine, SamplingParams
from llm_mcp_amd.models import config as mc
from llm_mcp_amd.models.refolix import RefolixModel, tensor_shapes
from llm_mcp_amd.models.registry import model_class
from llm_mcp_amd.models.weights import load_weights, save_layer_list
from refolix_cases import (CASES, attention, config, delta, moe, par, ret, scaling, shapes,
                           tokens, weights)

GPU = pytest.mark.gpu
RUNS = [pytest.param("cpu", "float32", id="cpu-fp32"),
        pytest.param("cuda", "float32", id="gpu-fp32", marks=GPU),
        pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=GPU)]
# rms error over the vocabulary, relative to the logits' own rms
TOL = {"float32": 5e-5, "bfloat16": 0.08}
# positions that may be over: a near tie of a router falls the other way in bf16,
# and the tokens behind it see that one
STRAY = {"float32": 0.0, "bfloat16": 0.05}


def product_config(cfg, name="case"):
    return mc.RefolixConfig.from_json(json.loads(json.dumps(cfg)), name)


def engine(cfg, W, device, dtype, tokens=512, seqs=4, graphs=False, **kw):
    ecfg = dict(max_num_seqs=seqs, max_batched_tokens=512, mixed_prefill_tokens=0,
                max_model_len=512, kv_cache_tokens=tokens, use_graphs=graphs, dtype=dtype)
    ecfg.update(kw)
    return LLMEngine(EngineConfig(**ecfg), device=device, model_cfg=product_config(cfg), weights=W)


@pytest.fixture(autouse=True, scope="module")
def _one_thread():
    """Tiny tensors: intra-op threads only cost."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


_MADE = {}


def weights_for(cfg, dtype, seed=0):
    key = (json.dumps(cfg), dtype == "bfloat16", seed)
    if key not in _MADE:
        _MADE[key] = weights(cfg, seed, calm=key[1])
    return _MADE[key]


def reference(cfg, W, toks):
    key = (id(W), tuple(toks))            # W of ``weights_for``: kept
    if key not in _MADE:
        _MADE[key] = oracle.forward(cfg, W, toks)
    return _MADE[key]


def errors(got, want):
    got, want = got.double(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()


class Tally:
    """Errors of a test's positions, judged together."""

    def __init__(self, dtype):
        self.dtype, self.errs, self.where = dtype, [], []

    def add(self, got, want, what=""):
        e = errors(got, want)
        self.errs += e.tolist()
        self.where += [f"{what}+{k}" for k in range(len(e))]

    def done(self):
        bad = [(w, round(e, 6)) for w, e in zip(self.where, self.errs) if not e < TOL[self.dtype]]
        n = len(self.errs)
        assert n and len(bad) <= max(1, STRAY[self.dtype] * n) * (STRAY[self.dtype] > 0), \
            f"{len(bad)} of {n}: {bad[:6]}"


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", sorted(CASES))
def test_whole_prompt_and_decode(case, device, dtype):
    """Every position of one prompt in one step, then the same tokens with the
    tail one by one: the state and cache the prompt left must be the ones a
    longer prompt would have used."""
    cfg = CASES[case]
    W = weights_for(cfg, dtype)
    n, tail = 90, 12
    toks = tokens(cfg, n)
    want = reference(cfg, W, toks)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    t.add(e.feed([(1, toks, list(range(n)))], [1]), want, "whole")
    t.add(e.feed([(2, toks[:n - tail], list(range(n - tail)))]), want[:n - tail], "prompt")
    for i in range(n - tail, n):
        t.add(e.feed([(2, toks[i:i + 1], [0])], [2] if i == n - 1 else []), want[i:i + 1], f"at {i}")
    t.done()
    assert e.sched.kv_usage == 0.0


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "odd"])
def test_token_by_token_from_the_start(case, device, dtype):
    cfg = CASES[case]
    W = weights_for(cfg, dtype)
    toks = tokens(cfg, 50, seed=3)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    t.add(torch.cat([e.feed([(7, [x], [0])]) for x in toks]), reference(cfg, W, toks))
    t.done()


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "odd", "fast"])
def test_portions(case, device, dtype):
    """Portions cut inside pages, windows and chunks, down to two tokens and one."""
    cfg = CASES[case]
    W = weights_for(cfg, dtype)
    n = 150
    toks = tokens(cfg, n, seed=5)
    want = reference(cfg, W, toks)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    for k, cuts in enumerate([[2] * 20, [31, 1, 2, 33, 64, 3, 16], [65, 2, 2], [1, 149]]):
        at = 0
        for c in cuts:
            y = e.feed([(k + 1, toks[at:at + c], list(range(c)))])
            t.add(y, want[at:at + c], f"cuts {k} at {at}")
            at += c
        e.feed([], [k + 1])
    t.done()


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "beyond"])
def test_unequal_requests_share_steps_pages_and_slots(case, device, dtype):
    """Up to four live requests of unequal lengths in shared steps, portions
    beside decoded tokens, some left out of a step; requests end and their
    pages and slots go to the next ones (seven requests, a pool of four)."""
    cfg = CASES[case]
    W = weights_for(cfg, dtype)
    lens = [70, 1, 33, 64, 5, 90, 32]
    reqs = {i + 1: tokens(cfg, n, seed=10 + i) for i, n in enumerate(lens)}
    want = {i: reference(cfg, W, t) for i, t in reqs.items()}
    e, t = engine(cfg, W, device, dtype, tokens=288), Tally(dtype)
    rng = np.random.default_rng(0)
    at, live, waiting = {}, [], list(reqs)
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
            at[live[-1]] = 0
        ents, end, spans = [], [], []
        for r in live:
            if len(ents) and rng.random() < 0.25:
                continue                        # left out of this step
            left = len(reqs[r]) - at[r]
            n = int(min(left, rng.choice([1, 1, 2, 3, 17, 32, 40])))
            ents.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
            spans.append((r, at[r], n))
            at[r] += n
            if at[r] == len(reqs[r]):
                end.append(r)
        y = e.feed(ents, end)
        k = 0
        for r, a, n in spans:
            t.add(y[k:k + n], want[r][a:a + n], f"request {r} at {a}")
            k += n
        live = [r for r in live if r not in end]
    t.done()
    assert e.sched.kv_usage == 0.0


@pytest.mark.parametrize("device,dtype", RUNS)
def test_request_alone_and_in_a_batch_agree(device, dtype):
    cfg = CASES["beyond"]
    W = weights_for(cfg, dtype)
    toks = [tokens(cfg, n, seed=20 + n) for n in (3, 65, 40)]
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    alone = [e.feed([(9, x, list(range(len(x))))], [9]) for x in toks]
    both = e.feed([(i + 1, x, list(range(len(x)))) for i, x in enumerate(toks)], [1, 2, 3])
    t.add(both, torch.cat(alone))
    t.done()


@pytest.mark.parametrize("device,dtype", RUNS)
def test_long_decoding(device, dtype):
    """Decoded tokens pass over the windows and pages of the prompt."""
    cfg = CASES["mixed"]
    W = weights_for(cfg, dtype)
    toks = tokens(cfg, 240, seed=50)
    want = reference(cfg, W, toks)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    e.feed([(1, toks[:30], [])])
    for i in range(30, 240):
        y = e.feed([(1, toks[i:i + 1], [0] if i % 5 == 4 or i < 80 else [])])
        if y.shape[0]:
            t.add(y, want[i:i + 1], f"at {i}")
    t.done()


def sharp_window(window, back):
    """One layer whose attention looks for the token ``back`` places back and
    hardly anything else: constant queries and keys, and a rotation of the query
    that makes that distance the best match."""
    R = 32
    rot = dict(base=float(3 * window), dims=R, scaling=scaling(2.0, 4 * window, 8.0, 0.5))
    left = dict(heads=1, kv_heads=1, dim=R, vdim=16, mask=dict(size=window), rot=rot, scale=3.0,
                softcap=150.0)
    cfg = config([par(None, left, delta(heads=1, kv_heads=1, dim=8, vdim=8))], width=32, vocab=40,
                 scale=1.0, alpha=0.3)
    W = {k: v.float() for k, v in weights(cfg, 3).items()}
    a = oracle.frequencies(rot).float() * back
    # carried by an embedding column all tokens share
    W["embed"][:, 0] = 4.0
    x = "l0.mix.left."
    W[x + "q"], W[x + "k"] = torch.zeros(R, 32), torch.zeros(R, 32)
    W[x + "q"][:, 0] = torch.stack([a.cos(), -a.sin()], 1).reshape(-1)   # turned back by that many
    W[x + "k"][0::2, 0] = 1.0
    W[x + "q.norm"], W[x + "k.norm"] = torch.ones(R), torch.ones(R)
    W["l0.mix.right.out"] *= 0.0
    return cfg, {k: v.to(torch.bfloat16) for k, v in W.items()}


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("inside", [True, False], ids=["inside", "outside"])
@pytest.mark.parametrize("window", [31, 32, 33, 64, 65])
def test_the_edge_of_a_window(window, inside, device, dtype):
    """The best match is the oldest visible key, or the first one that is not
    visible any more, around page borders, in prompts, portions and decoding: a
    window one off moves the logits."""
    cfg, W = sharp_window(window, window - 1 if inside else window)
    n = window + 70
    toks = tokens(cfg, n, seed=9)
    want = oracle.forward(cfg, W, toks)
    c = json.loads(json.dumps(cfg))
    c["layers"][0]["mixer"]["left"]["mask"]["size"] += -1 if inside else 1
    e = errors(oracle.forward(c, W, toks)[window + 1:], want[window + 1:])
    assert float(e.median()) > 0.2          # the sharp weights would show it
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    t.add(e.feed([(1, toks, list(range(n)))], [1]), want, "whole")
    at = 0
    for k in (window - 1, 1, 1, 2, 5, 30):
        t.add(e.feed([(2, toks[at:at + k], list(range(k)))]), want[at:at + k], f"portion {at}")
        at += k
    for i in range(at, n):
        t.add(e.feed([(2, toks[i:i + 1], [0])]), want[i:i + 1], f"decoded {i}")
    t.done()


@pytest.mark.parametrize("device,dtype", RUNS)
def test_a_token_far_back(device, dtype):
    """The state carries a distant token: one token of a prompt is exchanged,
    and every later position must move as the reference's does, in the prompt
    and over portions and decoding."""
    slow = [1.0 - 2.0 ** -12] * 2
    right = delta(heads=2, kv_heads=1, dim=16, vdim=16)
    cfg = config([ret(None, heads=2, dim=16, vdim=16, dims=4, decay=slow),
                  par(None, attention(window=3), right)], alpha=0.2)
    W = dict(weights(cfg, 12))
    W["l1.mix.right.dt_bias"] = W["l1.mix.right.dt_bias"] * 0 - 9.0     # hardly any decay
    a = tokens(cfg, 200, seed=13)
    b = a[:3] + [(a[3] + 1) % cfg["vocab"]] + a[4:]
    want = [oracle.forward(cfg, W, x) for x in (a, b)]
    e = errors(want[0], want[1])
    assert float(e[20:60].median()) > 0.3 and float(e[150:].median()) > 0.08
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    for k, x in enumerate((a, b)):
        y = [e.feed([(k, x[i:j], list(range(j - i)))]) for i, j in ((0, 70), (70, 72), (72, 180))]
        y += [e.feed([(k, x[i:i + 1], [0])]) for i in range(180, 200)]
        t.add(torch.cat(y), want[k], f"text {k}")
        e.feed([], [k])
    t.done()


@pytest.mark.parametrize("device,dtype", RUNS)
def test_generation_is_greedy_of_the_reference(device, dtype):
    """The engine's own entry point: batches of unequal prompts through the
    scheduler, the sampler and (on the GPU) the captured decode graphs."""
    cfg = CASES["mixed"]
    W = weights_for(cfg, dtype, 4)
    e = engine(cfg, W, device, dtype, graphs=device == "cuda")
    prompts = [tokens(cfg, n, seed=30 + n) for n in (1, 5, 40, 66, 2, 31)]
    new = 24
    outs = e.generate(prompts, SamplingParams(temperature=0, max_tokens=new, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o) == new
        lg = oracle.forward(cfg, W, p + o)[len(p) - 1:-1]
        short = lg.max(-1).values - lg[torch.arange(new), torch.tensor(o)]
        # a token may only differ from the reference's where that is a near tie
        bad = int((short > 4 * TOL[dtype] * float(lg.std())).sum())
        assert bad <= STRAY[dtype] * new
    if device == "cuda":
        assert e.stats["graph_steps"] > 0


@pytest.mark.parametrize("device,dtype", RUNS)
def test_preemption_recomputes_the_state(device, dtype):
    """A pool too small for every request: preempted sequences lose pages and
    slot and come back through a recomputed prompt."""
    cfg = CASES["mixed"]
    W = weights_for(cfg, dtype, 6)
    e = engine(cfg, W, device, dtype, tokens=192, graphs=device == "cuda")
    prompts = [tokens(cfg, 50, seed=40 + i) for i in range(4)]
    outs = e.generate(prompts, SamplingParams(temperature=0, max_tokens=30, ignore_eos=True))
    assert e.sched.preemptions > 0
    for p, o in zip(prompts, outs):
        lg = oracle.forward(cfg, W, p + o)[len(p) - 1:-1]
        short = lg.max(-1).values - lg[torch.arange(len(o)), torch.tensor(o)]
        assert len(o) == 30
        assert int((short > 4 * TOL[dtype] * float(lg.std())).sum()) <= STRAY[dtype] * 30


@GPU
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_graphs_replay_what_eager_steps_compute(dtype):
    """The same streams through captured decode graphs and through eager steps,
    in batches that grow and shrink between replays."""
    cfg = CASES["fast"]
    W = weights_for(cfg, dtype, 8)
    prompts = [tokens(cfg, n, seed=60 + n) for n in (4, 35, 1, 140, 20, 9)]
    sp = SamplingParams(temperature=0, max_tokens=20, ignore_eos=True)
    outs = []
    for graphs in (True, False):
        e = engine(cfg, W, "cuda", dtype, seqs=3, graphs=graphs)
        outs.append(e.generate(prompts, sp))
    assert outs[0] == outs[1]


@pytest.mark.parametrize("device,dtype", RUNS)
def test_a_planted_mistake_shows(device, dtype):
    """The weights of the tests are sharp enough: the reference with one
    mechanism wrong is far outside the tolerance the product meets."""
    cfg = CASES["mixed"]
    W = weights_for(cfg, dtype)
    toks = tokens(cfg, 70)
    got = engine(cfg, W, device, dtype).feed([(1, toks, list(range(70)))])
    t = Tally(dtype)
    t.add(got, reference(cfg, W, toks))
    t.done()

    def changed(fn):
        c = json.loads(json.dumps(cfg))
        fn(c)
        return c, W
    left, right = (lambda c, n=n: c["layers"][1]["mixer"][n] for n in ("left", "right"))
    one = torch.ones(1, dtype=torch.bfloat16)
    wrong = {
        "embedding scale": changed(lambda c: c["embedding"].update(scale=12.0)),
        "alpha": changed(lambda c: c.update(postln_alpha=2.6)),
        "logit scale": changed(lambda c: c.update(logit_scale=0.6)),
        "logit cap": changed(lambda c: c.update(logit_softcap=3.0)),
        "retention rotation": changed(lambda c: c["layers"][0]["mixer"]["rot"].update(base=100.0)),
        "retention decay": changed(lambda c: c["layers"][2]["mixer"].update(decay=[0.6, 0.8, 0.9])),
        "rotation": changed(lambda c: left(c)["rot"].update(base=100.0)),
        "length scaling": changed(lambda c: left(c)["rot"].update(scaling=None)),
        "attention scale": changed(lambda c: left(c).update(scale=0.8)),
        "attention cap": changed(lambda c: left(c).update(softcap=1.0)),
        "top": changed(lambda c: [c["layers"][i]["mlp"]["router"].update(top=1) for i in (0, 1)]),
        "groups": changed(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=1)),
        "correction": (cfg, {**W, "l0.mlp.correction": W["l0.mlp.correction"] * 0}),
        "shared gate": (cfg, {**W, "l0.mlp.shared.sg": W["l0.mlp.shared.sg"] * 0}),
        "layer scale": (cfg, {**W, "l1.ls1": W["l1.ls1"] * 0 + one}),
        "feed-forward scale": (cfg, {**W, "l0.ls2": W["l0.ls2"] * 0 + one}),
        "query norm": (cfg, {**W, "l1.mix.left.q.norm": W["l1.mix.left.q.norm"] * 0 + one}),
        "branch gain": (cfg, {**W, "l1.mix.left.out": W["l1.mix.left.out"] * 0 + one}),
        "other branch": (cfg, {**W, "l1.mix.right.out": W["l1.mix.right.out"] * 0}),
        "decay": (cfg, {**W, "l1.mix.right.dt_bias": W["l1.mix.right.dt_bias"] + 2.0}),
        "step size": (cfg, {**W, "l1.mix.right.b": W["l1.mix.right.b"] * 0}),
        "oldest tap": (cfg, {**W, "l1.mix.right.k.conv": torch.cat(
            [W["l1.mix.right.k.conv"][:, :1] * 0, W["l1.mix.right.k.conv"][:, 1:]], 1)}),
        "output gate": (cfg, {**W, "l1.mix.right.g": W["l1.mix.right.g"] * 0 + one}),
    }
    for name, (c, w) in wrong.items():
        e = errors(got, oracle.forward(c, w, toks))
        assert float(e.median()) > TOL[dtype], f"{name}: {float(e.median()):.4f}"


@pytest.mark.parametrize("device,dtype", RUNS)
def test_residual_after_every_layer(device, dtype):
    cfg = CASES["mixed"]
    toks = tokens(cfg, 40, seed=2)
    W = weights_for(cfg, dtype)
    e = engine(cfg, W, device, dtype)
    got, run = [], e.model.forward

    def forward(*a, **k):
        return run(*a, layers_out=got, **k)
    e.model.forward = forward
    e.feed([(1, toks, [0])])
    want = []
    oracle.forward(cfg, W, toks, want)
    assert len(got) == len(want) == len(cfg["layers"])
    for a, b in zip(got, want):
        e_ = ((a.cpu().double() - b).pow(2).mean(-1).sqrt() / b.std())
        assert float(e_.median()) < TOL[dtype] / 2


@pytest.mark.parametrize("device,dtype", RUNS)
def test_a_wide_shared_expert(device, dtype):
    cfg = config([ret(moe(ff=20, shared=1100)), par(moe())])
    W = weights_for(cfg, dtype)
    toks = tokens(cfg, 40, seed=4)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    y = [e.feed([(1, toks[a:b], list(range(b - a)))]) for a, b in ((0, 17), (17, 18), (18, 40))]
    t.add(torch.cat(y), reference(cfg, W, toks))
    t.done()


# ------------------------------------------------- configuration, loading ----
def test_checkpoint_directory_round_trip(tmp_path):
    cfg = CASES["mixed"]
    W = weights(cfg)
    pc = product_config(cfg)
    assert {k: tuple(v) for k, v in tensor_shapes(pc).items()} == shapes(cfg)
    save_layer_list(W, pc, str(tmp_path))
    back = mc.resolve(str(tmp_path))
    assert back.family == "refolix" and model_class(back) is RefolixModel
    assert (back.layers, back.vocab_size, back.hidden_size, back.rms_eps, back.embed_scale,
            back.postln_alpha, back.logit_scale, back.logit_softcap) == \
        (pc.layers, pc.vocab_size, pc.hidden_size, pc.rms_eps, 3.0, 1.7, 0.7, 6.0)
    W2 = load_weights(str(tmp_path), back, "cpu")
    assert all(torch.equal(W[k], W2[k]) for k in W)
    assert back.params == sum(t.numel() for t in W.values())
    save_layer_list(dict(W, head=W["head"][:-1]), pc, str(tmp_path))
    with pytest.raises(ValueError, match="head"):
        load_weights(str(tmp_path), back, "cpu")


def test_unknown_mechanisms_are_refused():
    with pytest.raises(ValueError, match="mixer"):
        product_config(config([{**ret(), "type": "lightning"}]))
    with pytest.raises(ValueError, match="feed-forward"):
        product_config(config([ret(dict(kind="dense", ff=8))]))
    for bad in ([par(None, attention(window=0))], [par(None, attention(heads=3))],
                [par(None, attention(dims=26))], [par(None, None, delta(heads=3))],
                [ret(decay=[0.5])], [ret(dims=5)], [ret(moe(top=7))], [ret(moe(groups=4))],
                [ret(moe(keep=4))], [ret(moe(top=3, keep=1))]):
        with pytest.raises(ValueError):
            RefolixModel(product_config(config(bad)), "cpu")


def test_presets_and_layer_subsets():
    full = mc.resolve("refolix-8b")
    assert 7.5 < full.params_b < 8.5
    assert mc.resolve("refolix-8b@L3").num_layers == 3
    e = LLMEngine(EngineConfig(model="tiny-refolix", max_num_seqs=2, max_batched_tokens=64,
                               max_model_len=128, use_graphs=False), device="cpu")
    out = e.generate([[1, 2, 3], [9] * 40], SamplingParams(temperature=0.8, seed=3, max_tokens=5,
                                                          ignore_eos=True))
    assert [len(o) for o in out] == [5, 5] and e.sched.prefix_hits == 0
    assert e.model.weight_bytes() > 0


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("layers", [[ret()], [par(moe(), right=delta(conv=1))]],
                         ids=["states only", "no convolution state"])
def test_models_with_part_of_the_caches(layers, device, dtype):
    cfg = config(layers)
    W = weights_for(cfg, dtype)
    toks = tokens(cfg, 47)
    e, t = engine(cfg, W, device, dtype), Tally(dtype)
    y = torch.cat([e.feed([(1, toks[:20], list(range(20)))]),
                   e.feed([(1, toks[20:], list(range(27)))])])
    t.add(y, reference(cfg, W, toks))
    t.done()


def test_trace_replay(tmp_path):
    from llm_mcp_amd.engine import trace
    cfg = CASES["mixed"]
    W = weights_for(cfg, "float32")
    save_layer_list(W, product_config(cfg), str(tmp_path / "m"))
    e = trace.build_engine(str(tmp_path / "m"), "float32", 130, 4, "cpu")
    toks = tokens(cfg, 40)
    want = reference(cfg, W, toks)
    out = tmp_path / "out"
    out.mkdir()
    lines = [json.dumps(s) + "\n" for s in (
        {"step": 0, "entries": [{"id": "x", "tokens": toks[:11], "want": [10, 3]}], "end": []},
        {"step": 1, "entries": [{"id": "y", "tokens": toks[:2], "want": [1]},
                                {"id": "x", "tokens": toks[11:], "want": [0, 28]}],
         "end": ["x", "y"]})]
    said = []
    trace.replay(e, lines, str(out), said.append)
    assert said == ["done 0", "done 1"]
    t = Tally("float32")
    for step, places in ((0, [10, 3]), (1, [1, 11, 39])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        t.add(torch.from_numpy(got.copy()), want[places])
    t.done()
