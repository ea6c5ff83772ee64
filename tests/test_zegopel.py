"""Zegopel in the serving engine against the plain reference of
``zegopel_oracle``: whole prompts, token-by-token decoding, portions, batches,
slots and pages that are used again, generation -- on the CPU references and on
the GPU kernels, in bf16 and fp32."""
import json
import threading
import time

import numpy as np
import pytest
import torch

import zegopel_oracle as oracle
from llm_mcp_amd.engine.engine import EngineConfig, GenRequest, LLMEngine, SamplingParams
from llm_mcp_amd.models import config as mc
from llm_mcp_amd.models.registry import model_class
from llm_mcp_amd.models.weights import load_weights, save_layer_list
from llm_mcp_amd.models.zegopel import ZegopelModel, tensor_shapes
from zegopel_cases import CASES, config, layer, shapes, tokens, weights
from zegopel_cases import ATTN, LIGHT, MAMBA, MLP

GPU = pytest.mark.gpu
RUNS = [pytest.param("cpu", "float32", id="cpu-fp32"),
        pytest.param("cuda", "float32", id="gpu-fp32", marks=GPU),
        pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=GPU)]
# rms error over the vocabulary, relative to the logits' own rms
TOL = {"float32": 2e-5, "bfloat16": 0.04}


def product_config(cfg, name="case"):
    return mc.ZegopelConfig.from_json(cfg, name)


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


_REF = {}


def reference(case, seed, toks):
    cfg = CASES[case] if isinstance(case, str) else case
    key = (case if isinstance(case, str) else json.dumps(case), seed, tuple(toks))
    if key not in _REF:
        _REF[key] = oracle.forward(cfg, weights(cfg, seed), toks)
    return _REF[key]


def error(got, want):
    got, want = got.double(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.std()).max())


def check(got, want, dtype, what=""):
    e = error(got, want)
    assert e < TOL[dtype], f"{what}: {e:.2e}"


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", sorted(CASES))
def test_whole_prompt_and_decode(case, device, dtype):
    """Every position of one prompt in one step, then the same tokens with the
    tail one by one: the state and cache the prompt left must be the ones a
    longer prompt would have used."""
    cfg = CASES[case]
    n, tail = 90, 12
    toks = tokens(cfg, n)
    want = reference(case, 0, toks)
    e = engine(cfg, weights(cfg), device, dtype)
    check(e.feed([(1, toks, list(range(n)))], [1]), want, dtype, "whole")
    check(e.feed([(2, toks[:n - tail], list(range(n - tail)))]), want[:n - tail], dtype, "prompt")
    for t in range(n - tail, n):
        y = e.feed([(2, toks[t:t + 1], [0])], [2] if t == n - 1 else [])
        check(y, want[t:t + 1], dtype, f"decoded {t}")
    assert e.sched.kv_usage == 0.0


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "reordered", "odd"])
def test_token_by_token_from_the_start(case, device, dtype):
    cfg = CASES[case]
    toks = tokens(cfg, 40, seed=3)
    want = reference(case, 0, toks)
    e = engine(cfg, weights(cfg), device, dtype)
    got = torch.cat([e.feed([(7, [t], [0])]) for t in toks])
    check(got, want, dtype)


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "reordered", "fast"])
def test_portions(case, device, dtype):
    """Portions cut inside pages and chunks, down to two tokens and one."""
    cfg = CASES[case]
    n = 150
    toks = tokens(cfg, n, seed=5)
    want = reference(case, 0, toks)
    e = engine(cfg, weights(cfg), device, dtype)
    for k, cuts in enumerate([[2] * 20, [31, 1, 2, 33, 64, 3, 16], [65, 2, 2], [1, 149]]):
        at = 0
        for c in cuts:
            y = e.feed([(k + 1, toks[at:at + c], list(range(c)))])
            check(y, want[at:at + c], dtype, f"cuts {k} at {at}")
            at += c
        e.feed([], [k + 1])


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("case", ["mixed", "reordered"])
def test_unequal_requests_share_steps_pages_and_slots(case, device, dtype):
    """Up to four live requests of unequal lengths in shared steps, portions
    beside decoded tokens, some left out of a step; requests end and their
    pages and slots go to the next ones (seven requests, a pool of four)."""
    cfg = CASES[case]
    lens = [70, 1, 33, 64, 5, 90, 32]
    reqs = {i + 1: tokens(cfg, n, seed=10 + i) for i, n in enumerate(lens)}
    want = {i: reference(case, 0, t) for i, t in reqs.items()}
    e = engine(cfg, weights(cfg), device, dtype, tokens=288)
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
            check(y[k:k + n], want[r][a:a + n], dtype, f"request {r} at {a}")
            k += n
        live = [r for r in live if r not in end]
    assert e.sched.kv_usage == 0.0


@pytest.mark.parametrize("device,dtype", RUNS)
def test_request_alone_and_in_a_batch_agree(device, dtype):
    cfg = CASES["reordered"]
    W = weights(cfg)
    toks = [tokens(cfg, n, seed=20 + n) for n in (3, 65, 40)]
    e = engine(cfg, W, device, dtype)
    alone = [e.feed([(9, t, list(range(len(t))))], [9]) for t in toks]
    both = e.feed([(i + 1, t, list(range(len(t)))) for i, t in enumerate(toks)], [1, 2, 3])
    assert error(both, torch.cat(alone)) < TOL[dtype] / 2


@pytest.mark.parametrize("device,dtype", RUNS)
def test_generation_is_greedy_of_the_reference(device, dtype):
    """The engine's own entry point: batches of unequal prompts through the
    scheduler, the sampler and (on the GPU) the captured decode graphs."""
    cfg = CASES["mixed"]
    W = weights(cfg, 4)
    e = engine(cfg, W, device, dtype, graphs=device == "cuda")
    prompts = [tokens(cfg, n, seed=30 + n) for n in (1, 5, 40, 66, 2, 31)]
    new = 24
    outs = e.generate(prompts, SamplingParams(temperature=0, max_tokens=new, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o) == new
        lg = oracle.forward(cfg, W, p + o)[len(p) - 1:-1]
        short = lg.max(-1).values - lg[torch.arange(new), torch.tensor(o)]
        # a token may only differ from the reference's where that is a near tie
        assert float(short.max()) < 4 * TOL[dtype] * float(lg.std())
    if device == "cuda":
        assert e.stats["graph_steps"] > 0


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=GPU)])
def test_served_requests_come_and_go(device):
    """The engine thread with requests submitted while others run (lookahead
    stepping on the GPU): every stream equals the same request alone, whatever
    slots and pages it got; a stop token ends one early."""
    cfg = CASES["mixed"]
    W = weights(cfg, 8)
    e = engine(cfg, W, device, "float32", seqs=3, graphs=device == "cuda")
    prompts = [tokens(cfg, n, seed=60 + n) for n in (4, 35, 1, 70, 20, 9, 50)]
    sp = SamplingParams(temperature=0, max_tokens=20, ignore_eos=True)
    alone = [e.generate([p], sp)[0] for p in prompts]
    got, done = {}, threading.Event()

    def sink(evs):
        for v in evs:
            got.setdefault(v.req.user, []).append(v.token)
            if v.finish is not None and all(r.finished for r in reqs):
                done.set()
    reqs = []
    e.event_sink = sink
    stop = alone[3][7]
    e.start()
    try:
        for i, p in enumerate(prompts):
            params = sp if i != 3 else SamplingParams(temperature=0, max_tokens=20,
                                                      stop_token_ids=[stop])
            reqs.append(e.submit(GenRequest(p, params, user=i)))
            time.sleep(0.01)
        assert done.wait(60)
    finally:
        e.stop()
    want = dict(enumerate(alone))
    want[3] = alone[3][:alone[3].index(stop) + 1]
    assert got == want


@pytest.mark.parametrize("device,dtype", RUNS)
def test_preemption_recomputes_the_state(device, dtype):
    """A pool too small for every request: preempted sequences lose pages and
    slot and come back through a recomputed prompt."""
    cfg = CASES["mixed"]
    W = weights(cfg, 6)
    e = engine(cfg, W, device, dtype, tokens=192, graphs=device == "cuda")
    prompts = [tokens(cfg, 50, seed=40 + i) for i in range(4)]
    outs = e.generate(prompts, SamplingParams(temperature=0, max_tokens=30, ignore_eos=True))
    assert e.sched.preemptions > 0
    for p, o in zip(prompts, outs):
        lg = oracle.forward(cfg, W, p + o)[len(p) - 1:-1]
        short = lg.max(-1).values - lg[torch.arange(len(o)), torch.tensor(o)]
        assert len(o) == 30 and float(short.max()) < 4 * TOL[dtype] * float(lg.std())


@pytest.mark.parametrize("device,dtype", RUNS)
def test_long_decoding(device, dtype):
    cfg = CASES["mixed"]
    toks = tokens(cfg, 200, seed=50)
    want = reference("mixed", 0, toks)
    e = engine(cfg, weights(cfg), device, dtype)
    e.feed([(1, toks[:30], [])])
    for t in range(30, 200):
        y = e.feed([(1, toks[t:t + 1], [0] if t % 10 == 9 else [])])
        if t % 10 == 9:
            check(y, want[t:t + 1], dtype, f"decoded {t}")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_a_planted_mistake_shows(device, dtype):
    """The weights of the tests are sharp enough: the reference with one
    mechanism wrong is far outside the tolerance the product meets."""
    cfg = CASES["mixed"]
    W = weights(cfg)
    toks = tokens(cfg, 70)
    got = engine(cfg, W, device, dtype).feed([(1, toks, list(range(70)))])
    check(got, reference("mixed", 0, toks), dtype)

    def changed(i, **over):
        c = json.loads(json.dumps(cfg))
        c["layers"][i]["mixer"].update(over)
        return c
    wrong = {
        "decay": (changed(0, decay=[0.72, 0.985]), W),
        "temperature": (changed(2, q_temp=dict(coef=0.4, every=17)), W),
        "scale": (changed(2, scale=0.22), W),
        "part norms": (changed(1, norm_groups=1), W),
        "dt bias": (cfg, {**W, "l1.mix.dt_bias": W["l1.mix.dt_bias"] + 0.3}),
        "skip": (cfg, {**W, "l1.mix.D": W["l1.mix.D"] * 0.8}),
        "key bias": (cfg, {**W, "l2.mix.k.b": W["l2.mix.k.b"] * 0}),
        "oldest tap": (cfg, {**W, "l2.mix.v.conv": torch.cat(
            [W["l2.mix.v.conv"][:, :1] * 0, W["l2.mix.v.conv"][:, 1:]], 1)}),
    }
    for name, (c, w) in wrong.items():
        assert error(got, oracle.forward(c, w, toks)) > TOL[dtype], name


# ------------------------------------------------- configuration, loading ----
def test_checkpoint_directory_round_trip(tmp_path):
    cfg = CASES["reordered"]
    W = weights(cfg)
    pc = product_config(cfg)
    assert {k: tuple(v) for k, v in tensor_shapes(pc).items()} == shapes(cfg)
    save_layer_list(W, pc, str(tmp_path))
    back = mc.resolve(str(tmp_path))
    assert back.family == "zegopel" and model_class(back) is ZegopelModel
    assert (back.layers, back.vocab_size, back.hidden_size, back.rms_eps) == \
        (pc.layers, pc.vocab_size, pc.hidden_size, pc.rms_eps)
    W2 = load_weights(str(tmp_path), back, "cpu")
    assert all(torch.equal(W[k], W2[k]) for k in W)
    assert back.params == sum(t.numel() for t in W.values())
    bad = dict(W, head=W["head"][:-1])
    save_layer_list(bad, pc, str(tmp_path))
    with pytest.raises(ValueError, match="head"):
        load_weights(str(tmp_path), back, "cpu")


def test_unknown_mechanisms_are_refused():
    with pytest.raises(ValueError, match="mixer"):
        product_config(config([layer("recurrent", LIGHT)]))
    with pytest.raises(ValueError, match="feed-forward"):
        product_config(config([layer("lightning", LIGHT, dict(kind="experts", ff=8))]))
    with pytest.raises(ValueError, match="decay"):
        ZegopelModel(product_config(config([layer("lightning", LIGHT, decay=[0.5])])), "cpu")


def test_presets_and_layer_subsets():
    full = mc.resolve("zegopel-8b")
    assert 7.5 < full.params_b < 8.5
    assert mc.resolve("zegopel-8b@L3").num_layers == 3
    e = LLMEngine(EngineConfig(model="tiny-zegopel", max_num_seqs=2, max_batched_tokens=64,
                               max_model_len=128, use_graphs=False), device="cpu")
    out = e.generate([[1, 2, 3], [9] * 40], SamplingParams(temperature=0.8, seed=3, max_tokens=5,
                                                          ignore_eos=True))
    assert [len(o) for o in out] == [5, 5] and e.sched.prefix_hits == 0


def test_models_without_one_of_the_caches():
    """Only recurrent layers (no pages to hold), only attention layers."""
    for L in ([layer("lightning", LIGHT)], [layer("mamba2", MAMBA, MLP)],
              [layer("attention", ATTN), layer("attention", ATTN, MLP, conv=1)]):
        cfg = config(L)
        W = weights(cfg)
        toks = tokens(cfg, 37)
        e = engine(cfg, W, "cpu", "float32")
        y = torch.cat([e.feed([(1, toks[:20], list(range(20)))]),
                       e.feed([(1, toks[20:], list(range(17)))])])
        check(y, oracle.forward(cfg, W, toks), "float32")


# ------------------------------------------------------------ feed / trace ----
def test_feed_refuses_bad_steps():
    cfg = CASES["mixed"]
    e = engine(cfg, weights(cfg), "cpu", "float32", tokens=64)
    with pytest.raises(ValueError):
        e.feed([(1, [cfg["vocab"]], [])])
    with pytest.raises(ValueError):
        e.feed([(1, [3], [1])])
    with pytest.raises(ValueError):
        e.feed([(1, [3], []), (1, [4], [])])
    with pytest.raises(ValueError):
        e.feed([(1, [3] * 65, [])])          # more than the pool


def test_step_larger_than_the_budget_is_split():
    cfg = CASES["mixed"]
    toks = tokens(cfg, 100)
    e = engine(cfg, weights(cfg), "cpu", "float32", max_batched_tokens=24)
    y = e.feed([(1, toks[:60], list(range(60))), (2, toks[:9], [8, 0])])
    want = reference("mixed", 0, toks)
    check(y[:60], want[:60], "float32")
    check(y[60:], want[[8, 0]], "float32")


def test_trace_replay(tmp_path):
    from llm_mcp_amd.engine import trace
    cfg = CASES["mixed"]
    W = weights(cfg)
    save_layer_list(W, product_config(cfg), str(tmp_path / "m"))
    e = trace.build_engine(str(tmp_path / "m"), "float32", 130, 4, "cpu")
    assert e.num_blocks == 5 and len(e.states[0]) == 4
    toks = tokens(cfg, 40)
    want = reference("mixed", 0, toks)
    out = tmp_path / "out"
    out.mkdir()
    lines = [json.dumps(s) + "\n" for s in (
        {"step": 0, "entries": [{"id": "x", "tokens": toks[:11], "want": [10, 3]}], "end": []},
        {"step": 1, "entries": [{"id": "x", "tokens": toks[11:30], "want": []},
                                {"id": "y", "tokens": toks[:2], "want": [1]}], "end": ["y"]},
        {"step": 2, "entries": [{"id": "x", "tokens": toks[30:31], "want": []}], "end": []},
        {"step": 3, "entries": [{"id": "y", "tokens": toks[:1], "want": [0]},
                                {"id": "x", "tokens": toks[31:], "want": [0, 8]}],
         "end": ["x", "y"]})]
    said = []
    trace.replay(e, lines, str(out), said.append)
    assert said == ["done 0", "done 1", "done 2", "done 3"]
    assert sorted(p.name for p in out.iterdir()) == ["0.f32", "1.f32", "3.f32"]
    for step, places in ((0, [10, 3]), (1, [1]), (3, [0, 31, 39])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        check(torch.from_numpy(got.copy()), want[places], "float32")
    assert e.sched.kv_usage == 0.0


def test_feed_serves_other_families_too():
    """Teacher-forced steps are the engine's, not one model's: portions of a
    Llama sequence give the logits of the whole prompt."""
    e = LLMEngine(EngineConfig(model="tiny-llama", max_num_seqs=2, max_batched_tokens=256,
                               max_model_len=256, use_graphs=False), device="cpu")
    toks = list(range(20, 90))
    whole = e.feed([(1, toks, list(range(70)))], [1])
    parts = torch.cat([e.feed([(2, toks[a:b], list(range(b - a)))])
                       for a, b in ((0, 33), (33, 34), (34, 70))])
    assert float((whole - parts).abs().max()) < 0.05 * float(whole.std())
