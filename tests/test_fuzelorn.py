"""Fuzelorn through the engine, and its mechanisms one by one, against the
plain float64 model of tests/fuzelorn_oracle.py.

Engine cases write a small random checkpoint, build an engine on it and
replay a step plan with the product's trace replay (the scheduler's pages
and state slots, the runner's batches, the model's kernels); op cases drive
single ops with inputs made so that a fault shows (one key that must win
just inside, just outside and far from a window's edge; a sink that takes
nearly all the weight; a state that only an early token wrote; decays next
to 0 and 1; junk in slots and pages that are used again; corrections that
turn a choice of groups). CPU cases run the reference ops, gpu-marked ones
the HIP kernels in float32 and bfloat16.
"""

import io
import json
import os

import numpy as np
import pytest
import torch

import fuzelorn_oracle as O

CASES = [
    pytest.param("cpu", "float32", id="cpu-f32"),
    pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu),
]
GPU_CASES = [c for c in CASES if c.id != "cpu-f32"]
TOL = {"float32": 2e-4, "bfloat16": 8e-2}
TDT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64

A, R, MOE, DENSE, LAYER = (O.left_spec, O.right_spec, O.moe_spec, O.dense_spec,
                           O.layer_spec)


# ------------------------------------------------------------------ helpers
def write_checkpoint(path, cfg, seed=0):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    w = O.random_weights(cfg, seed)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()},
              os.path.join(path, "model.safetensors"))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    return w


def make_engine(path, device, dtype, max_tokens=256, **kw):
    from arks_amd.config import EngineConfig
    from arks_amd.engine import LLMEngine

    cfg = EngineConfig(model_path=str(path), device=device, dtype=dtype,
                       kv_cache_blocks=-(-max_tokens // 16), max_num_seqs=4,
                       max_model_len=max_tokens, max_num_batched_tokens=max_tokens,
                       enable_prefix_caching=False, **kw)
    return LLMEngine(cfg)


def replay(engine, tmp_path, steps):
    """steps: lists of (request id, tokens, end?); logits of every token.
    Returns {id: [n_tokens, vocab]}."""
    from arks_amd.engine.trace import replay as trace_replay

    out = tmp_path / "out"
    out.mkdir(exist_ok=True)
    lines = [json.dumps({
        "step": n,
        "entries": [{"id": i, "tokens": t, "want": list(range(len(t)))}
                    for i, t, _ in step],
        "end": [i for i, _, e in step if e]}) for n, step in enumerate(steps)]
    trace_replay(engine, lines, str(out), log=io.StringIO())
    got = {}
    V = engine.model_cfg.vocab_size
    for n, step in enumerate(steps):
        arr = np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, V)
        at = 0
        for i, t, _ in step:
            got.setdefault(i, []).append(arr[at:at + len(t)])
            at += len(t)
    return {i: np.concatenate(v) for i, v in got.items()}


def portions(tokens, sizes):
    out, at, k = [], 0, 0
    while at < len(tokens):
        n = sizes[k % len(sizes)]
        out.append(tokens[at:at + n])
        at += n
        k += 1
    return out


def toks(n, vocab=96, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


_WANT = {}


def wanted(cfg, w, t):
    """Oracle logits and router margins, once per model and sequence (id(w)
    names the model while its weights live, and the entry keeps them)."""
    key = (id(w), tuple(t))
    if key not in _WANT:
        margins = []
        _WANT[key] = (O.forward(cfg, w, t, margins)[0], margins, w)
    return _WANT[key][:2]


def assert_logits(got, cfg, w, t, dtype, note=None):
    """got [n, vocab] against the oracle's first n rows: every row, but in
    bfloat16 with routers that choose only the rows in front of the first
    close call. There a reduced-precision run may choose otherwise, which is
    another function, and the states carry that on to later rows; the
    typical row must be well inside all the same."""
    n = got.shape[0]
    want, margins = wanted(cfg, w, t)
    want = want[:n].numpy()
    err = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    if dtype == "bfloat16" and margins:
        assert np.median(err) < TOL[dtype] / 2, note
        err = err[:O.clear_rows(margins)]
    assert not err.size or err.max() < TOL[dtype], (note, int(err.argmax()))


# --------------------------------------------------- the model in the engine
def routed_config():
    """Every feed-forward kind, a looped pair of layers, windows from one
    token to longer than the prompt."""
    return O.make_config(
        [LAYER(mlp=DENSE()), LAYER(A(window=3), mlp=MOE()),
         LAYER(right=R(heads=3, kv_heads=3, conv=2)),
         LAYER(A(window=500, heads=6, kv_heads=1),
               mlp=MOE(top=1, groups=2, keep=1))], loop=(1, 3, 2))


def plain_config():
    """The same without routers, whose close calls make a comparison in
    bfloat16 blunt."""
    return O.make_config(
        [LAYER(mlp=DENSE()), LAYER(A(window=3)),
         LAYER(right=R(heads=3, kv_heads=3, conv=2), mlp=DENSE(17)),
         LAYER(A(window=500, heads=6, kv_heads=1))], loop=(1, 3, 3))


CONFIGS = {"routed": routed_config, "plain": plain_config}


@pytest.mark.parametrize("device,dtype", CASES)
def test_residual_after_every_layer_run(tmp_path, device, dtype):
    cfg = routed_config()
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(23)
    _, after = O.forward(cfg, w, t)
    eng = make_engine(tmp_path / "m", device, dtype)
    seen = {}
    eng.runner.model.residual_tap = lambda i, x: seen.__setitem__(
        i, x.detach().clone().float().cpu())
    replay(eng, tmp_path, [[("a", t, True)]])
    assert sorted(seen) == list(range(len(after))) and len(after) == 6
    for i, want in enumerate(after):
        row = (seen[i].double() - want).abs().amax(-1) / want.abs().max()
        # a close call of a router may flip a row in bfloat16
        worst = row.max() if dtype == "float32" else row.median()
        assert float(worst) < (1e-4 if dtype == "float32" else 3e-2), i


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_against_decode_and_portions(tmp_path, device, dtype, name):
    cfg = CONFIGS[name]()
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(70)
    for name, plan in {
        "whole": [t],
        "decode": [t[:9]] + [[x] for x in t[9:]],
        "small": portions(t, [2, 3, 5, 2, 7]),
        "pairs": portions(t, [2]),
        "odd": portions(t, [13, 1, 2, 17]),
        "tokens": [[x] for x in t[:40]],
    }.items():
        eng = make_engine(tmp_path / "m", device, dtype)
        steps = [[("a", p, False)] for p in plan]
        got = replay(eng, tmp_path, steps)["a"]
        assert_logits(got, cfg, w, t, dtype, name)


def mixed_plan(reqs, slots, pool_pages, sizes):
    """Steps in which unequal requests run side by side, portions beside
    single tokens, some sitting a step out; never more than `slots` live
    and never more pages than the pool holds."""
    at = {c: 0 for c in reqs}
    live, waiting, steps = [], list(reqs), []
    k = 0
    while live or waiting:
        while waiting and len(live) < slots and \
                sum(-(-len(reqs[c]) // 16) for c in live + waiting[:1]) <= pool_pages:
            live.append(waiting.pop(0))
        step = []
        for c in list(live):
            if (k + ord(c)) % 5 == 0 and len(live) > 1:
                k += 1
                continue  # this request sits the step out
            n = min(sizes[k % len(sizes)], len(reqs[c]) - at[c])
            k += 1
            part = reqs[c][at[c]:at[c] + n]
            at[c] += n
            done = at[c] == len(reqs[c])
            step.append((c, part, done))
            if done:
                live.remove(c)
        if step:
            steps.append(step)
    return steps


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches_and_reuse(tmp_path, device, dtype, name):
    """More requests than state slots over time and a pool just large
    enough, so pages and slots are given back and taken again."""
    cfg = CONFIGS[name]()
    w = write_checkpoint(tmp_path / "m", cfg)
    reqs = {c: toks(n, seed=s) for c, n, s in
            [("a", 61, 1), ("b", 18, 2), ("c", 33, 3), ("d", 5, 4),
             ("e", 47, 5), ("f", 29, 6), ("g", 40, 7)]}
    steps = mixed_plan(reqs, 4, 12, [7, 1, 2, 16, 1, 1, 3, 11])
    eng = make_engine(tmp_path / "m", device, dtype, max_tokens=192)
    got = replay(eng, tmp_path, steps)
    for c in reqs:
        assert got[c].shape[0] == len(reqs[c])
        assert_logits(got[c], cfg, w, reqs[c], dtype, c)


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_decode(tmp_path, device, dtype):
    """150 single tokens: the window passes over ten pages that filled up
    one token at a time, the state is carried by every one of them."""
    cfg = O.make_config([LAYER(A(window=37)),
                         LAYER(mlp=MOE(top=6, groups=2, keep=2))])
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(150)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", t[:5], False)]] + [[("a", [x], False)] for x in t[5:]]
    got = replay(eng, tmp_path, steps)["a"]
    assert_logits(got, cfg, w, t, dtype)


OTHER_SIZES = {
    "one-kv-head": dict(layers=[LAYER(A(heads=6, kv_heads=1),
                                      R(heads=6, kv_heads=1))]),
    "all-kv-heads": dict(layers=[LAYER(A(heads=3, kv_heads=3),
                                       R(heads=3, kv_heads=3))]),
    "one-head": dict(layers=[LAYER(A(heads=1, kv_heads=1),
                                   R(heads=1, kv_heads=1))]),
    "eighteen-heads": dict(layers=[LAYER(A(heads=18, kv_heads=1, dim=4),
                                         R(heads=10, kv_heads=5, dim=4))]),
    "dim-one": dict(layers=[LAYER(A(dim=1, vdim=1))]),
    "wide-values": dict(layers=[LAYER(A(dim=4, vdim=72), R(dim=4, vdim=72))]),
    "wide-keys": dict(layers=[LAYER(A(dim=140, vdim=6), R(dim=140, vdim=6))]),
    "wide-both": dict(layers=[LAYER(A(heads=2, dim=96, vdim=130),
                                    R(heads=1, kv_heads=1, dim=40, vdim=200))]),
    "no-history": dict(layers=[LAYER(right=R(conv=1))]),
    "two-taps": dict(layers=[LAYER(right=R(conv=2))]),
    "twelve-taps": dict(layers=[LAYER(right=R(conv=12, dim=16, vdim=16))]),
    "window-one": dict(layers=[LAYER(A(window=1))]),
    "window-two": dict(layers=[LAYER(A(window=2))]),
    "window-page": dict(layers=[LAYER(A(window=16))]),
    "window-above": dict(layers=[LAYER(A(window=500))]),
    "temperature-every-token": dict(layers=[LAYER(A(every=1, coef=1.5))]),
    "temperature-negative": dict(layers=[LAYER(A(every=5, coef=-0.2))]),
    "temperature-none": dict(layers=[LAYER(A(coef=0.0))]),
    "sharp-scores": dict(layers=[LAYER(A(scale=2.0))]),
    "scale-one": dict(layers=[LAYER(A(scale=1.0))]),
    "top-one": dict(layers=[LAYER(mlp=MOE(top=1))]),
    "top-all": dict(layers=[LAYER(mlp=MOE(experts=4, top=4, groups=2, keep=2))]),
    "one-group": dict(layers=[LAYER(mlp=MOE(groups=1, keep=1, top=3))]),
    "groups-of-one": dict(layers=[LAYER(mlp=MOE(experts=5, groups=5, keep=3))]),
    "one-expert": dict(layers=[LAYER(mlp=MOE(experts=1, top=1, groups=1, keep=1))]),
    "many-experts": dict(layers=[LAYER(mlp=MOE(experts=72, top=5, ff=8, groups=9,
                                               keep=4))]),
    "no-limit-in-reach": dict(layers=[LAYER(mlp=MOE(limit=90.0, shared_limit=70.0))]),
    "tight-limits": dict(layers=[LAYER(mlp=MOE(limit=0.1, shared_limit=0.2))]),
    "shared-wider": dict(layers=[LAYER(mlp=MOE(ff=8, shared_ff=50))]),
    "loop-all": dict(layers=[LAYER(mlp=DENSE(9)), LAYER()], loop=(0, 2, 3)),
    "loop-once": dict(layers=[LAYER(), LAYER()], loop=(1, 2, 1)),
    "loop-last": dict(layers=[LAYER(), LAYER(mlp=DENSE(5))], loop=(1, 2, 4)),
    "tight-cap": dict(layers=[LAYER()], cap=0.7),
    "scale-one-embedding": dict(layers=[LAYER()], scale=1.0),
    "one-bucket": dict(layers=[LAYER()], buckets=1),
    "many-buckets": dict(layers=[LAYER()], buckets=9001, mul_prev=90001,
                         mul_cur=70001),
    "hash-sees-one-token": dict(layers=[LAYER()], mul_prev=0),
    "odd-everything": dict(layers=[
        LAYER(A(heads=3, kv_heads=1, dim=7, vdim=11, window=5),
              R(heads=3, kv_heads=1, dim=5, vdim=7, conv=3),
              MOE(experts=6, top=2, ff=13, groups=2, keep=1, shared_ff=9)),
        LAYER(A(heads=9, kv_heads=3, dim=3, vdim=5),
              R(heads=5, kv_heads=5, dim=9, vdim=3, conv=5), DENSE(19))],
        width=43, vocab=97, eps=1e-3, loop=(0, 1, 2)),
}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(OTHER_SIZES))
def test_other_sizes(tmp_path, device, dtype, name):
    cfg = O.make_config(**OTHER_SIZES[name])
    w = write_checkpoint(tmp_path / "m", cfg, seed=3)
    t = toks(38, vocab=cfg["vocab"], seed=9)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", p, False)] for p in portions(t, [11, 2, 1, 6])]
    got = replay(eng, tmp_path, steps)["a"]
    assert_logits(got, cfg, w, t, dtype)


def fast_path_config(mlp=None):
    """Sizes the vectorised and matrix-core kernels are built for, with
    windows shorter than the prompts."""
    return O.make_config(
        [LAYER(A(heads=4, kv_heads=2, dim=64, vdim=64, window=70),
               R(heads=4, kv_heads=2, dim=64, vdim=64), mlp),
         LAYER(A(heads=6, kv_heads=1, dim=128, vdim=64, window=100),
               R(heads=2, kv_heads=2, dim=128, vdim=128)),
         LAYER(A(heads=2, kv_heads=2, dim=96, vdim=96, window=33),
               R(heads=3, kv_heads=1, dim=32, vdim=48), DENSE(64)),
         LAYER(A(heads=2, kv_heads=1, dim=64, vdim=32, window=65),
               R(heads=1, kv_heads=1, dim=96, vdim=16))], width=64)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
def test_fast_path_sizes(tmp_path, device, dtype):
    """Prompts across 64-row chunk and tile edges, single rows after them."""
    cfg = fast_path_config(MOE(experts=8, top=2, ff=32, groups=4, keep=2,
                               shared_ff=24))
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(470, seed=11)
    eng = make_engine(tmp_path / "m", device, dtype, max_tokens=512)
    plan = [t[:130], t[130:131], t[131:197], t[197:198], t[198:199],
            t[199:201], t[201:]]
    assert len(plan[-1]) > 256
    got = replay(eng, tmp_path, [[("a", p, False)] for p in plan])["a"]
    assert_logits(got, cfg, w, t, dtype)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
def test_decoded_rows_beside_long_portions(tmp_path, device, dtype):
    """Single rows of two requests, in front of and behind a portion that
    fills a 256-row tile."""
    cfg = fast_path_config()
    w = write_checkpoint(tmp_path / "m", cfg)
    ta, tb, tc = toks(95, seed=5), toks(560, seed=6), toks(40, seed=7)
    eng = make_engine(tmp_path / "m", device, dtype, max_tokens=768)
    steps = [[("a", ta[:93], False), ("c", tc[:38], False)],
             [("a", ta[93:94], False), ("b", tb[:300], False),
              ("c", tc[38:39], False)],
             [("b", tb[300:], False), ("c", tc[39:], False),
              ("a", ta[94:], False)]]
    got = replay(eng, tmp_path, steps)
    for c, t in (("a", ta), ("b", tb), ("c", tc)):
        assert_logits(got[c], cfg, w, t, dtype, c)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
def test_fast_path_sizes_in_mixed_batches(tmp_path, device, dtype):
    cfg = fast_path_config()
    w = write_checkpoint(tmp_path / "m", cfg)
    reqs = {c: toks(n, seed=s) for c, n, s in
            [("a", 350, 1), ("b", 70, 2), ("c", 201, 3), ("d", 9, 4),
             ("e", 66, 5)]}
    steps = mixed_plan(reqs, 3, 42, [67, 1, 1, 270, 2, 1, 33, 1, 90])
    eng = make_engine(tmp_path / "m", device, dtype, max_tokens=672)
    got = replay(eng, tmp_path, steps)
    for c in reqs:
        assert_logits(got[c], cfg, w, reqs[c], dtype, c)


@pytest.mark.parametrize("device,dtype", CASES)
def test_sorted_expert_segments(tmp_path, device, dtype, monkeypatch):
    """Steps above DENSE_TOKENS rows sort (row, expert) pairs by expert;
    below they run every expert with factor 0 where unused: same logits."""
    from arks_amd.models.feedforward import RoutedMoE

    monkeypatch.setattr(RoutedMoE, "DENSE_TOKENS", 6)
    cfg = O.make_config([LAYER(mlp=MOE(experts=6, top=3)),
                         LAYER(mlp=MOE(experts=4, top=1, groups=2, keep=1,
                                       ff=16, shared_ff=40))])
    w = write_checkpoint(tmp_path / "m", cfg)
    ta, tb = toks(50, seed=2), toks(31, seed=3)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", ta[:21], False)], [("a", ta[21:24], False), ("b", tb[:30], False)],
             [("a", ta[24:43], False), ("b", tb[30:31], True)],
             [("a", ta[43:], True)]]
    got = replay(eng, tmp_path, steps)
    assert_logits(got["a"], cfg, w, ta, dtype)
    assert_logits(got["b"], cfg, w, tb, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
def test_layers_without_router_extras(tmp_path, device, dtype):
    """A routed layer without groups and without a shared expert."""
    mlp = MOE(groups=1, keep=1)
    del mlp["router"]["groups"]
    mlp["shared"] = None
    cfg = O.make_config([LAYER(mlp=mlp)])
    w = write_checkpoint(tmp_path / "m", cfg)
    mlp["router"]["groups"] = {"count": 1, "keep": 1}  # what the oracle reads
    t = toks(30)
    eng = make_engine(tmp_path / "m", device, dtype)
    got = replay(eng, tmp_path, [[("a", t[:17], False)], [("a", t[17:], True)]])
    assert_logits(got["a"], cfg, w, t, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
def test_greedy_generation(tmp_path, device, dtype):
    """LLMEngine.generate (scheduler, sampler, captured decode steps on the
    GPU) picks the oracle's tokens; three prompts share the batch."""
    from arks_amd.engine import SamplingParams

    cfg = plain_config()
    w = write_checkpoint(tmp_path / "m", cfg)
    prompts = [toks(19, seed=4), toks(3, seed=5), toks(34, seed=6)]
    eng = make_engine(tmp_path / "m", device, dtype)
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True,
                                                temperature=0.0))
    for p, o in zip(prompts, outs):
        seq = list(p) + list(o)
        assert len(o) == 12
        logits = O.forward(cfg, w, seq)[0]
        for n, tok in enumerate(o, start=len(p)):
            top2 = torch.topk(logits[n - 1], 2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == "float32" else 0.6):
                assert tok == int(logits[n - 1].argmax()), (n, tok)


@pytest.mark.parametrize("device,dtype", CASES)
def test_preempted_requests_start_over(tmp_path, device, dtype):
    """A pool too small for all requests: the scheduler gives pages back and
    recomputes, and the tokens are the ones of a request alone."""
    from arks_amd.engine import SamplingParams

    cfg = plain_config()
    write_checkpoint(tmp_path / "m", cfg)
    prompts = [toks(30, seed=s) for s in (4, 5, 6)]
    sp = SamplingParams(max_tokens=24, ignore_eos=True, temperature=0.0)
    small = make_engine(tmp_path / "m", device, dtype, max_tokens=128)
    got = small.generate(prompts, sp)
    alone = make_engine(tmp_path / "m", device, dtype)
    want = [alone.generate([p], sp)[0] for p in prompts]
    if dtype == "float32":
        assert got == want
    assert [len(o) for o in got] == [24] * 3


def test_config_round_trip_and_registry(tmp_path):
    from arks_amd.config import PRESET_CONFIGS, HybridModelConfig, ModelConfig
    from arks_amd.models import create_model

    cfg = PRESET_CONFIGS["tiny-fuzelorn"]
    again = HybridModelConfig.from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.layers == cfg.layers and not again.tied_head
    assert again.bigram == cfg.bigram and again.loop == cfg.loop
    assert again.logit_softcap == 30.0
    model = create_model(again)
    # six layer runs with caches of their own and the model's own state
    layout = model.cache_layout(16)
    assert len(layout) == 7 and set(layout[-1]) == {"prev_token"}
    assert model.state_slot_bytes() > 4
    raw = O.make_config([LAYER(mlp=MOE())])
    write_checkpoint(tmp_path / "m", raw)
    got = ModelConfig.from_pretrained(str(tmp_path / "m"))
    assert got.num_local_experts == 6
    assert got.bigram == {"buckets": 53, "mul_prev": 11, "mul_cur": 5}
    for key, value in (("buckets", 0), ("mul_prev", -1)):
        bad = json.loads(json.dumps(raw))
        bad["embedding"]["bigram"][key] = value
        with pytest.raises(ValueError):
            HybridModelConfig.from_dict(bad)
    for bad in ({"type": "latent_attention"}, {"mlp": {"kind": "other"}}):
        broken = json.loads(json.dumps(raw))
        broken["layers"][0].update(bad)
        with pytest.raises(ValueError):
            create_model(HybridModelConfig.from_dict(broken))


def test_preset_generates_with_random_weights():
    """The engine configuration of the command line builds the preset, and the
    random-init model generates."""
    from arks_amd.config import EngineConfig
    from arks_amd.engine import LLMEngine, SamplingParams

    eng = LLMEngine(EngineConfig(preset="tiny-fuzelorn", device="cpu",
                                 kv_cache_blocks=16, max_num_seqs=2,
                                 max_model_len=128, dtype="float32"))
    outs = eng.generate([[1, 2, 3], [4] * 20],
                        SamplingParams(max_tokens=4, ignore_eos=True))
    assert [len(o) for o in outs] == [4, 4]


# ------------------------------------------------------- mechanisms alone
def _dev(device):
    return torch.device(device)


def _rounded(x, dtype):
    """What the op will see: the value after rounding to its row dtype."""
    return x.to(TDT[dtype]).to(F64)


def _i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [13, 40, 2056])
def test_hashed_embedding_state(device, dtype, W):
    """Portions of 1, 2 and more tokens of two sequences, single-row steps
    (one launch), a padding row, and a slot used again: the first token has
    the last row whatever the slot holds."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    g = torch.Generator().manual_seed(2)
    E = _rounded(torch.randn(31, W, generator=g, dtype=F64), dtype)
    table = _rounded(torch.randn(8, W, generator=g, dtype=F64), dtype)
    spec = {"scale": 1.5, "bigram": {"buckets": 7, "mul_prev": 40000001,
                                     "mul_cur": 60000011}}
    seqs = {s: toks(30, vocab=31, seed=s) for s in (0, 1, 2)}
    want = {s: O.embed(t, {"embed": E, "bigram": table}, spec)
            for s, t in seqs.items()}
    prev = torch.full((4,), 29, dtype=torch.int32, device=dev)
    at = {0: 0, 1: 0, 2: 0}
    slot = {0: 3, 1: 1, 2: 3}
    for step in [[(0, 1), (1, 5)], [(0, 1), (1, 1)], [(1, 2), (0, 2)], [(0, 1)],
                 [(1, 1), (0, 1)], [(0, 9)], [(1, 4), (2, 1)], [(2, 1)],
                 [(2, 3), (1, 1)], [(1, 1), (2, 1)]]:
        cu = [0]
        for _, n in step:
            cu.append(cu[-1] + n)
        ids = sum([seqs[s][at[s]:at[s] + n] for s, n in step], [])
        x = ops.hashed_embed(
            torch.tensor(ids, device=dev), E.to(dt).to(dev),
            table.to(dt).to(dev), prev, _i32(cu, dev),
            _i32([at[s] + n for s, n in step], dev),
            _i32([slot[s] for s, _ in step], dev),
            _i32(sum([[j] * n for j, (_, n) in enumerate(step)], []), dev),
            1.5, 40000001, 60000011, max(n for _, n in step))
        assert x.dtype == torch.float32
        x = x.double().cpu()
        for j, (s, n) in enumerate(step):
            assert torch.allclose(x[cu[j]:cu[j + 1]], want[s][at[s]:at[s] + n],
                                  atol=1e-5, rtol=1e-6), (step, s)
            at[s] += n
    assert prev.tolist()[0] == 29 and prev.tolist()[2] == 29
    # a padding row (slot -1) reads no state and leaves none
    before = prev.clone()
    ops.hashed_embed(torch.zeros(1, dtype=torch.int64, device=dev),
                     E.to(dt).to(dev), table.to(dt).to(dev), prev,
                     _i32([0, 1], dev), _i32([1], dev), _i32([-1], dev),
                     _i32([0], dev), 1.5, 1, 1, 1)
    assert torch.equal(before, prev)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("sizes", [(3, 1, 7, 5), (4, 2, 8, 16), (8, 8, 24, 8),
                                   (32, 8, 128, 64), (40, 2, 128, 128),
                                   (70, 1, 128, 8)],
                         ids=lambda s: "x".join(map(str, s)))
def test_whole_row_norm_temperature_and_pages(device, dtype, sizes):
    """One root mean square for all heads of a row (a head of its own size
    would show: head 0 is much larger), the factor at its steps, only the
    row's own places in the pages."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    H, G, D, V = sizes
    T, first = 10, 6  # positions 6 .. 15 cross the factor's steps at 7 and 15
    nq, nk, nv = H * D, G * D, G * V
    g = torch.Generator().manual_seed(9)
    p = torch.randn(T, nq + nk + nv + (3 if D == 7 else 8), generator=g, dtype=F64)
    p[:, :D] *= 20.0
    p[4] = 0.0  # eps alone under the root
    p = _rounded(p, dtype)
    qw, kw = (torch.randn(n, generator=g, dtype=F64).float().double()
              for n in (nq, nk))
    temp = {"coef": 0.7, "every": 8}
    kc = torch.full((3, G, 16, D), 3.0, dtype=dt, device=dev)
    vc = torch.full((3, G, 16, V), 3.0, dtype=dt, device=dev)
    pos = torch.arange(first, first + T)
    slots = pos + 16
    slots[2] = -1
    pd = p.to(dt).to(dev)
    q = ops.row_norm_qk_cache(
        pd[:, :nq], pd[:, nq:nq + nk], pd[:, nq + nk:nq + nk + nv],
        qw.float().to(dev), kw.float().to(dev), 1e-4, pos.to(dev), 0.7, 8, kc,
        vc, slots.to(dev)).double().cpu()
    factor = O.query_factor(first + T, temp)[first:]
    assert len(set(factor.tolist())) == 3
    tol = 2e-5 if dtype == "float32" else 2e-2
    want_q = O.rms_norm(p[:, :nq], qw, 1e-4) * factor[:, None]
    assert torch.allclose(q, want_q, atol=tol, rtol=tol)
    want_k = O.rms_norm(p[:, nq:nq + nk], kw, 1e-4)
    want_v = p[:, nq + nk:nq + nk + nv]
    for cache, want, n in ((kc, want_k, D), (vc, want_v, V)):
        flat = cache.double().cpu().transpose(1, 2).reshape(-1, G * n)
        ok = slots >= 0
        assert torch.allclose(flat[slots[ok]], want[ok], atol=tol, rtol=tol)
        rest = torch.ones(flat.shape[0], dtype=torch.bool)
        rest[slots[ok]] = False
        assert float((flat[rest] - 3.0).abs().max()) == 0.0
    # no factor at all
    q = ops.row_norm_qk_cache(
        pd[:, :nq], pd[:, nq:nq + nk], pd[:, nq + nk:nq + nk + nv],
        qw.float().to(dev), kw.float().to(dev), 1e-4, pos.to(dev), 0.7, 0, kc,
        vc, slots.to(dev)).double().cpu()
    assert torch.allclose(q, O.rms_norm(p[:, :nq], qw, 1e-4), atol=tol, rtol=tol)


def test_slopes_of_any_head_count():
    from arks_amd.models.mixers import distance_slopes

    for H in (1, 3, 8, 12, 96):
        assert torch.allclose(distance_slopes(H).double(),
                              torch.tensor(O.bias_slopes(H), dtype=F64), rtol=1e-7)


class Pages:
    """One sequence's keys and values in pages handed out in a scrambled
    order, junk elsewhere."""

    def __init__(self, dev, dtype, k, v):
        n, G = k.shape[:2]
        nblk = -(-n // 16)
        g = torch.Generator().manual_seed(7)
        self.dev, self.dt = dev, TDT[dtype]
        self.table = torch.randperm(nblk + 3, generator=g)[:nblk].to(torch.int32)
        self.k, self.v = (torch.full((nblk + 3, G, 16, x.shape[2]), 9.0,
                                     dtype=self.dt, device=dev) for x in (k, v))
        pos = torch.arange(n)
        page = self.table[pos // 16].long().to(dev)
        for cache, x in ((self.k, k), (self.v, v)):
            cache[page, :, (pos % 16).to(dev)] = x.to(self.dt).to(dev)

    def attend(self, q, total, scale, window, slopes, sinks):
        from arks_amd import ops

        n = q.shape[0]
        f = lambda x: None if x is None else torch.tensor(
            [float(y) for y in x]).to(self.dev)
        out = ops.attention_sink_paged(
            q.to(self.dt).to(self.dev).contiguous(), self.k, self.v,
            self.table[None].to(self.dev), _i32([total], self.dev),
            _i32([0, n], self.dev), _i32([0] * n, self.dev), scale, False,
            None, False, n, None, sink_w=f(sinks), window=window,
            slopes=f(slopes))
        return out.double().cpu()


ATT_SIZES = [(3, 1, 10, 6), (8, 2, 64, 64), (4, 4, 128, 128), (6, 2, 128, 64),
             (18, 1, 96, 96), (5, 1, 64, 32), (4, 2, 96, 64)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("size", ATT_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_distance_bias_and_sink(device, dtype, size):
    """Every row of a prompt and the last row alone, random scores; the bias
    and the sink both matter (without either the outputs differ)."""
    H, G, D, V = size
    n, scale, window = 83, D ** -0.5, 50
    g = torch.Generator().manual_seed(3)
    q = _rounded(torch.randn(n, H, D, generator=g, dtype=F64) * 1.5, dtype)
    k = _rounded(torch.randn(n, G, D, generator=g, dtype=F64), dtype)
    v = _rounded(torch.randn(n, G, V, generator=g, dtype=F64), dtype)
    slopes, sinks = O.bias_slopes(H), (torch.randn(H, generator=g) + 1.0).tolist()
    of = [h // (H // G) for h in range(H)]
    want = O.biased_attend(q, k[:, of], v[:, of], scale, window, slopes, sinks)
    for s, z in (([0.0] * H, sinks), (slopes, [-60.0] * H)):
        other = O.biased_attend(q, k[:, of], v[:, of], scale, window, s, z)
        assert float((other - want).abs().max()) > 0.1
    pg = Pages(_dev(device), dtype, k, v)
    tol = 1e-4 if dtype == "float32" else 2e-2
    for first in (0, 18, n - 2, n - 1):
        got = pg.attend(q[first:], n, scale, window, slopes, sinks)
        assert torch.allclose(got, want[first:], atol=tol, rtol=tol), first


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size", [(4, 2, 10, 6), (4, 2, 64, 64), (8, 1, 128, 128)],
                         ids=lambda s: "x".join(map(str, s)))
def test_window_edges(device, dtype, decode, size):
    """One key carries a huge score: it takes all the weight as the last key
    inside the window, at a page border, far back and at the row itself
    (whatever the bias takes off), and leaves no trace as the first key
    outside."""
    H, G, D, V = size
    n, scale = 300, 0.5
    g = torch.Generator().manual_seed(5)
    i = n - 1
    q = torch.zeros(n, H, D, dtype=F64)
    q[i, :, 3] = 64.0
    slopes, sinks = O.bias_slopes(H), [0.5] * H
    of = [h // (H // G) for h in range(H)]
    v = _rounded(torch.randn(n, G, V, generator=g, dtype=F64), dtype)
    base = torch.randn(n, G, D, generator=g, dtype=F64) * 0.1
    for window, hot, seen in [(37, i - 36, True), (37, i - 37, False),
                              (37, 2, False), (300, 2, True), (300, 0, True),
                              (299, 0, False), (29, 271, True), (28, 271, False),
                              (28, 272, True), (1, i, True), (1, i - 1, False)]:
        k = base.clone()
        k[hot, :, 3] += 40.0
        k = _rounded(k, dtype)
        want = O.biased_attend(q, k[:, of], v[:, of], scale, window, slopes,
                               sinks, rows=[i])[i]
        assert torch.allclose(want[0], v[hot, 0], atol=1e-6) == seen
        pg = Pages(_dev(device), dtype, k, v)
        first = i if decode else n - 41
        got = pg.attend(q[first:], n, scale, window, slopes, sinks)[-1]
        tol = 1e-4 if dtype == "float32" else 1e-2
        assert torch.allclose(got, want, atol=tol, rtol=tol), (window, hot)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("D,V", [(10, 6), (64, 64), (64, 32)])
def test_sink_takes_its_share_at_the_first_tokens(device, dtype, D, V):
    """Equal scores 0: row i's output is the mean over i + 1 values shrunk by
    the sink's share, from the very first row on; a sink far above leaves
    next to nothing, one far below nothing of itself."""
    H, n = 3, 40
    g = torch.Generator().manual_seed(5)
    q = torch.zeros(n, H, D, dtype=F64)
    k = _rounded(torch.randn(n, 1, D, generator=g, dtype=F64), dtype)
    v = _rounded(torch.randn(n, 1, V, generator=g, dtype=F64), dtype)
    sinks = [1.0, 50.0, -50.0]
    pg = Pages(_dev(device), dtype, k, v)
    tol = 1e-4 if dtype == "float32" else 1e-2
    mean = v[:, 0].cumsum(0)
    count = torch.arange(1, n + 1, dtype=F64)[:, None]
    for first in (0, n - 1):
        got = pg.attend(q[first:], n, 1.0, 0, [0.0] * H, sinks)
        want = mean[first:] / (count[first:] + np.exp(1.0))
        assert torch.allclose(got[:, 0], want, atol=tol, rtol=tol)
        assert float(got[:, 1].abs().max()) < 1e-6
        assert torch.allclose(got[:, 2], mean[first:] / count[first:], atol=tol,
                              rtol=tol)


@pytest.mark.gpu
@pytest.mark.parametrize("size", [s for s in ATT_SIZES if s[2] in (64, 96, 128)],
                         ids=lambda s: "x".join(map(str, s)))
def test_matrix_core_attention_against_the_general_kernel(size, monkeypatch):
    """Long prompt with a window over several tiles, a portion in the middle
    and single rows."""
    from arks_amd import ops

    H, G, D, V = size
    n = 260
    g = torch.Generator().manual_seed(3)
    q, k, v = (_rounded(torch.randn(n, *s, generator=g, dtype=F64), "bfloat16")
               for s in ((H, D), (G, D), (G, V)))
    pg = Pages(_dev("cuda"), "bfloat16", k, v)
    args = (D ** -0.5, 90, O.bias_slopes(H), torch.randn(H, generator=g).tolist())
    for first in (0, 131, n - 1):
        fast = pg.attend(q[first:], n, *args)
        monkeypatch.setattr(ops, "use_masked_mfma", False)
        slow = pg.attend(q[first:], n, *args)
        monkeypatch.setattr(ops, "use_masked_mfma", True)
        assert torch.allclose(fast, slow, atol=1e-2, rtol=1e-2), first


@pytest.mark.gpu
@pytest.mark.parametrize("window", [1, 63, 64, 90, 300, 0])
@pytest.mark.parametrize("singles", [False, True], ids=["tiles", "single-rows"])
@pytest.mark.parametrize("H,G,D", [(8, 2, 64), (5, 1, 128), (3, 3, 64)])
def test_prefill_kernel_with_bias_and_sinks(H, G, D, singles, window):
    """The 256-row kernel over sequences of 1, 2, 70, 300 and 513 rows with
    contexts in front of them, one launch (a few heads: key ranges are split;
    the sink is counted once), the single row in it or on the decode kernel:
    against the oracle's attention, every row."""
    from arks_amd import ops

    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(D + window)
    rows, ctx = [1, 300, 2, 70, 513], [40, 0, 17, 130, 33]
    total = [a + b for a, b in zip(rows, ctx)]
    blocks = [-(-n // 16) for n in total]
    order = torch.randperm(sum(blocks) + 2, generator=g).to(torch.int32)
    kc = torch.full((sum(blocks) + 2, G, 16, D), 9.0, dtype=torch.bfloat16)
    vc = kc.clone()
    table = torch.zeros(5, max(blocks), dtype=torch.int32)
    slopes, sinks = O.bias_slopes(H), (torch.randn(H, generator=g) + 1.0).tolist()
    scale, of = D ** -0.5, [h // (H // G) for h in range(H)]
    qs, want, at = [], [], 0
    for s, n in enumerate(total):
        table[s, :blocks[s]] = order[at:at + blocks[s]]
        at += blocks[s]
        q, k, v = (_rounded(torch.randn(n, x, D, generator=g, dtype=F64) * 1.5,
                            "bfloat16") for x in (H, G, G))
        pos = torch.arange(n)
        page = table[s][pos // 16].long()
        kc[page, :, pos % 16], vc[page, :, pos % 16] = k.bfloat16(), v.bfloat16()
        qs.append(q[ctx[s]:])
        seen = sorted({ctx[s], n - 1, *range(ctx[s], n, 37)})
        want.append((seen, O.biased_attend(q, k[:, of], v[:, of], scale,
                                           window or n, slopes, sinks, rows=seen)))
    f = lambda x: torch.tensor([float(y) for y in x]).to(dev)
    cu = [0]
    for n in rows:
        cu.append(cu[-1] + n)
    tiles = ops.build_extend_tiles(rows, total, False, dev, num_q_heads=H,
                                   flash_decode=singles, min_ladder=1)
    assert (tiles[2][0] is not None) == singles
    assert tiles[3].numel() and not tiles[0].numel()  # split, no 64-row tiles
    out = ops.attention_extend_paged(
        torch.cat(qs).bfloat16().to(dev), kc.to(dev), vc.to(dev), table.to(dev),
        _i32(total, dev), _i32(cu, dev), None, scale, window=window, tiles=tiles,
        native=ops.seq_extension(), sink_w=f(sinks), slopes=f(slopes))
    out = out.double().cpu()
    for s, (seen, w) in enumerate(want):
        for i in seen:
            assert torch.allclose(out[cu[s] + i - ctx[s]], w[i], atol=2e-2,
                                  rtol=2e-2), (s, i)


class DeltaRun:
    """Steps of ops.channel_delta with one decay per head, over slots filled
    with junk."""

    def __init__(self, device, dtype, H, G, D, V, T, decay_shift=-1.0, seed=4):
        self.dev, self.dtype = _dev(device), dtype
        self.H, self.G, self.D, self.V = H, G, D, V
        g = torch.Generator().manual_seed(seed)

        def rn(*s):
            return torch.randn(*s, generator=g, dtype=F64)

        self.u = _rounded(rn(T, 2 * G * D + H * V), dtype)
        self.decay = _rounded(rn(T, H) + decay_shift, dtype)
        self.beta = _rounded(rn(T, H), dtype)
        self.gate = _rounded(rn(T, H * V), dtype)
        self.rate = torch.exp(rn(H) * 0.5).float().double()
        self.dt_bias = rn(H).float().double()
        self.norm = (1.0 + 0.3 * rn(V)).float().double()
        self.state = torch.full((4, H, D, V), 7.0, device=self.dev)

    def want(self, lo, hi):
        """Outputs of the sequence made of rows [lo, hi)."""
        H, G, D, V = self.H, self.G, self.D, self.V
        u = self.u[lo:hi]
        of = [h // (H // G) for h in range(H)]
        q = O.unit_vector(u[:, :G * D].view(-1, G, D)) * D ** -0.5
        k = O.unit_vector(u[:, G * D:2 * G * D].view(-1, G, D))
        v = u[:, 2 * G * D:].view(-1, H, V)
        decay = torch.exp(-self.rate * O.softplus(self.decay[lo:hi] + self.dt_bias))
        o = O.delta_rule(q[:, of], k[:, of], v, decay,
                         O.sigmoid(self.beta[lo:hi]))
        return (O.rms_norm(o, self.norm, 1e-5)
                * O.silu(self.gate[lo:hi]).view(-1, H, V)).reshape(hi - lo, -1)

    def step(self, spans):
        """spans: (first row, rows, position of the first row, slot)."""
        from arks_amd import ops

        dt, dev, H = TDT[self.dtype], self.dev, self.H
        rows = torch.cat([torch.arange(a, a + n) for a, n, _, _ in spans])
        cu, most = [0], max(n for _, n, _, _ in spans)
        for _, n, _, _ in spans:
            cu.append(cu[-1] + n)
        out = torch.zeros(cu[-1], H * self.V + 8, dtype=dt, device=dev)
        chunks = None
        if dev.type == "cuda" and most > ops.DELTA_CHUNK:
            chunks = ops.scan_chunks([n for _, n, _, _ in spans], dev,
                                     ops.DELTA_CHUNK)
        f = lambda x: x.float().to(dev)
        # gate, write strength and decay as slices of one projection's rows
        p = torch.cat([self.gate, self.beta, self.decay], 1)[rows]
        p = torch.cat([p, torch.full((p.shape[0], -p.shape[1] % 8), 9.0)], 1)
        p = p.to(dt).to(dev)
        at = H * self.V
        ops.channel_delta(
            self.u[rows].to(dt).to(dev), p[:, at + H:at + 2 * H],
            p[:, at:at + H], p[:, :at], f(self.rate), f(self.dt_bias),
            f(self.norm), 1e-5, self.state, _i32(cu, dev),
            _i32([p_ + n for _, n, p_, _ in spans], dev),
            _i32([s for _, _, _, s in spans], dev), H, self.G, self.D,
            self.V, out[:, :at], most, chunks, head_decay=True, silu_gate=True)
        res = out.double().cpu()
        assert float(res[:, at:].abs().max()) == 0.0
        return [res[a:b, :at] for a, b in zip(cu, cu[1:])]


DELTA_SIZES = [(4, 2, 8, 12), (2, 2, 32, 32), (3, 1, 64, 48), (2, 1, 96, 64),
               (2, 2, 128, 128), (1, 1, 140, 20), (2, 1, 16, 200), (3, 3, 1, 1)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("size", DELTA_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_delta_portions_and_slots(device, dtype, size):
    """Two sequences in portions of 1, 2, 70, 65, 64 and more rows beside
    each other, in slots filled with junk; then a third in a slot that is
    used again."""
    r = DeltaRun(device, dtype, *size, T=420)
    want_a, want_b, want_c = r.want(0, 205), r.want(205, 341), r.want(341, 420)
    tol = 1e-4 if dtype == "float32" else 4e-2
    got_a, got_b = [], []

    def run(a=None, b=None):
        spans, sinks = [], []
        for part, base, slot, sink in ((a, 0, 2, got_a), (b, 205, 0, got_b)):
            if part:
                at = sum(x.shape[0] for x in sink)
                spans.append((base + at, part, at, slot))
                sinks.append(sink)
        for sink, o in zip(sinks, r.step(spans)):
            sink.append(o)

    run(a=1, b=2)
    run(a=2)
    run(a=70, b=1)
    run(b=65)
    run(a=65, b=3)
    run(a=64, b=65)
    run(a=3)
    a, b = torch.cat(got_a), torch.cat(got_b)
    assert a.shape[0] == 205 and b.shape[0] == 136
    assert torch.allclose(a, want_a, atol=tol, rtol=tol)
    assert torch.allclose(b, want_b, atol=tol, rtol=tol)
    c = torch.cat(r.step([(341, 79, 0, 2)]))
    assert torch.allclose(c, want_c, atol=tol, rtol=tol)
    assert float((r.state[1] - 7.0).abs().max()) == 0.0
    assert float((r.state[3] - 7.0).abs().max()) == 0.0


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("shift", [-30.0, 3.0, 25.0],
                         ids=["no-decay", "strong", "gone-at-once"])
@pytest.mark.parametrize("D,V", [(64, 32), (128, 64), (20, 12)])
def test_delta_decays_of_every_strength(device, dtype, shift, D, V):
    """Decays next to 1 (a token's write stays for the whole prompt), ones
    that forget at once, and a stretch of strong ones in front of weak ones
    (sums of logarithms far from 0 whose differences are small)."""
    r = DeltaRun(device, dtype, 2, 1, D, V, T=150, decay_shift=shift)
    r.decay[:40, 0] = 30.0
    r.decay[40:, 0] = -9.0
    want = r.want(0, 150)
    got = torch.cat(r.step([(0, 150, 0, 1)]))
    tol = 1e-4 if dtype == "float32" else 4e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("D,V", [(32, 16), (128, 128), (12, 20)])
@pytest.mark.parametrize("cut", [140, 141, 190, 199])
def test_delta_asks_for_an_early_token(device, dtype, D, V, cut):
    """Hardly any decay, orthogonal keys: the row at the end asks with the
    key of ONE early row and must get that row's value, wherever the prompt
    was cut (the last portion is a prompt's or a single token)."""
    n = 200
    r = DeltaRun(device, dtype, 1, 1, D, V, T=n, decay_shift=-30.0)
    r.beta[:] = 30.0  # what is written is the value itself
    at = min(9, D - 2)
    for t in range(n):
        q, k = torch.zeros(D, dtype=F64), torch.zeros(D, dtype=F64)
        q[at] = 1.0
        k[at if t == 3 else D - 1] = 1.0
        r.u[t, :D], r.u[t, D:2 * D] = q, k
    want = r.want(0, n)
    got = torch.cat(r.step([(0, cut, 0, 0)]) + r.step([(cut, n - cut, cut, 0)]))
    v = r.u[3, 2 * D:]
    plain = O.rms_norm(v * D ** -0.5, r.norm, 1e-5) * O.silu(r.gate[-1])
    assert torch.allclose(want[-1], plain, atol=1e-2)
    tol = 1e-4 if dtype == "float32" else 3e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol)


@pytest.mark.gpu
@pytest.mark.parametrize("size", [(2, 2, 32, 32), (3, 1, 64, 48), (2, 1, 96, 64),
                                  (2, 2, 128, 128), (1, 1, 128, 256)])
def test_delta_matrix_cores_against_row_by_row(size, monkeypatch):
    from arks_amd import ops

    spans = [(0, 191, 0, 2), (191, 1, 0, 0), (192, 108, 0, 3)]
    r = DeltaRun("cuda", "bfloat16", *size, T=300)
    fast = torch.cat(r.step(spans))
    s_fast = r.state.clone()
    r.state.fill_(7.0)
    monkeypatch.setattr(ops, "use_delta_mfma", False)
    slow = torch.cat(r.step(spans))
    assert not torch.equal(fast, slow)  # two paths
    assert torch.allclose(fast, slow, atol=3e-2, rtol=3e-2)
    assert torch.allclose(s_fast, r.state, atol=1e-4, rtol=1e-4)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("width", [37, 64, 2056, 4096, 6016, 8200])
def test_two_results_join_the_residual(device, dtype, width):
    """Both results normed, one or neither; a result without a weight is
    added as it is."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    T = 6
    g = torch.Generator().manual_seed(8)
    x = torch.randn(T, width, generator=g, dtype=F64).float().double() * 3.0
    y, z = (_rounded(torch.randn(T, width, generator=g, dtype=F64) * m, dtype)
            for m in (20.0, 0.1))
    x[2], y[3], z[4] = 0.0, 0.0, 0.0  # eps alone under the root
    wy, wz, wp = (torch.randn(width, generator=g, dtype=F64).float().double()
                  for _ in range(3))
    f = lambda t: None if t is None else t.float().to(dev)
    for a, b, wa, wb, pre in [(y, z, wy, wz, wp), (y, None, None, None, wp),
                              (y, z, None, wz, wp), (y, z, wy, None, None),
                              (None, None, None, None, wp)]:
        new = x.clone()
        for r, w in ((a, wa), (b, wb)):
            if r is not None:
                new = new + 0.5 * (r if w is None else O.rms_norm(r, w, 1e-5))
        xs = f(x)
        act = lambda t: None if t is None else t.to(dt).to(dev)
        h = ops.residual_sandwich_norm(xs, act(a), f(wa), 0.5, f(pre), 1e-5, dt,
                                       act(b), f(wb))
        assert torch.allclose(xs.double().cpu(), new, atol=2e-5, rtol=1e-5)
        assert (h is None) == (pre is None)
        if pre is not None:
            tol = 2e-5 if dtype == "float32" else 2e-2
            assert torch.allclose(h.double().cpu(), O.rms_norm(new, pre, 1e-5),
                                  atol=tol, rtol=tol)


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("E,top,groups,keep", [(12, 3, 4, 2), (16, 2, 2, 1),
                                               (6, 4, 6, 5), (5, 5, 1, 1),
                                               (256, 8, 8, 4), (72, 6, 9, 3)])
def test_grouped_choice_by_corrected_scores(device, E, top, groups, keep):
    """Corrections are far below 0, so choice scores are negative and an
    excluded expert must not beat them; the weights do not see them; the
    shared expert's column rides along."""
    from arks_amd import ops

    g = torch.Generator().manual_seed(E)
    z = torch.randn(40, E + 1, generator=g) * 2.0
    corr = torch.randn(E, generator=g) - 4.0
    w, ids, mat = ops.moe_route_grouped(
        z.to(device), top, groups, keep, "sigmoid", True, matrix=True,
        correction=corr.to(device), group_top=2, shared_gate=True)
    w, ids, mat = w.double().cpu(), ids.cpu(), mat.double().cpu()
    assert mat.shape == (40, E + 1)
    s = O.sigmoid(z.double())
    seen_negative = turned = 0
    for t in range(40):
        choice = s[t, :E] + corr.double()
        want, margin = O.choose_experts(choice, top, groups, keep)
        if margin < 1e-6:
            continue
        assert ids[t].tolist() == want
        weights = s[t, want] / (s[t, want].sum() + 1e-20)
        assert torch.allclose(w[t], weights, atol=1e-6)
        row = torch.zeros(E + 1, dtype=F64)
        row[want], row[E] = weights, s[t, E]
        assert torch.allclose(mat[t], row, atol=1e-6)
        seen_negative += float(choice[want[-1]]) < 0.0
        turned += O.choose_experts(s[t, :E], top, groups, keep)[0] != want
    assert seen_negative and (turned or top == E)


def test_a_group_counts_its_two_best():
    """Group 0 has the single best expert, group 1 the best pair."""
    from arks_amd import ops

    z = torch.tensor([[3.0, -6.0, -6.0, 1.5, 1.4, -6.0]])
    _, one = ops.moe_route_grouped(z, 1, 2, 1, "sigmoid", True)
    _, two = ops.moe_route_grouped(z, 1, 2, 1, "sigmoid", True, group_top=2)
    assert one.tolist() == [[0]] and two.tolist() == [[3]]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("ff,sff", [(8, 16), (9, 5), (16, 0)])
def test_clamped_experts_with_their_weights(device, dtype, ff, sff):
    """Gate and up far beyond the limits on both sides; an unused expert's
    columns are exactly 0; the shared expert has a limit and a weight of its
    own."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    E, T, alpha = 3, 5, 1.702
    g = torch.Generator().manual_seed(10)
    gu = _rounded(torch.randn(T, E * 2 * ff + 2 * sff, generator=g, dtype=F64) * 3,
                  dtype)
    scale = torch.rand(T, E + bool(sff), generator=g)
    scale[1, 2] = scale[3, 0] = 0.0
    got = ops.moe_glu_scaled(gu.to(dt).to(dev), scale.to(dev), E, ff, sff, False,
                             "clamped", 1.3, 0.7, alpha, bool(sff)).double().cpu()

    def act(a, b, limit):
        a, b = a.clamp(max=limit), b.clamp(-limit, limit)
        return a * O.sigmoid(alpha * a) * (b + 1.0)

    tol = 1e-5 if dtype == "float32" else 2e-2
    for e in range(E):
        a = gu[:, e * 2 * ff:e * 2 * ff + ff]
        b = gu[:, e * 2 * ff + ff:(e + 1) * 2 * ff]
        want = scale[:, e:e + 1].double() * act(a, b, 1.3)
        assert torch.allclose(got[:, e * ff:(e + 1) * ff], want, atol=tol, rtol=tol)
    assert float(got[1, 2 * ff:3 * ff].abs().max()) == 0.0
    if sff:
        a, b = gu[:, E * 2 * ff:].split(sff, 1)
        want = scale[:, E:].double() * act(a, b, 0.7)
        assert torch.allclose(got[:, E * ff:], want, atol=tol, rtol=tol)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("shape", [(3, 7), (5, 64)])
def test_relu_square(device, dtype, shape):
    from arks_amd import ops

    x = _rounded(torch.linspace(-4, 4, shape[0] * shape[1], dtype=F64).view(shape),
                 dtype)
    got = ops.relu_square(x.to(TDT[dtype]).to(device)).double().cpu()
    tol = 1e-6 if dtype == "float32" else 1e-2
    assert torch.allclose(got, x.clamp(min=0.0) ** 2, atol=tol, rtol=tol)


@pytest.mark.gpu
def test_captured_decode_steps_equal_eager_ones(tmp_path):
    """The captured decode step, replayed many times with eager prompt steps
    in between, gives the logits of eager decode steps."""
    cfg = fast_path_config()
    write_checkpoint(tmp_path / "m", cfg)
    ta, tb = toks(120, seed=2), toks(90, seed=3)
    steps = [[("a", ta[:80], False)], [("a", ta[80:81], False)],
             [("a", ta[81:82], False), ("b", tb[:66], False)]]
    steps += [[("a", [x], False), ("b", [y], False)]
              for x, y in zip(ta[82:100], tb[66:84])]
    steps += [[("a", ta[100:103], False)]]
    steps += [[("a", [x], False), ("b", [y], False)]
              for x, y in zip(ta[103:109], tb[84:90])]
    got = {}
    for eager in (False, True):
        eng = make_engine(tmp_path / "m", "cuda", "bfloat16", enforce_eager=eager)
        got[eager] = replay(eng, tmp_path, steps)
    for c in ("a", "b"):
        a, b = got[False][c], got[True][c]
        err = np.sqrt(((a - b) ** 2).mean(-1)) / np.sqrt((b ** 2).mean())
        assert err.max() < 2e-2
