"""Pazilorn through the engine, and its mechanisms one by one, against the
plain float64 model of tests/pazilorn_oracle.py.

Engine cases write a small random checkpoint, build an engine on it and
replay a step plan with the product's trace replay (the scheduler's pages
and state slots, the runner's batches, the model's kernels); op cases drive
single ops with inputs made so that a fault shows (one key that must win
just inside, just outside and far from a window's edge; a state that only an
early token wrote; decays next to 0 and 1; junk in slots and pages that are
used again; a router whose bias decides). CPU cases run the reference ops,
gpu-marked ones the HIP kernels in float32 and bfloat16.
"""

import io
import json
import math
import os

import numpy as np
import pytest
import torch

import pazilorn_oracle as O

CASES = [
    pytest.param("cpu", "float32", id="cpu-f32"),
    pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu),
]
GPU_CASES = [c for c in CASES if c.id != "cpu-f32"]
TOL = {"float32": 2e-4, "bfloat16": 8e-2}
TDT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64

C, L, MOE = O.delta_spec, O.latent_spec, O.moe_spec


# ------------------------------------------------------------------ helpers
def write_checkpoint(path, cfg, seed=0, ranks=(5, 7)):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    w = O.random_weights(cfg, seed, ranks)
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


def rel_err(got, want):
    """Largest row error over the rms of all logits."""
    want = want.numpy() if isinstance(want, torch.Tensor) else want
    d = got - want
    return float((np.sqrt((d ** 2).mean(-1)) / np.sqrt((want ** 2).mean())).max())


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


def oracle_logits(cfg, w, t):
    return O.forward(cfg, w, t)[0]


def assert_logits(got, cfg, w, t, dtype, note=None):
    """got [n, vocab] against the oracle's first n rows: every row, but in
    bfloat16 with routers that choose only the rows in front of the first
    close call. There a reduced-precision run may choose otherwise, which is
    another function, and the states carry that on to later rows; the
    typical row must be well inside all the same."""
    n = got.shape[0]
    margins = []
    want = O.forward(cfg, w, t, margins)[0][:n].numpy()
    err = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    if dtype == "bfloat16" and margins:
        assert np.median(err) < TOL[dtype] / 3, note
        err = err[:O.clear_rows(margins)]
    assert not err.size or err.max() < TOL[dtype], (note, int(err.argmax()))


# --------------------------------------------------- the model in the engine
ONE_LAYER = {
    "delta": [C()],
    "delta-alone": [C(mlp=None)],
    "latent": [L()],
    "latent-alone": [L(mlp=None)],
    "borrowed-delta": [C(), C(weights_of=0)],
    "borrowed-latent": [L(mlp=None), L(mlp=None, weights_of=0)],
    "borrowed-from-later": [L(weights_of=1), L()],
}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(ONE_LAYER))
def test_one_mixer(tmp_path, device, dtype, name):
    cfg = O.make_config(ONE_LAYER[name])
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(45)
    eng = make_engine(tmp_path / "m", device, dtype)
    got = replay(eng, tmp_path, [[("a", t, True)]])["a"]
    assert_logits(got, cfg, w, t, dtype)


def model_config():
    """Both mixers with and without feed-forward, and layers on other
    layers' weights whose caches and states are their own."""
    return O.make_config([C(), L(), C(conv=2, heads=3, kv_heads=3, mlp=None),
                          C(weights_of=0), L(weights_of=1),
                          L(window=3, mlp=MOE(top=1))])


def plain_config():
    """The same without routers, whose close calls make a comparison in
    bfloat16 blunt."""
    return O.make_config([C(mlp=None), L(mlp=None),
                          C(conv=2, heads=3, kv_heads=3, mlp=None),
                          C(weights_of=0, mlp=None), L(weights_of=1, mlp=None),
                          L(window=3, mlp=None)])


CONFIGS = {"routed": model_config, "plain": plain_config}


@pytest.mark.parametrize("device,dtype", CASES)
def test_residual_after_every_layer(tmp_path, device, dtype):
    cfg = model_config()
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(23)
    _, after = O.forward(cfg, w, t)
    eng = make_engine(tmp_path / "m", device, dtype)
    seen = {}
    eng.runner.model.residual_tap = lambda i, x: seen.__setitem__(
        i, x.detach().clone().float().cpu())
    replay(eng, tmp_path, [[("a", t, True)]])
    assert sorted(seen) == list(range(len(after)))
    for i, want in enumerate(after):
        row = (seen[i].double() - want).abs().amax(-1) / want.abs().max()
        # a close call of a router may flip a row in bfloat16
        worst = row.max() if dtype == "float32" else row.median()
        assert float(worst) < (1e-4 if dtype == "float32" else 2e-2), i


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_against_decode_and_portions(tmp_path, device, dtype, name):
    cfg = CONFIGS[name]()
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(70)
    for name, plan in {
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
    cfg = O.make_config([C(mlp=None), L(window=37, mlp=None), C(mlp=MOE(top=6))])
    w = write_checkpoint(tmp_path / "m", cfg)
    t = toks(150)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", t[:5], False)]] + [[("a", [x], False)] for x in t[5:]]
    got = replay(eng, tmp_path, steps)["a"]
    assert_logits(got, cfg, w, t, dtype)


OTHER_SIZES = {
    "one-kv-head": dict(layers=[C(heads=6, kv_heads=1, dim=8, vdim=12)]),
    "all-kv-heads": dict(layers=[C(heads=3, kv_heads=3, dim=12, vdim=4)]),
    "one-head": dict(layers=[C(heads=1, kv_heads=1), L(heads=1)]),
    "wide-values": dict(layers=[C(heads=2, kv_heads=1, dim=4, vdim=72)]),
    "wide-keys": dict(layers=[C(heads=2, kv_heads=2, dim=140, vdim=6)]),
    "wide-both": dict(layers=[C(heads=1, kv_heads=1, dim=40, vdim=200)]),
    "no-history": dict(layers=[C(conv=1)]),
    "two-taps": dict(layers=[C(conv=2)]),
    "twelve-taps": dict(layers=[C(conv=12, dim=16, vdim=16)]),
    "rank-one": dict(layers=[C()], ranks=(1, 1)),
    "wide-ranks": dict(layers=[C()], ranks=(33, 9)),
    "window-one": dict(layers=[L(window=1)]),
    "window-page": dict(layers=[L(window=16)]),
    "window-above": dict(layers=[L(window=500)]),
    "rotary-two-dims": dict(layers=[L(rot_dim=2, base=7.0)]),
    "rotary-wide": dict(layers=[L(dim=4, rot_dim=24)]),
    "rotary-unscaled": dict(layers=[L(scaling=None)]),
    "rotary-all-scaled": dict(layers=[L(rot_dim=16, scaling={
        "factor": 16.0, "original": 4, "fast": 64.0, "slow": 32.0})]),
    "rotary-ramp-inside": dict(layers=[L(rot_dim=32, base=100.0, scaling={
        "factor": 3.0, "original": 64, "fast": 6.0, "slow": 0.5})]),
    "sharp-scores": dict(layers=[L(scale=4.0)]),
    "latent-wider-than-model": dict(layers=[L(kv_rank=90, q_rank=70)]),
    "top-one": dict(layers=[C(mlp=MOE(top=1))]),
    "top-all": dict(layers=[L(mlp=MOE(experts=3, top=3))]),
    "one-expert": dict(layers=[L(mlp=MOE(experts=1, top=1))]),
    "many-experts": dict(layers=[C(mlp=MOE(experts=70, top=5, ff=8))]),
    "tight-cap": dict(layers=[C(), L()], cap=0.7),
    "mult-one": dict(layers=[C(), L()], mult=1.0, scale=1.0),
    "large-embedding": dict(layers=[C(), L()], scale=40.0, mult=0.1),
    "odd-everything": dict(layers=[
        C(heads=3, kv_heads=1, dim=7, vdim=11, conv=3,
          mlp=MOE(experts=5, top=2, ff=13)),
        L(heads=5, dim=7, rot_dim=10, vdim=9, kv_rank=19, q_rank=11, window=5,
          mlp=MOE(experts=7, top=3, ff=9)),
        C(heads=3, kv_heads=1, dim=7, vdim=11, conv=3,
          mlp=MOE(experts=5, top=2, ff=13), weights_of=0),
        C(heads=9, kv_heads=3, dim=3, vdim=5, conv=5, mlp=None)],
        width=43, vocab=97, eps=1e-3, ranks=(3, 11)),
}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(OTHER_SIZES))
def test_other_sizes(tmp_path, device, dtype, name):
    spec = dict(OTHER_SIZES[name])
    ranks = spec.pop("ranks", (5, 7))
    cfg = O.make_config(**spec)
    w = write_checkpoint(tmp_path / "m", cfg, seed=3, ranks=ranks)
    t = toks(38, vocab=cfg["vocab"], seed=9)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", p, False)] for p in portions(t, [11, 2, 1, 6])]
    got = replay(eng, tmp_path, steps)["a"]
    assert_logits(got, cfg, w, t, dtype)


def fast_path_config(mlp=None):
    """Sizes the vectorised and matrix-core kernels are built for, with a
    window shorter than the prompts."""
    return O.make_config(
        [C(heads=4, kv_heads=2, dim=64, vdim=64, mlp=mlp),
         L(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=64,
           window=100, mlp=mlp),
         C(heads=2, kv_heads=2, dim=128, vdim=128, mlp=None),
         C(heads=3, kv_heads=1, dim=32, vdim=48, mlp=None),
         L(heads=4, dim=48, rot_dim=16, vdim=64, kv_rank=256, q_rank=40,
           window=70, mlp=None),
         C(heads=1, kv_heads=1, dim=96, vdim=16, mlp=None)], width=64)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
def test_fast_path_sizes(tmp_path, device, dtype):
    """Prompts across 64-row chunk and tile edges, single rows after them,
    portions long enough for the per-head form of the latents (with pages
    behind the window skipped) and short ones on the latents themselves."""
    cfg = fast_path_config(MOE(experts=8, top=2, ff=32))
    w = write_checkpoint(tmp_path / "m", cfg, ranks=(16, 24))
    t = toks(470, seed=11)
    eng = make_engine(tmp_path / "m", device, dtype, max_tokens=512)
    plan = [t[:130], t[130:131], t[131:197], t[197:198], t[198:199],
            t[199:201], t[201:]]
    assert len(plan[-1]) > 256
    got = replay(eng, tmp_path, [[("a", p, False)] for p in plan])["a"]
    assert_logits(got, cfg, w, t, dtype)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
def test_fast_path_sizes_in_mixed_batches(tmp_path, device, dtype):
    cfg = fast_path_config()
    w = write_checkpoint(tmp_path / "m", cfg, ranks=(8, 8))
    reqs = {c: toks(n, seed=s) for c, n, s in
            [("a", 250, 1), ("b", 70, 2), ("c", 301, 3), ("d", 9, 4),
             ("e", 66, 5)]}
    steps = mixed_plan(reqs, 3, 42, [67, 1, 1, 200, 2, 1, 33, 1, 90])
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
    cfg = O.make_config([C(mlp=MOE(experts=5, top=3)),
                         L(mlp=MOE(experts=4, top=1))])
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
def test_latent_forms_agree(tmp_path, device, dtype, monkeypatch):
    """Portions on the latents themselves and portions on per-head keys of
    the reachable pages (mid-page window edges included) give the oracle's
    logits in one replay, two requests at different lengths side by side."""
    from arks_amd.models.mixers import LatentAttention

    monkeypatch.setattr(LatentAttention, "EXPAND_ROWS", 12)
    cfg = O.make_config([L(window=21), L(window=5, mlp=None),
                         L(window=300, mlp=None)])
    w = write_checkpoint(tmp_path / "m", cfg)
    ta, tb = toks(90, seed=2), toks(61, seed=3)
    eng = make_engine(tmp_path / "m", device, dtype)
    steps = [[("a", ta[:13], False)], [("a", ta[13:16], False)],
             [("a", ta[16:47], False), ("b", tb[:1], False)],
             [("a", ta[47:48], False), ("b", tb[1:40], False)],
             [("a", ta[48:75], False), ("b", tb[40:41], False)],
             [("a", ta[75:], True), ("b", tb[41:], True)]]
    got = replay(eng, tmp_path, steps)
    assert_logits(got["a"], cfg, w, ta, dtype)
    assert_logits(got["b"], cfg, w, tb, dtype)


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
        seq = list(p)
        assert len(o) == 12
        for tok in o:
            logits = oracle_logits(cfg, w, seq)[-1]
            top2 = torch.topk(logits, 2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == "float32" else 0.6):
                assert tok == int(logits.argmax()), (len(seq), tok)
            seq.append(tok)


def test_config_borrowed_weights_and_shape_sizes(tmp_path):
    from arks_amd.config import PRESET_CONFIGS, HybridModelConfig, ModelConfig
    from arks_amd.models import create_model

    cfg = PRESET_CONFIGS["tiny-pazilorn"]
    again = HybridModelConfig.from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.layers == cfg.layers and again.tied_head
    assert (again.logit_softcap, again.residual_mult) == (30.0, 0.5)
    model = create_model(again)
    assert model.layers[2] is model.layers[0]
    assert len(model.cache_layout(16)) == 4  # a cache of its own per layer
    assert not any(k.startswith(("l2.", "l3.")) for k in model._wmap)
    raw = O.make_config([C(), L(), C(weights_of=0)])
    write_checkpoint(tmp_path / "m", raw, ranks=(3, 9))
    got = ModelConfig.from_pretrained(str(tmp_path / "m"))
    for i in (0, 2):
        m = got.layers[i]["mixer"]
        assert (m["decay_rank"], m["gate_rank"]) == (3, 9)
    with pytest.raises(ValueError):  # ranks neither in the dict nor on disk
        HybridModelConfig.from_dict(raw)
    for owner in (1, 2, 7):  # another type, itself, none
        bad = json.loads(json.dumps(cfg.to_dict()))
        bad["layers"][2]["weights_of"] = owner
        with pytest.raises((ValueError, IndexError)):
            HybridModelConfig.from_dict(bad)


# ------------------------------------------------------- mechanisms alone
def _dev(device):
    return torch.device(device)


def _rounded(x, dtype):
    """What the op will see: the value after rounding to its row dtype."""
    return x.to(TDT[dtype]).to(F64)


def _i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


class DeltaRun:
    """Steps of ops.channel_delta over slots filled with junk."""

    def __init__(self, device, dtype, H, G, D, V, T, decay_shift=-1.0, seed=4,
                 gate_f32=False):
        self.dev, self.dtype = _dev(device), dtype
        self.H, self.G, self.D, self.V = H, G, D, V
        g = torch.Generator().manual_seed(seed)

        def rn(*s):
            return torch.randn(*s, generator=g, dtype=F64)

        self.u = _rounded(rn(T, 2 * G * D + H * V), dtype)
        self.decay = (rn(T, H * D) + decay_shift).float().double()
        self.beta = _rounded(rn(T, H), dtype)
        self.gate_dt = torch.float32 if gate_f32 else TDT[dtype]
        self.gate = rn(T, H * V).to(self.gate_dt).double()
        self.rate = torch.exp(rn(H) * 0.5).float().double()
        self.dt_bias = rn(H * D).float().double()
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
        z = (self.decay[lo:hi] + self.dt_bias).view(-1, H, D)
        decay = torch.exp(-self.rate[:, None] * O.softplus(z))
        o = O.delta_rule(q[:, of], k[:, of], v, decay,
                         O.sigmoid(self.beta[lo:hi]))
        return (O.rms_norm(o, self.norm, 1e-5)
                * O.sigmoid(self.gate[lo:hi]).view(-1, H, V)).reshape(hi - lo, -1)

    def step(self, spans):
        """spans: (first row, rows, position of the first row, slot)."""
        from arks_amd import ops

        dt, dev = TDT[self.dtype], self.dev
        rows = torch.cat([torch.arange(a, a + n) for a, n, _, _ in spans])
        cu, most = [0], max(n for _, n, _, _ in spans)
        for _, n, _, _ in spans:
            cu.append(cu[-1] + n)
        out = torch.zeros(cu[-1], self.H * self.V + 8, dtype=dt, device=dev)
        chunks = None
        if dev.type == "cuda" and most > ops.DELTA_CHUNK:
            chunks = ops.scan_chunks([n for _, n, _, _ in spans], dev,
                                     ops.DELTA_CHUNK)
        f = lambda x: x.float().to(dev)
        ops.channel_delta(
            self.u[rows].to(dt).to(dev), f(self.decay[rows]),
            self.beta[rows].to(dt).to(dev), self.gate[rows].to(self.gate_dt).to(dev),
            f(self.rate), f(self.dt_bias), f(self.norm), 1e-5, self.state,
            _i32(cu, dev), _i32([p + n for _, n, p, _ in spans], dev),
            _i32([s for _, _, _, s in spans], dev), self.H, self.G, self.D,
            self.V, out[:, :self.H * self.V], most, chunks)
        res = out.double().cpu()
        assert float(res[:, self.H * self.V:].abs().max()) == 0.0
        return [res[a:b, :self.H * self.V] for a, b in zip(cu, cu[1:])]


DELTA_SIZES = [(4, 2, 8, 12), (2, 2, 32, 32), (3, 1, 64, 48), (2, 1, 96, 64),
               (2, 2, 128, 128), (1, 1, 140, 20), (2, 1, 16, 200)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("size", DELTA_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_delta_portions_and_slots(device, dtype, size):
    """Two sequences in portions of 1, 2, 70, 65, 64 and 130 rows beside
    each other, in slots filled with junk; then a third in a slot that is
    used again."""
    r = DeltaRun(device, dtype, *size, T=420)
    want_a, want_b, want_c = r.want(0, 205), r.want(205, 341), r.want(341, 420)
    tol = 1e-4 if dtype == "float32" else 4e-2
    got_a, got_b = [], []

    def run(a=None, b=None, c=None):
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
    """Decays next to 1 (a token's write stays for the whole prompt), strong
    ones (a 16-row block's summed logarithm is far below what an fp32
    exponential can hold the inverse of) and a few of each side by side."""
    r = DeltaRun(device, dtype, 2, 1, D, V, T=150, decay_shift=shift)
    r.decay[:, ::3] = -9.0  # some channels decay slowly all the same
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
    plain = O.rms_norm(v * D ** -0.5, r.norm, 1e-5) * O.sigmoid(r.gate[-1])
    assert torch.allclose(want[-1], plain, atol=1e-2)
    tol = 1e-4 if dtype == "float32" else 3e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol)


@pytest.mark.parametrize("device,dtype", GPU_CASES)
@pytest.mark.parametrize("size", [(2, 2, 32, 32), (3, 1, 64, 48), (2, 1, 96, 64),
                                  (2, 2, 128, 128), (1, 1, 128, 256)])
def test_delta_matrix_cores_against_row_by_row(device, dtype, size, monkeypatch):
    from arks_amd import ops

    r = DeltaRun(device, dtype, *size, T=300)
    fast = torch.cat(r.step([(0, 191, 0, 2), (191, 1, 0, 0), (192, 108, 0, 3)]))
    s_fast = r.state.clone()
    r.state.fill_(7.0)
    monkeypatch.setattr(ops, "use_delta_mfma", False)
    slow = torch.cat(r.step([(0, 191, 0, 2), (191, 1, 0, 0), (192, 108, 0, 3)]))
    assert torch.allclose(fast, slow, atol=3e-2, rtol=3e-2)
    assert torch.allclose(s_fast, r.state, atol=1e-4, rtol=1e-4)


@pytest.mark.gpu
def test_delta_matrix_core_sizes_are_taken():
    from arks_amd import ops

    for D, V, takes in [(32, 32, True), (64, 48, True), (96, 16, True),
                        (128, 128, True), (40, 32, False), (128, 24, False)]:
        r = DeltaRun("cuda", "bfloat16", 2, 1, D, V, T=70)
        dev = torch.device("cuda")
        c = ops.scan_chunks([70], dev, ops.DELTA_CHUNK)
        bf = lambda x: x.to(torch.bfloat16).to(dev)
        f = lambda x: x.float().to(dev)
        out = torch.zeros(70, 2 * V, dtype=torch.bfloat16, device=dev)
        took = ops._native_seq().channel_delta_chunks(
            out, bf(r.u), f(r.decay), bf(r.beta), bf(r.gate), f(r.rate),
            f(r.dt_bias), f(r.norm), 1e-5, 1e-6, r.state, c["off"], c["cu"],
            _i32([0, 70], dev), _i32([70], dev), _i32([0], dev), 2, 1, D, V)
        assert took == takes, (D, V)


@pytest.mark.parametrize("device,dtype", CASES)
def test_delta_gate_rows_in_float32(device, dtype):
    """Short steps hand the gate over in float32."""
    r = DeltaRun(device, dtype, 4, 2, 16, 24, T=9, gate_f32=True)
    got = torch.cat(r.step([(0, 9, 0, 1)]))
    tol = 1e-4 if dtype == "float32" else 2e-2
    assert torch.allclose(got, r.want(0, 9), atol=tol, rtol=tol)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("taps,C_", [(4, 24), (1, 16), (3, 13), (9, 40), (20, 32)])
def test_convolution_without_bias_one_row_steps(device, dtype, taps, C_):
    """Single rows of two sequences (the history is replaced by the launch
    that reads it), then portions, in slots filled with junk."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    g = torch.Generator().manual_seed(6)
    w = torch.randn(C_, taps, generator=g, dtype=F64).float().double()
    x = {s: _rounded(torch.randn(40, C_, generator=g, dtype=F64), dtype)
         for s in (0, 1)}
    want = {s: O.conv_silu(x[s], w) for s in x}
    state = torch.full((3, max(taps - 1, 1), C_), 5.0, device=dev)
    at = {0: 0, 1: 0}
    tol = 1e-5 if dtype == "float32" else 3e-2
    for step in [[(0, 1), (1, 1)], [(1, 1), (0, 1)], [(0, 1)], [(0, 6), (1, 1)],
                 [(0, 1), (1, 1)], [(1, 12)], [(0, 1), (1, 1)]]:
        cu = [0]
        for _, n in step:
            cu.append(cu[-1] + n)
        y = ops.causal_conv_silu(
            torch.cat([x[s][at[s]:at[s] + n] for s, n in step]).to(dt).to(dev),
            w.float().to(dev), None, state if taps > 1 else None, _i32(cu, dev),
            _i32([at[s] + n for s, n in step], dev),
            _i32([2 * s for s, _ in step], dev),
            _i32(sum([[j] * n for j, (_, n) in enumerate(step)], []), dev),
            w.float().t().contiguous().to(dev), max(n for _, n in step))
        y = y.double().cpu()
        for j, (s, n) in enumerate(step):
            assert torch.allclose(y[cu[j]:cu[j + 1]], want[s][at[s]:at[s] + n],
                                  atol=tol, rtol=tol), (step, s)
            at[s] += n
    assert float((state[1] - 5.0).abs().max()) == 0.0


class LatentPages:
    """One sequence's latent rows in pages handed out in a scrambled order."""

    def __init__(self, dev, dtype, rank, R, n):
        nblk = -(-n // 16)
        g = torch.Generator().manual_seed(7)
        self.dev, self.dt = dev, TDT[dtype]
        self.table = torch.randperm(nblk + 3, generator=g)[:nblk].to(torch.int32)
        self.ckv = torch.full((nblk + 3, 1, 16, rank + R), 9.0, dtype=self.dt,
                              device=dev)
        self.rank = rank

    def put(self, rows, first=0):
        pos = torch.arange(first, first + rows.shape[0])
        self.ckv[self.table[pos // 16].long().to(self.dev), 0,
                 (pos % 16).to(self.dev)] = rows.to(self.dt).to(self.dev)

    def attend(self, q, total, scale, window):
        from arks_amd import ops

        n = q.shape[0]
        out = ops.attention_sink_paged(
            q.to(self.dt).to(self.dev).contiguous(), self.ckv,
            self.ckv[..., :self.rank], self.table[None].to(self.dev),
            _i32([total], self.dev), _i32([0, n], self.dev),
            _i32([0] * n, self.dev), scale, False, None, True, n, None,
            window=window)
        return out.double().cpu()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("rank,R", [(24, 8), (512, 64), (256, 64), (128, 16)])
def test_window_edges_over_latents(device, dtype, decode, rank, R):
    """One key carries a huge score: it takes all the weight as the last key
    inside the window, at a page border, and at the row itself, and leaves
    no trace as the first key outside or far back."""
    dev = _dev(device)
    H, n, scale = 4, 300, 0.5
    g = torch.Generator().manual_seed(5)
    base = torch.randn(n, rank + R, generator=g, dtype=F64) * 0.1
    i = n - 1
    e = torch.zeros(rank + R, dtype=F64)
    e[rank + 3] = 1.0
    q = torch.zeros(n, H, rank + R, dtype=F64)
    q[i] = 8.0 * e
    for window, hot, seen in [(37, i - 36, True), (37, i - 37, False),
                              (37, 2, False), (300, 2, True), (300, 0, True),
                              (299, 0, False), (29, 271, True), (28, 271, False),
                              (28, 272, True), (1, i, True), (1, i - 1, False)]:
        row = base.clone()
        row[hot] = row[hot] + 40.0 * e
        row = _rounded(row, dtype)
        k = row[:, None].expand(n, H, rank + R)
        v = row[:, None, :rank].expand(n, H, rank)
        want = O.window_attend(q, k, v, scale, window)[i]
        assert torch.allclose(want[0], v[hot, 0], atol=1e-6) == seen
        pg = LatentPages(dev, dtype, rank, R, n)
        pg.put(row)
        first = i if decode else n - 41
        got = pg.attend(q[first:], n, scale, window)[-1]
        tol = 1e-4 if dtype == "float32" else 1e-2
        assert torch.allclose(got, want, atol=tol, rtol=tol), (window, hot)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("sizes", [(6, 10, 14, 8), (8, 24, 40, 16), (64, 1536, 512, 64)],
                         ids=["odd", "vector", "large"])
def test_latent_rows_norm_turn_and_pages(device, dtype, interleaved, sizes):
    """The latent is normed and not turned, the shared key part turned (with
    the scaling's magnitude) and not normed; only the row's own place in the
    pages changes; the query's plain part passes unchanged."""
    from arks_amd import ops
    from arks_amd.models.mixers import ramp_scaled_inv_freq

    dev, dt = _dev(device), TDT[dtype]
    D, Rq, Rk, R = sizes
    rot = {"base": 100.0, "dims": R,
           "scaling": {"factor": 4.0, "original": 16, "fast": 4.0, "slow": 0.5}}
    f, mag = ramp_scaled_inv_freq(rot["base"], rot["dims"], rot["scaling"])
    of, omag = O.ramped_freqs(rot)
    assert torch.allclose(f.double(), of, rtol=1e-6) and math.isclose(mag, omag)
    assert mag > 1.1
    T, H, W = 45, 3, Rk + R
    g = torch.Generator().manual_seed(9)
    p = _rounded(torch.randn(T, Rq + W + 3 if D == 6 else Rq + W + 8, generator=g,
                             dtype=F64), dtype)
    qw, kw = (torch.randn(k, generator=g, dtype=F64).float().double()
              for k in (Rq, Rk))
    q = _rounded(torch.randn(T, H, D + R, generator=g, dtype=F64), dtype)
    q_abs = _rounded(torch.randn(H, T, Rk, generator=g, dtype=F64), dtype)

    def turn(x):  # rows are positions 0 .. T-1
        if interleaved:
            x = torch.cat([x[..., 0::2], x[..., 1::2]], -1)
        y = O.rotate_half(x, rot)
        if interleaved:
            y = torch.stack([y[..., :R // 2], y[..., R // 2:]], -1).flatten(-2)
        return y

    cache = torch.full((4, 1, 16, W), 3.0, dtype=dt, device=dev)
    pos = torch.arange(T)
    slots = (pos + 16).to(dev)
    slots[7] = -1  # a padding row writes no page
    pd, fd = p.to(dt).to(dev), f.to(dev)
    cq = ops.latent_prepare(pd[:, :Rq], pd[:, Rq:Rq + W],
                            qw.float().to(dev), kw.float().to(dev), 1e-5,
                            pos.to(dev), fd, cache, slots, interleaved, mag)
    tol = 1e-5 if dtype == "float32" else 2e-2
    assert torch.allclose(cq.double().cpu(), O.rms_norm(p[:, :Rq], qw, 1e-5),
                          atol=tol, rtol=tol)
    got = cache.double().cpu().reshape(-1, W)
    assert float((got[:16] - 3.0).abs().max()) == 0.0
    assert float((got[16 + T:] - 3.0).abs().max()) == 0.0
    assert float((got[16 + 7] - 3.0).abs().max()) == 0.0
    keep = pos != 7
    got = got[16:16 + T][keep]
    assert torch.allclose(got[:, :Rk], O.rms_norm(p[:, Rq:Rq + Rk], kw, 1e-5)[keep],
                          atol=tol, rtol=tol)
    want = turn(p[:, None, Rq + Rk:Rq + W])[:, 0]
    assert torch.allclose(got[:, Rk:], want[keep], atol=tol, rtol=tol)
    for absorbed in (True, False):
        plain = q_abs.transpose(0, 1) if absorbed else q[..., :D]
        qd = q.to(dt).to(dev)
        out = (torch.zeros(T, H, W, dtype=dt, device=dev) if absorbed
               else torch.zeros_like(qd))
        for o in (out, qd)[:1 if absorbed else 2]:  # a new tensor, then in place
            ops.latent_query(qd, q_abs.to(dt).to(dev) if absorbed else None,
                             pos.to(dev), fd, o, interleaved, mag)
            res = o.double().cpu()
            n = plain.shape[-1]
            assert torch.equal(res[..., :n], plain)
            assert torch.allclose(res[..., n:], turn(q[..., D:]), atol=tol, rtol=tol)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("sizes", [(3, 6, 4, 5, 10), (4, 24, 8, 16, 32), (1, 1, 2, 1, 1)])
def test_latent_pages_of_single_heads(device, dtype, sizes):
    from arks_amd import ops

    H, D, R, V, rank = sizes
    NB, bs = 5, 16
    g = torch.Generator().manual_seed(3)
    k, v, lat = (torch.randn(NB * bs, n, generator=g).to(TDT[dtype]).to(device)
                 for n in (H * D, H * V, rank + R))
    kt, vt = (x.cpu() for x in ops.latent_pages(k, v, lat, H, R, bs))
    assert kt.shape == (NB, H, bs, D + R) and vt.shape == (NB, H, bs, V)
    for n in range(NB * bs):
        for h in range(H):
            at = (n // bs, h, n % bs)
            assert torch.equal(kt[at][:D], k[n, h * D:(h + 1) * D].cpu())
            assert torch.equal(kt[at][D:], lat[n, rank:].cpu())
            assert torch.equal(vt[at], v[n, h * V:(h + 1) * V].cpu())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("V", [10, 64])
def test_head_gate(device, dtype, V):
    """Each head by its own number; heads-first inputs, strided rows, in
    place, and no gate at all."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    T, H = 5, 6
    g = torch.Generator().manual_seed(3)
    o = _rounded(torch.randn(H, T, V, generator=g, dtype=F64), dtype)
    p = _rounded(torch.randn(T, H + 9, generator=g, dtype=F64), dtype)
    p[:, 4] = -40.0
    want = o.transpose(0, 1) * O.sigmoid(p[:, 2:2 + H])[:, :, None] * 0.5
    out = torch.zeros(T, H * V + 8, dtype=dt, device=dev)
    view = out[:, :H * V].unflatten(-1, (H, V))
    gate = p.to(dt).to(dev)[:, 2:2 + H]
    ops.head_gate(o.to(dt).to(dev).transpose(0, 1), gate, view, 0.5)
    tol = 1e-5 if dtype == "float32" else 1e-2
    got = out.double().cpu()
    assert torch.allclose(got[:, :H * V].view(T, H, V), want, atol=tol, rtol=tol)
    assert float(got[:, H * V:].abs().max()) == 0.0
    assert float(got.view(T, -1)[:, 2 * V:3 * V].abs().max()) < 1e-12
    ops.head_gate(view, gate, view, 1.0)
    again = want * O.sigmoid(p[:, 2:2 + H])[:, :, None]
    assert torch.allclose(out.double().cpu()[:, :H * V].view(T, H, V), again,
                          atol=tol, rtol=2 * tol)
    ops.head_gate(o.to(dt).to(dev).transpose(0, 1), None, view, 1.0)
    assert torch.equal(out.double().cpu()[:, :H * V].view(T, H, V),
                       o.transpose(0, 1))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("width", [37, 64, 2056, 4096, 6016, 8200])
def test_residual_sandwich_norm(device, dtype, width):
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    T = 7
    g = torch.Generator().manual_seed(8)
    x = torch.randn(T, width, generator=g, dtype=F64).float().double() * 3.0
    y = _rounded(torch.randn(T, width, generator=g, dtype=F64) * 20.0, dtype)
    x[2], y[3] = 0.0, 0.0  # eps alone under the root
    w1, w2 = (torch.randn(width, generator=g, dtype=F64).float().double()
              for _ in range(2))
    f = lambda t: t.float().to(dev)
    for have_y, have_w in [(True, True), (False, True), (True, False)]:
        new = x + 0.3 * O.rms_norm(y, w1, 1e-5) if have_y else x
        xs = f(x)
        h = ops.residual_sandwich_norm(
            xs, y.to(dt).to(dev) if have_y else None, f(w1), 0.3,
            f(w2) if have_w else None, 1e-5, dt)
        assert torch.allclose(xs.double().cpu(), new, atol=1e-5, rtol=1e-5)
        assert (h is None) == (not have_w)
        if have_w:
            tol = 2e-5 if dtype == "float32" else 2e-2
            assert torch.allclose(h.double().cpu(), O.rms_norm(new, w2, 1e-5),
                                  atol=tol, rtol=tol)


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("shape", [(3, 8), (5, 97), (1, 1)])
def test_softcap(device, shape):
    from arks_amd import ops

    z = torch.linspace(-90, 90, shape[0] * shape[1]).reshape(shape)
    got = ops.softcap_(z.clone().to(device), 7.0).double().cpu()
    assert torch.allclose(got, 7.0 * torch.tanh(z.double() / 7.0), atol=1e-5)


@pytest.mark.parametrize("device,dtype", CASES)
def test_router_bias_decides_and_outputs_are_weighed(device, dtype):
    """Rows whose choice the bias turns; the weights are the softmax over
    the chosen logits alone; weighing an expert's output differs from
    weighing its input."""
    from arks_amd import ops

    dev, dt = _dev(device), TDT[dtype]
    z = torch.tensor([[3.0, -1.0, 0.5, 2.0, -4.0], [-2.0, -3.0, -1.0, -5.0, -2.5],
                      [0.1, 0.0, -0.1, -0.2, 7.0]])
    bias = torch.tensor([0.0, 6.0, 0.0, -3.0, 0.5])
    wts, ids, mat = ops.moe_route_grouped(z.to(dev), 2, 1, 1, "softmax", True,
                                          matrix=True, bias=bias.to(dev))
    assert ids.cpu().tolist() == [[1, 0], [1, 2], [4, 1]]
    picked = torch.gather(z + bias, 1, ids.cpu().long())
    assert torch.allclose(wts.cpu(), torch.softmax(picked, -1), atol=1e-6)
    dense = torch.zeros_like(z).scatter(1, ids.cpu().long(), wts.cpu())
    assert torch.allclose(mat.cpu(), dense, atol=1e-6)
    for ff in (8, 9):
        g = torch.Generator().manual_seed(10)
        gu = _rounded(torch.randn(3, 5 * 2 * ff, generator=g, dtype=F64), dtype)
        act = ops.moe_glu_scaled(gu.to(dt).to(dev), mat, 5, ff, 0, False)
        act = act.double().cpu()
        tol = 1e-5 if dtype == "float32" else 3e-2
        for t in range(3):
            for e in range(5):
                a = gu[t, e * 2 * ff:e * 2 * ff + ff]
                b = gu[t, e * 2 * ff + ff:(e + 1) * 2 * ff]
                sc = float(dense[t, e])
                got = act[t, e * ff:(e + 1) * ff]
                assert torch.allclose(got, sc * O.silu(a) * b, atol=tol, rtol=tol)
                if sc == 0.0:
                    assert float(got.abs().max()) == 0.0


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("T,k,E", [(1, 1, 1), (7, 2, 3), (300, 4, 16),
                                   (1111, 3, 70), (5000, 1, 2), (2050, 8, 300)])
def test_pairs_sorted_by_expert(device, T, k, E):
    """Stable order, places and counts, with an expert nobody chose and rows
    of one expert only."""
    from arks_amd import ops

    g = torch.Generator().manual_seed(T)
    ids = torch.randint(0, E, (T, k), generator=g, dtype=torch.int32)
    if E > 2:
        ids[ids == 1] = 2
        ids[T // 2:T // 2 + 70] = 0
    rows, place, counts = (t.cpu().long() for t in
                           ops.moe_sort_pairs(ids.to(device), E, 5))
    flat = ids.reshape(-1).long()
    order = torch.argsort(flat, stable=True)
    assert torch.equal(counts, torch.bincount(flat, minlength=E))
    assert torch.equal(rows[:T * k], order // k)
    assert torch.equal(rows[T * k:], torch.zeros(5, dtype=torch.long))
    assert torch.equal(place.reshape(-1)[order], torch.arange(T * k))


@pytest.mark.gpu
def test_captured_decode_steps_equal_eager_ones(tmp_path):
    """The captured decode step, replayed many times with eager prompt steps
    in between, gives the logits of eager decode steps."""
    cfg = fast_path_config()
    write_checkpoint(tmp_path / "m", cfg, ranks=(16, 16))
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
        assert rel_err(got[False][c], got[True][c]) < 2e-2
