"""GPU: whole layer-list models through the library's own step function, caches, generation loop and
trace replay, against the float64 reference (tests/ref_stack.py)."""
import importlib
import io
import json
import os

import numpy as np
import pytest

import ref_stack as R
import stack_models as M
import synth
import util

pytestmark = pytest.mark.gpu

NAMES = sorted(M.CONFIGS)


class Dut:
    """A model on the device; feed() takes a sequence's next tokens in one step."""

    def __init__(self, orn, ctx, cfg, w, act, rows=256, window=4):
        self.ws, self.model = M.load(orn, ctx, cfg, w, act)
        self.model.set_max_rows(rows)
        self.caches = self.model.make_cache(64, window)

    def feed(self, toks, capture=False, caches=None):
        return self.model.logits_f32(self.model.forward(caches or self.caches, toks, capture))

    def feed_in(self, toks, cuts):
        out, at = [], 0
        for n in cuts:
            out.append(self.feed(toks[at:at + n]))
            at += n
        assert at == len(toks)
        return np.concatenate(out)

    def close(self):
        self.caches.close()
        self.model.close()
        self.ws.close()


def _err(got, want):
    """rms over the vocabulary of the mean-free difference, relative to the logits' own rms; per row"""
    d = got - want
    d = d - d.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt(np.mean((want - want.mean(axis=-1, keepdims=True)) ** 2))


# What the precisions leave at an ordinary position; where the model itself is touchy (a denominator near
# zero, two maps that cancel), three times what disturbances of that size do to the reference's logits.
LIMIT = {0: 2e-5, 1: 0.03}


class Want:
    """Logits of a sequence and how far rounding may take them, position by position."""

    def __init__(self, cfg, w, toks, act):
        rng = np.random.default_rng(99)
        self.act, self.logits = act, R.Run(cfg, w).feed(toks)
        size = 2.0 ** -22 if act == 0 else 2.0 ** -9
        moved = [_err(R.Run(cfg, w, lambda x: x * (1 + size * rng.uniform(-1, 1, np.shape(x)))).feed(toks),
                self.logits) for _ in range(4)]
        self.limit = np.maximum(LIMIT[act], 3 * np.max(moved, axis=0))

    def check(self, got, what, at=0):
        """got: logits of the rows from `at` on (or at the rows listed)."""
        rows = at if isinstance(at, list) else slice(at, at + len(got))
        e = _err(np.asarray(got, np.float64), self.logits[rows]) / self.limit[rows]
        # (four disturbed runs do not find every touchy position)
        assert e.max() < 2 and np.sum(e > 1) <= max(1, len(e) // 50), (what, float(e.max()), int(e.argmax()),
                int(np.sum(e > 1)))


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("name", NAMES)
def test_prompt_portions_and_decoding(orn, ctx, name, act):
    """A prompt at once, in portions down to two tokens, its end token by token, token by token from the
    start; caches reset and used again in between, growing past their first capacity."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 11)
    toks = np.random.default_rng(12).integers(0, cfg["vocab"], 171)
    want = Want(cfg, w, toks, act)
    d = Dut(orn, ctx, cfg, w, act)
    for cuts in ([171], [2, 64, 2, 33, 2, 31, 37], [150] + [1] * 21, [65, 64, 42], [1] * 171):
        d.caches.reset()
        want.check(d.feed_in(toks, cuts), (name, cuts[:4]))
    d.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("name", ["even", "rv_even"])
def test_every_prefix_length_around_the_edges(orn, ctx, name, act):
    """Last-token logits of prompts whose length passes the windows', blocks' and chunks' edges one by one,
    the shortest included; one cache for all of them."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 21)
    toks = np.random.default_rng(22).integers(0, cfg["vocab"], 131)
    want = Want(cfg, w, toks, act)
    d = Dut(orn, ctx, cfg, w, act)
    for n in [1, 2, 3, 4, 8, 9, 10, 31, 32, 33, 34, 63, 64, 65, 95, 96, 97, 127, 128, 129, 131]:
        d.caches.reset()
        want.check(d.feed(toks[:n])[-1:], n, at=n - 1)
    d.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("name", ["odd", "rv_odd", "rv_latent"])
def test_sequences_take_turns(orn, ctx, name, act):
    """Two sequences with caches of their own, step by step in turn, then a third in a cache given back:
    each as if alone."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 31)
    rng = np.random.default_rng(32)
    d = Dut(orn, ctx, cfg, w, act)
    other = d.model.make_cache(16, 1)
    a, b, c = (rng.integers(0, cfg["vocab"], n) for n in (120, 57, 90))
    got = {0: [], 1: []}
    for i, (n, m) in enumerate([(40, 1), (1, 50), (70, 2), (8, 3), (1, 1)]):
        at, bt = sum(map(len, got[0])), sum(map(len, got[1]))
        got[0].append(d.feed(a[at:at + n]))
        got[1].append(d.feed(b[bt:bt + m], caches=other))
    for toks, g in ((a, got[0]), (b, got[1])):
        Want(cfg, w, toks, act).check(np.concatenate(g), len(toks))
    other.reset()
    Want(cfg, w, c, act).check(d.feed(c, caches=other), "reused")
    other.close()
    d.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("name", ["even", "rv_even"])
def test_long_decoding(orn, ctx, name, act):
    """Three hundred tokens one by one: windows slide over decoded tokens, the cache grows twice."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 41, gate_bias=4.0)
    toks = np.random.default_rng(42).integers(0, cfg["vocab"], 310)
    want = Want(cfg, w, toks, act)
    d = Dut(orn, ctx, cfg, w, act)
    want.check(d.feed_in(toks, [10] + [1] * 300), "long")
    assert d.caches.capacity >= 310
    d.close()


@pytest.mark.parametrize("name", NAMES)
def test_rewind(orn, ctx, name):
    """A captured step of which only the first rows are kept: what follows is as if the rest had never been."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 51)
    toks = np.random.default_rng(52).integers(0, cfg["vocab"], 60)
    d = Dut(orn, ctx, cfg, w, 0)
    for keep in (1, 2, 4):
        d.caches.reset()
        d.feed(toks[:40])
        d.feed(toks[40:44], capture=True)
        d.model.rewind(d.caches, keep)
        follow = np.concatenate([toks[:40 + keep], toks[50:60]])
        Want(cfg, w, follow, 0).check(d.feed(toks[50:60]), (name, keep), at=40 + keep)
        d.feed(toks[44:47], capture=True)
        d.model.rewind(d.caches, 3)
        Want(cfg, w, np.concatenate([follow, toks[44:48]]), 0).check(d.feed(toks[47:48]), (name, keep, "again"),
                at=len(follow) + 3)
    d.close()


@pytest.mark.parametrize("name", ["even", "odd", "memory", "rv_even", "rv_odd"])
def test_greedy_generation(orn, ctx, name):
    """The library's generation loop in 32-bit: the reference's argmax at every step, as far as bf16 logits
    (what the samplers read) can tell it from the runner-up; and the same from short prefill chunks. In
    bf16 the loop emits what stepping the model by hand gives."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 61)
    prompt = np.random.default_rng(62).integers(0, cfg["vocab"], 75).astype(np.uint32)
    d = Dut(orn, ctx, cfg, w, 0, rows=64)
    toks = orn.generate_step(d.model, d.caches, prompt, 24)
    run = R.Run(cfg, w)
    logits = run.feed(prompt)[-1]
    for i, t in enumerate(toks):
        assert logits.max() - logits[t] <= 2.0 ** -7 * np.abs(logits).max(), i
        logits = run.feed([t])[-1]
    assert d.caches.offset == 75 + 24
    d.caches.reset()
    again = orn.generate_step(d.model, d.caches, prompt, 24, prefill_step=7)
    assert again[:4] == toks[:4]
    d.close()
    d = Dut(orn, ctx, cfg, w, 1, rows=64)
    toks = orn.generate_step(d.model, d.caches, prompt, 16)
    d.caches.reset()
    h = d.model.forward(d.caches, prompt[:64])
    h = d.model.forward(d.caches, prompt[64:74])
    h = d.model.forward(d.caches, prompt[74:])
    for t in toks:
        assert int(np.argmax(util.bf16_to_f32(d.model.logits(h[-1:]))[0])) == t
        h = d.model.forward(d.caches, [t])
    smp = orn.Sampler(1, 0.8, 0.9, 20, 5, 0, 0)
    d.caches.reset()
    sampled = orn.generate_step(d.model, d.caches, prompt, 12, sampler=smp)
    d.caches.reset()
    assert sampled == orn.generate_step(d.model, d.caches, prompt, 12, sampler=smp) and max(sampled) < cfg["vocab"]
    d.close()


def _write_model(tmp_path, cfg, w, orn):
    d = str(tmp_path / "m")
    os.mkdir(d)
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    synth.write_safetensors(os.path.join(d, "model.safetensors"), {n: (util.f32_to_bf16(a), orn.DT_BF16) for n,
            a in w.items()})
    return d


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "rv_even"])
def test_trace_replay(orn, ctx, tmp_path, monkeypatch, capsys, name, dtype):
    """bin/trace_run's program on a model read from files: portions, wanted places in any order, a request
    that ends and another that takes its cache, steps in which nothing is wanted."""
    trace = importlib.import_module("ornith-rs_amd.trace")
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 71)
    d = _write_model(tmp_path, cfg, w, orn)
    rng = np.random.default_rng(72)
    a, b = rng.integers(0, cfg["vocab"], 50).tolist(), rng.integers(0, cfg["vocab"], 9).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [39, 0, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[40:42], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[42:], "want": list(range(8))}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [8]}], "end": ["b"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    out = tmp_path / "out"
    out.mkdir()
    assert trace.main(["--model", d, "--dtype", dtype, "--out", str(out), "--max-tokens", "60"]) == 0
    assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = (Want(cfg, w, t, 0 if dtype == "float32" else 1) for t in (a, b))
    for n, want, at in ((0, wa, [39, 0, 7]), (2, wa, 42), (3, wb, 8)):
        want.check(np.fromfile(str(out / f"{n}.f32"), np.float32).reshape(-1, cfg["vocab"]), n, at)
    assert not (out / "1.f32").exists()


def _refuses(orn, ctx, name):
    """What a config.json or a tensor must not be is an error that names it: fails(edit of the configuration, ..)."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 81)

    def fails(edit, drop=None, match=None, shape=None):
        c = json.loads(json.dumps(cfg))
        edit(c)
        ws = orn.WeightStore(ctx)
        for n, a in w.items():
            if n != drop:
                ws.put(n, util.f32_to_bf16(a if n != shape else a[:-1]), orn.DT_BF16)
        with pytest.raises(orn.OrnithError, match=match):
            orn.TextModel.from_json(ctx, ws, c)
        ws.close()

    fails(lambda c: c.update(architecture="Nobody"), match="Nobody")
    fails(lambda c: c["layers"][0].update(type="conv"), match="conv")
    fails(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), match="rot")
    fails(lambda c: c["layers"][1]["mixer"].update(heads=5), match="decay" if name == "rv_even" else "mix.q")
    fails(lambda c: c["layers"][1]["mlp"].update(kind="moe"), match="mlp")
    fails(lambda c: c.pop("norm"), match="eps")
    return fails


def test_config_is_checked(orn, ctx):
    fails = _refuses(orn, ctx, "even")
    fails(lambda c: c["layers"][0]["mixer"].pop("diff"), match="diff")
    fails(lambda c: None, drop="l2.mix.f.b", match="l2.mix.f.b")
    fails(lambda c: None, shape="l0.mix.k", match="l0.mix.k")


def test_config_is_checked_side_by_side(orn, ctx):
    fails = _refuses(orn, ctx, "rv_even")
    fails(lambda c: c.pop("residual_mult"), match="residual_mult")
    fails(lambda c: c["layers"][0]["mixer"].pop("kv_rank"), match="kv_rank")
    fails(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), match="slow")
    fails(lambda c: c["layers"][2]["mixer"].update(kv_from=1), match="kv_from")
    fails(lambda c: c["layers"][2]["mixer"].update(kv_from=2), match="kv_from")
    fails(lambda c: c["layers"][2]["mixer"]["rot"].update(base=999.0), match="rot")
    fails(lambda c: None, drop="l0.mix.sink", match="l0.mix.sink")
    fails(lambda c: None, drop="embed.norm", match="embed.norm")
    fails(lambda c: None, shape="l0.mix.uk", match="l0.mix.uk")


def test_a_draft_head_is_refused(orn, ctx):
    cfg = M.CONFIGS["memory"]
    ws, model = M.load(orn, ctx, cfg, M.weights(cfg, 1), 1)
    with pytest.raises(orn.OrnithError, match="draft head"):
        orn.MtpHead(model, ws, 16)
    with pytest.raises(orn.OrnithError, match="draft head"):
        orn.FrSpec(model, ids=[1, 2])
    model.close()
    ws.close()
