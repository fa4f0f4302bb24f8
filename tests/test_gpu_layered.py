"""Layered decoders with plain weights on the device against their numpy statement: products, experts, whole models in
32-bit and in bf16, prompts cut anywhere, states used again, far keys, long decoding, greedy generation through the
library's entry points."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from joshua_amd import capi
from joshua_amd.synth import layered as sl
from joshua_amd.synth import normal
from oracle import layered as ol
from tests import layered_cases as lc
from tests.layered_cases import build, check, error, feed, tokens

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32, BF16, BOUND = lc.F32, lc.BF16, lc.BOUND


# ---- products and experts alone --------------------------------------------------------------------------

@pytest.mark.parametrize("m", [1, 2, 3, 5, 8, 9, 64, 65, 200])
@pytest.mark.parametrize("n,k", [(7, 10), (33, 64), (130, 200), (64, 1100), (260, 2050)])
@pytest.mark.parametrize("qtype", [capi.F32, capi.BF16])
def test_products_with_plain_rows(qtype, n, k, m):
    w, x = normal(1, (n, k), k ** -0.5), normal(2, (m, k))
    b = sl.to_bf16(w) if qtype == capi.BF16 else w
    w = sl.from_bf16(b) if qtype == capi.BF16 else w
    got = capi.Weight.upload(qtype, b, n, k).matmul_t(m, x)
    if qtype == capi.BF16 and m > 8:
        x = sl.from_bf16(sl.to_bf16(x))          # what the matrix cores multiply
    want = x.astype(np.float64) @ w.astype(np.float64).T
    scale = np.abs(x).astype(np.float64) @ np.abs(w).astype(np.float64).T
    assert np.all(np.abs(got - want) <= 2e-6 * scale + 1e-7)


def test_plain_rows_dequantize_gather_and_view():
    n, k = 9, 70
    w = normal(3, (n, k))
    for qtype, b, ref in ((capi.F32, w, w), (capi.BF16, sl.to_bf16(w), sl.from_bf16(sl.to_bf16(w)))):
        wt = capi.Weight.upload(qtype, b, n, k)
        assert np.array_equal(wt.dequantize(), ref)
        assert np.array_equal(wt.embedding(np.array([8, 0, 3], np.uint32)), ref[[8, 0, 3]])
        part = wt.view(2 * k * b.itemsize, 4, k)
        x = normal(4, (2, k))
        assert np.allclose(part.matmul_t(2, x), x @ ref[2:6].T, atol=1e-4)
        with pytest.raises(capi.JoshuaHipError, match="range of its rows"):
            wt.view(b.itemsize, 1, k)
        with pytest.raises(capi.JoshuaHipError, match="exceeds"):
            wt.view(6 * k * b.itemsize, 4, k)


@pytest.mark.parametrize("tokens_n", [1, 2, 8, 9, 33, 150])
@pytest.mark.parametrize("E,top,h,inter,qtype", [(5, 2, 100, 44, capi.BF16), (5, 2, 100, 44, capi.F32), (16, 3, 64, 96, capi.BF16),
                                                 (3, 1, 41, 22, capi.BF16), (3, 2, 50, 30, capi.F32), (130, 9, 64, 24, capi.BF16), (300, 4, 32, 16, capi.BF16),
                                                 (6, 6, 256, 128, capi.F32)])
def test_experts_with_plain_rows(E, top, h, inter, qtype, tokens_n):
    limit, alpha, shift = 0.9, 1.702, 1.0
    mats = {p: normal(s, shape, shape[-1] ** -0.5) for s, (p, shape) in
            enumerate([("gate", (E * inter, h)), ("up", (E * inter, h)), ("down", (E * h, inter))], 10)}
    bits = {p: sl.to_bf16(v) if qtype == capi.BF16 else v for p, v in mats.items()}
    mats = {p: sl.from_bf16(b) if qtype == capi.BF16 else b for p, b in bits.items()}
    router, bias = normal(20, (E, h), 2.0 * h ** -0.5), normal(21, (E,))
    cfg = capi.MoeConfig(E, top, h, inter, 2, 1, 0.0, 0, 0, limit, 0.0, alpha, shift)
    wts = {p: capi.Weight.upload(qtype, b, mats[p].shape[0], mats[p].shape[1]) for p, b in bits.items()}
    layer = capi.Moe(cfg, router, wts["gate"], wts["up"], wts["down"], router_bias=bias)
    x = normal(22 + tokens_n, (tokens_n, h))
    w = {"router": router.astype(np.float64), "router.b": bias.astype(np.float64)}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"] = mats["gate"][e * inter:(e + 1) * inter], mats["up"][e * inter:(e + 1) * inter]
        w[f"e{e}.down"] = mats["down"][e * h:(e + 1) * h]
    want = ol.moe_mlp(x.astype(np.float64), w, {"router": {"top": top}, "expert": {"limit": limit}})
    got = layer.forward(x)
    d = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    assert np.all(d <= (3e-6 if qtype == capi.F32 else 2e-2)), float(d.max())
    ids, p = layer.route(x)
    oid, op = ol.route(x.astype(np.float64), w["router"], w["router.b"], top)
    assert np.array_equal(ids, oid) and np.allclose(p, op, atol=2e-6)


def test_dense_experts_refuse_what_they_cannot_run():
    w = capi.Weight.upload(capi.BF16, sl.to_bf16(normal(1, (8, 8))), 8, 8)
    q = capi.Weight.upload(capi.F32, normal(1, (8, 8)), 8, 8)
    router = normal(2, (1, 8))
    with pytest.raises(capi.JoshuaHipError, match="no kernels for expert tensors"):
        capi.Moe(capi.MoeConfig(1, 1, 8, 8, 2, 1), router, w, q, w)
    with pytest.raises(capi.JoshuaHipError, match="unknown gating"):
        capi.Moe(capi.MoeConfig(1, 1, 8, 8, 3, 1), router, w, w, w)


# ---- whole models ----------------------------------------------------------------------------------------

@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("name", list(lc.ALL))
def test_prompts_and_steps_match(tmp_path, name, compute):
    """One prompt whole, and cut so that steps of 1, 2, 8, 9 and more tokens follow each other."""
    cfg = lc.ALL[name]
    m, o, _ = build(tmp_path, cfg, 11, compute)
    toks = tokens(cfg, 12, 83)
    want = o.forward(toks)
    check(feed(m, toks, []), want, compute, "whole", o)
    check(feed(m, toks, [1, 2, 3, 5, 13, 22, 24, 55, 56, 57, 65, 67]), want, compute, "cut", o)


LAYERS = {
    "attention": lc.attention(6, 3, 28, 20, dims=12),
    "attention, no rotation scaling": lc.attention(4, 4, 32, 64, scaling=None),
    "mamba": lc.mamba(80, 12, 5, 4),
    "dense": lc.dense(lc.mamba(16, 2, 2, 2), 60, limit=0.4),
    "moe": lc.moe(lc.mamba(16, 2, 2, 2), 7, 3, 28, limit=0.4),
}


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("kind", list(LAYERS))
def test_one_layer_of_a_kind(tmp_path, kind, compute):
    cfg = lc.model(56, 77, [LAYERS[kind]], residual_mult=1.5)
    m, o, _ = build(tmp_path, cfg, 13, compute)
    toks = tokens(cfg, 14, 70)
    want = o.forward(toks)
    check(feed(m, toks, []), want, compute, "whole", o)
    check(feed(m, toks, [40, 41, 42, 50]), want, compute, "cut", o)


@pytest.mark.parametrize("size", [1, 2, 3, 7, 8, 9, 16, 31, 33, 64, 65])
def test_portions_of_one_size_equal_the_whole_prompt(tmp_path, size):
    cfg = lc.MIXED
    toks = tokens(cfg, 15, 70 if size < 16 else 140)
    for compute, bound in ((F32, 2e-5), (BF16, BOUND[BF16])):
        m, _, _ = build(tmp_path, cfg, 16, compute)
        whole = feed(m, toks, [])
        parts = feed(m, toks, range(size, len(toks), size))
        assert np.all(error(parts, whole) <= bound), size


@pytest.mark.parametrize("compute", [F32, BF16])
def test_a_sequence_leaves_nothing_behind(tmp_path, compute):
    """Caches, convolution tails and recurrent states are those of a new model after reset, whatever ran before, and a
    model with a larger cache gives the same bits."""
    cfg = lc.MIXED
    m, o, path = build(tmp_path, cfg, 17, compute)
    a, b, c = tokens(cfg, 18, 90), tokens(cfg, 19, 3), tokens(cfg, 20, 41)
    first = {i: feed(m, t, [2, 30]) for i, t in enumerate((a, b, c))}
    for order in ((2, 0, 1), (1, 1, 2, 0)):
        for i in order:
            assert np.array_equal(feed(m, (a, b, c)[i], [2, 30]), first[i]), (order, i)
    fresh = capi.Model(path, 1000, compute)
    for i, t in enumerate((a, b, c)):
        assert np.array_equal(feed(fresh, t, [2, 30]), first[i])
    o.reset()
    check(first[1], o.forward(b), compute)


def far_key_model():
    """One attention layer whose last, unrotated head dimension gives token 1 (asking) and token 0 (the key) a score that
    takes most of the softmax among hundreds of other keys."""
    cfg = lc.model(64, 120, [lc.attention(2, 1, 48, 32, dims=8, scaling=lc.YARN, scale=0.25)], residual_mult=1.0, scale=1.0)
    rng = np.random.default_rng(5)
    embed = rng.standard_normal((120, 64)).astype(np.float32)
    embed[:, :2] = 0.0
    embed[0, 0] = embed[1, 1] = 6.0
    proj = (0.5 * rng.standard_normal((3, 48, 64)) * 64 ** -0.5).astype(np.float32)
    proj[:, 47] = 0.0
    proj[0, 47, 1] = proj[1, 47, 1] = proj[2, 47, 0] = 1.5
    return cfg, {"embed": embed, "l0.mix.q": np.concatenate([proj[0], proj[1]]), "l0.mix.k": proj[2],
                 "l0.norm1": np.ones(64, np.float32), "l0.norm1.b": np.zeros(64, np.float32)}


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("place", [0, 1, 63, 64, 65, 127, 128, 191, 192, 255])
def test_a_far_key_at_the_edges_of_the_kernels_key_runs(tmp_path, place, compute):
    cfg, over = far_key_model()
    m, o, _ = build(tmp_path, cfg, 23, compute, override=over)
    toks = np.random.default_rng(100 + place).integers(2, cfg["vocab"], 290)
    asks = [260, 261, 289]
    toks[place], toks[asks] = 0, 1
    want = o.forward(toks)
    o.reset()
    moved = toks.copy()
    moved[place] = 2
    assert np.all(error(o.forward(moved), want)[asks] > 4 * BOUND[BF16])   # the key shows in the logits
    for cuts in ([], [200, 259] + list(range(260, 290)), sorted({place, place + 2, 250, 258, 266})):
        check(feed(m, toks, cuts), want, compute, cuts)


@pytest.mark.parametrize("compute", [F32, BF16])
def test_the_first_tokens_and_the_convolutions_reach(tmp_path, compute):
    """A prompt's first tokens see zeros in front of the convolution and a zero state; with 5 taps a step of one or two
    tokens hands a tail on that is older than the step."""
    cfg = lc.model(40, 50, [lc.mamba(64, 8, 6, 5), lc.mamba(48, 3, 2, 2)], residual_mult=1.0)
    m, o, _ = build(tmp_path, cfg, 25, compute)
    toks = tokens(cfg, 26, 24)
    want = o.forward(toks)
    for cuts in ([], [1], [1, 2, 3, 4, 5, 6], [2, 4, 6, 8], [1, 3, 12, 13, 15], [9, 10]):
        check(feed(m, toks, cuts), want, compute, cuts)


@pytest.mark.parametrize("compute", [F32, BF16])
def test_slow_states_are_carried_over_hundreds_of_tokens(tmp_path, compute):
    """Decays near 1 and a first token that differs: the difference still shows 250 tokens on."""
    cfg = lc.model(40, 50, [lc.mamba(64, 8, 6, 4)], residual_mult=1.0)
    over = {"l0.mix.A_log": np.full((64, 8), -7.0, np.float32), "l0.mix.dt.b": np.full((64,), -1.0, np.float32)}
    m, o, _ = build(tmp_path, cfg, 27, compute, override=over)
    a = tokens(cfg, 28, 260)
    b = a.copy()
    b[:6] = (b[:6] + 7) % cfg["vocab"]
    wa = o.forward(a)
    o.reset()
    wb = o.forward(b)
    assert error(wb, wa)[-1] > 20 * BOUND[F32]
    for toks, want in ((a, wa), (b, wb)):
        check(feed(m, toks, []), want, compute)
        check(feed(m, toks, [100, 101, 230] + list(range(240, 260))), want, compute)


@pytest.mark.parametrize("compute", [F32, BF16])
def test_long_decoding(tmp_path, compute):
    cfg = lc.MIXED
    m, o, _ = build(tmp_path, cfg, 29, compute)
    toks = tokens(cfg, 30, 300)
    want = o.forward(toks)
    check(feed(m, toks, range(20, 300)), want, compute, oracle=o)


def test_wanted_places_in_any_order(tmp_path):
    cfg = lc.MIXED
    m, _, _ = build(tmp_path, cfg, 31, F32)
    toks = tokens(cfg, 32, 40)
    every = feed(m, toks, [])
    m.reset()
    assert m.logits_at(toks[:10], 0, []).shape == (0, cfg["vocab"])
    got = m.logits_at(toks[10:], 10, [29, 3, 3, 0])
    assert np.all(error(got, every[[39, 13, 13, 10]]) < 2e-5) and np.array_equal(got[1], got[2])
    m.reset()
    m.logits_at(toks[:39], 0, [])
    one = m.logits_at(toks[39:], 39, [0, 0])
    assert np.array_equal(one[0], one[1]) and np.all(error(one, every[[39, 39]]) < 2e-5)


def test_greedy_generation_through_the_entry_points(tmp_path):
    """generate(), and the plugin's four symbols with the pick on the host, against greedy picks from the numpy statement (where
    its best two tokens lie apart)."""
    cfg = lc.MIXED
    m, o, path = build(tmp_path, cfg, 33, F32)
    prompt = tokens(cfg, 34, 21)
    got = m.generate(prompt, 40)
    o.reset()
    logits = o.forward(prompt)[-1]
    for i, t in enumerate(got):
        top = np.sort(logits)[-2:]
        if top[1] - top[0] > 1e-3:
            assert t == int(logits.argmax()), i
        logits = o.forward([t])[-1]
    assert m.generate(prompt, 40) == got
    plug = capi.NpuPlugin(path, 64)
    assert plug.rc == 0 and plug.vocab == cfg["vocab"]
    m16 = capi.Model(path, 64)
    picks = m16.generate(prompt, 40)
    step, pos = list(prompt), 0
    for t in picks:
        rc, logits = plug.forward(step, pos)
        pos += len(step)
        assert rc == 0 and logits[t] == logits.max()
        step = [t]
    assert plug.forward(step, pos + 1)[0] == -3 and plug.forward([0] * 9, pos)[0] == -4
    assert plug.reset() == 0 and plug.forward(prompt, 0)[0] == 0


def test_steps_that_are_refused(tmp_path):
    cfg = lc.ONES
    m, _, path = build(tmp_path, cfg, 35, BF16, n_ctx=12)
    assert (m.vocab, m.context, m.cached_tokens) == (cfg["vocab"], 12, 0)
    m.forward([1, 2, 3], 0)
    for call, text in ((lambda: m.forward([1], 2), "does not match the 3 tokens"), (lambda: m.forward([1] * 10, 3), "exceed the context of 12"),
                       (lambda: m.forward([cfg["vocab"]], 3), "out of range"), (lambda: m.forward([], 3), "at least one token"),
                       (lambda: m.logits_at([1, 2], 3, [2]), "wanted at place 2 of 2")):
        with pytest.raises(capi.JoshuaHipError, match=text):
            call()
    assert m.cached_tokens == 3
    m.forward([4], 3)


def test_tensors_that_are_missing_or_misshapen(tmp_path):
    cfg = lc.ONES
    tensors = sl.layered_tensors(cfg, 36)
    for name in ("head", "l0.mix.vmix", "l1.mix.conv.b", "l2.mix.vmix", "l2.mlp.e1.down", "l3.norm1b.b"):
        if name == "l0.mix.vmix":
            continue                                   # the first mixing layer's is not read
        sl.write_folder(str(tmp_path), cfg, {k: v for k, v in tensors.items() if k != name})
        with pytest.raises(capi.JoshuaHipError, match=name.replace(".", r"\.")):
            capi.Model(str(tmp_path), 16)
    sl.write_folder(str(tmp_path), cfg, {**tensors, "l1.mix.D": np.zeros(34, np.uint16)})
    with pytest.raises(capi.JoshuaHipError, match="shape the configuration implies"):
        capi.Model(str(tmp_path), 16)
    # f32 tensors load, too
    sl.write_folder(str(tmp_path), cfg, {k: sl.from_bf16(v).reshape(v.shape) for k, v in tensors.items()})
    a = capi.Model(str(tmp_path), 16).forward([1, 2, 3], 0)
    sl.write_folder(str(tmp_path), cfg, tensors)
    assert np.array_equal(capi.Model(str(tmp_path), 16).forward([1, 2, 3], 0), a)


def test_trace_runner_replays_requests(tmp_path):
    cfg = lc.MIXED
    m, o, path = build(tmp_path, cfg, 37, F32)
    a, b = tokens(cfg, 38, 30), tokens(cfg, 39, 12)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:19].tolist(), "want": [4, 18]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[19:21].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:].tolist(), "want": [8]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b.tolist(), "want": [0, 11]}], "end": ["b"]}]
    out = tmp_path / "out"
    out.mkdir()
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(out),
                          "--max-tokens", "40"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert run.returncode == 0, run.stderr[-500:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    wa = o.forward(a)
    o.reset()
    wb = o.forward(b)
    for name, want in (("0.f32", wa[[4, 18]]), ("2.f32", wa[[29]]), ("3.f32", wb[[0, 11]])):
        check(np.fromfile(out / name, "<f4").reshape(len(want), -1), want, F32, name)
