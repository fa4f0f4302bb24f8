"""Fasesun on the device against its numpy statement: each mixer and the experts alone, whole stacks in 32-bit and in bf16,
prompts cut anywhere, states and caches used again, far keys, sinks, gates at their limits, long decoding, greedy generation
through the library's entry points."""
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
from tests.layered_cases import BF16, BOUND, F32, build, check, error, feed, oracle_of, tokens

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BOTH = pytest.mark.parametrize("compute", [F32, BF16])


# ---- experts alone ---------------------------------------------------------------------------------------

@pytest.mark.parametrize("tokens_n", [1, 2, 8, 9, 33, 150])
@pytest.mark.parametrize("E,top,h,inter,shared,gated,qtype",
                         [(5, 2, 100, 44, 28, True, capi.BF16), (5, 2, 100, 44, 44, False, capi.F32), (16, 3, 64, 20, 96, True, capi.BF16),
                          (3, 1, 41, 22, 7, True, capi.BF16), (3, 2, 50, 30, 31, True, capi.F32), (130, 9, 64, 24, 1, True, capi.BF16),
                          (300, 4, 32, 16, 16, True, capi.BF16), (6, 6, 256, 128, 200, True, capi.F32), (4, 2, 36, 20, 0, False, capi.BF16)])
def test_sigmoid_routed_experts_with_a_gated_shared_one(E, top, h, inter, shared, gated, qtype, tokens_n):
    def matrix(seed, n, k):
        x = normal(seed, (n, k), k ** -0.5)
        b = sl.to_bf16(x) if qtype == capi.BF16 else x
        return capi.Weight.upload(qtype, b, n, k), (sl.from_bf16(b) if qtype == capi.BF16 else x).astype(np.float64)

    (wg, g), (wu, u), (wd, d) = matrix(10, E * inter, h), matrix(11, E * inter, h), matrix(12, E * h, inter)
    router, correction, sg = normal(20, (E, h), 2.0 * h ** -0.5), normal(21, (E,), 0.2), normal(22, (1, h), 2.0 * h ** -0.5)
    w = {"router": router.astype(np.float64), "correction": correction.astype(np.float64)}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"] = g[e * inter:(e + 1) * inter], u[e * inter:(e + 1) * inter]
        w[f"e{e}.down"] = d[e * h:(e + 1) * h]
    mlp, sh = {"router": {"top": top}}, None
    if shared:
        (sgw, sgm), (suw, sum_), (sdw, sdm) = matrix(13, shared, h), matrix(14, shared, h), matrix(15, h, shared)
        sh, mlp["shared"] = (sgw, suw, sdw), {"ff": shared}
        # (without a gate of its own the shared expert counts whole)
        w.update({"shared.gate": sgm, "shared.up": sum_, "shared.down": sdm, "shared.sg": sg.astype(np.float64)})
    layer = capi.Moe(capi.MoeConfig(E, top, h, inter, 1, 0), router, wg, wu, wd, router_bias=correction, shared=sh,
                     shared_gate=sg if gated and shared else None)
    x = normal(23 + tokens_n, (tokens_n, h))
    x64 = x.astype(np.float64)
    want = ol.shared_moe_mlp(x64, w, mlp)
    if shared and not gated:
        want += (1.0 - ol.sigmoid(x64 @ w["shared.sg"].T)) * ol.swiglu_mlp(x64, {k: w[f"shared.{k}"] for k in ("gate", "up", "down")})
    got = layer.forward(x)
    err = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    assert np.all(err <= (3e-6 if qtype == capi.F32 else 2e-2)), float(err.max())
    ids, p = layer.route(x)
    oid, op = ol.route_sigmoid(x64, w["router"], w["correction"], top)
    assert np.array_equal(ids, oid) and np.allclose(p, op, atol=2e-6)


def test_a_gate_needs_a_shared_expert():
    w = capi.Weight.upload(capi.BF16, sl.to_bf16(normal(1, (8, 8))), 8, 8)
    with pytest.raises(capi.JoshuaHipError, match="no shared expert"):
        capi.Moe(capi.MoeConfig(1, 1, 8, 8, 1, 0), normal(2, (1, 8)), w, w, w, shared_gate=np.ones(8, np.float32))


# ---- whole models ----------------------------------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("name", list(lc.FASE_ALL))
def test_prompts_and_steps_match(tmp_path, name, compute):
    """One prompt whole, and cut so that steps of 1, 2, 8, 9 and more tokens follow each other."""
    cfg = lc.FASE_ALL[name]
    m, o, _ = build(tmp_path, cfg, 11, compute)
    toks = tokens(cfg, 12, 83)
    want = o.forward(toks)
    check(feed(m, toks, []), want, compute, "whole", o)
    check(feed(m, toks, [1, 2, 3, 5, 13, 22, 24, 55, 56, 57, 65, 67]), want, compute, "cut", o)


LAYERS = {
    "latent": lc.latent(6, 28, 20, 24, 30, 52),
    "latent, heads of odd sizes": lc.latent(3, 13, 6, 11, 9, 70),
    "latent, one head": lc.latent(1, 32, 32, 32, 32, 32),
    "latent, 17 heads": lc.latent(17, 12, 4, 8, 40, 24),
    "matrix memory": lc.mlstm(3, 40, 28),
    "matrix memory, keys past the values": lc.mlstm(2, 130, 12),
    "matrix memory, two runs of rows": lc.mlstm(2, 20, 100),
    "constant decay": lc.lightning(44, 36, [0.9, 0.4, 1.0]),
    "constant decay, wide values": lc.lightning(12, 140, [0.7, 0.0]),
    "experts": lc.experts(lc.lightning(8, 8, [0.5]), 7, 3, 28, shared=40),
}


@BOTH
@pytest.mark.parametrize("kind", list(LAYERS))
def test_one_layer_of_a_kind(tmp_path, kind, compute):
    cfg = lc.fasesun(56, 77, [LAYERS[kind]])
    m, o, _ = build(tmp_path, cfg, 13, compute)
    toks = tokens(cfg, 14, 150)
    want = o.forward(toks)
    check(feed(m, toks, []), want, compute, "whole", o)
    check(feed(m, toks, [40, 41, 42, 50, 63, 64, 65, 67, 130]), want, compute, "cut", o)


def test_heads_of_one_element(tmp_path):
    """(In 32-bit: a normed number of one element is its sign.)"""
    cfg = lc.fasesun(56, 77, [lc.mlstm(2, 1, 1), lc.lightning(1, 1, [0.9]), lc.latent(2, 1, 2, 1, 1, 1)])
    m, o, _ = build(tmp_path, cfg, 13, F32)
    toks = tokens(cfg, 14, 70)
    want = o.forward(toks)
    for cuts in ([], [1, 2, 30, 38, 39]):
        check(feed(m, toks, cuts), want, F32, cuts)


@pytest.mark.parametrize("size", [1, 2, 3, 7, 8, 9, 16, 31, 33, 63, 64, 65, 127])
def test_portions_of_one_size_equal_the_whole_prompt(tmp_path, size):
    """(In 16 bits without experts: another choice by one token would show in the tokens behind it.)"""
    mixers = {**lc.FASE_MIXED, "layers": [{**layer, "mlp": None} for layer in lc.FASE_MIXED["layers"]]}
    for cfg, compute, bound in ((lc.FASE_MIXED, F32, 2e-5), (mixers, BF16, BOUND[BF16])):
        toks = tokens(cfg, 15, 70 if size < 16 else 140)
        m, _, _ = build(tmp_path, cfg, 16, compute)
        whole = feed(m, toks, [])
        parts = feed(m, toks, range(size, len(toks), size))
        assert np.all(error(parts, whole) <= bound), size


@BOTH
def test_a_sequence_leaves_nothing_behind(tmp_path, compute):
    """Caches, states and running maxima are those of a new model after reset, whatever ran before, and a model with a
    larger cache gives the same bits."""
    cfg = lc.FASE_MIXED
    m, o, path = build(tmp_path, cfg, 17, compute)
    a, b, c = tokens(cfg, 18, 90), tokens(cfg, 19, 3), tokens(cfg, 20, 41)
    first = {i: feed(m, t, [2, 30]) for i, t in enumerate((a, b, c))}
    for order in ((2, 0, 1), (1, 1, 2, 0)):
        for i in order:
            assert np.array_equal(feed(m, (a, b, c)[i], [2, 30]), first[i]), (order, i)
    fresh = capi.Model(path, 1000, compute)
    for i, t in enumerate((a, b, c)):
        assert np.array_equal(feed(fresh, t, [2, 30]), first[i])
    check(first[1], o.forward(b), compute, oracle=o)


# ---- latent attention ------------------------------------------------------------------------------------

def far_key_model(gain=6.0, sink=0.0):
    """One latent layer in which token 1 asks and token 0 answers: the last unrotated dimension of query and key is made
    of their marks alone, through latents of which the first element is nothing else."""
    cfg = lc.fasesun(64, 120, [lc.latent(2, 16, 8, 24, 20, 28, scale=0.25)])
    rng = np.random.default_rng(5)

    def rand(n, k, f=1.0):
        return (f * rng.standard_normal((n, k)) * k ** -0.5).astype(np.float32)

    embed = rng.standard_normal((120, 64)).astype(np.float32)
    embed[:, :2] = 0.0
    embed[0, 0] = embed[1, 1] = 8.0
    dq, dkv, uq, uk = rand(20, 64), rand(36, 64), rand(48, 20, 0.5), rand(32, 28, 0.5)
    dq[0], dkv[0] = 0.0, 0.0
    dq[0, 1], dkv[0, 0] = 1.5, 1.5
    for h in (0, 1):
        uq[24 * h + 15], uk[16 * h + 15] = 0.0, 0.0
        uq[24 * h + 15, 0] = uk[16 * h + 15, 0] = gain ** 0.5
    one = {"l0.norm1": 64, "l0.mix.dq.norm": 20, "l0.mix.dkv.norm": 28}
    return cfg, {"embed": embed, "l0.mix.dq": dq, "l0.mix.dkv": dkv, "l0.mix.uq": uq, "l0.mix.uk": uk,
                 "l0.mix.sink": np.full(2, sink, np.float32), "l0.mix.o": rand(64, 48, 4.0), **{k: np.ones(n, np.float32) for k, n in one.items()}}


@BOTH
@pytest.mark.parametrize("place", [0, 1, 2, 63, 64, 65, 127, 128, 191, 192, 255])
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
    assert np.all(error(o.forward(moved), want)[asks] > 3 * BOUND[BF16])   # the key shows in the logits
    for cuts in ([], [200, 259] + list(range(260, 290)), sorted({place, place + 2, 250, 258, 266})):
        check(feed(m, toks, cuts), want, compute, cuts)


@BOTH
@pytest.mark.parametrize("sink", [-30.0, 5.0, 30.0])
def test_the_sink_takes_its_share(tmp_path, sink, compute):
    """A sink below, among and far above the scores, in a prompt and token by token; without it the logits are others."""
    cfg, over = far_key_model(gain=2.0, sink=sink)
    m, o, _ = build(tmp_path, cfg, 24, compute, override=over)
    toks = tokens(cfg, 25, 80)
    want = o.forward(toks)
    if sink == 5.0:
        bare = oracle_of(cfg, 24, {**over, "l0.mix.sink": np.full(2, -1e4, np.float32)}).forward(toks)
        assert np.median(error(bare, want)) > 3 * BOUND[BF16]
    for cuts in ([], range(1, 80), [30, 37, 70]):
        check(feed(m, toks, cuts), want, compute, cuts)


@BOTH
def test_rotated_keys_know_their_places(tmp_path, compute):
    """Scores made by the rotated parts alone: a token that says the same at two places is two keys."""
    cfg = lc.fasesun(48, 60, [lc.latent(2, 4, 16, 20, 24, 16, base=50.0, scale=1.5)])
    over = {"l0.mix.uk": np.zeros((8, 16), np.float32), "l0.mix.o": normal(3, (48, 40), 0.6)}
    m, o, _ = build(tmp_path, cfg, 26, compute, override=over)
    toks = tokens(cfg, 27, 140)
    toks[1::3] = 7
    want = o.forward(toks)
    still = ol.FasesunOracle({**cfg, "layers": [{**cfg["layers"][0], "mixer": {**cfg["layers"][0]["mixer"], "rot": {"dims": 0, "base": 50.0}}}]}, o.w)
    assert np.median(error(still.forward(toks), want)) > 2 * BOUND[BF16]
    for cuts in ([], [60, 61, 70], list(range(64, 140))):
        check(feed(m, toks, cuts), want, compute, cuts)


# ---- matrix memory and constant decay --------------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("kind", ["mlstm", "lightning"])
def test_slow_states_are_carried_over_hundreds_of_tokens(tmp_path, kind, compute):
    """Gates that hardly forget and first tokens that differ: the difference still shows 250 tokens on."""
    layer = lc.mlstm(2, 24, 32, gate_cap=15.0) if kind == "mlstm" else lc.lightning(24, 32, [0.999, 1.0])
    cfg = lc.fasesun(40, 50, [layer])
    over = {"l0.mix.f.b": np.full(2, 12.0, np.float32), "l0.mix.i.b": np.zeros(2, np.float32)} if kind == "mlstm" else {}
    m, o, _ = build(tmp_path, cfg, 28, compute, override=over)
    a = tokens(cfg, 29, 260)
    b = a.copy()
    b[:40] = (b[:40] + 7) % cfg["vocab"]
    wa = o.forward(a)
    o.reset()
    wb = o.forward(b)
    assert error(wb, wa)[-1] > 100 * BOUND[F32]
    for toks, want in ((a, wa), (b, wb)):
        check(feed(m, toks, []), want, compute)
        check(feed(m, toks, [100, 101, 230] + list(range(240, 260))), want, compute)


@BOTH
@pytest.mark.parametrize("i_b,f_b,cap", [(-12.0, 2.0, 13.0), (12.0, -12.0, 13.0), (0.0, 0.0, 1.0), (6.0, 6.0, 30.0), (-5.0, -5.0, 5.0)])
def test_gates_at_their_limits(tmp_path, i_b, f_b, cap, compute):
    """Input gates that open and shut by many powers of e from token to token, so that the running maximum moves up and
    down and the normaliser lies above and below its floor; gates pressed against their cap."""
    cfg = lc.fasesun(40, 50, [lc.mlstm(3, 20, 24, gate_cap=cap)])
    over = {"l0.mix.i.b": np.array([i_b, i_b + 1, i_b - 1], np.float32), "l0.mix.f.b": np.array([f_b, f_b + 2, f_b - 2], np.float32),
            "l0.mix.i": normal(5, (3, 40), 0.6), "l0.mix.f": normal(6, (3, 40), 0.4)}
    m, o, _ = build(tmp_path, cfg, 30, compute, override=over)
    toks = tokens(cfg, 31, 140)
    want = o.forward(toks)
    for cuts in ([], [1, 2, 3, 40, 49, 64, 65], list(range(70, 140))):
        check(feed(m, toks, cuts), want, compute, cuts)


def test_a_first_token_with_a_shut_gate(tmp_path):
    """The running maximum starts at 0 and not below: an input gate of e^-12 leaves a first token almost nothing."""
    cfg = lc.fasesun(40, 50, [lc.mlstm(2, 20, 24, gate_cap=20.0)])
    over = {"l0.mix.i.b": np.full(2, -14.0, np.float32), "l0.mix.f.b": np.full(2, 8.0, np.float32), "l0.mix.i": np.zeros((2, 40), np.float32)}
    for compute in (F32, BF16):
        m, o, _ = build(tmp_path, cfg, 32, compute, override=over)
        toks = tokens(cfg, 33, 30)
        want = o.forward(toks)
        open_gate = oracle_of(cfg, 32, {**over, "l0.mix.i.b": np.zeros(2, np.float32)}).forward(toks)
        assert error(open_gate, want).min() > 2 * BOUND[BF16]
        for cuts in ([], [1, 2, 3, 4], [1, 12]):
            check(feed(m, toks, cuts), want, compute, cuts)


@BOTH
@pytest.mark.parametrize("cuts", [[1], [1, 2, 3, 4, 5, 6], [2, 4, 6, 8], [9, 10], [63], [64], [65], [128, 130]])
def test_first_tokens_and_chunk_edges(tmp_path, cuts, compute):
    cfg = lc.fasesun(40, 50, [lc.mlstm(2, 20, 24), lc.lightning(16, 24, [0.95, 0.5]), lc.latent(2, 12, 4, 8, 16, 12)])
    m, o, _ = build(tmp_path, cfg, 34, compute)
    toks = tokens(cfg, 35, 133)
    check(feed(m, toks, cuts), o.forward(toks), compute, cuts)


def test_a_prompt_longer_than_one_segment_of_chunks(tmp_path):
    cfg = lc.fasesun(24, 40, [lc.mlstm(1, 8, 12), lc.lightning(8, 12, [0.999])])
    m, o, _ = build(tmp_path, cfg, 36, BF16, n_ctx=4400)
    toks = tokens(cfg, 37, 4300)
    check(feed(m, toks, []), o.forward(toks), BF16)


# ---- the rest of the model -------------------------------------------------------------------------------

@BOTH
def test_long_decoding(tmp_path, compute):
    cfg = lc.FASE_MIXED
    m, o, _ = build(tmp_path, cfg, 38, compute)
    toks = tokens(cfg, 39, 300)
    want = o.forward(toks)
    check(feed(m, toks, range(20, 300)), want, compute, oracle=o)


@pytest.mark.parametrize("loop", [None, (0, 0, 5), (0, 3, 1), (0, 3, 2), (2, 3, 4)])
def test_repeated_layers_keep_a_state_a_pass(tmp_path, loop):
    layers = [lc.experts(lc.mlstm(2, 12, 16), 4, 2, 12, shared=8), lc.latent(2, 12, 4, 8, 16, 12), lc.lightning(16, 24, [0.95, 0.5])]
    cfg = lc.fasesun(40, 50, layers, loop=loop)
    m, o, _ = build(tmp_path, cfg, 40, F32)
    toks = tokens(cfg, 41, 50)
    want = o.forward(toks)
    for cuts in ([], [20, 21, 22, 40]):
        check(feed(m, toks, cuts), want, F32, cuts)


def test_wanted_places_in_any_order(tmp_path):
    cfg = lc.FASE_MIXED
    m, _, _ = build(tmp_path, cfg, 42, F32)
    toks = tokens(cfg, 43, 40)
    every = feed(m, toks, [])
    m.reset()
    assert m.logits_at(toks[:10], 0, []).shape == (0, cfg["vocab"])
    got = m.logits_at(toks[10:], 10, [29, 3, 3, 0])
    assert np.all(error(got, every[[39, 13, 13, 10]]) < 2e-5) and np.array_equal(got[1], got[2])


def test_greedy_generation_through_the_entry_points(tmp_path):
    """generate(), and the plugin's four symbols with the pick on the host, against greedy picks from the numpy statement
    (where its best two tokens lie apart)."""
    cfg = lc.FASE_MIXED
    m, o, path = build(tmp_path, cfg, 44, F32)
    prompt = tokens(cfg, 45, 21)
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
    picks = capi.Model(path, 64).generate(prompt, 40)
    step, pos = list(prompt), 0
    for t in picks:
        rc, logits = plug.forward(step, pos)
        pos += len(step)
        assert rc == 0 and logits[t] == logits.max()
        step = [t]
    assert plug.reset() == 0 and plug.forward(prompt, 0)[0] == 0


def test_tensors_that_are_missing_or_misshapen(tmp_path):
    cfg = lc.FASE_ONES
    tensors = sl.layered_tensors(cfg, 46)
    for name in ("embed", "l0.mix.sink", "l0.mix.dkv.norm", "l1.mix.f.b", "l1.mlp.correction", "l1.mlp.shared.sg", "l2.mix.norm", "l2.norm1", "final.norm"):
        sl.write_folder(str(tmp_path), cfg, {k: v for k, v in tensors.items() if k != name})
        with pytest.raises(capi.JoshuaHipError, match=name.replace(".", r"\.")):
            capi.Model(str(tmp_path), 16)
    sl.write_folder(str(tmp_path), cfg, {**tensors, "l0.mix.uk": np.zeros((16, 15), np.uint16)})
    with pytest.raises(capi.JoshuaHipError, match="shape the configuration implies"):
        capi.Model(str(tmp_path), 16)


def test_trace_runner_replays_requests(tmp_path):
    cfg = lc.FASE_MIXED
    m, o, path = build(tmp_path, cfg, 47, F32)
    a, b = tokens(cfg, 48, 30), tokens(cfg, 49, 12)
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
    wa = o.forward(a)
    o.reset()
    wb = o.forward(b)
    for name, want in (("0.f32", wa[[4, 18]]), ("2.f32", wa[[29]]), ("3.f32", wb[[0, 11]])):
        check(np.fromfile(out / name, "<f4").reshape(len(want), -1), want, F32, name)
