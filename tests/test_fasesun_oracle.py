"""The numpy statement of Fasesun's mechanisms pinned by what their mathematics fixes, and what its configuration reader
refuses before any device call."""
import copy
import json
import math

import numpy as np
import pytest

from joshua_amd import capi
from joshua_amd.synth import layered as sl
from oracle import layered as ol
from tests import layered_cases as lc
from tests.layered_cases import error, oracle_of, tokens


def test_rms_norm_of_a_known_row():
    assert np.allclose(ol.rms_norm(np.array([[3.0, 4.0]]), 0.0), np.array([[3.0, 4.0]]) / math.sqrt(12.5))
    assert np.allclose(ol.rms_norm(np.zeros((1, 3)), 1e-5), 0.0)


def test_decayed_memory_of_constant_input():
    """S after t tokens is the geometric sum; with decay 1 it counts, with decay 0 only the last token is left."""
    k, v, q = np.array([1.0, 2.0]), np.array([3.0]), np.array([0.5, 0.25])
    for decay in (0.0, 0.5, 1.0):
        S = np.zeros((2, 1))
        for t in range(6):
            S, o = ol.decayed_memory_step(S, k, v, q, decay)
            assert o[0] == pytest.approx(sum(decay ** j for j in range(t + 1)) * (k @ q) * 3.0)


def test_matrix_memory_equals_its_sum_without_a_running_maximum():
    """o = sum_s w_s (k_s . q) v_s / (max(|sum_s w_s (k_s . q)|, 1) + 1e-6 exp(m)) with w_s = exp(sum of f after s + i_s)."""
    rng = np.random.default_rng(1)
    T, d, dv = 9, 3, 4
    q, k, v = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, dv))
    i, f = 3.0 * rng.standard_normal(T), -np.abs(rng.standard_normal(T))
    S, n, m = np.zeros((d, dv)), np.zeros(d), 0.0
    floored = 0
    for t in range(T):
        S, n, m, o = ol.matrix_memory_step(S, n, m, q[t], k[t], v[t], i[t], f[t])
        w = np.array([math.exp(f[s + 1:t + 1].sum() + i[s]) for s in range(t + 1)]) * (k[:t + 1] @ q[t])
        floored += abs(w.sum()) < 1
        assert np.allclose(o, w @ v[:t + 1] / (max(abs(w.sum()), 1.0) + 1e-6 * math.exp(m)), rtol=1e-12)
        assert m >= i[t]
    assert 0 < floored < T


def test_the_running_maximum_starts_at_zero():
    S, n, m, _ = ol.matrix_memory_step(np.zeros((1, 1)), np.zeros(1), 0.0, np.ones(1), np.ones(1), np.ones(1), -5.0, -2.0)
    assert m == -2.0 and S[0, 0] == pytest.approx(math.exp(-3.0))


def test_the_sink_counts_once_and_takes_no_value():
    s = np.array([0.3, -1.0])
    p = ol.softmax_with_sink(s, 2.0)
    assert np.allclose(p, np.exp(s) / (np.exp(s).sum() + math.exp(2.0)))
    assert np.allclose(ol.softmax_with_sink(s + 900.0, 902.0), p)        # no overflow
    assert ol.softmax_with_sink(s, -1e4).sum() == pytest.approx(1.0)


def test_the_correction_moves_the_choice_and_not_the_weights():
    router, h = np.array([[1.0], [2.0], [0.5]]), np.array([[1.0]])
    ids, w = ol.route_sigmoid(h, router, np.array([0.0, -0.9, 0.0]), 2)
    assert list(ids[0]) == [0, 2] and np.allclose(w[0], ol.sigmoid(np.array([1.0, 0.5])))
    ids, w = ol.route_sigmoid(h, router, np.zeros(3), 2)
    assert list(ids[0]) == [1, 0] and np.allclose(w[0], ol.sigmoid(np.array([2.0, 1.0])))


def test_one_latent_token_attends_to_itself_and_the_sink():
    m = {"heads": 1, "dim": 2, "rot_dim": 2, "vdim": 3, "q_rank": 2, "kv_rank": 2, "scale": 0.7, "rot": {"dims": 2, "base": 10.0}}
    rng = np.random.default_rng(2)
    w = {k: rng.standard_normal(s) for k, s in {"dq": (2, 4), "dq.norm": (2,), "uq": (4, 2), "dkv": (4, 4), "dkv.norm": (2,), "uk": (2, 2),
                                                "uv": (3, 2), "sink": (1,), "g": (3, 4), "o": (4, 3)}.items()}
    h, cache = rng.standard_normal((1, 4)), {}
    got = ol.latent_attention(h, w, m, cache, 0, 1e-6)
    cq, down = ol.rms_norm(w["dq"] @ h[0], 1e-6) * w["dq.norm"], w["dkv"] @ h[0]
    c, q = ol.rms_norm(down[:2], 1e-6) * w["dkv.norm"], w["uq"] @ cq
    s = 0.7 * (q[:2] @ (w["uk"] @ c) + q[2:] @ down[2:])               # at position 0 nothing turns
    p = math.exp(s) / (math.exp(s) + math.exp(w["sink"][0]))
    assert np.allclose(got[0], w["o"] @ (p * (w["uv"] @ c) * ol.sigmoid(w["g"] @ h[0])))
    assert cache["c"].shape == (1, 2) and np.allclose(cache["r"][0], down[2:])


@pytest.mark.parametrize("name", ["mixed", "ones", "odd"])
def test_prefill_equals_token_by_token(name):
    cfg = lc.FASE_ALL[name]
    toks = tokens(cfg, 3, 19)
    o = oracle_of(cfg, 5)
    whole = o.forward(toks)
    o.reset()
    steps = np.concatenate([o.forward(toks[i:j]) for i, j in ((0, 1), (1, 2), (2, 4), (4, 9), (9, 10), (10, 19))])
    assert np.allclose(whole, steps, rtol=1e-9, atol=1e-9)


def test_a_repeated_run_of_layers_is_those_layers_written_out():
    cfg = lc.FASE_MIXED
    tensors = {k: sl.from_bf16(v) for k, v in sl.layered_tensors(cfg, 6).items()}
    order = [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    flat = {**cfg, "loop": None, "layers": [cfg["layers"][i] for i in order]}
    out = {k: v for k, v in tensors.items() if not k.startswith("l")}
    for at, i in enumerate(order):
        out.update({f"l{at}." + k.split(".", 1)[1]: v for k, v in tensors.items() if k.startswith(f"l{i}.")})
    toks = tokens(cfg, 7, 12)
    a, b = ol.FasesunOracle(cfg, tensors), ol.FasesunOracle(flat, out)
    assert a.runs() == order
    for lo, hi in ((0, 5), (5, 6), (6, 12)):
        assert np.allclose(a.forward(toks[lo:hi]), b.forward(toks[lo:hi]))
    # with one state for all passes of a layer the logits are others
    shared = ol.FasesunOracle(cfg, tensors)
    shared.state = [shared.state[order.index(i)] for i in order]
    a.reset()
    assert error(shared.forward(toks), a.forward(toks)).max() > 4 * lc.BOUND[lc.BF16]


def attempt(tmp_path, cfg, expect):
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(capi.JoshuaHipError) as e:
        capi.Model(str(tmp_path), 16)
    assert expect in str(e.value), str(e.value)


def test_configurations_are_checked_before_any_device_call(tmp_path):
    def broken(change):
        cfg = copy.deepcopy(lc.FASE_MIXED)
        change(cfg)
        return cfg

    attempt(tmp_path, broken(lambda c: c.pop("vocab")), "vocab is not a number")
    attempt(tmp_path, broken(lambda c: c.update(norm=None)), "norm is not an object")
    attempt(tmp_path, broken(lambda c: c["layers"][1].update(type="attention")), "layers[1].type names no mixer")
    attempt(tmp_path, broken(lambda c: c["layers"][1]["mixer"].pop("kv_rank")), "layers[1].kv_rank is not a number")
    attempt(tmp_path, broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=14)), "layer 1: 14 of 12 dimensions rotated")
    attempt(tmp_path, broken(lambda c: c["layers"][0]["mixer"].update(gate_cap=0)), "layer 0: gates capped at 0")
    attempt(tmp_path, broken(lambda c: c["layers"][2]["mixer"].update(decay=[0.5])), "layer 2: 1 decays for 2 heads")
    attempt(tmp_path, broken(lambda c: c["layers"][2]["mixer"].update(decay=[0.5, 1.5])), "layer 2: a decay of 1.5")
    attempt(tmp_path, broken(lambda c: c["layers"][2]["mixer"].update(decay=0.5)), "layers[2].decay is not a list")
    attempt(tmp_path, broken(lambda c: c["layers"][2]["mixer"].update(dim=0)), "layer 2: zero in the mixer")
    attempt(tmp_path, broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=6)), "layer 0: 6 experts used of 5")
    attempt(tmp_path, broken(lambda c: c["layers"][0]["mlp"].update(kind="dense")), "names no feed-forward block")
    attempt(tmp_path, broken(lambda c: c["loop"].update(stop=6)), "layers 1 to 6 of 5 run 3 times")
    attempt(tmp_path, broken(lambda c: c["loop"].update(times=0)), "run 0 times")
    attempt(tmp_path, broken(lambda c: c["loop"].pop("times")), "times is not a number")
