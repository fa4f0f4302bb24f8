"""The numpy statement of the layered decoder pinned by what its mathematics fixes, and the parts of the loader that
need no GPU: configuration errors and the synthetic folders."""
import copy
import json
import math

import numpy as np
import pytest

from joshua_amd import capi
from joshua_amd.synth import layered as sl
from oracle import layered as ol
from tests import layered_cases as lc
from tests.layered_cases import oracle_of


def test_layer_norm_of_a_known_row():
    y = ol.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 2.0]), np.array([0.5, -0.5]), 0.0)
    assert np.allclose(y, [[-2.0 + 0.5, 2.0 - 0.5]])
    assert np.allclose(ol.layer_norm(np.full((1, 4), 7.0), np.ones(4), np.arange(4.0), 1e-5), [np.arange(4.0)])


def test_clamped_unit_at_its_limits():
    # past the limit: g = L, u = +-L; below it g is free
    L = 0.75
    top = L / (1 + math.exp(-1.702 * L))
    assert ol.clamped_swiglu(np.array(9.0), np.array(9.0), L) == pytest.approx(top * (L + 1))
    assert ol.clamped_swiglu(np.array(9.0), np.array(-9.0), L) == pytest.approx(top * (1 - L))
    assert ol.clamped_swiglu(np.array(-4.0), np.array(0.0), L) == pytest.approx(-4.0 / (1 + math.exp(1.702 * 4.0)))


def test_rotation_pairs_neighbours_and_keeps_the_rest():
    rot = {"dims": 4, "base": 100.0}
    v = np.arange(1.0, 7.0).reshape(1, 1, 6)
    r = ol.rotate_interleaved(v, 3, rot)[0, 0]
    for i, f in enumerate((1.0, 0.1)):
        c, s = math.cos(3 * f), math.sin(3 * f)
        u, w = v[0, 0, 2 * i], v[0, 0, 2 * i + 1]
        assert r[2 * i] == pytest.approx(u * c - w * s) and r[2 * i + 1] == pytest.approx(w * c + u * s)
    assert np.array_equal(r[4:], v[0, 0, 4:])


def test_yarn_leaves_fast_pairs_and_slows_slow_ones():
    rot = {"dims": 32, "base": 10000.0, "scaling": {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 1.0}}
    plain, one = ol.rotary_frequencies({"dims": 32, "base": 10000.0})
    f, mag = ol.rotary_frequencies(rot)
    assert one == 1.0 and mag == pytest.approx(0.1 * math.log(4.0) + 1.0)
    assert f[0] == plain[0] and f[-1] == pytest.approx(plain[-1] / 4.0)
    ratio = f / plain
    assert np.all(np.diff(ratio) <= 1e-12) and np.any((ratio > 0.26) & (ratio < 0.99))


def test_scan_of_constant_input_reaches_its_fixed_point():
    # S <- a S + dt x B converges to dt x B / (1 - a)
    T, dt, A = 400, 0.3, -0.5
    y, S = ol.selective_scan(np.full((T, 1), 2.0), np.full((T, 1), dt), np.full((1, 1), A), np.full((T, 1), 0.7), np.full((T, 1), 1.5),
                             np.array([0.25]), np.zeros((1, 1)))
    fixed = dt * 2.0 * 0.7 / (1 - math.exp(dt * A))
    assert S[0, 0] == pytest.approx(fixed) and y[-1, 0] == pytest.approx(1.5 * fixed + 0.25 * 2.0)


def test_router_weights_are_a_softmax_over_the_chosen_biased_logits():
    ids, w = ol.route(np.array([[1.0]]), np.array([[0.0], [1.0], [2.0], [0.5]]), np.array([3.0, 0.0, 0.5, 0.0]), 2)
    assert list(ids[0]) == [0, 2]
    assert np.allclose(w[0], np.exp([3.0, 2.5]) / np.exp([3.0, 2.5]).sum())


@pytest.mark.parametrize("name", ["mixed", "ones"])
def test_prefill_equals_token_by_token(name):
    cfg = lc.ALL[name]
    toks = np.random.default_rng(3).integers(0, cfg["vocab"], 19)
    o = oracle_of(cfg, 5)
    whole = o.forward(toks)
    o.reset()
    steps = np.concatenate([o.forward(toks[i:j]) for i, j in ((0, 1), (1, 2), (2, 4), (4, 9), (9, 10), (10, 19))])
    assert np.allclose(whole, steps, rtol=1e-9, atol=1e-9)


def test_values_are_mixed_with_those_of_the_first_mixing_layer():
    """Layer 1 is the first of the mixing layers: its own `vmix` means nothing, a later layer's moves the logits,
    and at lambda = 1 that layer's value projection means nothing."""
    cfg = lc.MIXED
    toks = np.random.default_rng(4).integers(0, cfg["vocab"], 9)
    base = oracle_of(cfg, 6).forward(toks)
    assert np.array_equal(oracle_of(cfg, 6, {"l1.mix.vmix": np.float32(0.9)}).forward(toks), base)
    assert not np.allclose(oracle_of(cfg, 6, {"l4.mix.vmix": np.float32(0.9)}).forward(toks), base, atol=1e-3)
    v = np.zeros((48, 100), np.float32)
    one = {"l4.mix.vmix": np.float32(1.0)}
    assert np.allclose(oracle_of(cfg, 6, one).forward(toks), oracle_of(cfg, 6, {**one, "l4.mix.v": v}).forward(toks))


def test_bf16_rounding_of_the_synthetic_tensors():
    x = np.array([1.0, 1.00390625, 1.01171875, -3.1415927, 1e-30], np.float32)   # ties go to even
    assert np.array_equal(sl.from_bf16(sl.to_bf16(x))[:3], np.array([1.0, 1.0, 1.015625], np.float32))
    assert np.all(np.abs(sl.from_bf16(sl.to_bf16(x)) - x) <= np.abs(x) * 2.0 ** -8)


def attempt(tmp_path, cfg, expect):
    (tmp_path / "config.json").write_text(cfg if isinstance(cfg, str) else json.dumps(cfg))
    with pytest.raises(capi.JoshuaHipError) as e:
        capi.Model(str(tmp_path), 16)
    assert expect in str(e.value), str(e.value)
    plug = capi.NpuPlugin(str(tmp_path), 16)
    assert plug.rc == -2


def test_configurations_are_checked_before_any_device_call(tmp_path):
    with pytest.raises(capi.JoshuaHipError, match="no such file"):
        capi.Model(str(tmp_path / "nothing"), 16)
    with pytest.raises(capi.JoshuaHipError, match="config.json"):
        capi.Model(str(tmp_path), 16)
    attempt(tmp_path, "{\"architecture\": ", "JSON")
    attempt(tmp_path, {"vocab": 3}, "no \"architecture\"")
    attempt(tmp_path, {"architecture": "Other"}, "no model of architecture `Other`: expected `Bozosun`, `Fasesun`")

    def broken(change):
        cfg = copy.deepcopy(lc.MIXED)
        change(cfg)
        return cfg

    attempt(tmp_path, broken(lambda c: c.pop("vocab")), "vocab is not a number")
    attempt(tmp_path, broken(lambda c: c.update(width=12.5)), "width is not a whole number")
    attempt(tmp_path, broken(lambda c: c.update(layers=3)), "layers is not a list")
    attempt(tmp_path, broken(lambda c: c["layers"][2].update(type="ring")), "layers[2].type names no mixer")
    attempt(tmp_path, broken(lambda c: c["layers"][1]["mixer"].pop("vdim")), "layers[1].vdim is not a number")
    attempt(tmp_path, broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=4)), "layer 1: 6 query heads over 4 kv heads")
    attempt(tmp_path, broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=22)), "layer 0: 22 of 20 dimensions rotated")
    attempt(tmp_path, broken(lambda c: c["layers"][6]["mixer"].update(vdim=20)), "layers 1 and 6 mix values of different sizes")
    attempt(tmp_path, broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=6)), "layer 1: 6 experts used of 5")
    attempt(tmp_path, broken(lambda c: c["layers"][3]["mlp"].update(kind="wide")), "names no feed-forward block")
    attempt(tmp_path, broken(lambda c: c["layers"][3]["mixer"].update(state=0)), "layer 3: zero in the mixer")


@pytest.mark.parametrize("text,bad", [("[1, 2", True), ("{\"a\" 1}", True), ("{\"a\": tru}", True), ("{} x", True), ("[" * 80 + "]" * 80, True),
                                      ("\"\\ud83d\\ude00\"", False), ("{\"architecture\": 1}", False)])
def test_malformed_json_is_refused(tmp_path, text, bad):
    attempt(tmp_path, text, "JSON" if bad else "no \"architecture\"")
