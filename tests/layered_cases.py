"""Small configurations of layered decoders that the tests share, and what compares a model with its numpy statement."""
from __future__ import annotations

import numpy as np

from joshua_amd import capi
from joshua_amd.synth import layered as sl
from oracle import layered as ol

YARN = {"factor": 3.0, "original": 40, "fast": 8.0, "slow": 0.5}


def attention(heads, kv_heads, dim, vdim, dims=None, base=5000.0, scaling=YARN, scale=None, v_mix=False):
    return {"type": "attention", "mlp": None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "v_mix": v_mix,
                      "scale": dim ** -0.5 if scale is None else scale,
                      "rot": {"dims": dim if dims is None else dims, "base": base, **({"scaling": dict(scaling)} if scaling else {})}}}


def mamba(inner, state, dt_rank, conv):
    return {"type": "mamba1", "mlp": None, "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}}


def dense(layer, ff, limit=1.1):
    return {**layer, "mlp": {"kind": "dense", "ff": ff, "limit": limit}}


def moe(layer, experts, top, ff, limit=0.8):
    return {**layer, "mlp": {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}}


def model(width, vocab, layers, eps=1e-5, residual_mult=0.6, scale=3.0):
    return {"architecture": "Bozosun", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "residual_mult": residual_mult, "layers": layers}


# every branch in one stack: values mixed in some attention layers (not the first), a feed-forward block of every
# kind and none, partly rotated heads, with and without YaRN
MIXED = model(100, 131, [
    attention(3, 3, 20, 52, dims=8, scaling=None),
    moe(attention(6, 2, 40, 24, dims=16, v_mix=True), 5, 2, 44),
    mamba(72, 5, 7, 3),
    dense(mamba(136, 20, 12, 4), 90),
    dense(attention(4, 1, 72, 48, v_mix=True), 100, limit=0.5),
    moe(mamba(64, 16, 3, 2), 9, 4, 20, limit=2.0),
    attention(2, 2, 36, 24, dims=36, base=100.0, v_mix=True),
])
# values that are often 1 or equal
ONES = model(64, 70, [
    moe(attention(1, 1, 16, 32, v_mix=True), 3, 1, 16),
    dense(mamba(33, 1, 1, 1), 17),
    moe(attention(9, 1, 32, 32, dims=2, v_mix=True), 2, 2, 33),
    mamba(128, 37, 130, 5),
], eps=1e-3, residual_mult=1.0, scale=1.0)
# long heads: key and value classes of 256, and past what the tiled kernels take
WIDE = model(72, 90, [
    dense(attention(4, 2, 160, 130, dims=64, v_mix=True), 70),
    dense(attention(2, 1, 300, 260, dims=300, v_mix=True), 50),
    attention(18, 1, 96, 80),
    mamba(40, 140, 9, 4),
], eps=1e-4, residual_mult=0.25, scale=8.0)
# many experts: gating past one wave's reach
CROWD = model(48, 60, [moe(attention(2, 1, 24, 24), 300, 5, 8), moe(mamba(48, 8, 4, 4), 70, 66, 12)], residual_mult=0.9)

# sizes that are no multiple of anything
ODD = model(51, 33, [
    moe(attention(3, 1, 10, 7, dims=6, v_mix=True), 6, 3, 30),
    dense(mamba(21, 3, 5, 4), 13),
    moe(attention(2, 1, 5, 7, dims=2, v_mix=True), 70, 2, 9),
])

ALL = {"mixed": MIXED, "ones": ONES, "wide": WIDE, "crowd": CROWD, "odd": ODD}


# ---- Fasesun ---------------------------------------------------------------------------------------------

def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=3000.0, scale=None):
    return {"type": "latent_attention", "mlp": None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"dims": rot_dim, "base": base}}}


def mlstm(heads, dim, vdim, gate_cap=9.0):
    return {"type": "mlstm", "mlp": None, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}}


def lightning(dim, vdim, decay):
    return {"type": "lightning", "mlp": None, "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay}}


def experts(layer, n, top, ff, shared=None):
    return {**layer, "mlp": {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top},
                             **({"shared": {"ff": shared}} if shared else {})}}


def fasesun(width, vocab, layers, eps=1e-5, loop=None):
    return {"architecture": "Fasesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None}


# every mixer with and without experts, with and without a shared one, the middle run three times
FASE_MIXED = fasesun(100, 131, [
    experts(mlstm(3, 24, 40), 5, 2, 44, shared=28),
    latent(5, 20, 12, 28, 36, 44),
    experts(lightning(48, 20, [0.5, 0.97]), 7, 3, 20),
    experts(latent(2, 40, 8, 52, 70, 24, scale=0.3), 4, 1, 36, shared=36),
    mlstm(2, 36, 72, gate_cap=4.0),
], loop=(1, 4, 3))
# values that are often 1 or equal
FASE_ONES = fasesun(64, 70, [
    experts(latent(1, 16, 2, 16, 16, 16), 3, 3, 16, shared=1),
    experts(mlstm(1, 16, 16, gate_cap=1.0), 1, 1, 17, shared=64),
    experts(lightning(16, 16, [1.0]), 2, 1, 33),
    mlstm(1, 64, 64),
], eps=1e-3, loop=(0, 1, 2))
# long heads and latents: past the classes of the tiled kernels
FASE_WIDE = fasesun(72, 90, [
    latent(2, 150, 70, 130, 90, 600),
    latent(17, 130, 62, 128, 40, 300),
    latent(2, 200, 90, 270, 33, 1100, scale=0.1),
    mlstm(2, 300, 130),
    lightning(600, 70, [0.9, 0.2]),
])
# many experts, and more pairs than experts in a short step
FASE_CROWD = fasesun(48, 60, [experts(latent(2, 24, 8, 24, 20, 16), 300, 5, 8, shared=12), experts(lightning(24, 24, [0.8, 0.99]), 70, 66, 12, shared=8),
                              experts(mlstm(2, 16, 16), 3, 2, 10)])
# sizes that are no multiple of anything
FASE_ODD = fasesun(51, 33, [
    experts(latent(3, 10, 6, 7, 13, 19), 6, 3, 30, shared=11),
    experts(mlstm(3, 5, 9), 9, 2, 13, shared=7),
    experts(lightning(7, 3, [0.3, 0.6, 0.999, 0.0, 1e-3]), 70, 2, 9),
    latent(2, 9, 4, 5, 21, 33),
], loop=(1, 3, 2))

FASE_ALL = {"mixed": FASE_MIXED, "ones": FASE_ONES, "wide": FASE_WIDE, "crowd": FASE_CROWD, "odd": FASE_ODD}

# ---- a model beside its statement ------------------------------------------------------------------------

F32, BF16 = capi.COMPUTE_F32, capi.COMPUTE_DEFAULT
# root mean square of a position's difference over that of its logits: f32 against f64; bf16 activations through the
# small stacks here
BOUND = {F32: 5e-5, BF16: 0.06}
# how far apart the last expert chosen and the first left out may lie (in logits; in scores) for 16-bit activations to
# choose another one
CLOSE_CALL = {"Bozosun": 0.05, "Fasesun": 0.015}
ORACLES = {"Bozosun": ol.LayeredOracle, "Fasesun": ol.FasesunOracle}


def oracle_of(cfg, seed, override=None):
    return ORACLES[cfg["architecture"]](cfg, {k: sl.from_bf16(v) for k, v in sl.layered_tensors(cfg, seed, override).items()})


def build(tmp_path, cfg, seed, compute, n_ctx=320, override=None):
    """(model on the device, its statement, the folder)"""
    path = sl.write_folder(str(tmp_path / "model"), cfg, sl.layered_tensors(cfg, seed, override))
    return capi.Model(path, n_ctx, compute), oracle_of(cfg, seed, override), path


def error(got, want):
    """Per position: rms of the difference (mean taken off) over the rms of the logits."""
    d = got - want
    d = d - d.mean(axis=-1, keepdims=True)
    w = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1) / (w ** 2).mean())


def check(got, want, compute, what="", oracle=None):
    """`oracle`: in bf16 a token of which its margins say that the choice of experts was close may run another expert."""
    e = error(got, want)
    bound = np.full(e.shape, BOUND[compute])
    if oracle is not None and compute == BF16:
        close = oracle.margin < CLOSE_CALL[oracle.cfg["architecture"]]
        bound[close] = 1.0
        assert close.mean() < 0.9
    assert np.all(e <= bound), (what, float((e / bound).max()), int((e / bound).argmax()))


def feed(m, toks, cuts):
    """The logits of every token, the tokens cut into steps at `cuts`."""
    m.reset()
    edges = [0] + [c for c in cuts if 0 < c < len(toks)] + [len(toks)]
    return np.concatenate([m.logits_at(toks[a:b], a, range(b - a)) for a, b in zip(edges, edges[1:])])


def tokens(cfg, seed, n):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n)
