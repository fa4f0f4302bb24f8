"""Small configurations of layered decoders that the tests share."""
from __future__ import annotations

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
