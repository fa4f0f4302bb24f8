"""Random-weight folders (config.json, model.safetensors in bf16) of layered decoders, for tests and benchmarks."""
from __future__ import annotations

import json
import os
import re
import struct

import numpy as np

from . import normal


def to_bf16(x) -> np.ndarray:
    """f32 values as bf16 bit patterns, rounded to nearest even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16)).astype(np.uint16)


def from_bf16(b: np.ndarray) -> np.ndarray:
    return (b.astype(np.uint32) << np.uint32(16)).view(np.float32)


def bozosun_shapes(cfg: dict) -> dict:
    """name -> shape of every tensor of a Bozosun model."""
    w, out = cfg["width"], {}

    def norm(name):
        out[name], out[name + ".b"] = (w,), (w,)

    def gated(p, ff):
        out[p + "gate"], out[p + "up"], out[p + "down"] = (ff, w), (ff, w), (w, ff)

    out["embed"] = (cfg["vocab"], w)
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        norm(p + "norm1"), norm(p + "norm1b")
        if layer["type"] == "attention":
            out[p + "mix.q"], out[p + "mix.k"] = (m["heads"] * m["dim"], w), (m["kv_heads"] * m["dim"], w)
            out[p + "mix.v"], out[p + "mix.o"] = (m["kv_heads"] * m["vdim"], w), (w, m["heads"] * m["vdim"])
            if m.get("v_mix"):
                out[p + "mix.vmix"] = ()
        else:
            C, N, R = m["inner"], m["state"], m["dt_rank"]
            out.update({p + "mix.in": (2 * C, w), p + "mix.conv": (C, m["conv"]), p + "mix.conv.b": (C,), p + "mix.x": (R + 2 * N, C),
                        p + "mix.dt": (C, R), p + "mix.dt.b": (C,), p + "mix.A_log": (C, N), p + "mix.D": (C,), p + "mix.o": (w, C)})
        if not mlp:
            continue
        norm(p + "norm2"), norm(p + "norm2b")
        if mlp["kind"] == "dense":
            gated(p + "mlp.", mlp["ff"])
        else:
            E = mlp["router"]["experts"]
            for e in range(E):
                gated(p + f"mlp.e{e}.", mlp["expert"]["ff"])
            out[p + "mlp.router"], out[p + "mlp.router.b"] = (E, w), (E,)
    norm("final.norm")
    out["head"] = (cfg["vocab"], w)
    return out


def bozosun_tensor(name: str, shape, seed: int) -> np.ndarray:
    """Seeded f32 values of one tensor: matrices keep their input's scale, norms lie around 1, step sizes around
    0.01 to 1, decays spread from slow to fast."""
    role = name.split(".", 1)[-1] if name[0] == "l" and name[1].isdigit() else name
    n = normal(seed, shape if shape else (1,))
    if name == "embed":
        return n
    if "norm" in role:
        return (0.1 * n if role.endswith(".b") else 1.0 + 0.2 * n).astype(np.float32)
    if role == "mix.vmix":
        return np.float32(0.35 + 0.2 * np.tanh(n)).reshape(())
    if role == "mix.A_log":
        return (np.log(1.0 + np.arange(shape[1], dtype=np.float32))[None, :] * 0.7 - 1.0 + 0.3 * n).astype(np.float32)
    if role == "mix.dt.b":
        return (-2.0 + 1.0 * n).astype(np.float32)
    if role in ("mix.conv", "mix.D"):
        return (0.6 * n).astype(np.float32)
    if role.endswith(".b"):
        return (0.3 * n).astype(np.float32)
    return (n / np.sqrt(np.float32(shape[-1]))).astype(np.float32)


def fasesun_shapes(cfg: dict) -> dict:
    """name -> shape of every tensor of a Fasesun model."""
    w, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}

    def gated(p, ff):
        out[p + "gate"], out[p + "up"], out[p + "down"] = (ff, w), (ff, w), (w, ff)

    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        H, d, nv = m["heads"], m["dim"], m["heads"] * m["vdim"]
        out[p + "norm1"] = (w,)
        x = p + "mix."
        if layer["type"] == "latent_attention":
            Q, R, rd = m["q_rank"], m["kv_rank"], m["rot_dim"]
            out.update({x + "dq": (Q, w), x + "dq.norm": (Q,), x + "uq": (H * (d + rd), Q), x + "dkv": (R + rd, w), x + "dkv.norm": (R,),
                        x + "uk": (H * d, R), x + "uv": (nv, R), x + "sink": (H,)})
        else:
            out.update({x + "q": (H * d, w), x + "k": (H * d, w), x + "v": (nv, w), x + "norm": (nv,)})
            if layer["type"] == "mlstm":
                out.update({x + "i": (H, w), x + "i.b": (H,), x + "f": (H, w), x + "f.b": (H,)})
        out[x + "g"], out[x + "o"] = (nv, w), (w, nv)
        if not mlp:
            continue
        E = mlp["router"]["experts"]
        for e in range(E):
            gated(p + f"mlp.e{e}.", mlp["expert"]["ff"])
        out[p + "mlp.router"], out[p + "mlp.correction"] = (E, w), (E,)
        if mlp.get("shared"):
            gated(p + "mlp.shared.", mlp["shared"]["ff"])
            out[p + "mlp.shared.sg"] = (1, w)
    out["final.norm"] = (w,)
    return out


def fasesun_tensor(name: str, shape, seed: int) -> np.ndarray:
    """Seeded f32 values of one tensor: matrices keep their input's scale, norms lie around 1, forget gates mostly open."""
    role = name.split(".", 1)[-1] if name[0] == "l" and name[1].isdigit() else name
    n = normal(seed, shape)
    if name == "embed":
        return n
    if "norm" in role:
        return (1.0 + 0.2 * n).astype(np.float32)
    if role == "mix.f.b":
        return (3.0 + 1.5 * n).astype(np.float32)
    if role in ("mix.i.b", "mix.sink"):
        return n
    if role == "mlp.correction":
        return (0.1 * n).astype(np.float32)
    return (n / np.sqrt(np.float32(shape[-1]))).astype(np.float32)


SHAPES = {"Bozosun": bozosun_shapes, "Fasesun": fasesun_shapes}
VALUES = {"Bozosun": bozosun_tensor, "Fasesun": fasesun_tensor}


def layered_tensors(cfg: dict, seed: int, override: "dict | None" = None, share: bool = False) -> dict:
    """name -> bf16 bit patterns of a whole model; `override` gives f32 values of some tensors instead.  `share`: layers
    and experts repeat the values of the first tensor of their role and shape (for benchmarks: faster to make)."""
    out, made = {}, {}
    shapes, values = SHAPES[cfg["architecture"]], VALUES[cfg["architecture"]]
    for i, (name, shape) in enumerate(shapes(cfg).items()):
        key = (re.sub(r"^l\d+\.|\be\d+\.", "", name), shape)
        if share and key in made:
            out[name] = made[key]
            continue
        x = override[name] if override and name in override else values(name, shape, seed * 100003 + i)
        assert tuple(np.shape(x)) == tuple(shape), (name, np.shape(x), shape)
        out[name] = made[key] = to_bf16(x).reshape(shape)
    return out


def write_safetensors(path: str, tensors) -> None:
    """`tensors`: name -> bf16 bit patterns (uint16) or float32 arrays."""
    header, at = {}, 0
    for name, a in tensors.items():
        header[name] = {"dtype": "BF16" if a.dtype == np.uint16 else "F32", "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
    h = json.dumps(header).encode()
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for a in tensors.values():
            f.write(np.ascontiguousarray(a).data if a.ndim else a.tobytes())


def write_folder(path: str, cfg: dict, tensors: dict) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), tensors)
    return str(path)
