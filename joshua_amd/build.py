"""Builds the native libraries in-tree: libjoshua_hip.so (HIP, gfx950), its subset for the models that hold no
quantized blocks, and the host-only synthetic-input library."""
from __future__ import annotations

import concurrent.futures
import fcntl
import hashlib
import os
import shutil
import subprocess
import tempfile

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
HIP_LIB = os.path.join(HERE, "libjoshua_hip.so")
# The translation units behind jq_model_* for the architectures of plain BF16 / F32 weights, without the kernels of
# the block formats (api.hip): all that a folder of config.json and model.safetensors needs, in a fraction of the build.
LAYERS_LIB = os.path.join(HERE, "libjoshua_layers.so")
LAYERS_SOURCES = ("core.hip", "moe.hip", "model.hip", "dense.hip", "layers.hip")

HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function",
    # keep the compiler from forming packed-f32 instructions out of scalar float code
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    # the leading kernel arguments arrive in scalar registers with the wave instead of by a scalar load
    # from memory at its entry (0.4 us sooner to the first global load of a kernel that starts cold)
    "-mllvm", "-amdgpu-kernarg-preload-count=16",
]


def hip_sources() -> list[str]:
    return sorted(os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".hip"))


def _run(cmd: list[str]) -> str:
    res = subprocess.run(cmd, capture_output=True, text=True)
    noise = ("is not a recognized feature for this target", "warning generated", "warnings generated")
    err = "\n".join(l for l in res.stderr.splitlines() if not any(n in l for n in noise))
    if res.returncode != 0:
        raise RuntimeError(f"{os.path.basename(cmd[0])} failed:\n{err}")
    return err.strip()


def _stamp(sources: list[str]) -> str:
    """A digest of everything that goes into a library: flags, the sources, every header beside them."""
    h = hashlib.sha256(repr((HIPCC_FLAGS, [os.path.basename(s) for s in sources])).encode())
    headers = [os.path.join(CSRC, f) for f in sorted(os.listdir(CSRC)) if f.endswith((".hpp", ".h"))]
    for path in [*sources, *headers, os.path.join(HERE, "..", "include", "joshua_hip.h")]:
        with open(path, "rb") as f:
            h.update(f.read() + b"\0")
    return h.hexdigest()


def up_to_date(lib: str, sources: list[str]) -> bool:
    try:
        with open(lib + ".stamp") as f:
            return os.path.exists(lib) and f.read() == _stamp(sources)
    except OSError:
        return False


def _link(lib: str, sources: list[str], verbose: bool) -> str:
    """One object a source, side by side, then the library in one move."""
    stamp = _stamp(sources)
    tmp = tempfile.mkdtemp(prefix=".build-", dir=HERE)
    try:
        def compile_one(src: str) -> str:
            return _run(["hipcc", *HIPCC_FLAGS, "-c", "-o", os.path.join(tmp, os.path.basename(src) + ".o"), src])
        with concurrent.futures.ThreadPoolExecutor(min(len(sources), 8)) as pool:
            logs = list(pool.map(compile_one, sources))
        out = os.path.join(tmp, "lib.so")
        logs.append(_run(["hipcc", "--offload-arch=gfx950", "-shared", "-fPIC", "-o", out,
                          *(os.path.join(tmp, os.path.basename(s) + ".o") for s in sources)]))
        os.replace(out, lib)
        with open(os.path.join(tmp, "stamp"), "w") as f:
            f.write(stamp)
        os.replace(os.path.join(tmp, "stamp"), lib + ".stamp")
    finally:
        shutil.rmtree(tmp, ignore_errors=True)
    if verbose:
        for log in logs:
            if log:
                print(log)
    return lib


def build_hip(verbose: bool = False) -> str:
    return _link(HIP_LIB, hip_sources(), verbose)


def layers_library() -> str:
    """A library that runs the models of plain weights: the whole one where it is built and current, else the subset,
    compiled if it is not there or its sources have changed."""
    if up_to_date(HIP_LIB, hip_sources()):
        return HIP_LIB
    sources = [os.path.join(CSRC, f) for f in LAYERS_SOURCES]
    with open(os.path.join(HERE, ".layers.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not up_to_date(LAYERS_LIB, sources):
            _link(LAYERS_LIB, sources, False)
    return LAYERS_LIB


CALIB_SRC = os.path.join(HERE, "calib", "copy_kernel.hip")
CALIB_BIN = os.path.join(HERE, "calib", "copy_kernel")


PROBE_SRC = os.path.join(HERE, "calib", "read_probe.hip")
PROBE_BIN = os.path.join(HERE, "calib", "read_probe")
MIX_SRC = os.path.join(HERE, "calib", "gemm_mix_probe.hip")
MIX_BIN = os.path.join(HERE, "calib", "gemm_mix_probe")


def build_calibration() -> str:
    """The copy kernel that calibrates the FETCH_SIZE / WRITE_SIZE counters, the plain-read probe that gives
    the floor of one launch over a matrix of the benchmark's size, and the probe that runs the int8 GEMM's
    instruction mix of a super-block iteration with nothing else around it."""
    for src, out in ((CALIB_SRC, CALIB_BIN), (PROBE_SRC, PROBE_BIN), (MIX_SRC, MIX_BIN)):
        res = subprocess.run(["hipcc", "--offload-arch=gfx950", "-O3", "-o", out, src], capture_output=True, text=True)
        if res.returncode != 0:
            raise RuntimeError(f"hipcc failed:\n{res.stderr}")
    return CALIB_BIN


def build_all(verbose: bool = False) -> None:
    """The library and the synthetic-data helper: what tests, smoke and the benchmark load.  The counter
    calibration program is a profiling aid, built on request (`python -m joshua_amd.build --calibration`)."""
    from . import synth
    build_hip(verbose)
    synth.build()


if __name__ == "__main__":
    import sys
    if "--calibration" in sys.argv[1:]:
        print("built", build_calibration())
    else:
        build_all(verbose=True)
        print("built", HIP_LIB)
