"""Builds the HIP kernels + C ABI for gfx950 with hipcc, in-tree.

``build()`` makes ``libgptoss_mi355.so``, everything.  ``ensure_for(architecture)`` is for programs
that open one checkpoint in a fresh checkout: it returns a library that serves that model class,
compiling only the sources the class needs if none is up to date."""
from __future__ import annotations

import fcntl
import glob
import hashlib
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
OBJ = os.path.join(HERE, "build")
LIB = os.path.join(HERE, "libgptoss_mi355.so")

HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
COMMON = ["-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function", "-Wno-unused-variable",
          "-Wno-unused-command-line-argument"]
# packed fp32 VALU ops are kept off for every device translation unit
DEVICE = ["--offload-arch=gfx950", "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

#: sources every model class links
CORE = ("common.cpp", "engine.cpp", "model_registry.cpp", "glue.hip", "precise.hip", "gemm_dense.cpp",
        "gemm_bf16.hip", "gemm_mixed_bf16.hip", "gemm_tall.hip")
#: architecture -> sources of its class beside CORE (None: all of them)
MODELS = {"gpt-oss": None, "Nezavik": ("model_nezavik.cpp", "recurrent.hip", "window_attn.hip"),
          "Netinex": ("model_netinex.cpp", "retention.hip", "recurrent.hip", "window_attn.hip", "rotary.hip", "moe_layer.cpp",
                      "moe_route.hip", "moe_gemm.hip", "gemm_gather_bf16.hip", "gemm_tall_grouped.hip")}


def sources():
    return sorted(glob.glob(os.path.join(CSRC, "*.hip")) + glob.glob(os.path.join(CSRC, "*.cpp")))


def _stamp(srcs) -> str:
    """Digest of what a library of these sources is made from."""
    h = hashlib.sha256(" ".join(COMMON + DEVICE).encode())
    headers = glob.glob(os.path.join(CSRC, "*.hpp")) + glob.glob(os.path.join(HERE, "..", "include", "*.h"))
    for path in sorted(srcs) + sorted(headers):
        h.update(os.path.basename(path).encode())
        with open(path, "rb") as f:
            h.update(f.read())
    return h.hexdigest()


def _current(lib, srcs) -> bool:
    try:
        with open(lib + ".stamp") as f:
            return os.path.exists(lib) and f.read().strip() == _stamp(srcs)
    except OSError:
        return False


def _compile(src: str, obj_dir: str) -> str:
    obj = os.path.join(obj_dir, os.path.basename(src) + ".o")
    cmd = [HIPCC] + COMMON + DEVICE
    if src.endswith(".cpp"):
        cmd += ["-x", "hip"]
    cmd += ["-c", src, "-o", obj]
    r = subprocess.run(cmd, capture_output=True, text=True)
    noise = "packed-fp32-ops"
    err = "\n".join(l for l in r.stderr.splitlines() if noise not in l)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{err}")
    if err.strip():
        sys.stderr.write(err + "\n")
    return obj


def _build(lib, srcs, obj_dir, jobs):
    os.makedirs(obj_dir, exist_ok=True)
    stamp = _stamp(srcs)
    # the longest compilations first
    order = sorted(srcs, key=lambda s: (not os.path.basename(s).startswith(("gemm", "attn", "window", "recurrent")), s))
    with ThreadPoolExecutor(max_workers=jobs) as ex:
        objs = list(ex.map(lambda s: _compile(s, obj_dir), order))
    part = lib + f".{os.getpid()}.tmp"
    r = subprocess.run([HIPCC, "-shared", "-fPIC", "--offload-arch=gfx950", "-o", part] + objs,
                       capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError("link failed:\n" + r.stderr)
    os.replace(part, lib)
    with open(lib + ".stamp", "w") as f:
        f.write(stamp + "\n")


def build(jobs: int = 8, verbose: bool = True) -> str:
    srcs = sources()
    _build(LIB, srcs, OBJ, jobs)
    if verbose:
        print(f"built {LIB} from {len(srcs)} sources")
    return LIB


def ensure_for(architecture: str, jobs: int = 8) -> str:
    """Path of an up-to-date library that serves `architecture`."""
    if _current(LIB, sources()):
        return LIB
    own = MODELS.get(architecture)
    if own is None:
        srcs, lib = sources(), LIB
    else:
        srcs = [os.path.join(CSRC, s) for s in CORE + own]
        lib = os.path.join(OBJ, architecture, os.path.basename(LIB))
    os.makedirs(os.path.dirname(lib), exist_ok=True)
    with open(lib + ".lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not _current(lib, srcs):
            _build(lib, srcs, os.path.join(OBJ, architecture), jobs)
    return lib


if __name__ == "__main__":
    build()
