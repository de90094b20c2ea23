"""Builds libespresso_hip.so for gfx950 with hipcc (cross-compiles without a GPU).

Every source is compiled to an object of its own, several at a time, and the objects are linked into the shared
library.  build() recompiles everything; build(incremental=True) keeps objects that are newer than their source and
every header (a convenience while developing); build(component=...) builds a part of the library that stands alone.
"""
from __future__ import annotations

import glob
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB_DIR = os.path.join(HERE, "lib")
OBJ_DIR = os.path.join(HERE, "build")
LIB_PATH = os.path.join(LIB_DIR, "libespresso_hip.so")

# Parts of the library that can be built alone (a checkout with nothing built that serves one model): the sources under csrc/.
COMPONENTS = {
    "layered": [
        "context.cpp", "decoder_runtime.cpp", "generation.cpp", "layered_runtime.cpp", "layered_mixers.cpp", "capi_runtime.cpp", "capi_engine.cpp", "capi_layered.cpp",
        "host/engine.cpp", "host/runtime_registry.cpp", "host/layered_loader.cpp", "host/layered_config.cpp", "host/safetensors.cpp", "host/json_min.cpp",
        "host/model_support.cpp", "host/tokenizer.cpp", "host/regex_min.cpp", "kernels/decode_ops.hip", "kernels/dense_gemv.hip", "kernels/dense_gemm.hip",
        "kernels/layer_ops.hip", "kernels/retention.hip", "kernels/mamba2.hip",
        "kernels/latent_attention.hip", "kernels/window_attention.hip", "kernels/block_attention.hip",
    ],
}

# -packed-fp32-ops is switched off on purpose: packed fp32 VALU forms are not used in this library.
HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-mllvm", "-amdgpu-kernarg-preload-count=14",
    "-Wall", "-Wno-unused-function", "-Wno-c++20-extensions",   # templated lambdas (compile-time piece indices in gemm_split.hip)
]
NOISE = "is not a recognized feature for this target"


def sources() -> list[str]:
    return sorted(glob.glob(os.path.join(CSRC, "*.cpp")) + glob.glob(os.path.join(CSRC, "host", "*.cpp")) +
                  glob.glob(os.path.join(CSRC, "kernels", "*.hip")))


def headers() -> list[str]:
    return (glob.glob(os.path.join(CSRC, "**", "*.h"), recursive=True) +
            glob.glob(os.path.join(HERE, "..", "include", "*.h")))


def _object_path(src: str) -> str:
    return os.path.join(OBJ_DIR, os.path.relpath(src, CSRC).replace(os.sep, "__") + ".o")


def _run(cmd: list[str]) -> str:
    proc = subprocess.run(cmd, capture_output=True, text=True)
    err = "\n".join(l for l in proc.stderr.splitlines() if NOISE not in l)
    if proc.returncode != 0:
        raise RuntimeError(f"hipcc failed: {' '.join(cmd)}\n{err}")
    return err


def component_path(component: str) -> str:
    return os.path.join(LIB_DIR, f"libespresso_{component}.so")


def build(verbose: bool = False, incremental: bool = False, jobs: int = 8, component: str | None = None) -> str:
    """Builds the library (or one component of it) and returns its path."""
    chosen = sources() if component is None else [os.path.join(CSRC, s) for s in COMPONENTS[component]]
    path = LIB_PATH if component is None else component_path(component)
    os.makedirs(LIB_DIR, exist_ok=True)
    os.makedirs(OBJ_DIR, exist_ok=True)
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    newest_header = max(os.path.getmtime(h) for h in headers())
    todo = []
    for src in chosen:
        obj = _object_path(src)
        fresh = incremental and os.path.exists(obj) and os.path.getmtime(obj) > max(os.path.getmtime(src), newest_header)
        if not fresh:
            todo.append([hipcc, *HIPCC_FLAGS, "-I", os.path.join(HERE, "..", "include"), "-c", "-x", "hip", src, "-o", obj])
    with ThreadPoolExecutor(max_workers=max(1, jobs)) as pool:
        for cmd, err in zip(todo, pool.map(_run, todo)):
            if verbose:
                print(" ".join(cmd))
                if err.strip():
                    print(err, file=sys.stderr)
    part = f"{path}.{os.getpid()}"   # two processes may build at once
    err = _run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,-z,defs", "-o", part, *[_object_path(s) for s in chosen]])
    os.replace(part, path)
    if verbose and err.strip():
        print(err, file=sys.stderr)
    return path


if __name__ == "__main__":
    print(build(verbose="-v" in sys.argv, incremental="--incremental" in sys.argv))
