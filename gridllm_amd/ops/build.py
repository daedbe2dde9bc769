"""In-tree build of the HIP kernel libraries for gfx950.

Each entry of LIBS is one source under csrc/ and the shared library it
becomes next to this file, by a direct hipcc invocation (no hipify, no
CUDA-compat layer). The libraries are git-ignored. Libraries are compiled in
parallel; a file lock keeps two processes from building the same one.
"""

from __future__ import annotations

import fcntl
import glob
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from typing import Iterable, Optional

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
REPO_ROOT = os.path.dirname(os.path.dirname(PKG_DIR))
CSRC = os.path.join(REPO_ROOT, "csrc")
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")

# library name -> source. "hip": what every model shares and the Llama
# family's attention; "hybrid": layer-list models (paged attention, mLSTM,
# gated linear and lightning attention, routed experts, residual streams);
# "latent": their latent attention;
# "talk": their talking-heads attention
LIBS = {"hip": "gridllm_kernels.hip", "hybrid": "gridllm_hybrid.hip",
        "latent": "gridllm_latent.hip", "talk": "gridllm_talk.hip"}

# hipcc otherwise forms packed-FP32 instructions from plain float code; some
# of their forms give wrong results on this hardware, so all HIP code is
# compiled without the feature (the host pass warns that it does not know it)
FLAGS = [f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-shared", "-fPIC",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def lib_path(name: str) -> str:
    return os.path.join(PKG_DIR, f"libgridllm_{name}.so")


def libs_of(spec) -> list[str]:
    """The libraries that a model of this spec calls."""
    from gridllm_amd.models.registry import (HybridSpec, LatentMixer,
                                             TalkingMixer)
    if not isinstance(spec, HybridSpec):
        return ["hip"]
    mixers = [ly.mixer for ly in spec.layers]
    return ["hip", "hybrid"] + [
        lib for lib, kind in (("latent", LatentMixer), ("talk", TalkingMixer))
        if any(isinstance(m, kind) for m in mixers)]


def needs_build(name: str) -> bool:
    out = lib_path(name)
    if not os.path.exists(out):
        return True
    srcs = [os.path.join(CSRC, LIBS[name])] + glob.glob(
        os.path.join(CSRC, "*.h"))
    return max(map(os.path.getmtime, srcs)) > os.path.getmtime(out)


def _build_one(name: str, force: bool) -> str:
    out = lib_path(name)
    if not force and not needs_build(name):
        return out
    with open(out + ".lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not force and not needs_build(name):
            return out                  # another process has just built it
        tmp = f"{out}.{os.getpid()}"
        proc = subprocess.run(
            [HIPCC, *FLAGS, os.path.join(CSRC, LIBS[name]), "-o", tmp],
            capture_output=True, text=True)
        if proc.returncode != 0:
            raise RuntimeError(f"hipcc build of {LIBS[name]} failed "
                               f"(rc={proc.returncode}):\n"
                               f"{proc.stderr[-4000:]}")
        os.replace(tmp, out)
    return out


def build(force: bool = False,
          names: Optional[Iterable[str]] = None) -> list[str]:
    """Build the named libraries (all by default); returns their paths."""
    names = list(LIBS if names is None else names)
    with ThreadPoolExecutor(max_workers=len(names)) as ex:
        return list(ex.map(lambda n: _build_one(n, force), names))


if __name__ == "__main__":
    for path in build(force="--force" in sys.argv):
        print(f"built {path}")
