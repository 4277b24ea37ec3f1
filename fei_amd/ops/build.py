"""Build the gfx950 HIP kernel library in-tree.

The .so lives at fei_amd/ops/libfei_kernels.so so it travels with the repo
snapshot to GPU boxes (JIT caches under ~/.cache do not). hipcc
cross-compiles gfx950 without a GPU, so this runs on CPU-only machines too.
"""

from __future__ import annotations

import os
import subprocess
import sys
import tempfile
from concurrent.futures import ThreadPoolExecutor

CSRC = os.path.join(os.path.dirname(os.path.abspath(__file__)), "csrc")
OUT = os.path.join(os.path.dirname(os.path.abspath(__file__)), "libfei_kernels.so")
SOURCES = ["fei_kernels.hip", "attn_prefill.hip", "gemv.hip", "attn_decode_fused.hip", "gemv_fp8.hip", "stream_layer.hip",
           "hybrid.hip", "latent_attn.hip", "gla.hip", "sigmoid_attn.hip", "moe.hip"]
HEADERS = ["fei_common.h", "fei_epilogue.h", "fei_mma.h", "fei_attn.h"]
HIPCC = os.environ.get("HIPCC", "hipcc")
ARCH = os.environ.get("FEI_AMD_ARCH", "gfx950")
# Packed fp32 VALU instructions are off: some of their forms have returned
# wrong values on this hardware, and -O3 forms them from plain float code.
FLAGS = [f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def needs_build() -> bool:
    if not os.path.exists(OUT):
        return True
    out_mtime = os.path.getmtime(OUT)
    for src in SOURCES + HEADERS:
        if os.path.getmtime(os.path.join(CSRC, src)) > out_mtime:
            return True
    return False


def build(force: bool = False, verbose: bool = True) -> str:
    """Compile every HIP source into one shared library. Returns the path."""
    if not force and not needs_build():
        return OUT
    with tempfile.TemporaryDirectory() as tmp:
        def compile_one(src: str) -> str:
            obj = os.path.join(tmp, src + ".o")
            _run([HIPCC, *FLAGS, "-c", os.path.join(CSRC, src), "-o", obj],
                 verbose)
            return obj

        jobs = min(len(SOURCES), int(os.environ.get("MAX_JOBS", "8")))
        with ThreadPoolExecutor(max(jobs, 1)) as pool:
            objs = list(pool.map(compile_one, SOURCES))
        # link beside the target and rename: a reader never sees half a file
        part = f"{OUT}.{os.getpid()}.part"
        try:
            _run([HIPCC, *FLAGS, "-shared", *objs, "-o", part], verbose)
            os.replace(part, OUT)
        finally:
            if os.path.exists(part):
                os.unlink(part)
    return OUT


def _run(cmd, verbose: bool) -> None:
    if verbose:
        print("[fei_amd.ops.build]", " ".join(cmd), file=sys.stderr)
    result = subprocess.run(cmd, capture_output=True, text=True)
    if result.returncode != 0:
        raise RuntimeError(
            f"hipcc failed (rc={result.returncode}):\n{result.stderr[-4000:]}")


if __name__ == "__main__":
    build(force="--force" in sys.argv)
    print(OUT)
