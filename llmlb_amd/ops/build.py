"""Compiles the HIP kernel libraries for gfx950, in-tree.

Each library is built from its own sources, so a program that needs one
model family compiles only that family's kernels:

  kernels   csrc/*.hip          Llama-family ops and decode GEMMs
  hybrid    csrc/hybrid/*.hip   latent, differential, windowed and
                                chunked attention, recurrences, the
                                32-bit residual stream

Command line: ``python -m llmlb_amd.ops.build [name ...]`` (all without
a name).
"""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

OPS = Path(__file__).resolve().parent

LIBRARIES = {
    "kernels": ("libllmlb_kernels.so", "csrc"),
    "hybrid": ("libllmlb_hybrid.so", "csrc/hybrid"),
}

# packed FP32 instructions stay off: some of their forms have returned
# wrong results on this hardware
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def library_path(name: str) -> Path:
    return OPS / LIBRARIES[name][0]


def build_library(name: str) -> Path:
    """Compile one library (sources in parallel) and move it in place."""
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    out = library_path(name)
    srcs = sorted((OPS / LIBRARIES[name][1]).glob("*.hip"))
    work = OPS / "csrc" / "build" / f"{name}-{os.getpid()}"
    work.mkdir(parents=True, exist_ok=True)

    def compile_one(src: Path) -> Path:
        obj = work / (src.stem + ".o")
        subprocess.run([hipcc, *FLAGS, "-c", str(src), "-o", str(obj)],
                       check=True, stdout=sys.stderr)
        return obj

    try:
        with ThreadPoolExecutor(max_workers=min(8, len(srcs))) as pool:
            objs = list(pool.map(compile_one, srcs))
        part = work / out.name
        subprocess.run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC",
                        *map(str, objs), "-o", str(part)],
                       check=True, stdout=sys.stderr)
        os.replace(part, out)
    finally:
        for f in work.glob("*"):
            f.unlink()
        work.rmdir()
    return out


def ensure_library(name: str) -> Path:
    """The built library's path; compiles it only if it is not there."""
    out = library_path(name)
    return out if out.exists() else build_library(name)


if __name__ == "__main__":
    for lib in sys.argv[1:] or list(LIBRARIES):
        print("built", build_library(lib), flush=True)
