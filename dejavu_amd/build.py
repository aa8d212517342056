"""Builds the kernel libraries in-tree with hipcc for gfx950.

    libdejavu_hip.so     csrc/dejavu_hip.hip   contextual-sparsity decode path
    libdejavu_mixers.so  csrc/mixers.hip       latent, windowed and chunk-local attention, gated delta rule, Mamba-2

Run as ``python -m dejavu_amd.build``; tests and benchmarks only load the
libraries that this step leaves next to the package.
"""
from __future__ import annotations

import os
import shutil
import subprocess
import sys

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(PKG_DIR, "csrc")
LIB_NAME = "libdejavu_hip.so"
LIB_PATH = os.path.join(PKG_DIR, LIB_NAME)
MIXERS_LIB_NAME = "libdejavu_mixers.so"
MIXERS_LIB_PATH = os.path.join(PKG_DIR, MIXERS_LIB_NAME)
SOURCES = {LIB_NAME: "dejavu_hip.hip", MIXERS_LIB_NAME: "mixers.hip"}

HIPCC_FLAGS = [
    "--offload-arch=gfx950",
    "-O3",
    "-std=c++17",
    "-fPIC",
    "-shared",
    "-fvisibility=hidden",
    "-Wall",
    "-Wno-unused-function",
    # packed fp32 ALU forms are kept out of the generated code
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]


def hipcc_path() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found; it is needed to build " + LIB_NAME)
    return exe


def build_library(verbose: bool = True, name: str = LIB_NAME) -> str:
    """Compiles one library; the finished file replaces the old one in one step."""
    path = os.path.join(PKG_DIR, name)
    part = f"{path}.{os.getpid()}.tmp"
    cmd = [hipcc_path(), *HIPCC_FLAGS, "-I", os.path.join(PKG_DIR, "..", "include"),
           os.path.join(CSRC, SOURCES[name]), "-o", part]
    if verbose:
        print(" ".join(cmd), flush=True)
    try:
        subprocess.run(cmd, check=True, stdout=None if verbose else sys.stderr)
        os.replace(part, path)
    finally:
        if os.path.exists(part):
            os.unlink(part)
    return path


def ensure_built(name: str = LIB_NAME) -> str:
    """The library's path; compiled first if it is not there."""
    path = os.path.join(PKG_DIR, name)
    return path if os.path.exists(path) else build_library(verbose=False, name=name)


if __name__ == "__main__":
    for lib_name in SOURCES:
        print("built", build_library(name=lib_name))
    sys.exit(0)
