"""Loading of the in-tree kernel libraries with ctypes.  There is no fallback: a missing library raises."""
from __future__ import annotations

import ctypes
import os

import torch  # noqa: F401  (loads the HIP runtime that the libraries bind to)


class DejavuHipError(RuntimeError):
    """An entry point of a kernel library returned a non-zero status."""


def load_library(path: str, signatures: dict) -> ctypes.CDLL:
    """signatures: name -> (restype, argtypes)."""
    if not os.path.exists(path):
        raise ImportError(f"{path} is missing: build it with `python -m dejavu_amd.build` "
                          "(there is no fallback implementation)")
    lib = ctypes.CDLL(path)
    for name, (restype, argtypes) in signatures.items():
        fn = getattr(lib, name)
        fn.restype = restype
        fn.argtypes = argtypes
    return lib
