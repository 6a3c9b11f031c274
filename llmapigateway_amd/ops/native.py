"""The built HIP extensions and who needs them.

``_C`` holds the dense-transformer kernels and sampling, ``_H`` those of the
hybrid decoders; kernels both kinds of model run (skinny GEMM, SwiGLU, the
block allocator) are built into both. A GPU tensor that reaches an op whose
extension is missing raises: there is no fallback."""

from __future__ import annotations

import importlib
from typing import Dict

_loaded: Dict[str, object] = {}
_errors: Dict[str, str] = {}


def _load(name: str):
    """The extension module, or None (CPU-only trees are fine)."""
    if name not in _loaded:
        try:
            _loaded[name] = importlib.import_module(f"llmapigateway_amd.ops.{name}")
        except ImportError as e:
            _errors[name] = str(e)
            return None
    return _loaded[name]


def _require(name: str):
    ext = _load(name)
    if ext is None:
        raise RuntimeError(
            f"llmapigateway_amd.ops.{name} (gfx950 HIP extension) is not built but a GPU "
            "tensor reached the ops layer. Build it with `python setup.py build_ext "
            f"--inplace` (import error: {_errors[name]})"
        )
    return ext


def have_native() -> bool:
    return _load("_C") is not None and _load("_H") is not None


def dense_native():
    return _require("_C")


def hybrid_native():
    return _require("_H")


def shared_native():
    """Either extension: for kernels that are in both."""
    return _load("_C") or _require("_H")
