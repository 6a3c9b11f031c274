"""The built HIP extensions and who needs them.

``_C`` holds the dense-transformer kernels and sampling, ``_H`` those of the
hybrid decoders; kernels both kinds of model run (skinny GEMM, SwiGLU, the
block allocator) are built into both. A GPU tensor that reaches an op whose
extension is missing raises: there is no fallback."""

from __future__ import annotations

import importlib
from typing import Optional

_C = None
_C_ERR: Optional[str] = None
_H = None
_H_ERR: Optional[str] = None

try:
    _C = importlib.import_module("llmapigateway_amd.ops._C")
except ImportError as e:  # extension not built (CPU-only envs are fine)
    _C_ERR = str(e)
try:
    _H = importlib.import_module("llmapigateway_amd.ops._H")
except ImportError as e:
    _H_ERR = str(e)


def _missing(name: str, err: Optional[str]):
    raise RuntimeError(
        f"llmapigateway_amd.ops.{name} (gfx950 HIP extension) is not built but a GPU "
        "tensor reached the ops layer. Build it with `python setup.py build_ext "
        f"--inplace` (import error: {err})"
    )


def dense_native():
    return _C if _C is not None else _missing("_C", _C_ERR)


def hybrid_native():
    return _H if _H is not None else _missing("_H", _H_ERR)


def shared_native():
    """Either extension: for kernels that are in both."""
    return _C if _C is not None else hybrid_native()
