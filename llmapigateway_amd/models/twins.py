"""Weight twins in the layouts the hand-written decode GEMMs read."""

from __future__ import annotations

import os
from typing import Dict

import torch

from .. import ops


def add_decode_twins(
    layer: Dict[str, torch.Tensor], names=("qkv", "o", "gate_up", "down")
) -> None:
    """Fragment-major twins of the decode projections for the macro-tile
    LDS-staged GEMM (ops/csrc/gemm_m256.hip) — ON by default: the twin copy
    costs ~weights-again for the projections (~14 GB for llama-3-8b, cheap
    against 288 GB HBM) and buys the decode step its dominant GEMM time back
    from the library. LLMAPI_NO_FRAG_WEIGHTS=1 opts out;
    LLMAPI_SWZ_WEIGHTS=1 selects the legacy k-major twins (gemm_skinny
    streaming form) for comparison runs."""
    if os.environ.get("LLMAPI_NO_FRAG_WEIGHTS"):
        return
    legacy = bool(os.environ.get("LLMAPI_SWZ_WEIGHTS"))
    for name in names:
        w = layer.get(name)
        if w is None or not w.is_cuda or w.dtype != torch.bfloat16:
            continue
        N, K = w.shape
        if legacy:
            if N % 64 == 0 and K % 32 == 0:
                layer[name + "_swz"] = ops.swizzle_weight(w)
            continue
        fused = name == "gate_up" and ops._m256_swiglu_config(256, N, K) is not None
        # only shapes the measured dispatch actually routes to the custom
        # kernel get a twin — qkv/gate_up twins would be dead HBM (the
        # library wins those shapes), ~9 GB at 8B and ~89 GB at 70B; a
        # gate_up with a fused-swiglu twin never uses the plain twin
        if (
            N % 64 == 0 and K % 64 == 0 and not fused
            and ops._m256_config(256, N, K) is not None
        ):
            layer[name + "_swz"] = ops.swizzle_weight_frag(w)
        if fused:
            # block-16 interleaved twin for the FUSED gate_up+swiglu
            # decode path (ops.swiglu_linear)
            layer["gate_up_int"] = ops.swizzle_weight_frag(ops.interleave_gate_up(w))
