"""Build the gfx950 HIP extension in-tree:

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

Produces llmapigateway_amd/ops/_C*.so and _H*.so (git-ignored).
"""

import os

from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils.cpp_extension import BuildExtension, CUDAExtension  # noqa: E402

ROOT = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(ROOT, "llmapigateway_amd", "ops", "csrc")

# dense transformers and sampling / hybrid decoders; activation.hip and
# gemm_skinny.hip serve both. LLMAPI_EXT=_H (or _C) builds one of them only.
SOURCES = {
    "_C": ["ext.cpp", "elementwise.hip", "activation.hip", "attention_decode.hip",
           "attention_prefill.hip", "sampling.hip", "gemm_skinny.hip", "gemm_m256.hip"],
    "_H": ["ext_hybrid.cpp", "hybrid_rows.hip", "head_linear.hip", "attention_latent.hip",
           "recurrence.hip", "recurrence_chunked.hip", "bind_parallel.cpp", "tanh_rows.hip",
           "attention_paged.hip", "recurrence_decay.hip", "experts.hip", "bind_sigmoid.cpp",
           "rms_rows.hip", "attention_sigmoid.hip", "bind_streams.cpp", "stream_rows.hip",
           "attention_window.hip", "recurrence_delta.hip", "activation.hip",
           "gemm_skinny.hip"],
}
wanted = os.environ.get("LLMAPI_EXT", "_C,_H").split(",")

# mfma-vgpr-form: keep MFMA accumulators in arch VGPRs — the AGPR form
# copies every accumulator through v_accvgpr_read/write pairs each loop
# iteration. No packed fp32 (v_pk_*_f32): some of its forms have given wrong
# results on this hardware now and then.
HIP_FLAGS = ["-O3", "-std=c++17", "--offload-arch=gfx950",
             "-mllvm", "-amdgpu-mfma-vgpr-form",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

setup(
    name="llmapigateway_amd_ext",
    ext_modules=[
        CUDAExtension(
            name=f"llmapigateway_amd.ops.{name}",
            sources=[os.path.join(CSRC, f) for f in SOURCES[name]],
            extra_compile_args={"cxx": ["-O3", "-std=c++17"], "nvcc": HIP_FLAGS},
        )
        for name in wanted
    ],
    cmdclass={"build_ext": BuildExtension.with_options(no_python_abi_suffix=False)},
)
