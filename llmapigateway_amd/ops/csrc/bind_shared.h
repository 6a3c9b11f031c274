// Binding helpers, and the bindings of what every extension holds.
#pragma once

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <vector>

#include "kv_manager.cpp"

extern "C" {
hipError_t launch_swiglu(void*, const void*, int, int, int, hipStream_t);
hipError_t launch_gemm_skinny(void*, float*, const void*, const void*, int, int, int, int, int, hipStream_t);
}

namespace {

#define CHECK_HIP(call)                                                        \
    do {                                                                       \
        hipError_t err = (call);                                               \
        TORCH_CHECK(err == hipSuccess, "HIP kernel failed: ",                  \
                    hipGetErrorString(err));                                   \
    } while (0)

inline hipStream_t current_stream() {
    return at::hip::getCurrentHIPStream().stream();
}

inline void check_bf16(const torch::Tensor& t, const char* name) {
    TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
    TORCH_CHECK(t.scalar_type() == torch::kBFloat16, name, " must be bf16");
}

void swiglu(torch::Tensor out, torch::Tensor x) {
    TORCH_CHECK(x.is_cuda() && out.is_cuda());
    TORCH_CHECK(x.scalar_type() == torch::kBFloat16 || x.scalar_type() == torch::kFloat32,
                "swiglu: bf16 or fp32");
    TORCH_CHECK(out.scalar_type() == x.scalar_type());
    TORCH_CHECK(x.is_contiguous() && out.is_contiguous());
    const int I = out.size(-1);
    TORCH_CHECK(x.size(-1) == 2 * I, "x last dim must be 2*I");
    const int T = x.numel() / (2 * I);
    TORCH_CHECK(out.numel() == (int64_t)T * I);
    CHECK_HIP(launch_swiglu(out.data_ptr(), x.data_ptr(), T, I,
                            x.scalar_type() == torch::kFloat32, current_stream()));
}

void gemm_skinny(torch::Tensor y, torch::Tensor x, torch::Tensor w,
                 c10::optional<torch::Tensor> workspace, int64_t nsk,
                 bool swizzled) {
    check_bf16(x, "x");
    check_bf16(w, "w");
    check_bf16(y, "y");
    TORCH_CHECK(x.is_contiguous() && w.is_contiguous() && y.is_contiguous());
    TORCH_CHECK(x.dim() == 2 && y.dim() == 2);
    const int M = x.size(0), K = x.size(1);
    int N;
    if (swizzled) {  // w is [K/32, N, 32]
        TORCH_CHECK(w.dim() == 3 && w.size(0) == K / 32 && w.size(2) == 32);
        N = w.size(1);
    } else {
        TORCH_CHECK(w.dim() == 2 && w.size(1) == K);
        N = w.size(0);
    }
    TORCH_CHECK(y.size(0) == M && y.size(1) == N);
    float* ws = nullptr;
    if (workspace.has_value() && workspace->defined()) {
        TORCH_CHECK(workspace->scalar_type() == torch::kFloat32 &&
                    workspace->numel() >= nsk * (int64_t)M * N,
                    "workspace must be fp32 with >= nsk*M*N elements");
        ws = workspace->data_ptr<float>();
    }
    CHECK_HIP(launch_gemm_skinny(y.data_ptr(), ws, x.data_ptr(), w.data_ptr(),
                                 M, N, K, (int)nsk, swizzled ? 1 : 0,
                                 current_stream()));
}

// module_local: every extension registers its own copies
inline void bind_shared(pybind11::module_& m) {
    m.def("swiglu", &swiglu, "fused SiLU-gate multiply");
    m.def("gemm_skinny", &gemm_skinny,
          "skinny-M weight-streaming GEMM y = x @ w.T (decode projections)");
    pybind11::class_<BlockAllocator>(m, "BlockAllocator", pybind11::module_local())
        .def(pybind11::init<int64_t>())
        .def("num_free", &BlockAllocator::num_free)
        .def("allocate", &BlockAllocator::allocate)
        .def("free", &BlockAllocator::free_blocks)
        .def_property_readonly("num_blocks", &BlockAllocator::capacity);
}

}  // namespace
