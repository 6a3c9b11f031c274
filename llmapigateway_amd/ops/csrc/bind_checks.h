// Checks of what the hybrid kernels assume of their operands.
#pragma once

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

namespace {

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;

inline bool has(const OptTensor& t) { return t.has_value() && t->defined(); }

// compute dtype of an activation; returns whether it is fp32
inline bool is_f32(const Tensor& t, const char* name) {
    TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
    TORCH_CHECK(t.scalar_type() == torch::kBFloat16 || t.scalar_type() == torch::kFloat32,
                name, " must be bf16 or fp32");
    return t.scalar_type() == torch::kFloat32;
}
inline const float* f32_ptr(const Tensor& t, int64_t numel, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 && t.is_contiguous() &&
                t.numel() == numel, name, ": fp32, dense, ", numel, " elements");
    return t.data_ptr<float>();
}
inline const int* i32_ptr(const Tensor& t, int64_t at_least, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 && t.is_contiguous() &&
                t.numel() >= at_least, name, ": int32, dense, >= ", at_least, " elements");
    return t.data_ptr<int>();
}
inline const int64_t* i64_ptr(const Tensor& t, int64_t at_least, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt64 && t.is_contiguous() &&
                t.numel() >= at_least, name, ": int64, dense, >= ", at_least, " elements");
    return t.data_ptr<int64_t>();
}
inline void same_type(const Tensor& a, const Tensor& b, const char* what) {
    TORCH_CHECK(a.is_cuda() && b.is_cuda() && a.scalar_type() == b.scalar_type(), what,
                ": dtypes differ");
}
// rows of a 2D tensor whose last dimension is dense
inline void check_rows(const Tensor& t, int64_t rows, int64_t width, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == rows && t.size(1) == width &&
                (t.stride(1) == 1 || width <= 1), name, ": [", rows, ", ", width,
                "] with dense rows");
}
// 8-element accesses possible: base 16-byte aligned, strides multiples of 8
inline bool vec8(std::initializer_list<const Tensor*> ts, std::initializer_list<int64_t> dims) {
    for (int64_t d : dims)
        if (d % 8) return false;
    for (const Tensor* t : ts) {
        if (reinterpret_cast<uintptr_t>(t->data_ptr()) % 16) return false;
        for (int64_t i = 0; i + 1 < t->dim(); ++i)
            if (t->stride(i) % 8) return false;
    }
    return true;
}

}  // namespace
