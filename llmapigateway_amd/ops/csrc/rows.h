// Row-kernel helpers: vector access in either compute dtype, block sums, and
// the choice of a launch's form.
#pragma once

#include "common.h"

namespace {

template <int VEC>
__device__ __forceinline__ void load_vec(const float* p, float* f) {
    if (VEC == 8) {
        const float4 a = reinterpret_cast<const float4*>(p)[0];
        const float4 b = reinterpret_cast<const float4*>(p)[1];
        f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
        f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
    } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] = p[j];
    }
}
template <int VEC>
__device__ __forceinline__ void load_vec(const bf16* p, float* f) {
    if (VEC == 8) {
        const uint4 v = *reinterpret_cast<const uint4*>(p);
        unpack2(v.x, f[0], f[1]);
        unpack2(v.y, f[2], f[3]);
        unpack2(v.z, f[4], f[5]);
        unpack2(v.w, f[6], f[7]);
    } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] = ldf(p + j);
    }
}
template <int VEC>
__device__ __forceinline__ void store_vec(float* p, const float* f) {
    if (VEC == 8) {
        reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
        reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
    } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) p[j] = f[j];
    }
}
template <int VEC>
__device__ __forceinline__ void store_vec(bf16* p, const float* f) {
    if (VEC == 8) {
        uint4 v;
        v.x = pack2(f[0], f[1]);
        v.y = pack2(f[2], f[3]);
        v.z = pack2(f[4], f[5]);
        v.w = pack2(f[6], f[7]);
        *reinterpret_cast<uint4*>(p) = v;
    } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) stf(p + j, f[j]);
    }
}

__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_reduce_sum(v);
    const int wave = threadIdx.x >> 6, n = (blockDim.x + 63) >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (int w = 0; w < n; ++w) t += red[w];
    return t;
}

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

// g sigmoid(1.702 g) (u + 1) of g <= limit and u within +-limit
template <typename T>
__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    const float z = 1.702f * g;
    const float s = sizeof(T) == 4 ? sigmoid_f(z) : 1.f / (1.f + __expf(-z));
    return g * s * (u + 1.f);
}

template <typename T>
__device__ __forceinline__ float silu_glu(float g, float u) {
    return g * (sizeof(T) == 4 ? sigmoid_f(g) : 1.f / (1.f + __expf(-g))) * u;
}

// threads per row: enough for VEC elements each, whole waves, at most 512
inline int row_threads(int width, int vec) {
    int t = (width + vec - 1) / vec;
    t = (t + 63) / 64 * 64;
    return t < 64 ? 64 : (t > 512 ? 512 : t);
}

}  // namespace

// f32: compute dtype is fp32; vec8: widths, strides and addresses allow
// 8-element accesses
template <typename T_, int V_>
struct Form {
    using T = T_;
    static constexpr int V = V_;
};

// run launch(Form<compute dtype, elements per access>)
template <typename F>
static hipError_t pick(int f32, int vec8, F launch) {
    if (f32) {
        if (vec8) launch(Form<float, 8>{});
        else launch(Form<float, 1>{});
    } else {
        if (vec8) launch(Form<bf16, 8>{});
        else launch(Form<bf16, 1>{});
    }
    HIP_CHECK_LAST();
    return hipSuccess;
}
#define FORM(f)                                                                \
    using T = typename decltype(f)::T;                                         \
    constexpr int V = decltype(f)::V;                                          \
    (void)V
