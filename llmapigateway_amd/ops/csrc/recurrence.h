// Gate arithmetic and state access shared by the recurrence kernels (fp32).
#pragma once

#include "common.h"

// log(1 + e^z) without overflow
__device__ __forceinline__ float softplus_f(float z) {
    return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}
__device__ __forceinline__ float log_sigmoid_f(float z) {
    return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}
__device__ __forceinline__ float soft_cap_f(float z, float cap) {
    return cap * tanhf(z / cap);
}

// a 16-lane group shares a state row; lane's key dims: 64 * e4 + 4 * l16 + j
template <typename T, int E4>
__device__ __forceinline__ void load_dims(const T* p, int l16, int dk, float (*f)[4]) {
#pragma unroll
    for (int e = 0; e < E4; ++e)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int i = 64 * e + 4 * l16 + j;
            f[e][j] = i < dk ? ldf(p + i) : 0.f;
        }
}
template <int E4>
__device__ __forceinline__ void load_state(
    const float* p, int l16, int dk, bool vec, float (*f)[4]) {
#pragma unroll
    for (int e = 0; e < E4; ++e) {
        const int i = 64 * e + 4 * l16;
        if (vec) {
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i < dk) v = *reinterpret_cast<const float4*>(p + i);
            f[e][0] = v.x; f[e][1] = v.y; f[e][2] = v.z; f[e][3] = v.w;
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) f[e][j] = i + j < dk ? p[i + j] : 0.f;
        }
    }
}
template <int E4>
__device__ __forceinline__ void store_state(
    float* p, int l16, int dk, bool vec, float (*f)[4]) {
#pragma unroll
    for (int e = 0; e < E4; ++e) {
        const int i = 64 * e + 4 * l16;
        if (vec) {
            if (i < dk)
                *reinterpret_cast<float4*>(p + i) =
                    make_float4(f[e][0], f[e][1], f[e][2], f[e][3]);
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (i + j < dk) p[i + j] = f[e][j];
        }
    }
}
