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
// STREAM: state that a step reads and writes once, past the caches
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float state4;
template <int E4, bool STREAM = false>
__device__ __forceinline__ void load_state(
    const float* p, int l16, int dk, bool vec, float (*f)[4]) {
#pragma unroll
    for (int e = 0; e < E4; ++e) {
        const int i = 64 * e + 4 * l16;
        if (vec) {
            state4 v = {0.f, 0.f, 0.f, 0.f};
            const state4* at = reinterpret_cast<const state4*>(p + i);
            if (i < dk) v = STREAM ? __builtin_nontemporal_load(at) : *at;
#pragma unroll
            for (int j = 0; j < 4; ++j) f[e][j] = v[j];
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
            if (i < dk) {
                const state4 v = {f[e][0], f[e][1], f[e][2], f[e][3]};
                __builtin_nontemporal_store(v, reinterpret_cast<state4*>(p + i));
            }
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (i + j < dk) p[i + j] = f[e][j];
        }
    }
}
