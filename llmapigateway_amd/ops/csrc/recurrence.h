// Gate arithmetic shared by the recurrence kernels (fp32).
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
