// Gated activations for gfx950 (built into every extension: dense and hybrid
// decoders run them).

#include "common.h"

// ---------------------------------------------------------------------------
// SwiGLU: out[t, i] = silu(x[t, i]) * x[t, I + i]  (x contiguous [T, 2I])
// ---------------------------------------------------------------------------

__global__ void swiglu_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x, int I) {
    const int row = blockIdx.x;
    const uint4* grow = reinterpret_cast<const uint4*>(x + (size_t)row * 2 * I);
    const uint4* urow = reinterpret_cast<const uint4*>(x + (size_t)row * 2 * I + I);
    uint4* orow = reinterpret_cast<uint4*>(out + (size_t)row * I);
    const int nvec = I / 8;
    for (int i = threadIdx.x; i < nvec; i += blockDim.x) {
        uint4 vg = grow[i];
        uint4 vu = urow[i];
        float g[8], u[8];
        unpack2(vg.x, g[0], g[1]);
        unpack2(vg.y, g[2], g[3]);
        unpack2(vg.z, g[4], g[5]);
        unpack2(vg.w, g[6], g[7]);
        unpack2(vu.x, u[0], u[1]);
        unpack2(vu.y, u[2], u[3]);
        unpack2(vu.z, u[4], u[5]);
        unpack2(vu.w, u[6], u[7]);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float s = g[j] / (1.f + __expf(-g[j]));
            g[j] = s * u[j];
        }
        uint4 vo;
        vo.x = pack2(g[0], g[1]);
        vo.y = pack2(g[2], g[3]);
        vo.z = pack2(g[4], g[5]);
        vo.w = pack2(g[6], g[7]);
        orow[i] = vo;
    }
}

// any width, bf16 or fp32
template <typename E>
__global__ void swiglu_any_kernel(E* __restrict__ out, const E* __restrict__ x, int I) {
    const E* g = x + (size_t)blockIdx.x * 2 * I;
    for (int i = threadIdx.x; i < I; i += blockDim.x) {
        const float a = ldf(g + i);
        stf(out + (size_t)blockIdx.x * I + i, a / (1.f + expf(-a)) * ldf(g + I + i));
    }
}

extern "C" hipError_t launch_swiglu(
    void* out, const void* x, int T, int I, int is_f32, hipStream_t stream) {
    if (T <= 0) return hipSuccess;
    if (!is_f32 && I % 8 == 0)
        swiglu_kernel<<<T, 256, 0, stream>>>((bf16*)out, (const bf16*)x, I);
    else if (is_f32)
        swiglu_any_kernel<float><<<T, 256, 0, stream>>>((float*)out, (const float*)x, I);
    else
        swiglu_any_kernel<bf16><<<T, 256, 0, stream>>>((bf16*)out, (const bf16*)x, I);
    HIP_CHECK_LAST();
    return hipSuccess;
}
