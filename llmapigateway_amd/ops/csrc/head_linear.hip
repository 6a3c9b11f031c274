// Per-head products for gfx950: y[t, h, :] = W[h] x[t, h, :], W [H, N, K].
//
// They take queries into the latent space and latent sums out of it
// (latent attention, folded form). bf16: v_mfma_f32_16x16x32_bf16, fragments
// loaded 16 B a lane straight from global memory (an activation fragment is
// used for four column tiles; W is read once per 64 rows and lives in L2
// between them). fp32 and shapes that are no multiple of 8: one output a
// thread.

#include "mfma.h"

// WM waves along rows, 4/WM along columns; a wave owns 16 rows x 16*NJ columns
template <int WM, int NJ>
__launch_bounds__(256)
__global__ void head_linear_mfma_kernel(
    bf16* __restrict__ y, int64_t yt, int64_t yh, const bf16* __restrict__ x, int64_t xt,
    int64_t xh, const bf16* __restrict__ w, int M, int N, int K) {
    const int h = blockIdx.z;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int r = lane & 15, g = lane >> 4;
    const int m0 = (blockIdx.x * WM + wave % WM) * 16;
    const int n0 = (blockIdx.y * (4 / WM) + wave / WM) * (16 * NJ);
    if (m0 >= M || n0 >= N) return;
    // rows and columns past the end read the last one; nothing of them is kept
    const bf16* xr = x + (size_t)min(m0 + r, M - 1) * xt + h * xh;
    const bf16* wr[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j)
        wr[j] = w + ((size_t)h * N + min(n0 + j * 16 + r, N - 1)) * K;
    f32x4 acc[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) acc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    // U k-steps of loads in flight; past K the activations are 0
    constexpr int U = NJ == 1 ? 8 : 4;
    for (int k0 = 0; k0 < K; k0 += 32 * U) {
        uint4 av[U], bv[U][NJ];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const bool in = k0 + u * 32 + g * 8 < K;  // K is a multiple of 8
            const int k = in ? k0 + u * 32 + g * 8 : 0;
            av[u] = *reinterpret_cast<const uint4*>(xr + k);
            if (!in) av[u] = (uint4){0, 0, 0, 0};
#pragma unroll
            for (int j = 0; j < NJ; ++j)
                bv[u][j] = *reinterpret_cast<const uint4*>(wr[j] + k);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int j = 0; j < NJ; ++j)
                acc[j] = mfma16(as_frag(av[u]), as_frag(bv[u][j]), acc[j]);
    }
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int n = n0 + j * 16 + r;
        if (n >= N) continue;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            const int m = m0 + g * 4 + q;
            if (m < M) stf(y + (size_t)m * yt + h * yh + n, acc[j][q]);
        }
    }
}

template <typename T>
__global__ void head_linear_any_kernel(
    T* __restrict__ y, int64_t yt, int64_t yh, const T* __restrict__ x, int64_t xt,
    int64_t xh, const T* __restrict__ w, int N, int K) {
    const size_t t = blockIdx.x;
    const int h = blockIdx.z;
    const int n = blockIdx.y * blockDim.x + threadIdx.x;
    if (n >= N) return;
    const T* xr = x + t * xt + h * xh;
    const T* wr = w + ((size_t)h * N + n) * K;
    float acc = 0.f;
    for (int k = 0; k < K; ++k) acc = fmaf(ldf(xr + k), ldf(wr + k), acc);
    stf(y + t * yt + h * yh + n, acc);
}

template <int WM, int NJ>
static void head_linear_go(
    bf16* y, int64_t yt, int64_t yh, const bf16* x, int64_t xt, int64_t xh, const bf16* w,
    int M, int N, int K, int H, hipStream_t stream) {
    const dim3 grid(ceil_div_i(M, 16 * WM), ceil_div_i(N, 16 * NJ * (4 / WM)), H);
    head_linear_mfma_kernel<WM, NJ><<<grid, 256, 0, stream>>>(
        y, yt, yh, x, xt, xh, w, M, N, K);
}
#define ARGS (bf16*)y, yt, yh, (const bf16*)x, xt, xh, (const bf16*)w, M, N, K, H, stream

extern "C" hipError_t launch_head_linear(
    void* y, int64_t yt, int64_t yh, const void* x, int64_t xt, int64_t xh, const void* w,
    int M, int N, int K, int H, int f32, int vec8, hipStream_t stream) {
    if (M <= 0) return hipSuccess;
    if (f32)
        head_linear_any_kernel<float><<<dim3(M, ceil_div_i(N, 64), H), 64, 0, stream>>>(
            (float*)y, yt, yh, (const float*)x, xt, xh, (const float*)w, N, K);
    else if (!vec8)
        head_linear_any_kernel<bf16><<<dim3(M, ceil_div_i(N, 64), H), 64, 0, stream>>>(
            (bf16*)y, yt, yh, (const bf16*)x, xt, xh, (const bf16*)w, N, K);
    else if (M <= 16) {
        // narrower column tiles until the chip is filled
        if (ceil_div_i(N, 256) * H >= 256) head_linear_go<1, 4>(ARGS);
        else if (ceil_div_i(N, 128) * H >= 256) head_linear_go<1, 2>(ARGS);
        else head_linear_go<1, 1>(ARGS);
    } else {
        const int mt = ceil_div_i(M, 64);
        if (mt * ceil_div_i(N, 64) * H >= 512) head_linear_go<4, 4>(ARGS);
        else if (mt * ceil_div_i(N, 32) * H >= 512) head_linear_go<4, 2>(ARGS);
        else head_linear_go<4, 1>(ARGS);
    }
    HIP_CHECK_LAST();
    return hipSuccess;
}
