// Latent attention for gfx950: softmax attention with a sink over cached
// latent rows [c (rank) | rotated key part | zero pad].
//
// Folded form: queries are already in the latent space, one cached row is
// key and value of every head.

#include "common.h"

#define LA_THREADS 256

// ---------------------------------------------------------------------------
// Any size, bf16 or fp32: one workgroup per (row, head), keys in tiles of
// 256, one key a thread for the scores, one latent dimension a thread for
// the sums. The softmax starts from the sink: running maximum = sink,
// denominator = 1, sum = 0.
// ---------------------------------------------------------------------------
template <typename T, int ND>  // ND: latent dimensions per thread
__launch_bounds__(LA_THREADS)
__global__ void latent_folded_any_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ latent,
    const float* __restrict__ sink, float scale, const int64_t* __restrict__ positions,
    const int* __restrict__ row_seg, const int* __restrict__ tables, int max_blocks,
    int block_size, int H, int rank, int row_w) {
    extern __shared__ float lds[];  // [row_w] query, [256] weights
    float* qs = lds;
    float* ps = lds + row_w;
    __shared__ float red[8];
    const size_t t = blockIdx.x;
    const int h = blockIdx.y;
    const int n = (int)positions[t] + 1;
    const int* bt = tables + (size_t)row_seg[t] * max_blocks;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    for (int i = tid; i < row_w; i += LA_THREADS)
        qs[i] = ldf(q + (t * H + h) * row_w + i);
    float m = sink[h], l = 1.f, acc[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[d] = 0.f;
    for (int k0 = 0; k0 < n; k0 += LA_THREADS) {
        __syncthreads();
        const int key = k0 + tid;
        float s = -INFINITY;
        if (key < n) {
            const T* kr = latent +
                ((size_t)bt[key / block_size] * block_size + key % block_size) * row_w;
            s = 0.f;
            for (int i = 0; i < row_w; ++i) s = fmaf(qs[i], ldf(kr + i), s);
            s *= scale;
        }
        float v = wave_reduce_max(s);
        if (lane == 0) red[wave] = v;
        __syncthreads();
        const float m_new =
            fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float p = key < n ? expf(s - m_new) : 0.f;
        ps[tid] = p;
        v = wave_reduce_sum(p);
        if (lane == 0) red[4 + wave] = v;
        __syncthreads();
        const float f = expf(m - m_new);
        l = l * f + red[4] + red[5] + red[6] + red[7];
        m = m_new;
#pragma unroll
        for (int d = 0; d < ND; ++d) acc[d] *= f;
        const int here = min(LA_THREADS, n - k0);
        for (int j = 0; j < here; ++j) {
            const int kj = k0 + j;
            const T* kr = latent +
                ((size_t)bt[kj / block_size] * block_size + kj % block_size) * row_w;
            const float pj = ps[j];
#pragma unroll
            for (int d = 0; d < ND; ++d) {
                const int i = tid + d * LA_THREADS;
                if (i < rank) acc[d] = fmaf(pj, ldf(kr + i), acc[d]);
            }
        }
    }
#pragma unroll
    for (int d = 0; d < ND; ++d) {
        const int i = tid + d * LA_THREADS;
        if (i < rank) stf(out + (t * H + h) * rank + i, acc[d] / l);
    }
}

template <typename T>
static hipError_t folded_any(
    void* out, const void* q, const void* latent, const float* sink, float scale,
    const int64_t* positions, const int* row_seg, const int* tables, int rows, int H,
    int rank, int row_w, int block_size, int max_blocks, hipStream_t stream) {
    const int nd = ceil_div_i(rank, LA_THREADS);
    const size_t lds = (row_w + LA_THREADS) * sizeof(float);
    if (lds > 48 * 1024) return hipErrorInvalidValue;
    const dim3 grid(rows, H);
#define GO(ND)                                                                          \
    latent_folded_any_kernel<T, ND><<<grid, LA_THREADS, lds, stream>>>(                 \
        (T*)out, (const T*)q, (const T*)latent, sink, scale, positions, row_seg, tables, \
        max_blocks, block_size, H, rank, row_w)
    if (nd == 1) GO(1);
    else if (nd == 2) GO(2);
    else if (nd <= 4) GO(4);
    else if (nd <= 8) GO(8);
    else return hipErrorInvalidValue;
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}

extern "C" hipError_t launch_latent_folded_any(
    void* out, const void* q, const void* latent, const float* sink, float scale,
    const int64_t* positions, const int* row_seg, const int* tables, int rows, int H,
    int rank, int row_w, int block_size, int max_blocks, int f32, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return f32 ? folded_any<float>(out, q, latent, sink, scale, positions, row_seg, tables,
                                   rows, H, rank, row_w, block_size, max_blocks, stream)
               : folded_any<bf16>(out, q, latent, sink, scale, positions, row_seg, tables,
                                  rows, H, rank, row_w, block_size, max_blocks, stream);
}
