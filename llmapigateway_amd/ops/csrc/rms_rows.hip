// Row kernels of decoders with RMS norms for gfx950: pending sublayer outputs
// onto the fp32 stream with one or two norms of it in the same pass; norms of
// whole query and key rows with the values' blend and the page write.
//
// Templated on the compute dtype like hybrid_rows.hip; arithmetic is fp32. A
// row stays in registers between its sum and its norm: up to 16384 values.

#include "rows.h"

#define MAX_ROW 16384

// ---------------------------------------------------------------------------
// x += d1 + d2 + sum_j weights[t, j] * rows[slot[t, j]]  (each may be absent)
// out1 = x / rms(x) * w1, out2 = x / rms(x) * w2 (absent: null)
// ---------------------------------------------------------------------------
struct RmsArgs {
    void *out1, *out2;
    float* x;
    const void *d1, *d2, *rows;
    const int* slot;       // null: no experts
    const float* weights;
    int top;
    const float *w1, *w2;
    float eps;
    int W;
};

template <typename T, int VEC>
__launch_bounds__(512)
__global__ void add_rms_norm_kernel(RmsArgs a) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    float* xr = a.x + t * a.W;
    const int step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    const bool add = a.d1 != nullptr || a.slot != nullptr;
    float held[HELD][VEC];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= a.W) continue;
        float* f = held[k];
        float g[VEC];
        load_vec<VEC>(xr + i, f);
        if (a.d1 != nullptr) {
            load_vec<VEC>((const T*)a.d1 + t * a.W + i, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] += g[j];
        }
        if (a.d2 != nullptr) {
            load_vec<VEC>((const T*)a.d2 + t * a.W + i, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] += g[j];
        }
        if (a.slot != nullptr) {
            float y[VEC];
#pragma unroll
            for (int j = 0; j < VEC; ++j) y[j] = 0.f;
            for (int c = 0; c < a.top; ++c) {
                const float p = a.weights[t * a.top + c];
                load_vec<VEC>((const T*)a.rows + (size_t)a.slot[t * a.top + c] * a.W + i, g);
#pragma unroll
                for (int j = 0; j < VEC; ++j) y[j] = fmaf(p, g[j], y[j]);
            }
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] += y[j];
        }
        if (add) store_vec<VEC>(xr + i, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss += f[j] * f[j];
    }
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.W + a.eps);
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= a.W) continue;
        float w[VEC], o[VEC];
        load_vec<VEC>(a.w1 + i, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            held[k][j] *= inv;
            o[j] = held[k][j] * w[j];
        }
        store_vec<VEC>((T*)a.out1 + t * a.W + i, o);
        if (a.out2 != nullptr) {
            load_vec<VEC>(a.w2 + i, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) o[j] = held[k][j] * w[j];
            store_vec<VEC>((T*)a.out2 + t * a.W + i, o);
        }
    }
}

// ---------------------------------------------------------------------------
// out = q / rms(q) * q_norm over the whole row; keys likewise, and values
// (blended with v_first's rows if given), into the row's cache slot (-1: not
// kept)
// ---------------------------------------------------------------------------
struct QkvArgs {
    void* out;
    const void *q, *k, *v, *v_first;
    int64_t ldq, ldk, ldv, ld_first;
    const float *q_norm, *k_norm;
    float eps, blend;
    void *k_pages, *v_pages;
    const int64_t* slot_mapping;
    int wq, wk, wv;
};

template <typename T, int VEC>
__launch_bounds__(512)
__global__ void qkv_rows_kernel(QkvArgs a) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    const T *qr = (const T*)a.q + t * a.ldq, *kr = (const T*)a.k + t * a.ldk;
    const int W = a.wq + a.wk, step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int c = 0; c < HELD; ++c) {
        const int i = i0 + c * step;
        if (i >= W) continue;
        load_vec<VEC>(i < a.wq ? qr + i : kr + i - a.wq, held[c]);
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss += held[c][j] * held[c][j];
        if (i < a.wq) sq += ss;
        else sk += ss;
    }
    const int64_t slot = a.slot_mapping[t];
    if (slot >= 0) {
        for (int i = i0; i < a.wv; i += step) {
            float f[VEC], g[VEC];
            load_vec<VEC>((const T*)a.v + t * a.ldv + i, f);
            if (a.v_first != nullptr) {
                load_vec<VEC>((const T*)a.v_first + t * a.ld_first + i, g);
#pragma unroll
                for (int j = 0; j < VEC; ++j) f[j] = (1.f - a.blend) * f[j] + a.blend * g[j];
            }
            store_vec<VEC>((T*)a.v_pages + (size_t)slot * a.wv + i, f);
        }
    }
    const float iq = 1.f / sqrtf(block_sum(sq, red) / (float)a.wq + a.eps);
    const float ik = 1.f / sqrtf(block_sum(sk, red) / (float)a.wk + a.eps);
#pragma unroll
    for (int c = 0; c < HELD; ++c) {
        const int i = i0 + c * step;
        if (i >= W) continue;
        const bool is_q = i < a.wq;
        if (!is_q && slot < 0) continue;
        float w[VEC];
        load_vec<VEC>(is_q ? a.q_norm + i : a.k_norm + i - a.wq, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[c][j] *= (is_q ? iq : ik) * w[j];
        if (is_q) store_vec<VEC>((T*)a.out + t * a.wq + i, held[c]);
        else store_vec<VEC>((T*)a.k_pages + (size_t)slot * a.wk + i - a.wq, held[c]);
    }
}

// ---------------------------------------------------------------------------
// launchers (vec8: all widths, strides and addresses allow 8-element accesses)
// ---------------------------------------------------------------------------
extern "C" hipError_t launch_add_rms_norm(
    void* out1, void* out2, float* x, const void* d1, const void* d2, const void* rows,
    const int* slot, const float* weights, int top, const float* w1, const float* w2, float eps,
    int T_rows, int W, int f32, int vec8, hipStream_t stream) {
    if (T_rows <= 0) return hipSuccess;
    if (W > MAX_ROW) return hipErrorInvalidValue;
    const RmsArgs a = {out1, out2, x, d1, d2, rows, slot, weights, top, w1, w2, eps, W};
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        add_rms_norm_kernel<T, V><<<T_rows, row_threads(W, V), 0, stream>>>(a);
    });
}

extern "C" hipError_t launch_qkv_rows(
    void* out, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const void* v_first, int64_t ld_first, const float* q_norm,
    const float* k_norm, float eps, float blend, void* k_pages, void* v_pages,
    const int64_t* slot_mapping, int T_rows, int wq, int wk, int wv, int f32, int vec8,
    hipStream_t stream) {
    if (T_rows <= 0) return hipSuccess;
    if (wq + wk > MAX_ROW) return hipErrorInvalidValue;
    const QkvArgs a = {out, q, k, v, v_first, ldq, ldk, ldv, ld_first, q_norm, k_norm, eps,
                       blend, k_pages, v_pages, slot_mapping, wq, wk, wv};
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        qkv_rows_kernel<T, V><<<T_rows, row_threads(wq + wk, V), 0, stream>>>(a);
    });
}
