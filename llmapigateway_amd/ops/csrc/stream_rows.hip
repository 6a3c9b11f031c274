// Row kernels of decoders with hyper-connected streams and rotary attention
// for gfx950: combinations of streams and pending sublayer outputs with the
// norm of what a sublayer reads, the norm of the embedding, per-head norms
// with rotation and the page write, xIELU, silu.
//
// Templated on the compute dtype like hybrid_rows.hip; arithmetic is fp32. A
// row stays in registers between its sum and its norm: up to 16384 values.

#include "rows.h"

#define MAX_ROW 16384
#define MAX_PENDING 8

// ---------------------------------------------------------------------------
// Rows z_r of one token: S stored streams x [T, S, W] (fp32), then n pending
// outputs, each times its scale. Column c of the result is sum_r coef[r, c]
// z_r: column 0 is normed to h, the others (if out is given) are the new
// streams [T, C - 1, W]. out may be x if it has as many streams: a thread
// reads all rows of its coordinates before it writes them.
// ---------------------------------------------------------------------------
struct MixArgs {
    void* h;
    float* out;
    const float* x;
    const void* y[MAX_PENDING];
    const float* scale[MAX_PENDING];  // null: 1
    const float *coef, *w;
    float eps;
    int S, n, C, W;
};

template <typename T, int VEC, int MAXC>
__launch_bounds__(512)
__global__ void mix_streams_kernel(MixArgs a) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    const int step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= a.W) continue;
        float acc[MAXC][VEC];
#pragma unroll
        for (int c = 0; c < MAXC; ++c)
#pragma unroll
            for (int j = 0; j < VEC; ++j) acc[c][j] = 0.f;
        auto add = [&](int r, const float* f) {
#pragma unroll
            for (int c = 0; c < MAXC; ++c) {  // (columns past the last repeat it, unused)
                const float p = a.coef[r * a.C + min(c, a.C - 1)];
#pragma unroll
                for (int j = 0; j < VEC; ++j) acc[c][j] = fmaf(p, f[j], acc[c][j]);
            }
        };
        const float* xr = a.x + t * a.S * a.W + i;
#pragma unroll 4
        for (int s = 0; s < a.S; ++s) {
            float f[VEC];
            load_vec<VEC>(xr + (size_t)s * a.W, f);
            add(s, f);
        }
#pragma unroll
        for (int p = 0; p < MAX_PENDING; ++p) {
            if (p >= a.n) break;
            float f[VEC], g[VEC];
            load_vec<VEC>((const T*)a.y[p] + t * a.W + i, f);
            if (a.scale[p] != nullptr) {
                load_vec<VEC>(a.scale[p] + i, g);
#pragma unroll
                for (int j = 0; j < VEC; ++j) f[j] *= g[j];
            }
            add(a.S + p, f);
        }
        if (MAXC > 1) {
#pragma unroll
            for (int c = 1; c < MAXC; ++c)
                if (c < a.C) store_vec<VEC>(a.out + (t * (a.C - 1) + c - 1) * a.W + i, acc[c]);
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            held[k][j] = acc[0][j];
            ss += acc[0][j] * acc[0][j];
        }
    }
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.W + a.eps);
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= a.W) continue;
        float w[VEC];
        load_vec<VEC>(a.w + i, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[k][j] *= inv * w[j];
        store_vec<VEC>((T*)a.h + t * a.W + i, held[k]);
    }
}

// x[t] = embed[token] / rms * w (fp32)
template <typename T, int VEC>
__launch_bounds__(512)
__global__ void embed_rms_kernel(
    float* __restrict__ x, const int64_t* __restrict__ tokens, const T* __restrict__ embed,
    const float* __restrict__ w, float eps, int W) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    const T* src = embed + (size_t)tokens[t] * W;
    const int step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        load_vec<VEC>(src + i, held[k]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss += held[k][j] * held[k][j];
    }
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        float g[VEC];
        load_vec<VEC>(w + i, g);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[k][j] *= inv * g[j];
        store_vec<VEC>(x + t * W + i, held[k]);
    }
}

// ---------------------------------------------------------------------------
// z = pos z^2 + z/2 above 0, neg (e^z - 1 - z) + z/2 below, in place
// ---------------------------------------------------------------------------
template <typename T>
__device__ __forceinline__ float xielu_f(float z, float pos, float neg) {
    const float n = fminf(z, 0.f);
    float e;  // e^n - 1 - n
    if (sizeof(T) == 4) {
        e = expm1f(n) - n;
    } else {
        const float series =
            n * n * (0.5f + n * (1.f / 6.f + n * (1.f / 24.f + n * (1.f / 120.f))));
        e = n > -0.25f ? series : __expf(n) - 1.f - n;
    }
    return (z > 0.f ? pos * z * z : neg * e) + 0.5f * z;
}
template <typename T, int VEC>
__launch_bounds__(256)
__global__ void xielu_kernel(T* __restrict__ z, float pos, float neg, size_t n) {
    const size_t step = (size_t)gridDim.x * 256 * VEC;
    for (size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * VEC; i < n; i += step) {
        float f[VEC];
        load_vec<VEC>(z + i, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] = xielu_f<T>(f[j], pos, neg);
        store_vec<VEC>(z + i, f);
    }
}

// silu of rows of a strided matrix, in place
template <typename T, int VEC>
__launch_bounds__(256)
__global__ void silu_kernel(T* __restrict__ x, int64_t ld, int W) {
    T* row = x + (size_t)blockIdx.x * ld;
    const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (i >= W) return;
    float f[VEC];
    load_vec<VEC>(row + i, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j)
        f[j] *= sizeof(T) == 4 ? sigmoid_f(f[j]) : 1.f / (1.f + __expf(-f[j]));
    store_vec<VEC>(row + i, f);
}

// ---------------------------------------------------------------------------
// Heads of q (to out) and k (to the row's cache slot, -1: not kept): RMS norm
// of a head's dim values times w, then dimensions i and i + half turn by the
// position's angle i for i < half. Values are copied to the cache.
// ---------------------------------------------------------------------------
struct RotaryArgs {
    void* out;
    const void *q, *k, *v;  // k null: queries alone
    int64_t ldq, ldk, ldv;
    const float *q_norm, *k_norm, *cos_sin;
    float eps;
    const int64_t *positions, *slot_mapping;
    void *k_pages, *v_pages;
    int T, nq, nk, dim, half, wv;
};

// lg lanes a head, 8 values a lane; items of a token: nq + nk heads, then
// pieces of 8*lg values
template <typename T>
__launch_bounds__(256)
__global__ void rotary_rows_kernel(RotaryArgs a, int lg, int per_token) {
    const size_t item = ((size_t)blockIdx.x * 256 + threadIdx.x) / lg;
    const int c = threadIdx.x % lg * 8;
    const size_t t = item / per_token;
    const int id = item % per_token, heads = a.nq + a.nk;
    const bool live = t < (size_t)a.T;
    const int64_t slot = live && a.k != nullptr ? a.slot_mapping[t] : -1;
    if (live && id >= heads) {
        const int i = (id - heads) * lg * 8 + c;
        float f[8];
        if (i >= a.wv || slot < 0) return;
        load_vec<8>((const T*)a.v + t * a.ldv + i, f);
        store_vec<8>((T*)a.v_pages + (size_t)slot * a.wv + i, f);
        return;
    }
    const bool in = live && c < a.dim, is_q = id < a.nq;
    const T* src = is_q ? (const T*)a.q + t * a.ldq + (size_t)id * a.dim
                        : (const T*)a.k + t * a.ldk + (size_t)(id - a.nq) * a.dim;
    float f[8];
    float ss = 0.f;
    if (in) {
        load_vec<8>(src + c, f);
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += f[j] * f[j];
    }
    for (int off = lg / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE_SIZE);
    if (!in || (!is_q && slot < 0)) return;
    const float inv = 1.f / sqrtf(ss / (float)a.dim + a.eps);
    const float* w = is_q ? a.q_norm : a.k_norm;
    float g[8];
    load_vec<8>(w + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] *= inv * g[j];
    if (c < 2 * a.half) {
        const bool first = c < a.half;
        const int o = first ? c + a.half : c - a.half, i = first ? c : o;
        const float* cs = a.cos_sin + (size_t)a.positions[t] * 2 * a.half + i;
        float p[8], co[8], si[8];
        load_vec<8>(src + o, p);
        load_vec<8>(w + o, g);
        load_vec<8>(cs, co);
        load_vec<8>(cs + a.half, si);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float other = p[j] * inv * g[j];
            f[j] = f[j] * co[j] + (first ? -other : other) * si[j];
        }
    }
    if (is_q) store_vec<8>((T*)a.out + (t * a.nq + id) * a.dim + c, f);
    else store_vec<8>((T*)a.k_pages + ((size_t)slot * a.nk + id - a.nq) * a.dim + c, f);
}

// any size: a wave per head or per 64 values to copy
template <typename T>
__launch_bounds__(256)
__global__ void rotary_rows_any_kernel(RotaryArgs a, int per_token) {
    const size_t item = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    const size_t t = item / per_token;
    const int id = item % per_token, heads = a.nq + a.nk;
    if (t >= (size_t)a.T) return;
    const int64_t slot = a.k != nullptr ? a.slot_mapping[t] : -1;
    if (id >= heads) {
        const int i = (id - heads) * 64 + lane;
        if (i < a.wv && slot >= 0)
            ((T*)a.v_pages)[(size_t)slot * a.wv + i] = ((const T*)a.v)[t * a.ldv + i];
        return;
    }
    const bool is_q = id < a.nq;
    const T* src = is_q ? (const T*)a.q + t * a.ldq + (size_t)id * a.dim
                        : (const T*)a.k + t * a.ldk + (size_t)(id - a.nq) * a.dim;
    float ss = 0.f;
    for (int i = lane; i < a.dim; i += 64) {
        const float x = ldf(src + i);
        ss += x * x;
    }
    const float inv = 1.f / sqrtf(wave_reduce_sum(ss) / (float)a.dim + a.eps);
    if (!is_q && slot < 0) return;
    const float* w = is_q ? a.q_norm : a.k_norm;
    const float* cs = a.cos_sin + (size_t)a.positions[t] * 2 * a.half;
    T* dst = is_q ? (T*)a.out + (t * a.nq + id) * a.dim
                  : (T*)a.k_pages + ((size_t)slot * a.nk + id - a.nq) * a.dim;
    for (int i = lane; i < a.dim; i += 64) {
        float x = ldf(src + i) * inv * w[i];
        if (i < 2 * a.half) {
            const bool first = i < a.half;
            const int o = first ? i + a.half : i - a.half, j = first ? i : o;
            const float other = ldf(src + o) * inv * w[o];
            x = x * cs[j] + (first ? -other : other) * cs[a.half + j];
        }
        stf(dst + i, x);
    }
}

// ---------------------------------------------------------------------------
// launchers (vec8: all widths, strides and addresses allow 8-element accesses)
// ---------------------------------------------------------------------------
extern "C" hipError_t launch_mix_streams(
    void* h, float* out, const float* x, const void* const* y, const float* const* scale,
    const float* coef, const float* w, float eps, int rows, int S, int n, int C, int W, int f32,
    int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (W > MAX_ROW || n > MAX_PENDING || C < 1 || C > 17 || (C > 1) != (out != nullptr))
        return hipErrorInvalidValue;
    MixArgs a = {};
    a.h = h; a.out = out; a.x = x; a.coef = coef; a.w = w; a.eps = eps;
    a.S = S; a.n = n; a.C = C; a.W = W;
    for (int i = 0; i < n; ++i) {
        a.y[i] = y[i];
        a.scale[i] = scale[i];
    }
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const int th = row_threads(W, V);
#define GO(MAXC) mix_streams_kernel<T, V, MAXC><<<rows, th, 0, stream>>>(a)
        if (C == 1) GO(1);
        else if (C <= 3) GO(3);
        else if (C <= 5) GO(5);
        else if (C <= 9) GO(9);
        else GO(17);
#undef GO
    });
}

extern "C" hipError_t launch_embed_rms(
    float* x, const int64_t* tokens, const void* embed, const float* w, float eps, int rows,
    int W, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (W > MAX_ROW) return hipErrorInvalidValue;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        embed_rms_kernel<T, V><<<rows, row_threads(W, V), 0, stream>>>(
            x, tokens, (const T*)embed, w, eps, W);
    });
}

extern "C" hipError_t launch_xielu(
    void* z, float pos, float neg, size_t n, int f32, int vec8, hipStream_t stream) {
    if (n == 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const size_t want = (n + 256 * V - 1) / (256 * V);
        const unsigned blocks = want < 16384 ? want : 16384;
        xielu_kernel<T, V><<<blocks, 256, 0, stream>>>((T*)z, pos, neg, n);
    });
}

extern "C" hipError_t launch_silu(
    void* x, int64_t ld, int rows, int W, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0 || W <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        silu_kernel<T, V><<<dim3(rows, ceil_div_i(W, 256 * V)), 256, 0, stream>>>((T*)x, ld, W);
    });
}

// vec8 also: dim (at most 512) and half multiples of 8
extern "C" hipError_t launch_rotary_rows(
    void* out, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* q_norm, const float* k_norm, float eps, const float* cos_sin,
    const int64_t* positions, void* k_pages, void* v_pages, const int64_t* slot_mapping,
    int rows, int nq, int nk, int dim, int half, int wv, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (2 * half > dim || (k == nullptr && (nk || wv))) return hipErrorInvalidValue;
    const RotaryArgs a = {out, q, k, v, ldq, ldk, ldv, q_norm, k_norm, cos_sin, eps, positions,
                          slot_mapping, k_pages, v_pages, rows, nq, nk, dim, half, wv};
    if (vec8 && (dim % 8 || half % 8 || wv % 8)) return hipErrorInvalidValue;
    if (vec8 && dim <= 512) {
        int lg = 1;
        while (lg * 8 < dim) lg *= 2;
        const int per_token = nq + nk + ceil_div_i(wv, lg * 8);
        const unsigned blocks = (unsigned)(((size_t)rows * per_token * lg + 255) / 256);
        return pick(f32, 1, [&](auto form) {
            FORM(form);
            rotary_rows_kernel<T><<<blocks, 256, 0, stream>>>(a, lg, per_token);
        });
    }
    const int per_token = nq + nk + ceil_div_i(wv, 64);
    const unsigned blocks = (unsigned)(((size_t)rows * per_token + 3) / 4);
    return pick(f32, 0, [&](auto form) {
        FORM(form);
        rotary_rows_any_kernel<T><<<blocks, 256, 0, stream>>>(a, per_token);
    });
}
