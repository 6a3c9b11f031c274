// Row kernels of decoders with dynamic-tanh norms for gfx950: a sublayer's
// output (a tensor, or the experts' parts of it) through its own norm onto
// the fp32 stream and the next norm of the stream in one pass; token shift;
// head-wise norm with a silu gate; page writes; clamped GLU; soft cap.
//
// Templated on the compute dtype like hybrid_rows.hip; arithmetic is fp32.

#include "rows.h"

// tanh: the library's in fp32, the short one in bf16 steps
template <typename T>
__device__ __forceinline__ float tanh_of(float z) {
    return sizeof(T) == 4 ? tanhf(z) : tanh_fast(z);
}
template <typename T>
__device__ __forceinline__ float sigmoid_of(float z) {
    return sizeof(T) == 4 ? sigmoid_f(z) : 1.f / (1.f + __expf(-z));
}
template <typename T>
__device__ __forceinline__ float silu_of(float z) {
    return sizeof(T) == 4 ? z * sigmoid_f(z) : z / (1.f + __expf(-z));
}

struct TanhNorm {
    const float *w, *b;  // null: no norm
    float alpha;
};

// ---------------------------------------------------------------------------
// x = (replace ? 0 : x) + post(d);  out = norm(x), or x itself
// d: delta, or sum_j weights[t, j] * rows[slot[t, j]] + shared[t]
// ---------------------------------------------------------------------------
struct StreamArgs {
    void* out;
    int64_t ld_out;
    float* x;
    const void* delta;  // null: nothing to add
    const void *rows, *shared;
    const int* slot;    // non-null: the experts' form
    const float* weights;
    int top;
    TanhNorm post, norm;
    int replace, W;
};

template <typename T, typename D, int VEC, bool EXPERTS>
__launch_bounds__(256)
__global__ void stream_tanh_kernel(StreamArgs a) {
    const size_t t = blockIdx.x;
    const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (i >= a.W) return;
    float* xr = a.x + t * a.W + i;
    float f[VEC], d[VEC], u[VEC], v[VEC];
    if (a.replace) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] = 0.f;
    } else {
        load_vec<VEC>(xr, f);
    }
    const bool add = EXPERTS || a.delta != nullptr;
    if (EXPERTS) {
        if (a.shared != nullptr) {
            load_vec<VEC>((const T*)a.shared + t * a.W + i, d);
        } else {
#pragma unroll
            for (int j = 0; j < VEC; ++j) d[j] = 0.f;
        }
        for (int k = 0; k < a.top; ++k) {
            const float p = a.weights[t * a.top + k];
            load_vec<VEC>((const T*)a.rows + (size_t)a.slot[t * a.top + k] * a.W + i, u);
#pragma unroll
            for (int j = 0; j < VEC; ++j) d[j] = fmaf(p, u[j], d[j]);
        }
    } else if (add) {
        load_vec<VEC>((const D*)a.delta + t * a.W + i, d);
    }
    if (add) {
        if (a.post.w != nullptr) {
            load_vec<VEC>(a.post.w + i, u);
            load_vec<VEC>(a.post.b + i, v);
#pragma unroll
            for (int j = 0; j < VEC; ++j)
                d[j] = fmaf(tanh_of<T>(a.post.alpha * d[j]), u[j], v[j]);
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] += d[j];
        store_vec<VEC>(xr, f);
    }
    if (a.norm.w != nullptr) {
        load_vec<VEC>(a.norm.w + i, u);
        load_vec<VEC>(a.norm.b + i, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] = fmaf(tanh_of<T>(a.norm.alpha * f[j]), u[j], v[j]);
    }
    store_vec<VEC>((T*)a.out + t * a.ld_out + i, f);
}

// x[t] = norm(embed[token]) (fp32); x0[t] (compute dtype) the same
template <typename T, int VEC>
__launch_bounds__(256)
__global__ void embed_tanh_kernel(
    float* __restrict__ x, T* __restrict__ x0, int64_t ld0,
    const int64_t* __restrict__ tokens, const T* __restrict__ embed, TanhNorm norm, int W) {
    const size_t t = blockIdx.x;
    const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (i >= W) return;
    float f[VEC], u[VEC], v[VEC];
    load_vec<VEC>(embed + (size_t)tokens[t] * W + i, f);
    load_vec<VEC>(norm.w + i, u);
    load_vec<VEC>(norm.b + i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = fmaf(tanh_of<T>(norm.alpha * f[j]), u[j], v[j]);
    store_vec<VEC>(x + t * W + i, f);
    if (x0 != nullptr) store_vec<VEC>(x0 + t * ld0 + i, f);
}

// ---------------------------------------------------------------------------
// Token shift: out[m, t] = h_t + (h_{t-1} - h_t) mu_m. The row before a
// segment's first comes from prev[slot] (zeros at a sequence's start). With
// one row per segment (STEP) prev takes in the row here; otherwise
// shift_state_kernel does, after this one.
// ---------------------------------------------------------------------------
template <typename T, int VEC, bool STEP>
__launch_bounds__(256)
__global__ void token_shift_kernel(
    T* __restrict__ out, const T* __restrict__ h, const float* __restrict__ mu, int mixes,
    T* __restrict__ prev, const int64_t* __restrict__ positions, const int* __restrict__ cu,
    const int* __restrict__ slots, const int* __restrict__ row_seg, int rows, int W) {
    const size_t t = blockIdx.x;
    const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (i >= W) return;
    const int s = STEP ? (int)t : row_seg[t];
    const int slot = slots[s];
    float cur[VEC], last[VEC], u[VEC], v[VEC];
    load_vec<VEC>(h + t * W + i, cur);
    if (!STEP && (int)t > cu[s]) {
        load_vec<VEC>(h + (t - 1) * W + i, last);
    } else if (slot >= 0 && positions[t] > 0) {
        load_vec<VEC>(prev + (size_t)slot * W + i, last);
    } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) last[j] = 0.f;
    }
    if (STEP && slot >= 0) store_vec<VEC>(prev + (size_t)slot * W + i, cur);
#pragma unroll
    for (int j = 0; j < VEC; ++j) last[j] -= cur[j];
    for (int m = 0; m < mixes; ++m) {
        load_vec<VEC>(mu + (size_t)m * W + i, u);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = fmaf(last[j], u[j], cur[j]);
        store_vec<VEC>(out + ((size_t)m * rows + t) * W + i, v);
    }
}

template <typename T, int VEC>
__launch_bounds__(256)
__global__ void shift_state_kernel(
    const T* __restrict__ h, T* __restrict__ prev, const int* __restrict__ cu,
    const int* __restrict__ slots, int W) {
    const int s = blockIdx.x, i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    const int slot = slots[s];
    if (i >= W || slot < 0) return;
    float f[VEC];
    load_vec<VEC>(h + (size_t)(cu[s + 1] - 1) * W + i, f);
    store_vec<VEC>(prev + (size_t)slot * W + i, f);
}

// ---------------------------------------------------------------------------
// out = rms(y) * w * silu(gate) (or sigmoid(gate)) per head of gs values: LG
// lanes a head, 8 values a lane, several heads a wave
// ---------------------------------------------------------------------------
template <typename T, bool SIGMOID>
__launch_bounds__(256)
__global__ void head_norm_kernel(
    T* __restrict__ out, int64_t ld_out, const T* __restrict__ y, const T* __restrict__ gate,
    int64_t ld_gate, const float* __restrict__ w, float eps, int groups, int gs, int lg,
    size_t total) {
    const size_t item = ((size_t)blockIdx.x * 256 + threadIdx.x) / lg;
    const int l = threadIdx.x % lg;
    const bool in = item < total && l * 8 < gs;
    const size_t t = in ? item / groups : 0;
    const int c = in ? (int)(item % groups) * gs + l * 8 : 0;
    float f[8], z[8], wv[8];
    load_vec<8>(y + t * (size_t)groups * gs + c, f);
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += f[j] * f[j];
    if (!in) ss = 0.f;
    for (int off = lg / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE_SIZE);
    if (!in) return;
    const float inv = 1.f / sqrtf(ss / (float)gs + eps);
    load_vec<8>(gate + t * ld_gate + c, z);
    load_vec<8>(w + c, wv);
#pragma unroll
    for (int j = 0; j < 8; ++j)
        f[j] *= inv * wv[j] * (SIGMOID ? sigmoid_of<T>(z[j]) : silu_of<T>(z[j]));
    store_vec<8>(out + t * ld_out + c, f);
}

// ---------------------------------------------------------------------------
// a token's key and value rows into its cache page slot (-1: not kept)
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__launch_bounds__(256)
__global__ void page_write_kernel(
    T* __restrict__ k_pages, T* __restrict__ v_pages, const T* __restrict__ k, int64_t ldk,
    const T* __restrict__ v, int64_t ldv, const int64_t* __restrict__ slot_mapping, int wk,
    int wv) {
    const size_t t = blockIdx.x;
    const int64_t slot = slot_mapping[t];
    if (slot < 0) return;
    float f[VEC];
    for (int i = threadIdx.x * VEC; i < wk + wv; i += blockDim.x * VEC) {
        if (i < wk) {
            load_vec<VEC>(k + t * ldk + i, f);
            store_vec<VEC>(k_pages + (size_t)slot * wk + i, f);
        } else {
            load_vec<VEC>(v + t * ldv + i - wk, f);
            store_vec<VEC>(v_pages + (size_t)slot * wv + i - wk, f);
        }
    }
}

// out [rows, ff] from x [rows, 2 ff] = [gate | up]
template <typename T, int VEC>
__launch_bounds__(256)
__global__ void clamped_glu_kernel(
    T* __restrict__ out, const T* __restrict__ x, float limit, int ff) {
    const size_t t = blockIdx.x;
    const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (i >= ff) return;
    float g[VEC], u[VEC];
    load_vec<VEC>(x + t * 2 * ff + i, g);
    load_vec<VEC>(x + t * 2 * ff + ff + i, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) g[j] = clamped_glu<T>(g[j], u[j], limit);
    store_vec<VEC>(out + t * ff + i, g);
}

__global__ void soft_cap_kernel(float* __restrict__ x, float cap, size_t n) {
    const float inv = 1.f / cap;
    const size_t step = (size_t)gridDim.x * blockDim.x * 4;
    for (size_t i = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * 4; i < n; i += step) {
        if (i + 4 <= n) {
            float4 v = *reinterpret_cast<float4*>(x + i);
            v.x = cap * tanhf(v.x * inv);
            v.y = cap * tanhf(v.y * inv);
            v.z = cap * tanhf(v.z * inv);
            v.w = cap * tanhf(v.w * inv);
            *reinterpret_cast<float4*>(x + i) = v;
        } else {
            for (size_t j = i; j < n; ++j) x[j] = cap * tanhf(x[j] * inv);
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
static dim3 row_grid(int rows, int W, int vec) { return dim3(rows, ceil_div_i(W, 256 * vec)); }

extern "C" hipError_t launch_stream_tanh(
    void* out, int64_t ld_out, float* x, const void* delta, int delta_f32, const void* rows,
    const void* shared, const int* slot, const float* weights, int top, const float* post_w,
    const float* post_b, float post_alpha, const float* norm_w, const float* norm_b,
    float norm_alpha, int replace, int T_rows, int W, int f32, int vec8, hipStream_t stream) {
    if (T_rows <= 0) return hipSuccess;
    StreamArgs a = {out, ld_out, x, delta, rows, shared, slot, weights, top,
                    {post_w, post_b, post_alpha}, {norm_w, norm_b, norm_alpha}, replace, W};
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const dim3 grid = row_grid(T_rows, W, V);
        if (slot != nullptr) stream_tanh_kernel<T, T, V, true><<<grid, 256, 0, stream>>>(a);
        else if (delta_f32) stream_tanh_kernel<T, float, V, false><<<grid, 256, 0, stream>>>(a);
        else {
            stream_tanh_kernel<T, T, V, false><<<grid, 256, 0, stream>>>(a);
        }
    });
}

extern "C" hipError_t launch_embed_tanh(
    float* x, void* x0, int64_t ld0, const int64_t* tokens, const void* embed, const float* w,
    const float* b, float alpha, int rows, int W, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        embed_tanh_kernel<T, V><<<row_grid(rows, W, V), 256, 0, stream>>>(
            x, (T*)x0, ld0, tokens, (const T*)embed, TanhNorm{w, b, alpha}, W);
    });
}

extern "C" hipError_t launch_token_shift(
    void* out, const void* h, const float* mu, int mixes, void* prev,
    const int64_t* positions, const int* cu, const int* slots, const int* row_seg, int rows,
    int nseg, int W, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const dim3 grid = row_grid(rows, W, V);
        if (rows == nseg) {
            token_shift_kernel<T, V, true><<<grid, 256, 0, stream>>>(
                (T*)out, (const T*)h, mu, mixes, (T*)prev, positions, cu, slots, row_seg, rows, W);
        } else {
            token_shift_kernel<T, V, false><<<grid, 256, 0, stream>>>(
                (T*)out, (const T*)h, mu, mixes, (T*)prev, positions, cu, slots, row_seg, rows, W);
            shift_state_kernel<T, V><<<row_grid(nseg, W, V), 256, 0, stream>>>(
                (const T*)h, (T*)prev, cu, slots, W);
        }
    });
}

// gs a multiple of 8, at most 512; everything aligned for 8-element accesses
extern "C" hipError_t launch_head_norm(
    void* out, int64_t ld_out, const void* y, const void* gate, int64_t ld_gate,
    const float* w, float eps, int groups, int gs, int sigmoid, int rows, int f32,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (gs % 8 || gs > 512) return hipErrorInvalidValue;
    int lg = 1;
    while (lg * 8 < gs) lg *= 2;
    const size_t total = (size_t)rows * groups;
    const unsigned blocks = (unsigned)((total * lg + 255) / 256);
    return pick(f32, 1, [&](auto form) {
        FORM(form);
        auto kernel = sigmoid ? head_norm_kernel<T, true> : head_norm_kernel<T, false>;
        kernel<<<blocks, 256, 0, stream>>>(
            (T*)out, ld_out, (const T*)y, (const T*)gate, ld_gate, w, eps, groups, gs, lg, total);
    });
}

extern "C" hipError_t launch_page_write(
    void* k_pages, void* v_pages, const void* k, int64_t ldk, const void* v, int64_t ldv,
    const int64_t* slot_mapping, int rows, int wk, int wv, int f32, int vec8,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const int th = row_threads(wk + wv, V) < 256 ? row_threads(wk + wv, V) : 256;
        page_write_kernel<T, V><<<rows, th, 0, stream>>>(
            (T*)k_pages, (T*)v_pages, (const T*)k, ldk, (const T*)v, ldv, slot_mapping, wk, wv);
    });
}

extern "C" hipError_t launch_clamped_glu(
    void* out, const void* x, float limit, int rows, int ff, int f32, int vec8,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        clamped_glu_kernel<T, V><<<row_grid(rows, ff, V), 256, 0, stream>>>(
            (T*)out, (const T*)x, limit, ff);
    });
}

extern "C" hipError_t launch_soft_cap(float* x, float cap, size_t n, hipStream_t stream) {
    if (n == 0) return hipSuccess;
    const size_t want = (n + 1023) / 1024;
    const unsigned grid = want < 4096 ? (unsigned)want : 4096;
    soft_cap_kernel<<<grid, 256, 0, stream>>>(x, cap, n);
    HIP_CHECK_LAST();
    return hipSuccess;
}
