// Row kernels of the hybrid decoders for gfx950: scaled embedding, residual
// add + layer norm over an fp32 stream, latent norms + rotation + page
// write, gated group norm, causal convolution with carried state.
//
// Every kernel is templated on the compute dtype (bf16 or fp32) and takes
// any width; widths and strides that allow it are moved 16 bytes a lane.
// Sums and transcendentals are fp32.

#include "rows.h"


// ---------------------------------------------------------------------------
// x[t] = embed[token] * scale (fp32); x0[t] (compute dtype) the same
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void embed_scaled_kernel(
    float* __restrict__ x, T* __restrict__ x0, int64_t ld0,
    const int64_t* __restrict__ tokens, const T* __restrict__ embed, float scale, int W) {
    const size_t t = blockIdx.x;
    const T* src = embed + (size_t)tokens[t] * W;
    for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
        float f[VEC];
        load_vec<VEC>(src + i, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] *= scale;
        store_vec<VEC>(x + t * W + i, f);
        if (x0 != nullptr) store_vec<VEC>(x0 + t * ld0 + i, f);
    }
}

// ---------------------------------------------------------------------------
// x = (REPLACE ? 0 : x) + delta + vec, kept in the fp32 stream; then
//   norm:  out = (x - mean) / sqrt(var + eps) * w + b   (w given)
//   cast:  out = x                                      (w null)
// One pass over memory: a row stays in registers between the sums (widths
// beyond 16384 re-read it).
// ---------------------------------------------------------------------------
template <typename T, typename D, int VEC>
__launch_bounds__(512)
__global__ void stream_norm_kernel(
    T* __restrict__ out, int64_t ld_out, float* __restrict__ x,
    const D* __restrict__ delta, const float* __restrict__ vec,
    const float* __restrict__ w, const float* __restrict__ b, float eps, int replace,
    int W) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    float* xr = x + t * W;
    const D* dr = delta + t * W;
    T* orow = out + t * ld_out;
    const int step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        float* f = held[k];
        if (replace) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] = 0.f;
        } else {
            load_vec<VEC>(xr + i, f);
        }
        float g[VEC];
        if (delta != nullptr) {
            load_vec<VEC>(dr + i, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] += g[j];
        }
        if (vec != nullptr) {
            load_vec<VEC>(vec + i, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] += g[j];
        }
        if (delta != nullptr || vec != nullptr) store_vec<VEC>(xr + i, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) sum += f[j];
        if (w == nullptr) store_vec<VEC>(orow + i, f);
    }
    if (w == nullptr) return;
    const float mean = block_sum(sum, red) / (float)W;
    float ssq = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        if (i0 + k * step >= W) continue;
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            held[k][j] -= mean;
            ssq += held[k][j] * held[k][j];
        }
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, red) / (float)W + eps);
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        float wv[VEC], bv[VEC];
        load_vec<VEC>(w + i, wv);
        load_vec<VEC>(b + i, bv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[k][j] = held[k][j] * inv * wv[j] + bv[j];
        store_vec<VEC>(orow + i, held[k]);
    }
}

// ---------------------------------------------------------------------------
// One row of d = [query latent | kv latent | rotated key part]: RMS norm of
// the first two, pair rotation of the third; the query latent goes to cq,
// the rest to the row's cache page slot (-1: not kept).
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__launch_bounds__(512)
__global__ void latent_rows_kernel(
    T* __restrict__ cq, T* __restrict__ latent, int row_w, const T* __restrict__ d,
    const float* __restrict__ q_norm, const float* __restrict__ kv_norm, float eps,
    int q_rank, int rank, int rot, const int64_t* __restrict__ positions,
    const float* __restrict__ cos_sin, const int64_t* __restrict__ slot_mapping) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    const T* src = d + t * (q_rank + rank + rot);
    const int W = q_rank + rank, step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float sq = 0.f, sc = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        load_vec<VEC>(src + i, held[k]);
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss += held[k][j] * held[k][j];
        if (i < q_rank) sq += ss;
        else sc += ss;
    }
    const float iq = 1.f / sqrtf(block_sum(sq, red) / (float)q_rank + eps);
    const float ic = 1.f / sqrtf(block_sum(sc, red) / (float)rank + eps);
    const int64_t slot = slot_mapping[t];
    T* dst = latent + (size_t)(slot < 0 ? 0 : slot) * row_w;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= W) continue;
        const bool is_q = i < q_rank;
        float wv[VEC];
        load_vec<VEC>(is_q ? q_norm + i : kv_norm + i - q_rank, wv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[k][j] *= (is_q ? iq : ic) * wv[j];
        if (is_q) store_vec<VEC>(cq + t * q_rank + i, held[k]);
        else if (slot >= 0) store_vec<VEC>(dst + i - q_rank, held[k]);
    }
    if (slot < 0) return;
    const int half = rot / 2;
    const float* cs = cos_sin + (size_t)positions[t] * rot;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
        const float u = ldf(src + W + 2 * i);
        const float v = ldf(src + W + 2 * i + 1);
        stf(dst + rank + 2 * i, u * cs[i] - v * cs[half + i]);
        stf(dst + rank + 2 * i + 1, v * cs[i] + u * cs[half + i]);
    }
}

// ---------------------------------------------------------------------------
// out[t, h, :width] = pair rotation of x[t, h, :rot], zeros from rot on
// (x may be out). Strides in elements; the last dimension is dense.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void rotate_pairs_kernel(
    T* out, int64_t ot, int64_t oh, int width, const T* x, int64_t xt, int64_t xh, int rot,
    int H, const int64_t* __restrict__ positions, const float* __restrict__ cos_sin) {
    const size_t t = blockIdx.x;
    const int half = rot / 2;
    const float* cs = cos_sin + (size_t)positions[t] * rot;
    for (int e = threadIdx.x; e < H * half; e += blockDim.x) {
        const int h = e / half, i = e % half;
        const T* p = x + t * xt + h * xh + 2 * i;
        T* o = out + t * ot + h * oh + 2 * i;
        const float u = ldf(p), v = ldf(p + 1);
        stf(o, u * cs[i] - v * cs[half + i]);
        stf(o + 1, v * cs[i] + u * cs[half + i]);
    }
    const int pad = width - rot;
    for (int e = threadIdx.x; e < H * pad; e += blockDim.x)
        stf(out + t * ot + (e / pad) * oh + rot + e % pad, 0.f);
}

// ---------------------------------------------------------------------------
// Group norm with a gate: y (dense rows) in `groups` equal parts.
//   GATE 0: out = rms(y) * w * sigmoid(gate)
//   GATE 1: out = rms(y * silu(gate)) * w
//   GATE 2: out = rms(y) * w * silu(gate)
// One workgroup per (row, group).
// ---------------------------------------------------------------------------
template <typename T, int VEC, int GATE>
__launch_bounds__(512)
__global__ void gated_norm_kernel(
    T* __restrict__ out, int64_t ld_out, const T* __restrict__ y, const T* __restrict__ gate,
    int64_t ld_gate, const float* __restrict__ w, float eps, int groups, int gs) {
    __shared__ float red[8];
    constexpr int HELD = 32 / VEC;
    const size_t t = blockIdx.x;
    const int g = blockIdx.y;
    const size_t base = t * (size_t)groups * gs + (size_t)g * gs;
    const T* yr = y + base;
    const T* gr = gate + t * ld_gate + (size_t)g * gs;
    const float* wr = w + (size_t)g * gs;
    const int step = blockDim.x * VEC, i0 = threadIdx.x * VEC;
    float held[HELD][VEC];
    float ssq = 0.f;
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= gs) continue;
        load_vec<VEC>(yr + i, held[k]);
        if (GATE == 1) {
            float z[VEC];
            load_vec<VEC>(gr + i, z);
#pragma unroll
            for (int j = 0; j < VEC; ++j) held[k][j] *= z[j] * sigmoid_f(z[j]);
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) ssq += held[k][j] * held[k][j];
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, red) / (float)gs + eps);
#pragma unroll
    for (int k = 0; k < HELD; ++k) {
        const int i = i0 + k * step;
        if (i >= gs) continue;
        float wv[VEC];
        load_vec<VEC>(wr + i, wv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[k][j] *= inv * wv[j];
        if (GATE != 1) {
            float z[VEC];
            load_vec<VEC>(gr + i, z);
#pragma unroll
            for (int j = 0; j < VEC; ++j)
                held[k][j] *= sigmoid_f(z[j]) * (GATE == 2 ? z[j] : 1.f);
        }
        store_vec<VEC>(out + t * ld_out + (size_t)g * gs + i, held[k]);
    }
}

// ---------------------------------------------------------------------------
// Causal per-channel convolution + silu over the rows of each segment; taps
// before the segment come from state [slots, taps-1, C] (zeros when the
// segment starts its sequence). w_t is [taps, C].
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void causal_conv_kernel(
    T* __restrict__ y, const T* __restrict__ x, int64_t ldx, const float* __restrict__ w_t,
    const float* __restrict__ b, const T* __restrict__ state,
    const int64_t* __restrict__ positions, const int* __restrict__ cu,
    const int* __restrict__ slots, const int* __restrict__ row_seg, int C, int taps) {
    const size_t t = blockIdx.x;
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
    if (c >= C) return;
    const int s = row_seg[t];
    const int slot = slots[s];
    const int j0 = (int)t - cu[s];
    float acc[VEC];
    load_vec<VEC>(b + c, acc);
    const bool fresh = slot < 0 || positions[t] == j0;
    for (int k = 0; k < taps; ++k) {
        const int src = j0 - (taps - 1) + k;
        float f[VEC], wv[VEC];
        if (src >= 0)
            load_vec<VEC>(x + (t - j0 + src) * ldx + c, f);
        else if (!fresh)
            load_vec<VEC>(state + ((size_t)slot * (taps - 1) + src + taps - 1) * C + c, f);
        else
            continue;
        load_vec<VEC>(w_t + (size_t)k * C + c, wv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) acc[j] += wv[j] * f[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] *= sigmoid_f(acc[j]);
    store_vec<VEC>(y + t * C + c, acc);
}

// the same for CONV_ROWS consecutive rows a thread, the window in registers
#define CONV_ROWS 8
template <typename T, int TAPS>
__global__ void causal_conv_rows_kernel(
    T* __restrict__ y, const T* __restrict__ x, int64_t ldx, const float* __restrict__ w_t,
    const float* __restrict__ b, const T* __restrict__ state,
    const int64_t* __restrict__ positions, const int* __restrict__ cu,
    const int* __restrict__ slots, const int* __restrict__ row_seg, int rows, int C) {
    constexpr int P = TAPS - 1;  // rows of the past in the window
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * 8;
    if (c >= C) return;
    float w[TAPS][8], bias[8], win[TAPS][8];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) load_vec<8>(w_t + (size_t)k * C + c, w[k]);
    load_vec<8>(b + c, bias);
    int prev = -1;
    for (int i = 0; i < CONV_ROWS; ++i) {
        const int t = blockIdx.x * CONV_ROWS + i;
        if (t >= rows) return;
        const int s = row_seg[t];
        if (s != prev) {  // fill the window from the segment or the state
            prev = s;
            const int slot = slots[s], j0 = t - cu[s];
            const bool fresh = slot < 0 || positions[t] == j0;
#pragma unroll
            for (int k = 0; k < P; ++k) {
                const int src = j0 - P + k;
                if (src >= 0) {
                    load_vec<8>(x + (size_t)(t - P + k) * ldx + c, win[k]);
                } else if (!fresh) {
                    load_vec<8>(state + ((size_t)slot * P + src + P) * C + c, win[k]);
                } else {
#pragma unroll
                    for (int j = 0; j < 8; ++j) win[k][j] = 0.f;
                }
            }
        }
        load_vec<8>(x + (size_t)t * ldx + c, win[P]);
        float acc[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            acc[j] = bias[j];
#pragma unroll
            for (int k = 0; k < TAPS; ++k) acc[j] = fmaf(w[k][j], win[k][j], acc[j]);
            acc[j] *= sigmoid_f(acc[j]);
#pragma unroll
            for (int k = 0; k < P; ++k) win[k][j] = win[k + 1][j];
        }
        store_vec<8>(y + (size_t)t * C + c, acc);
    }
}

// the state after each segment: its last taps-1 inputs (ascending rows, so
// shifting within the state is safe in place)
template <typename T, int VEC>
__global__ void conv_state_kernel(
    const T* __restrict__ x, int64_t ldx, T* __restrict__ state,
    const int64_t* __restrict__ positions, const int* __restrict__ cu,
    const int* __restrict__ slots, int C, int taps) {
    const int s = blockIdx.x;
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
    const int slot = slots[s];
    if (c >= C || slot < 0) return;
    const int r0 = cu[s], n = cu[s + 1] - r0;
    const bool fresh = positions[r0] == 0;
    T* st = state + (size_t)slot * (taps - 1) * C + c;
    for (int r = 0; r < taps - 1; ++r) {
        const int src = n - (taps - 1) + r;
        float f[VEC];
        if (src >= 0) {
            load_vec<VEC>(x + (size_t)(r0 + src) * ldx + c, f);
        } else if (!fresh) {
            load_vec<VEC>(st + (size_t)(src + taps - 1) * C, f);
        } else {
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] = 0.f;
        }
        store_vec<VEC>(st + (size_t)r * C, f);
    }
}

// one row per segment: convolve and shift in one launch. TAPS 0: any number;
// otherwise all of a channel's inputs are loaded before the first is stored
template <typename T, int VEC, int TAPS>
__global__ void conv_step_kernel(
    T* __restrict__ y, const T* __restrict__ x, int64_t ldx, const float* __restrict__ w_t,
    const float* __restrict__ b, T* __restrict__ state,
    const int64_t* __restrict__ positions, const int* __restrict__ slots, int C, int any_taps) {
    const size_t t = blockIdx.x;
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
    if (c >= C) return;
    const int slot = slots[t], taps = TAPS ? TAPS : any_taps;
    const bool empty = slot < 0 || positions[t] == 0;
    float acc[VEC];
    load_vec<VEC>(b + c, acc);
    T* st = state + (size_t)(slot < 0 ? 0 : slot) * (taps - 1) * C + c;
    auto load = [&](int k, float* f) {
        if (k == taps - 1) {
            load_vec<VEC>(x + t * ldx + c, f);
        } else if (empty) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] = 0.f;
        } else {
            load_vec<VEC>(st + (size_t)k * C, f);
        }
    };
    auto take = [&](int k, const float* f) {
        float wv[VEC];
        load_vec<VEC>(w_t + (size_t)k * C + c, wv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) acc[j] += wv[j] * f[j];
        if (k > 0 && slot >= 0) store_vec<VEC>(st + (size_t)(k - 1) * C, f);
    };
    if (TAPS) {
        float f[TAPS ? TAPS : 1][VEC];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) load(k, f[k]);
#pragma unroll
        for (int k = 0; k < TAPS; ++k) take(k, f[k]);
    } else {
        for (int k = 0; k < taps; ++k) {
            float f[VEC];
            load(k, f);
            take(k, f);
        }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] *= sigmoid_f(acc[j]);
    store_vec<VEC>(y + t * C + c, acc);
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
extern "C" hipError_t launch_embed_scaled(
    float* x, void* x0, int64_t ld0, const int64_t* tokens, const void* embed, float scale,
    int rows, int W, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        embed_scaled_kernel<T, V><<<rows, row_threads(W, V), 0, stream>>>(
            x, (T*)x0, ld0, tokens, (const T*)embed, scale, W);
    });
}

extern "C" hipError_t launch_stream_norm(
    void* out, int64_t ld_out, float* x, const void* delta, int delta_f32, const float* vec,
    const float* w, const float* b, float eps, int replace, int rows, int W, int f32,
    int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (W > 512 * 32) return hipErrorInvalidValue;
    if (delta_f32)
        return pick(f32, vec8, [&](auto form) {
            FORM(form);
            stream_norm_kernel<T, float, V><<<rows, row_threads(W, V), 0, stream>>>(
                (T*)out, ld_out, x, (const float*)delta, vec, w, b, eps, replace, W);
        });
    else
        return pick(f32, vec8, [&](auto form) {
            FORM(form);
            stream_norm_kernel<T, T, V><<<rows, row_threads(W, V), 0, stream>>>(
                (T*)out, ld_out, x, (const T*)delta, vec, w, b, eps, replace, W);
        });
}

extern "C" hipError_t launch_latent_rows(
    void* cq, void* latent, int row_w, const void* d, const float* q_norm,
    const float* kv_norm, float eps, int q_rank, int rank, int rot,
    const int64_t* positions, const float* cos_sin, const int64_t* slot_mapping, int rows,
    int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (q_rank + rank > 512 * 32) return hipErrorInvalidValue;
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        latent_rows_kernel<T, V><<<rows, row_threads(q_rank + rank, V), 0, stream>>>(
            (T*)cq, (T*)latent, row_w, (const T*)d, q_norm, kv_norm, eps, q_rank, rank, rot,
            positions, cos_sin, slot_mapping);
    });
}

extern "C" hipError_t launch_rotate_pairs(
    void* out, int64_t ot, int64_t oh, int width, const void* x, int64_t xt, int64_t xh,
    int rot, int H, const int64_t* positions, const float* cos_sin, int rows, int f32,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    return pick(f32, 0, [&](auto form) {
        FORM(form);
        rotate_pairs_kernel<T><<<rows, 256, 0, stream>>>(
            (T*)out, ot, oh, width, (const T*)x, xt, xh, rot, H, positions, cos_sin);
    });
}

extern "C" hipError_t launch_gated_norm(
    void* out, int64_t ld_out, const void* y, const void* gate, int64_t ld_gate,
    const float* w, float eps, int groups, int gs, int mode, int rows, int f32, int vec8,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (gs > 512 * 32 || mode < 0 || mode > 2) return hipErrorInvalidValue;
    const dim3 grid(rows, groups);
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
#define GO(GATE)                                                                  \
    gated_norm_kernel<T, V, GATE><<<grid, row_threads(gs, V), 0, stream>>>(       \
        (T*)out, ld_out, (const T*)y, (const T*)gate, ld_gate, w, eps, groups, gs)
        if (mode == 0) GO(0);
        else if (mode == 1) GO(1);
        else GO(2);
#undef GO
    });
}

extern "C" hipError_t launch_causal_conv(
    void* y, const void* x, int64_t ldx, const float* w_t, const float* b, void* state,
    const int64_t* positions, const int* cu, const int* slots, const int* row_seg,
    int rows, int nseg, int C, int taps, int f32, int vec8, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    const int per = vec8 ? 8 : 1, th = 256;
    const int cb = ceil_div_i(C, per * th);
    if (rows == nseg)
        return pick(f32, vec8, [&](auto form) {
            FORM(form);
            auto kernel = taps == 4 ? conv_step_kernel<T, V, 4> : conv_step_kernel<T, V, 0>;
            kernel<<<dim3(rows, cb), th, 0, stream>>>(
                (T*)y, (const T*)x, ldx, w_t, b, (T*)state, positions, slots, C, taps);
        });
    return pick(f32, vec8, [&](auto form) {
        FORM(form);
        const dim3 grid(ceil_div_i(rows, CONV_ROWS), cb);
        if (vec8 && taps == 4)
            causal_conv_rows_kernel<T, 4><<<grid, th, 0, stream>>>(
                (T*)y, (const T*)x, ldx, w_t, b, (const T*)state, positions, cu, slots,
                row_seg, rows, C);
        else if (vec8 && taps == 3)
            causal_conv_rows_kernel<T, 3><<<grid, th, 0, stream>>>(
                (T*)y, (const T*)x, ldx, w_t, b, (const T*)state, positions, cu, slots,
                row_seg, rows, C);
        else if (vec8 && taps == 2)
            causal_conv_rows_kernel<T, 2><<<grid, th, 0, stream>>>(
                (T*)y, (const T*)x, ldx, w_t, b, (const T*)state, positions, cu, slots,
                row_seg, rows, C);
        else
            causal_conv_kernel<T, V><<<dim3(rows, cb), th, 0, stream>>>(
                (T*)y, (const T*)x, ldx, w_t, b, (const T*)state, positions, cu, slots,
                row_seg, C, taps);
        if (taps > 1)
            conv_state_kernel<T, V><<<dim3(nseg, cb), th, 0, stream>>>(
                (const T*)x, ldx, (T*)state, positions, cu, slots, C, taps);
    });
}
