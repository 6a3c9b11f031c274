// Grouped-query attention over the last `window` tokens in cache pages for
// gfx950, without softmax: key j weighs, for head h of the row at position p,
//   w_h(j) = sigmoid(scale * q_h.k_j + bias[p - j, h])
// and head h's output is sum_j m_h(j) v_j with m_h = sum_g talk[h, g] w_g: all
// heads' weights of a pair (row, key) are mixed before the values of head h's
// own key head h/(H/G) are summed. Every output value is multiplied by
// sigmoid(gate). Pages as in attention_paged.hip: a token's row holds the keys
// (or values) of all G key heads.
//
// Nothing is normalized, so partial sums over any keys add up.
//
// Three forms of one function: any size (fp32, or sizes that are no multiple
// of 8), rows (decoding and short portions: a row's heads side by side) and
// tiles (prompts: 16 rows, all heads).
//
// The weights are fp32; into their mix they go as the sum of two bf16 (talk is
// bf16 data), which keeps fp32-like accuracy. The mixed weights meet the bf16
// values in bf16.

#include "lds_dma.h"
#include "mfma.h"
#include "rows.h"

#define SA_THREADS 256
#define LOG2E 1.4426950408889634f

struct SigmoidArgs {
    void* out;
    int64_t ld_out;            // row stride; heads are vdim apart
    const void* q;
    int64_t ldq;
    const void *k, *v;         // pages
    const float* bias;         // [nbias, Hp] by distance; the last row for all beyond
    const void* talk;          // [H, H]
    const void* gate;          // [rows, H * vdim], row stride ld_gate
    int64_t ld_gate;
    float scale;
    const int64_t* positions;
    const int *row_seg, *tables;
    const int* rows;           // nullable: which rows of the batch
    int window, nbias, Hp, max_blocks, block_size, H, G, dim, vdim;
};

// ---------------------------------------------------------------------------
// Any size: one workgroup per row and slice of ND*256 outputs. 32 keys at a
// time: all heads' weights, their mix, then an output a thread.
// ---------------------------------------------------------------------------
#define ANY_ND 4
#define ANY_KEYS 32

template <typename T>
__launch_bounds__(SA_THREADS)
__global__ void sigmoid_any_kernel(SigmoidArgs a) {
    extern __shared__ float lds[];  // [H][32] weights, [H][32] their mix
    float *w = lds, *m = lds + a.H * ANY_KEYS;
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int pos = (int)a.positions[t], bs = a.block_size, per = a.H / a.G;
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const T *kp = (const T*)a.k, *vp = (const T*)a.v, *talk = (const T*)a.talk;
    const T* qr = (const T*)a.q + t * a.ldq;
    const int tid = threadIdx.x, o0 = blockIdx.y * ANY_ND * SA_THREADS, n_out = a.H * a.vdim;
    float acc[ANY_ND];
#pragma unroll
    for (int d = 0; d < ANY_ND; ++d) acc[d] = 0.f;
    for (int k0 = max(0, pos - a.window + 1); k0 <= pos; k0 += ANY_KEYS) {
        const int here = min(ANY_KEYS, pos + 1 - k0);
        __syncthreads();
        for (int e = tid; e < a.H * ANY_KEYS; e += SA_THREADS) {
            const int h = e / ANY_KEYS, j = e % ANY_KEYS, key = k0 + j;
            float p = 0.f;
            if (j < here) {
                const T* kr =
                    kp + (((size_t)bt[key / bs] * bs + key % bs) * a.G + h / per) * a.dim;
                float s = 0.f;
                for (int i = 0; i < a.dim; ++i) s = fmaf(ldf(qr + h * a.dim + i), ldf(kr + i), s);
                p = sigmoid_f(s * a.scale + a.bias[(size_t)min(pos - key, a.nbias - 1) * a.Hp + h]);
            }
            w[e] = p;
        }
        __syncthreads();
        for (int e = tid; e < a.H * ANY_KEYS; e += SA_THREADS) {
            const int h = e / ANY_KEYS, j = e % ANY_KEYS;
            float s = 0.f;
            for (int g = 0; g < a.H; ++g)
                s = fmaf(ldf(talk + (size_t)h * a.H + g), w[g * ANY_KEYS + j], s);
            m[e] = s;
        }
        __syncthreads();
        for (int j = 0; j < here; ++j) {
            const int key = k0 + j;
            const T* vr = vp + ((size_t)bt[key / bs] * bs + key % bs) * a.G * a.vdim;
#pragma unroll
            for (int d = 0; d < ANY_ND; ++d) {
                const int o = o0 + tid + d * SA_THREADS, h = o / a.vdim;
                if (o < n_out)
                    acc[d] = fmaf(m[h * ANY_KEYS + j],
                                  ldf(vr + (size_t)(h / per) * a.vdim + o % a.vdim), acc[d]);
            }
        }
    }
#pragma unroll
    for (int d = 0; d < ANY_ND; ++d) {
        const int o = o0 + tid + d * SA_THREADS;
        if (o < n_out)
            stf((T*)a.out + t * a.ld_out + o,
                acc[d] * sigmoid_f(ldf((const T*)a.gate + t * a.ld_gate + o)));
    }
}

// sigmoid(s) from s * log2(e): both exponentials' ends give 0 and 1
__device__ __forceinline__ float sigmoid_2(float s2) {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-s2));
}
__device__ __forceinline__ float gate_2(float z) { return sigmoid_2(z * LOG2E); }

// 8 fp32 as bf16 fragments of their leading and remaining halves
__device__ __forceinline__ void split_frag(const float* f, bf16x8& hi, bf16x8& lo) {
    uint4 h, l;
    uint32_t *hp = &h.x, *lp = &l.x;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        float a, b;
        hp[i] = cvt_pk_bf16(f[2 * i], f[2 * i + 1]);
        unpack2(hp[i], a, b);
        lp[i] = cvt_pk_bf16(f[2 * i] - a, f[2 * i + 1] - b);
    }
    hi = as_frag(h);
    lo = as_frag(l);
}
__device__ __forceinline__ bf16x8 masked(bool keep, const bf16x8& f) {
    uint4 v = *reinterpret_cast<const uint4*>(&f);
    if (!keep) v = (uint4){0, 0, 0, 0};
    return as_frag(v);
}

// ---------------------------------------------------------------------------
// Rows: one workgroup per (row, split of the keys); its 4 waves take 32 keys
// of all key heads in turn. A chain of products in which every result is the
// next one's operand as it stands:
//   S [head, key] = Q K^T: the operand Q holds 16 heads, zeros where a head
//     does not read this key head, so that one accumulator collects all of them
//   M^T [key, head] = W^T talk^T, W = sigmoid(S + bias): a lane's heads
//     (4g + r of two fragments of 16) are the k order of the operand
//   O^T [value, head] += V^T M^T, M^T zeroed like Q; key order as in
//     attention_paged.hip
// Keys go from global memory into the fragments, values through the wave's
// LDS tile. The waves' shares meet in LDS; several splits leave partial sums
// for sigmoid_combine_kernel.
// ---------------------------------------------------------------------------
template <int NB, int NDQ, int NDV>  // blocks of 16 heads; dim/32, vdim/16
__launch_bounds__(SA_THREADS)
__global__ void sigmoid_rows_kernel(SigmoidArgs a, int page_shift, int nsplit, float* part) {
    constexpr int LDV = NDV * 16 + 8, TILE = 32 * LDV, NK = (NB + 1) / 2;
    __shared__ __align__(16) bf16 v_lds[4][TILE];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int split = blockIdx.y, per = a.H / a.G;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pos = (int)a.positions[t];
    const int first = max(0, pos - a.window + 1), base = first & ~31;
    const int span = (pos + 1 - base + nsplit * 128 - 1) / (nsplit * 128) * 128;
    const int key_lo = base + split * span, key_hi = min(pos + 1, key_lo + span);
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const float scale2 = a.scale * LOG2E;

    int key_head[NB];  // of this lane's head in each block
    bf16x8 qf[NB][NDQ], tf[NB][NK];
#pragma unroll
    for (int b = 0; b < NB; ++b) {
        const int h = b * 16 + r16;
        key_head[b] = h < a.H ? h / per : -1;
        const bf16* qr = (const bf16*)a.q + t * a.ldq + (size_t)min(h, a.H - 1) * a.dim;
#pragma unroll
        for (int c = 0; c < NDQ; ++c) {
            uint4 x = {0, 0, 0, 0};
            if (c * 32 + g * 8 < a.dim) x = *reinterpret_cast<const uint4*>(qr + c * 32 + g * 8);
            qf[b][c] = as_frag(x);
        }
#pragma unroll
        for (int kb = 0; kb < NK; ++kb) {
            uint16_t x[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int from = kb * 32 + (j >> 2) * 16 + g * 4 + (j & 3);
                x[j] = h < a.H && from < a.H
                           ? reinterpret_cast<const uint16_t*>(a.talk)[(size_t)h * a.H + from]
                           : 0;
            }
            tf[b][kb] = *reinterpret_cast<const bf16x8*>(x);
        }
    }
    f32x4 acc[NB][NDV];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[b][j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    // rows of 16 keys from k0 in the pages; past the end any row that is there
    const int last = pos;
    auto page_row = [&](int k0) {
        return (size_t)bt[min(k0, last) >> page_shift] << page_shift;
    };
    auto load_k = [&](size_t b0, size_t b1, int k0, int gk, uint4* kreg) {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int key = min(k0 + u * 16 + r16, last);
            const size_t row = (u && k0 + 16 <= last ? b1 : b0) + (key & mask);
            const bf16* p = (const bf16*)a.k + (row * a.G + gk) * a.dim;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                kreg[u * NDQ + c] = (uint4){0, 0, 0, 0};
                if (c * 32 + g * 8 < a.dim)
                    kreg[u * NDQ + c] = *reinterpret_cast<const uint4*>(p + c * 32 + g * 8);
            }
        }
    };
    auto load_v = [&](size_t b0, size_t b1, int k0, int gk, uint4* vreg) {
#pragma unroll
        for (int u = 0; u < NDV; ++u) {
            const int e = lane + u * 64, o = e / (NDV * 2), d = e % (NDV * 2) * 8;
            const int key = min(k0 + o, last);
            const size_t row = (key >= k0 + 16 ? b1 : b0) + (key & mask);
            vreg[u] = (uint4){0, 0, 0, 0};
            if (d < a.vdim)
                vreg[u] = *reinterpret_cast<const uint4*>(
                    (const bf16*)a.v + (row * a.G + gk) * a.vdim + d);
        }
    };
    bf16* vt = v_lds[wave];
    uint4 kreg[2 * NDQ], vreg[NDV];
    int k0 = key_lo + wave * 32;
    size_t b0 = 0, b1 = 0;
    if (k0 < key_hi) {
        b0 = page_row(k0);
        b1 = page_row(k0 + 16);
        load_k(b0, b1, k0, 0, kreg);
    }
    for (; k0 < key_hi; k0 += 128) {
        f32x4 s[NB][2];
#pragma unroll
        for (int b = 0; b < NB; ++b) s[b][0] = s[b][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
        for (int gk = 0; gk < a.G; ++gk) {
            uint4 kf[2 * NDQ];
#pragma unroll
            for (int i = 0; i < 2 * NDQ; ++i) kf[i] = kreg[i];
            if (gk + 1 < a.G) load_k(b0, b1, k0, gk + 1, kreg);
            else load_v(b0, b1, k0, 0, vreg);
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                if (gk * per >= b * 16 + 16 || (gk + 1) * per <= b * 16) continue;
                const bool mine = key_head[b] == gk;
#pragma unroll
                for (int c = 0; c < NDQ; ++c) {
                    const bf16x8 qm = masked(mine, qf[b][c]);
#pragma unroll
                    for (int u = 0; u < 2; ++u)
                        s[b][u] = mfma16(qm, as_frag(kf[u * NDQ + c]), s[b][u]);
                }
            }
        }
        // weights of heads 16b + 4g + r, keys k0 + 16u + r16; their mix
        bf16x8 pf[NB];
        {
            f32x4 m[NB][2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int key = k0 + u * 16 + r16, dist = pos - key;
                const bool seen = key >= first && key < key_hi;
                const float* br = a.bias + (size_t)max(0, min(dist, a.nbias - 1)) * a.Hp + g * 4;
                bf16x8 hi[NK], lo[NK];
#pragma unroll
                for (int kb = 0; kb < NK; ++kb) {
                    float w[8];
#pragma unroll
                    for (int half = 0; half < 2; ++half) {
                        const int b = kb * 2 + half;
                        if (b < NB && b * 16 < a.Hp) {
                            const float4 bb = *reinterpret_cast<const float4*>(br + b * 16);
                            const float bv[4] = {bb.x, bb.y, bb.z, bb.w};
#pragma unroll
                            for (int r = 0; r < 4; ++r)
                                w[half * 4 + r] =
                                    seen ? sigmoid_2(fmaf(s[b < NB ? b : 0][u][r], scale2,
                                                          bv[r] * LOG2E))
                                         : 0.f;
                        } else {
#pragma unroll
                            for (int r = 0; r < 4; ++r) w[half * 4 + r] = 0.f;
                        }
                    }
                    split_frag(w, hi[kb], lo[kb]);
                }
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    m[b][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int kb = 0; kb < NK; ++kb) {
                        m[b][u] = mfma16(hi[kb], tf[b][kb], m[b][u]);
                        m[b][u] = mfma16(lo[kb], tf[b][kb], m[b][u]);
                    }
                }
            }
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                uint4 v;
                v.x = cvt_pk_bf16(m[b][0][0], m[b][0][1]);
                v.y = cvt_pk_bf16(m[b][0][2], m[b][0][3]);
                v.z = cvt_pk_bf16(m[b][1][0], m[b][1][1]);
                v.w = cvt_pk_bf16(m[b][1][2], m[b][1][3]);
                pf[b] = as_frag(v);
            }
        }
        const size_t c0 = b0, c1 = b1;  // this tile's pages
        if (k0 + 128 < key_hi) {
            b0 = page_row(k0 + 128);
            b1 = page_row(k0 + 144);
        }
        const bf16* r0 = vt + (g * 4 + (r16 >> 2)) * LDV + (r16 & 3) * 4;
        for (int gk = 0; gk < a.G; ++gk) {
#pragma unroll
            for (int u = 0; u < NDV; ++u) {
                const int e = lane + u * 64;
                *reinterpret_cast<uint4*>(vt + e / (NDV * 2) * LDV + e % (NDV * 2) * 8) = vreg[u];
            }
            if (gk + 1 < a.G) load_v(c0, c1, k0, gk + 1, vreg);
            else if (k0 + 128 < key_hi) load_k(b0, b1, k0 + 128, 0, kreg);
            bf16x8 pm[NB];
#pragma unroll
            for (int b = 0; b < NB; ++b) pm[b] = masked(key_head[b] == gk, pf[b]);
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16x8 vf = tr_pair(r0 + j * 16, r0 + 16 * LDV + j * 16);
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    if (gk * per >= b * 16 + 16 || (gk + 1) * per <= b * 16) continue;
                    acc[b][j] = mfma16(vf, pm[b], acc[b][j]);
                }
            }
        }
    }
    // the waves' shares, 16 heads at a time: [vdim][16 heads] in each wave's tile
    float* sh = reinterpret_cast<float*>(vt);
#pragma unroll
    for (int b = 0; b < NB; ++b) {
        if (b > 0) __syncthreads();
#pragma unroll
        for (int j = 0; j < NDV; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) sh[(j * 16 + g * 4 + r) * 16 + r16] = acc[b][j][r];
        __syncthreads();
        for (int e = tid; e < 16 * a.vdim; e += SA_THREADS) {
            const int c = e / a.vdim, d = e % a.vdim, h = b * 16 + c;
            if (h >= a.H) break;
            float o = 0.f;
#pragma unroll
            for (int w = 0; w < 4; ++w) o += reinterpret_cast<const float*>(v_lds[w])[d * 16 + c];
            const int at = h * a.vdim + d;
            if (nsplit == 1)
                stf((bf16*)a.out + t * a.ld_out + at,
                    o * gate_2(ldf((const bf16*)a.gate + t * a.ld_gate + at)));
            else
                part[((size_t)blockIdx.x * nsplit + split) * a.H * a.vdim + at] = o;
        }
    }
}

// the splits' sums, gated: 4 outputs a thread
__global__ void sigmoid_combine_kernel(SigmoidArgs a, int nsplit, const float* __restrict__ part) {
    const size_t i = blockIdx.x, t = a.rows ? a.rows[i] : i;
    const int at = (blockIdx.y * blockDim.x + threadIdx.x) * 4, n = a.H * a.vdim;
    if (at >= n) return;
    const float* p = part + i * nsplit * n + at;
    float4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < nsplit; ++s) {
        const float4 x = *reinterpret_cast<const float4*>(p + (size_t)s * n);
        o.x += x.x;
        o.y += x.y;
        o.z += x.z;
        o.w += x.w;
    }
    const bf16* z = (const bf16*)a.gate + t * a.ld_gate + at;
    *reinterpret_cast<uint2*>((bf16*)a.out + t * a.ld_out + at) = make_uint2(
        cvt_pk_bf16(o.x * gate_2(ldf(z)), o.y * gate_2(ldf(z + 1))),
        cvt_pk_bf16(o.z * gate_2(ldf(z + 2)), o.w * gate_2(ldf(z + 3))));
}

// ---------------------------------------------------------------------------
// Tiles: one workgroup of 8 waves per 16 rows of a segment, all heads; a wave
// holds HW heads that share a key head. 32 keys at a time:
//   S [row, key] of the wave's heads; weights to LDS, by row: [key][32 heads]
//   mix: each wave two rows, M^T [key, head] = W^T talk^T; back to LDS in
//     place of the weights, by row: [head][32 keys]
//   O^T [value, row] += V^T M^T of the wave's heads
// Keys go into the fragments, 32 ahead; values by transfers into the wave's
// own LDS tile, 32-byte pairs of chunks XOR-swizzled by row on the source
// address. 16-byte chunks of weights are swizzled likewise.
// ---------------------------------------------------------------------------
template <int HW, int NDQ, int NDV>
__launch_bounds__(512)
__global__ void sigmoid_tiles_kernel(
    SigmoidArgs a, int page_shift, const int* __restrict__ cu,
    const int* __restrict__ tile_seg, const int* __restrict__ tile_off, int ntiles) {
    constexpr int LDW = 32 * 32 + 8;  // a row's weights
    constexpr int LDB = 36;           // biases of a distance
    __shared__ __align__(16) bf16 w_lds[2][16][LDW], v_lds[8][32 * NDV * 16];
    __shared__ __align__(16) float b_lds[47][LDB];
    // each XCD (8, round robin) takes a contiguous part of the tiles, whose
    // windows overlap
    const int share = (ntiles + 7) / 8;
    const int tile = (blockIdx.x & 7) * share + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= share || tile >= ntiles) return;
    const int seg = tile_seg[tile], off = tile_off[tile];
    const int q0 = cu[seg] + off, nq = min(16, cu[seg + 1] - q0);
    const int pos0 = (int)a.positions[q0];  // of the tile's first row
    const int* bt = a.tables + (size_t)seg * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h0 = wave * HW;
    const bool active = h0 < a.H;
    const int gk = active ? h0 / (a.H / a.G) : 0;
    const float scale2 = a.scale * LOG2E;
    const bf16 *kp = (const bf16*)a.k + (size_t)gk * a.dim;
    const bf16 *vp = (const bf16*)a.v + (size_t)gk * a.vdim;
    const int key_end = pos0 + nq, key_lo = max(0, pos0 - a.window + 1) & ~31;

    for (int e = tid; e < 2 * 16 * LDW / 8; e += 512)  // heads that are not there: finite
        reinterpret_cast<uint4*>(w_lds)[e] = (uint4){0, 0, 0, 0};
    bf16x8 qf[HW][NDQ];
    if (active) {
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            const bf16* qr = (const bf16*)a.q + (size_t)(q0 + min(r16, nq - 1)) * a.ldq +
                             (size_t)(h0 + i) * a.dim;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                uint4 x = {0, 0, 0, 0};
                if (c * 32 + g * 8 < a.dim)
                    x = *reinterpret_cast<const uint4*>(qr + c * 32 + g * 8);
                qf[i][c] = as_frag(x);
            }
        }
    }
    bf16x8 tf[2];  // talk^T: column = head 16b + r16, k = head 8g + j
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const int h = b * 16 + r16;
        uint16_t x[8];
#pragma unroll
        for (int j = 0; j < 8; ++j)
            x[j] = h < a.H && g * 8 + j < a.H
                       ? reinterpret_cast<const uint16_t*>(a.talk)[(size_t)h * a.H + g * 8 + j]
                       : 0;
        tf[b] = *reinterpret_cast<const bf16x8*>(x);
    }
    f32x4 acc[HW][NDV];
#pragma unroll
    for (int i = 0; i < HW; ++i)
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    auto page_row = [&](int k0) {
        return (size_t)bt[min(k0, key_end - 1) >> page_shift] << page_shift;
    };
    uint4 kreg[2 * NDQ];
    auto load_k = [&](int k0, size_t b0, size_t b1) {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int key = min(k0 + u * 16 + r16, key_end - 1);
            const size_t row = (u && k0 + 16 < key_end ? b1 : b0) + (key & mask);
            const bf16* p = kp + row * a.G * a.dim;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                kreg[u * NDQ + c] = (uint4){0, 0, 0, 0};
                if (c * 32 + g * 8 < a.dim)
                    kreg[u * NDQ + c] = *reinterpret_cast<const uint4*>(p + c * 32 + g * 8);
            }
        }
    };
    bf16* vt = v_lds[wave];
    auto stage_v = [&](int k0, size_t b0, size_t b1) {
        constexpr int PER = 64 / (NDV * 2);  // rows a transfer
#pragma unroll
        for (int u = 0; u < 32 / PER; ++u) {
            const int o = u * PER + lane / (NDV * 2), c = lane % (NDV * 2);
            const int d = ((((c >> 1) ^ (o & (NDV - 1) & 7)) << 1) | (c & 1)) * 8;
            const int key = min(k0 + o, key_end - 1);
            const size_t row = (key >= k0 + 16 ? b1 : b0) + (key & mask);
            dma16(vp + row * a.G * a.vdim + (d < a.vdim ? d : 0), vt + u * 512);
        }
    };
    // biases of distances dmin .. dmin + 46
    auto fill_bias = [&](int dmin) {
        for (int e = tid; e < 47 * 32; e += 512) {
            const int x = e >> 5, h = e & 31;
            if (h < a.Hp)
                b_lds[x][h] =
                    a.bias[(size_t)max(0, min(dmin + x, a.nbias - 1)) * a.Hp + h] * LOG2E;
        }
    };
    size_t b0 = page_row(key_lo), b1 = page_row(key_lo + 16);
    if (active) load_k(key_lo, b0, b1);
    fill_bias(pos0 - key_lo - 31);
    __syncthreads();

    for (int k0 = key_lo; k0 < key_end; k0 += 32) {
        f32x4 s[HW][2];
        if (active) {
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int i = 0; i < HW; ++i) {
                    s[i][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int c = 0; c < NDQ; ++c)
                        s[i][u] = mfma16(qf[i][c], as_frag(kreg[u * NDQ + c]), s[i][u]);
                }
            __builtin_amdgcn_sched_barrier(0);  // the keys are in: transfers after them
            stage_v(k0, b0, b1);
        }
        lds_barrier();  // the last tile's mixed weights are read
        if (active) {
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int o = u * 16 + r16;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int row = g * 4 + r, dist = pos0 + row - (k0 + o);
                    const bool seen = dist >= 0 && dist < a.window;
                    const float* bv = &b_lds[row + 31 - o][h0];
                    float w[4];
#pragma unroll
                    for (int i = 0; i < HW; ++i)
                        w[i] = seen ? sigmoid_2(fmaf(s[i][u][r], scale2, bv[i])) : 0.f;
#pragma unroll
                    for (int i = HW; i < 4; ++i) w[i] = 0.f;
                    const uint32_t p0 = cvt_pk_bf16(w[0], w[1]), p1 = cvt_pk_bf16(w[2], w[3]);
                    float f[4];
                    unpack2(p0, f[0], f[1]);
                    unpack2(p1, f[2], f[3]);
                    const uint32_t l0 = cvt_pk_bf16(w[0] - f[0], w[1] - f[1]);
                    const uint32_t l1 = cvt_pk_bf16(w[2] - f[2], w[3] - f[3]);
                    auto at = [&](int h) {
                        return o * 32 + (((h >> 3) ^ ((o >> 2) & 3)) << 3) + (h & 7);
                    };
                    if (HW == 4) {
                        *reinterpret_cast<uint2*>(&w_lds[0][row][at(h0)]) = make_uint2(p0, p1);
                        *reinterpret_cast<uint2*>(&w_lds[1][row][at(h0)]) = make_uint2(l0, l1);
                    } else if (HW == 2) {
                        *reinterpret_cast<uint32_t*>(&w_lds[0][row][at(h0)]) = p0;
                        *reinterpret_cast<uint32_t*>(&w_lds[1][row][at(h0)]) = l0;
                    } else {
                        const uint16_t hs[4] = {(uint16_t)p0, (uint16_t)(p0 >> 16), (uint16_t)p1, 0};
                        const uint16_t ls[4] = {(uint16_t)l0, (uint16_t)(l0 >> 16), (uint16_t)l1, 0};
#pragma unroll
                        for (int i = 0; i < HW; ++i) {
                            *reinterpret_cast<uint16_t*>(&w_lds[0][row][at(h0 + i)]) = hs[i];
                            *reinterpret_cast<uint16_t*>(&w_lds[1][row][at(h0 + i)]) = ls[i];
                        }
                    }
                }
            }
        }
        lds_barrier();  // all weights are there
        // the next tile's biases, unless both are all beyond the table
        const int dmin = pos0 - k0 - 31;
        if (k0 + 32 < key_end && dmin - 32 < a.nbias - 1) fill_bias(dmin - 32);
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const int row = wave * 2 + i;
            bf16 *hi = w_lds[0][row], *lo = w_lds[1][row];
            f32x4 m[2][2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int o = u * 16 + r16, at = o * 32 + ((g ^ ((o >> 2) & 3)) << 3);
                const bf16x8 wh = *reinterpret_cast<const bf16x8*>(hi + at);
                const bf16x8 wl = *reinterpret_cast<const bf16x8*>(lo + at);
#pragma unroll
                for (int b = 0; b < 2; ++b) {
                    m[u][b] = mfma16(wh, tf[b], (f32x4){0.f, 0.f, 0.f, 0.f});
                    m[u][b] = mfma16(wl, tf[b], m[u][b]);
                }
            }
            // keys 16u + 4g + r of head 16b + r16, at 8g + 4u + r
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int b = 0; b < 2; ++b) {
                    const int h = b * 16 + r16;
                    *reinterpret_cast<uint2*>(
                        hi + h * 32 + ((g ^ ((h >> 2) & 3)) << 3) + u * 4) =
                        make_uint2(cvt_pk_bf16(m[u][b][0], m[u][b][1]),
                                   cvt_pk_bf16(m[u][b][2], m[u][b][3]));
                }
        }
        const bool more = k0 + 32 < key_end;
        if (more) {
            b0 = page_row(k0 + 32);
            b1 = page_row(k0 + 48);
        }
        dma_barrier();  // mixed weights and values are there
        if (active) {
            if (more) load_k(k0 + 32, b0, b1);
            bf16x8 pf[HW];
#pragma unroll
            for (int i = 0; i < HW; ++i) {
                const int h = h0 + i;
                pf[i] = *reinterpret_cast<const bf16x8*>(
                    &w_lds[0][r16][h * 32 + ((g ^ ((h >> 2) & 3)) << 3)]);
            }
            const int vr = g * 4 + (r16 >> 2), sw = vr & (NDV - 1) & 7;
            const bf16* r0 = vt + vr * NDV * 16 + (r16 & 3) * 4;
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16* p = r0 + ((j ^ sw) << 4);
                const bf16x8 vf = tr_pair(p, p + 16 * NDV * 16);
#pragma unroll
                for (int i = 0; i < HW; ++i) acc[i][j] = mfma16(vf, pf[i], acc[i][j]);
            }
            // the transfers of the next tile may overwrite what is read here
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        }
    }
    if (!active || r16 >= nq) return;
    const size_t t = q0 + r16;
#pragma unroll
    for (int i = 0; i < HW; ++i) {
        const size_t at = (size_t)(h0 + i) * a.vdim;
        const bf16* z = (const bf16*)a.gate + t * a.ld_gate + at;
        bf16* o = (bf16*)a.out + t * a.ld_out + at;
#pragma unroll
        for (int j = 0; j < NDV; ++j) {
            const int d = j * 16 + g * 4;  // vdim is a multiple of 8
            if (d >= a.vdim) continue;
            const uint2 zz = *reinterpret_cast<const uint2*>(z + d);
            float f[4];
            unpack2(zz.x, f[0], f[1]);
            unpack2(zz.y, f[2], f[3]);
            *reinterpret_cast<uint2*>(o + d) = make_uint2(
                cvt_pk_bf16(acc[i][j][0] * gate_2(f[0]), acc[i][j][1] * gate_2(f[1])),
                cvt_pk_bf16(acc[i][j][2] * gate_2(f[2]), acc[i][j][3] * gate_2(f[3])));
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
static SigmoidArgs sigmoid_args(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* bias, const void* talk, const void* gate, int64_t ld_gate, float scale,
    const int64_t* positions, const int* row_seg, const int* tables, const int* rows, int window,
    int nbias, int Hp, int max_blocks, int block_size, int H, int G, int dim, int vdim) {
    return SigmoidArgs{out, ld_out, q, ldq, k, v, bias, talk, gate, ld_gate, scale, positions,
                       row_seg, tables, rows, window, nbias, Hp, max_blocks, block_size, H, G,
                       dim, vdim};
}

// sizes of the MFMA forms; pages of a power of two, at least 16 tokens
static bool sigmoid_mfma_ok(const SigmoidArgs& a) {
    return a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 && a.vdim <= 256 && a.H <= 64 &&
           a.Hp % 16 == 0 && a.Hp >= a.H && a.block_size >= 16 &&
           (a.block_size & (a.block_size - 1)) == 0;
}

// nsplit 0: the any-size form
extern "C" hipError_t launch_sigmoid_rows(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* bias, const void* talk, const void* gate, int64_t ld_gate, float scale,
    const int64_t* positions, const int* row_seg, const int* tables, const int* rows, int window,
    int nbias, int Hp, int max_blocks, int block_size, int H, int G, int dim, int vdim,
    int nrows, int nsplit, float* part, int f32, hipStream_t stream) {
    if (nrows <= 0) return hipSuccess;
    const SigmoidArgs a = sigmoid_args(
        out, ld_out, q, ldq, k, v, bias, talk, gate, ld_gate, scale, positions, row_seg, tables,
        rows, window, nbias, Hp, max_blocks, block_size, H, G, dim, vdim);
    if (nsplit == 0) {
        const size_t lds = 2 * (size_t)H * ANY_KEYS * sizeof(float);
        if (lds > 64 * 1024) return hipErrorInvalidValue;
        const dim3 grid(nrows, ceil_div_i(H * vdim, ANY_ND * SA_THREADS));
        if (f32) sigmoid_any_kernel<float><<<grid, SA_THREADS, lds, stream>>>(a);
        else {
            sigmoid_any_kernel<bf16><<<grid, SA_THREADS, lds, stream>>>(a);
        }
        HIP_CHECK_LAST();
        return hipSuccess;
    }
    if (f32 || !sigmoid_mfma_ok(a) || (nsplit > 1 && !part)) return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size);
    const dim3 grid(nrows, nsplit);
#define GO(NB, A, B) \
    sigmoid_rows_kernel<NB, A, B><<<grid, SA_THREADS, 0, stream>>>(a, shift, nsplit, part)
#define SIZES(NB)                                   \
    {                                               \
        if (dim <= 64 && vdim <= 64) GO(NB, 2, 4);  \
        else if (dim <= 128 && vdim <= 128) GO(NB, 4, 8); \
        else GO(NB, 8, 16);                         \
    }
    if (H <= 16) SIZES(1)
    else if (H <= 32) SIZES(2)
    else SIZES(4)
#undef SIZES
#undef GO
    HIP_CHECK_LAST();
    if (nsplit > 1) {
        sigmoid_combine_kernel<<<dim3(nrows, ceil_div_i(H * vdim, 1024)), 256, 0, stream>>>(
            a, nsplit, part);
        HIP_CHECK_LAST();
    }
    return hipSuccess;
}

// dim and vdim up to 128; at most 32 heads, the H/8 (rounded up) of a wave all
// of one key head
extern "C" hipError_t launch_sigmoid_tiles(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* bias, const void* talk, const void* gate, int64_t ld_gate, float scale,
    const int64_t* positions, const int* tables, int window, int nbias, int Hp, int max_blocks,
    int block_size, int H, int G, int dim, int vdim, const int* cu, const int* tile_seg,
    const int* tile_off, int ntiles, hipStream_t stream) {
    if (ntiles <= 0) return hipSuccess;
    const SigmoidArgs a = sigmoid_args(
        out, ld_out, q, ldq, k, v, bias, talk, gate, ld_gate, scale, positions, nullptr, tables,
        nullptr, window, nbias, Hp, max_blocks, block_size, H, G, dim, vdim);
    const int hw = ceil_div_i(H, 8);
    if (!sigmoid_mfma_ok(a) || dim > 128 || vdim > 128 || hw > 4 || (H / G) % hw)
        return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size), grid = ceil_div_i(ntiles, 8) * 8;
#define GO(HW, A, B)                                                    \
    sigmoid_tiles_kernel<HW, A, B><<<grid, 512, 0, stream>>>(           \
        a, shift, cu, tile_seg, tile_off, ntiles)
#define SIZES(HW)                                  \
    {                                              \
        if (dim <= 64 && vdim <= 64) GO(HW, 2, 4); \
        else GO(HW, 4, 8);                         \
    }
    if (hw == 1) SIZES(1)
    else if (hw == 2) SIZES(2)
    else if (hw == 3) SIZES(3)
    else SIZES(4)
#undef SIZES
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}
