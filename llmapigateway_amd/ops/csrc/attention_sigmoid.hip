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

__device__ __forceinline__ bf16x8 masked(bool keep, const bf16x8& f) {
    uint4 v = *reinterpret_cast<const uint4*>(&f);
    if (!keep) v = (uint4){0, 0, 0, 0};
    return as_frag(v);
}

// columns past a row's end are read from its start: of keys they meet zeros of
// the query, of values they make outputs that nobody stores
__device__ __forceinline__ uint32_t col_of(int c, int width) { return c < width ? c : 0; }

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
// Keys, then values of 32 tokens and one key head at a time come by transfers
// through a ring of LDS buffers of the wave's own, RING - 1 ahead, 16-byte
// chunks (of values: pairs of them) XOR-swizzled by row on the source address.
// The waves' shares meet in LDS; several splits leave partial sums for
// sigmoid_combine_kernel.
// ---------------------------------------------------------------------------
template <int NB, int NDQ, int NDV>  // blocks of 16 heads; dim/32, vdim/16
__launch_bounds__(SA_THREADS)
__global__ void sigmoid_rows_kernel(SigmoidArgs a, int page_shift, int nsplit, float* part) {
    static_assert(NDV == 2 * NDQ, "rows of keys and values have one length in LDS");
    constexpr int LD = NDV * 16, CH = LD / 8, PER = 64 / CH;  // values, chunks; rows a transfer
    constexpr int RING = NDQ > 4 ? 2 : 4, AHEAD = (RING - 1) * (32 / PER);
    constexpr int NK = (NB + 1) / 2;
    __shared__ __align__(16) bf16 ring[4][RING][32 * LD];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int split = blockIdx.y, per = a.H / a.G;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pos = __builtin_amdgcn_readfirstlane((int)a.positions[t]);
    const int first = max(0, pos - a.window + 1), base = first & ~31;
    const int span = (pos + 1 - base + nsplit * 128 - 1) / (nsplit * 128) * 128;
    const int key_lo = base + split * span, key_hi = min(pos + 1, key_lo + span);
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int mask = (1 << page_shift) - 1, last = pos;
    const float scale2 = -a.scale * LOG2E;
    // this wave's steps of 32 keys: k_first, k_first + 128, ...
    const int k_first = key_lo + wave * 32;
    const int steps = k_first < key_hi ? (key_hi - k_first + 127) / 128 : 0;

    int key_head[NB];  // of this lane's head in each block
    bf16x8 qf[NB][NDQ], tf[NB][NK];
    f32x4 far[NB];     // biases beyond the table, of heads 16b + 4g + r
#pragma unroll
    for (int b = 0; b < NB; ++b) {
        const int h = b * 16 + r16;
        key_head[b] = h < a.H ? h / per : -1;
        const bf16* qr = (const bf16*)a.q + t * a.ldq + (size_t)min(h, a.H - 1) * a.dim;
#pragma unroll
        for (int c = 0; c < NDQ; ++c)
            qf[b][c] = masked(c * 32 + g * 8 < a.dim, *reinterpret_cast<const bf16x8*>(
                                                          qr + col_of(c * 32 + g * 8, a.dim)));
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
        far[b] = *reinterpret_cast<const f32x4*>(a.bias + (size_t)(a.nbias - 1) * a.Hp +
                                                 min(b * 16, a.Hp - 16) + g * 4);
    }
    f32x4 acc[NB][NDV];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[b][j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    // pages of 32 steps, two a step (past the end: of the last key)
    int pages = 0;
    auto load_pages = [&](int step) {
        const int k = k_first + (step + (lane >> 1)) * 128 + (lane & 1) * 16;
        pages = bt[min(k, last) >> page_shift];
    };
    // the next transfers: step, key head (G and up: values), ring buffer
    int p_step = 0, p_head = 0, p_buf = 0;
    auto issue = [&] {
        if (p_step >= steps) return false;
        if (p_head == 0 && (p_step & 31) == 0) load_pages(p_step);
        const bool is_v = p_head >= a.G;
        const int width = is_v ? a.vdim : a.dim, ld = a.G * width;
        const bf16* src = is_v ? (const bf16*)a.v + (size_t)(p_head - a.G) * a.vdim
                               : (const bf16*)a.k + (size_t)p_head * a.dim;
        const int k0 = k_first + p_step * 128, at = (p_step & 31) * 2;
        const bf16* b0 =
            src + ((size_t)__builtin_amdgcn_readlane(pages, at) << page_shift) * ld;
        const bf16* b1 =
            src + ((size_t)__builtin_amdgcn_readlane(pages, at + 1) << page_shift) * ld;
#pragma unroll
        for (int u = 0; u < 32 / PER; ++u) {
            const int o = u * PER + lane / CH, c = lane % CH;
            const int col = (is_v ? c ^ ((o & (NDV - 1) & 7) << 1) : c ^ (o & (CH - 1))) * 8;
            const int key = min(k0 + o, last);
            // (past the last key its own page: that of the first half, or both are one)
            const bf16* page = u * PER >= 16 && k0 + 16 <= last ? b1 : b0;
            dma16(page + (uint32_t)((key & mask) * ld + col_of(col, width)),
                  ring[wave][p_buf] + u * 512);
        }
        p_buf = (p_buf + 1) % RING;
        if (++p_head == 2 * a.G) {
            p_head = 0;
            ++p_step;
        }
        return true;
    };
    int buf = 0;
    // starts a transfer into the buffer that was read last; the next buffer to
    // read, once its transfer has landed
    auto next_buffer = [&] {
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if (issue()) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(AHEAD) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        const bf16* p = ring[wave][buf];
        buf = (buf + 1) % RING;
        return p;
    };
#pragma unroll
    for (int i = 0; i < RING - 1; ++i) issue();

    for (int step = 0; step < steps; ++step) {
        const int k0 = k_first + step * 128;
        f32x4 s[NB][2];
#pragma unroll
        for (int b = 0; b < NB; ++b) s[b][0] = s[b][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
        for (int gk = 0; gk < a.G; ++gk) {
            const bf16* kt = next_buffer();
            bf16x8 kf[2][NDQ];
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int c = 0; c < NDQ; ++c)
                    kf[u][c] = *reinterpret_cast<const bf16x8*>(
                        kt + (u * 16 + r16) * LD +
                        (((c * 4 + g) ^ ((u * 16 + r16) & (CH - 1))) << 3));
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                if (gk * per >= b * 16 + 16 || (gk + 1) * per <= b * 16) continue;
                const bool mine = key_head[b] == gk;
#pragma unroll
                for (int c = 0; c < NDQ; ++c) {
                    const bf16x8 qm = masked(mine, qf[b][c]);
#pragma unroll
                    for (int u = 0; u < 2; ++u) s[b][u] = mfma16(qm, kf[u][c], s[b][u]);
                }
            }
        }
        // weights of heads 16b + 4g + r, keys k0 + 16u + r16; their mix
        const bool near = pos - (k0 + 31) < a.nbias - 1;
        f32x4 m[NB][2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int key = k0 + u * 16 + r16;
            const bool seen = key >= first && key < key_hi;
            f32x4 bias[NB];
#pragma unroll
            for (int b = 0; b < NB; ++b) bias[b] = far[b];
            if (near) {
                const float* br = a.bias +
                                  (size_t)max(0, min(pos - key, a.nbias - 1)) * a.Hp + g * 4;
#pragma unroll
                for (int b = 0; b < NB; ++b)
                    bias[b] = *reinterpret_cast<const f32x4*>(br + min(b * 16, a.Hp - 16));
            }
            bf16x8 hi[NK], lo[NK];
#pragma unroll
            for (int kb = 0; kb < NK; ++kb) {
                float w[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int b = kb * 2 + j / 4, r = j % 4;
                    w[j] = b < NB && seen
                               ? __builtin_amdgcn_rcpf(
                                     1.f + __builtin_amdgcn_exp2f(
                                               fmaf(s[b < NB ? b : 0][u][r], scale2,
                                                    bias[b < NB ? b : 0][r] * -LOG2E)))
                               : 0.f;
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
        bf16x8 pf[NB];
#pragma unroll
        for (int b = 0; b < NB; ++b) {
            uint4 v;
            v.x = cvt_pk_bf16(m[b][0][0], m[b][0][1]);
            v.y = cvt_pk_bf16(m[b][0][2], m[b][0][3]);
            v.z = cvt_pk_bf16(m[b][1][0], m[b][1][1]);
            v.w = cvt_pk_bf16(m[b][1][2], m[b][1][3]);
            pf[b] = as_frag(v);
        }
        const int vr = g * 4 + (r16 >> 2), sw = vr & (NDV - 1) & 7;
        for (int gk = 0; gk < a.G; ++gk) {
            const bf16* r0 = next_buffer() + vr * LD + (r16 & 3) * 4;
            bf16x8 pm[NB];
#pragma unroll
            for (int b = 0; b < NB; ++b) pm[b] = masked(key_head[b] == gk, pf[b]);
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16* p = r0 + ((j ^ sw) << 4);
                const bf16x8 vf = tr_pair(p, p + 16 * LD);
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    if (gk * per >= b * 16 + 16 || (gk + 1) * per <= b * 16) continue;
                    acc[b][j] = mfma16(vf, pm[b], acc[b][j]);
                }
            }
        }
    }
    // the waves' shares, 16 heads at a time: [vdim][16 heads] in each wave's tile
    float* sh = reinterpret_cast<float*>(ring[wave][0]);
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
            for (int w = 0; w < 4; ++w) o += reinterpret_cast<const float*>(ring[w][0])[d * 16 + c];
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
// Keys go into the fragments, a step ahead; values by transfers into the wave's
// own LDS tile, 32-byte pairs of chunks XOR-swizzled by row on the source
// address. 16-byte chunks of weights are swizzled likewise.
//
// Queries and sums of 4 heads of 128 take 192 of a lane's 256 registers: the
// steps are kept apart (sched_barrier) so that their temporaries are, too.
// ---------------------------------------------------------------------------
template <int HW, int NDQ, int NDV>
__launch_bounds__(512)
__global__ void sigmoid_tiles_kernel(
    SigmoidArgs a, int page_shift, const int* __restrict__ cu,
    const int* __restrict__ tile_seg, const int* __restrict__ tile_off, int ntiles) {
    constexpr int LDW = 32 * 32 + 8;  // a row's weights
    constexpr int LDB = 36;           // biases of a distance
    constexpr bool FULL = HW * (NDQ + NDV) > 36;
    __shared__ __align__(16) bf16 w_lds[2][16][LDW], v_lds[8][32 * NDV * 16], t_lds[2][64 * 8];
    __shared__ __align__(16) float b_lds[47][LDB];
    // the last fragments of some heads' queries, where registers do not hold all
    constexpr int QL = FULL ? 2 : 0;
    __shared__ __align__(16) bf16 q_lds[8][QL > 0 ? QL : 1][64 * 8];
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
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    int lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    // what addresses are made of, made anew in every step: kept from one step
    // to the next they would fill the registers
    auto fresh_lane = [&] {
        lane = threadIdx.x & 63;
        asm volatile("" : "+v"(lane));
        r16 = lane & 15;
        g = lane >> 4;
    };
    const int h0 = wave * HW;
    const bool active = h0 < a.H;
    const int gk = active ? h0 / (a.H / a.G) : 0;
    const float scale2 = -a.scale * LOG2E;
    const bf16 *kp = (const bf16*)a.k + (size_t)gk * a.dim;
    const bf16 *vp = (const bf16*)a.v + (size_t)gk * a.vdim;
    const int ldk = a.G * a.dim, ldv = a.G * a.vdim;
    const int key_end = pos0 + nq, key_lo = max(0, pos0 - a.window + 1) & ~31;

    for (int e = tid; e < 2 * 16 * LDW / 8; e += 512)  // heads that are not there: finite
        reinterpret_cast<uint4*>(w_lds)[e] = (uint4){0, 0, 0, 0};
    if (wave < 2) {  // talk^T as fragments: column = head 16b + r16, k = head 8g + j
        const int h = wave * 16 + r16;
#pragma unroll
        for (int j = 0; j < 8; ++j)
            reinterpret_cast<uint16_t*>(t_lds[wave])[lane * 8 + j] =
                h < a.H && g * 8 + j < a.H
                    ? reinterpret_cast<const uint16_t*>(a.talk)[(size_t)h * a.H + g * 8 + j]
                    : 0;
    }
    bf16x8 qf[HW][NDQ];
    if (active) {
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            const bf16* qr = (const bf16*)a.q + (size_t)(q0 + min(r16, nq - 1)) * a.ldq +
                             (size_t)(h0 + i) * a.dim;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                qf[i][c] =
                    masked(c * 32 + g * 8 < a.dim, *reinterpret_cast<const bf16x8*>(
                                                       qr + col_of(c * 32 + g * 8, a.dim)));
                if (i < QL && c == NDQ - 1)
                    *reinterpret_cast<bf16x8*>(q_lds[wave][i < QL ? i : 0] + lane * 8) = qf[i][c];
            }
        }
    }
    f32x4 acc[HW][NDV];
#pragma unroll
    for (int i = 0; i < HW; ++i)
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    // the page of 16 keys from k0 (past the end: of the last key)
    auto page_of = [&](int k0) { return bt[min(k0, key_end - 1) >> page_shift]; };
    auto row_of = [&](int page) {
        return (size_t)__builtin_amdgcn_readfirstlane(page) << page_shift;
    };
    auto load_k = [&](bf16x8* kreg, int k0, size_t page) {
        const bf16* base = kp + page * ldk;
        const uint32_t at = (uint32_t)((min(k0 + r16, key_end - 1) & mask) * ldk);
#pragma unroll
        for (int c = 0; c < NDQ; ++c)
            kreg[c] =
                *reinterpret_cast<const bf16x8*>(base + at + col_of(c * 32 + g * 8, a.dim));
    };
    bf16* vt = v_lds[wave];
    auto stage_v = [&](int k0, size_t b0, size_t b1) {
        constexpr int PER = 64 / (NDV * 2);  // rows a transfer
#pragma unroll
        for (int u = 0; u < 32 / PER; ++u) {
            const int o = u * PER + lane / (NDV * 2), c = lane % (NDV * 2);
            const int d = ((((c >> 1) ^ (o & (NDV - 1) & 7)) << 1) | (c & 1)) * 8;
            const int key = min(k0 + o, key_end - 1);
            const bf16* base = vp + (u * PER >= 16 && k0 + 16 < key_end ? b1 : b0) * ldv;
            dma16(base + (uint32_t)((key & mask) * ldv + col_of(d, a.vdim)), vt + u * 512);
        }
    };
    // -log2(e) times the biases of distances dmin .. dmin + 46
    auto fill_bias = [&](int dmin) {
        for (int e = tid; e < 47 * 32; e += 512) {
            const int x = e >> 5, h = e & 31;
            if (h < a.Hp)
                b_lds[x][h] =
                    a.bias[(size_t)max(0, min(dmin + x, a.nbias - 1)) * a.Hp + h] * -LOG2E;
        }
    };
    f32x4 s[2][HW];
    auto scores = [&](const bf16x8* kreg, int u) {
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            s[u][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                const bool spilt = i < QL && c == NDQ - 1;
                const bf16x8 x = spilt ? *reinterpret_cast<const bf16x8*>(
                                             q_lds[wave][spilt ? i : 0] + lane * 8)
                                       : qf[i][c];
                s[u][i] = mfma16(x, kreg[c], s[u][i]);
            }
        }
    };
    // s to weights of rows 4g + r, key k0 + 16u + r16, in LDS
    auto weights = [&](int k0, int u) {
        const int o = u * 16 + r16;
        const bool edge = k0 + u * 16 + 15 > pos0 || k0 + u * 16 < pos0 + 16 - a.window;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = g * 4 + r;
            const float* bv = &b_lds[row + 31 - o][h0];
            float w[4];
#pragma unroll
            for (int i = 0; i < HW; ++i)
                w[i] = __builtin_amdgcn_rcpf(
                    1.f + __builtin_amdgcn_exp2f(fmaf(s[u][i][r], scale2, bv[i])));
            if (edge) {
                const int dist = pos0 + row - (k0 + o);
                const bool seen = dist >= 0 && dist < a.window;
#pragma unroll
                for (int i = 0; i < HW; ++i) w[i] = seen ? w[i] : 0.f;
            }
#pragma unroll
            for (int i = HW; i < 4; ++i) w[i] = 0.f;
            if (FULL) __builtin_amdgcn_sched_barrier(0);
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
    };
    bf16x8 k_lo[NDQ], k_hi[NDQ];
    int n0, n1;
    // keys of the step at k0, which lie in pages p0 and p1; pages of the next one
    auto load_step = [&](int k0, size_t p0, size_t p1) {
        n0 = page_of(k0 + 32);
        n1 = page_of(k0 + 48);
        load_k(k_lo, k0, p0);
        load_k(k_hi, k0 + 16, k0 + 16 < key_end ? p1 : p0);
    };
    size_t b0 = row_of(page_of(key_lo)), b1 = row_of(page_of(key_lo + 16));
    load_step(key_lo, b0, b1);
    fill_bias(pos0 - key_lo - 31);
    __syncthreads();

    for (int k0 = key_lo; k0 < key_end; k0 += 32) {
        // Transfers are waited for by count: what load_step loads must be in
        // before they start (this uses it), the next step's comes after them.
#pragma unroll
        for (int c = 0; c < NDQ; ++c) asm volatile("" : "+v"(k_lo[c]), "+v"(k_hi[c]));
        asm volatile("" : "+v"(n0), "+v"(n1));
        const size_t next0 = row_of(n0), next1 = row_of(n1);
        fresh_lane();
        __builtin_amdgcn_sched_barrier(0);
        if (active) stage_v(k0, b0, b1);
        scores(k_lo, 0);
        scores(k_hi, 1);
        __builtin_amdgcn_sched_barrier(0);
        b0 = next0;
        b1 = next1;
        if (!FULL) load_step(k0 + 32, b0, b1);
        lds_barrier();  // the last tile's mixed weights are read
        if (active) {
            weights(k0, 0);
            weights(k0, 1);
        }
        __builtin_amdgcn_sched_barrier(0);
        if (FULL) load_step(k0 + 32, b0, b1);
        const bool more = k0 + 32 < key_end;
        lds_barrier();  // all weights are there
        fresh_lane();
        // the next tile's biases, unless both are all beyond the table
        const int dmin = pos0 - k0 - 31;
        if (more && dmin - 32 < a.nbias - 1) fill_bias(dmin - 32);
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            if (FULL) __builtin_amdgcn_sched_barrier(0);
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
                    const bf16x8 tf = *reinterpret_cast<const bf16x8*>(t_lds[b] + lane * 8);
                    m[u][b] = mfma16(wh, tf, (f32x4){0.f, 0.f, 0.f, 0.f});
                    m[u][b] = mfma16(wl, tf, m[u][b]);
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
        __builtin_amdgcn_sched_barrier(0);
        // mixed weights and values are there; the 2 NDQ keys after them need not be
        asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(2 * NDQ) : "memory");
        if (active) {
            fresh_lane();
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
                if (FULL && j % 2 == 0) __builtin_amdgcn_sched_barrier(0);
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
            const uint2 zz = *reinterpret_cast<const uint2*>(z + col_of(d, a.vdim));
            if (d >= a.vdim) continue;
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

// sizes of the MFMA forms: up to 64 heads of 128, or 32 of 256; pages of a
// power of two, at least 16 tokens
static bool sigmoid_mfma_ok(const SigmoidArgs& a) {
    const int most = a.H <= 32 ? 256 : 128;
    return a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= most && a.vdim <= most && a.H <= 64 &&
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
#define SIZES(GO1, GO2, GO4)    \
    {                           \
        if (H <= 16) GO1;       \
        else if (H <= 32) GO2;  \
        else GO4;               \
    }
    if (dim <= 64 && vdim <= 64) SIZES(GO(1, 2, 4), GO(2, 2, 4), GO(4, 2, 4))
    else if (dim <= 128 && vdim <= 128) SIZES(GO(1, 4, 8), GO(2, 4, 8), GO(4, 4, 8))
    else SIZES(GO(1, 8, 16), GO(2, 8, 16), return hipErrorInvalidValue)
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
