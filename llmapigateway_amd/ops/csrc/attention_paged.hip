// Grouped-query attention over cache pages for gfx950: soft-capped scores
// cap*tanh(scale*q.k/cap), a sink per head in the softmax's denominator, an
// output gate per head. A page holds block_size tokens, a token's row the
// keys (or values) of all G key heads; query head h reads key head h/(H/G).
// A row at position p sees keys 0..p, all of which are in the pages.
//
// Three forms of one function: any size (fp32, or sizes that are no multiple
// of 8), rows (decoding and short portions: one query row a workgroup) and
// tiles (prompts: 64 or 128 query rows of a head a workgroup).
//
// The MFMA forms compute S^T = K Q^T and O^T = V^T P^T: a lane keeps one
// query column (a head of the group, or a row of the tile), so its softmax
// state is one scalar, and with the key order
//   k slot (g, j): key 4g+j for j < 4, 16+4g+(j-4) above (g = lane/16)
// two 16-key score fragments are the P^T operand as they stand.

#include "mfma.h"

#define PA_THREADS 256
#define PA_NEG (-1e30f)
#define LOG2E 1.4426950408889634f

struct PagedArgs {
    void* out;
    int64_t ld_out;                // row stride; heads are vdim apart
    const void* q;
    int64_t ldq;
    const void *k, *v;             // pages
    const float* sink;
    const void* gate;              // [rows, H], row stride ld_gate
    int64_t ld_gate;
    float scale, cap, out_scale;
    const int64_t* positions;
    const int *row_seg, *tables;
    const int* rows;               // nullable: which rows of the batch
    int max_blocks, block_size, H, G, dim, vdim;
};

__device__ __forceinline__ float gate_of(float z, float scale) {
    return scale / (1.f + expf(-z));
}

// ---------------------------------------------------------------------------
// Any size: one workgroup per (row, head), a key a thread for the scores, a
// value dimension a thread for the sums; the softmax starts from the sink.
// ---------------------------------------------------------------------------
template <typename T, int ND>
__launch_bounds__(PA_THREADS)
__global__ void paged_any_kernel(PagedArgs a) {
    extern __shared__ float lds[];  // [dim] query, [256] weights
    float* qs = lds;
    float* ps = lds + a.dim;
    __shared__ float red[8];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int h = blockIdx.y, g = h / (a.H / a.G), bs = a.block_size;
    const int n = (int)a.positions[t] + 1;
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const T *kp = (const T*)a.k, *vp = (const T*)a.v;
    for (int i = tid; i < a.dim; i += PA_THREADS)
        qs[i] = ldf((const T*)a.q + t * a.ldq + (size_t)h * a.dim + i);
    float m = a.sink[h], l = 1.f, acc[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[d] = 0.f;
    for (int k0 = 0; k0 < n; k0 += PA_THREADS) {
        __syncthreads();
        const int key = k0 + tid;
        float s = -INFINITY;
        if (key < n) {
            const T* kr = kp + (((size_t)bt[key / bs] * bs + key % bs) * a.G + g) * a.dim;
            s = 0.f;
            for (int i = 0; i < a.dim; ++i) s = fmaf(qs[i], ldf(kr + i), s);
            s = a.cap * tanhf(s * a.scale / a.cap);
        }
        float v = wave_reduce_max(s);
        if (lane == 0) red[wave] = v;
        __syncthreads();
        const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
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
        const int here = min(PA_THREADS, n - k0);
        for (int j = 0; j < here; ++j) {
            const int kj = k0 + j;
            const T* vr = vp + (((size_t)bt[kj / bs] * bs + kj % bs) * a.G + g) * a.vdim;
            const float pj = ps[j];
#pragma unroll
            for (int d = 0; d < ND; ++d) {
                const int i = tid + d * PA_THREADS;
                if (i < a.vdim) acc[d] = fmaf(pj, ldf(vr + i), acc[d]);
            }
        }
    }
    const float f = gate_of(ldf((const T*)a.gate + t * a.ld_gate + h), a.out_scale) / l;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
        const int i = tid + d * PA_THREADS;
        if (i < a.vdim) stf((T*)a.out + t * a.ld_out + (size_t)h * a.vdim + i, acc[d] * f);
    }
}

// e^(score - m) is taken as 2^(.), everything scaled by log2 e beforehand:
//   2^(c2 tanh(x) - m2), tanh(x) = 1 - 2 / (1 + e^(2x)), x = q.k * scale/cap
struct CapExp {
    float in, c2;
    __device__ __forceinline__ CapExp(float scale, float cap)
        : in(2.f * LOG2E * scale / cap), c2(cap * LOG2E) {}
    __device__ __forceinline__ float score(float qk) const {
        const float e = __builtin_amdgcn_exp2f(qk * in);
        return fmaf(-2.f * c2, __builtin_amdgcn_rcpf(1.f + e), c2);
    }
};

__device__ __forceinline__ bf16x8 weights_frag(const float* lo, const float* hi) {
    uint4 v;
    v.x = cvt_pk_bf16(lo[0], lo[1]);
    v.y = cvt_pk_bf16(lo[2], lo[3]);
    v.z = cvt_pk_bf16(hi[0], hi[1]);
    v.w = cvt_pk_bf16(hi[2], hi[3]);
    return as_frag(v);
}

// ---------------------------------------------------------------------------
// Rows: one workgroup per (row, 16 query heads of a key head, split of the
// keys). Its 4 waves take tiles of 32 keys in turn, each with its own softmax
// state, without a barrier: keys go from global memory into the fragments,
// values through the wave's LDS tile (read back transposed), both loaded a
// tile ahead. The waves' shares meet in LDS at the end; several splits leave
// partials for paged_combine_kernel.
// ONLINE: running maximum; otherwise the maximum is fixed at max(cap, sink),
// which no score exceeds and, for caps up to 30, none is too far below.
// ---------------------------------------------------------------------------
template <int NDQ, int NDV, bool ONLINE>
__launch_bounds__(PA_THREADS)
__global__ void paged_rows_kernel(
    PagedArgs a, int page_shift, int nsplit, float* part_acc, float* part_ml) {
    constexpr int LDV = NDV * 16 + 8, TILE = 32 * LDV;
    constexpr int KV = 2 * NDQ, VV = NDV;  // 16-byte loads a lane and tile
    __shared__ __align__(16) bf16 v_lds[4][TILE];
    __shared__ float m_lds[4][16], l_lds[4][16];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int per = a.H / a.G, nht = (per + 15) / 16;
    const int g_kv = blockIdx.y / nht, h0 = blockIdx.y % nht * 16, split = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int n = (int)a.positions[t] + 1;
    const int span = (n + nsplit * 128 - 1) / (nsplit * 128) * 128;
    const int key_lo = split * span, key_hi = min(n, key_lo + span);
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const bf16 *kp = (const bf16*)a.k + (size_t)g_kv * a.dim;
    const bf16 *vp = (const bf16*)a.v + (size_t)g_kv * a.vdim;
    const int head = min(h0 + r16, per - 1);  // this lane's column
    const int h = g_kv * per + head;
    const CapExp ce(a.scale, a.cap);

    bf16x8 qf[NDQ];
    {
        const bf16* qr = (const bf16*)a.q + t * a.ldq + (size_t)h * a.dim;
#pragma unroll
        for (int c = 0; c < NDQ; ++c) {
            uint4 x = {0, 0, 0, 0};
            if (c * 32 + g * 8 < a.dim) x = *reinterpret_cast<const uint4*>(qr + c * 32 + g * 8);
            qf[c] = as_frag(x);
        }
    }
    float m = ONLINE ? PA_NEG : fmaxf(a.cap, a.sink[h]) * LOG2E, l = 0.f;
    f32x4 acc[NDV];
#pragma unroll
    for (int j = 0; j < NDV; ++j) acc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    uint4 kreg[KV], vreg[VV];
    // row of key k0 + o (o < 32) in the pages; past the end any row
    auto load_tile = [&](int k0) {
        const int last = key_hi - 1;
        const size_t b0 = (size_t)bt[k0 >> page_shift] << page_shift;
        const size_t b1 = (size_t)bt[min(k0 + 16, last) >> page_shift] << page_shift;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int key = min(k0 + u * 16 + r16, last);
            const size_t row = (u && k0 + 16 <= last ? b1 : b0) + (key & mask);
            const bf16* p = kp + row * a.G * a.dim;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                kreg[u * NDQ + c] = (uint4){0, 0, 0, 0};
                if (c * 32 + g * 8 < a.dim)
                    kreg[u * NDQ + c] = *reinterpret_cast<const uint4*>(p + c * 32 + g * 8);
            }
        }
#pragma unroll
        for (int u = 0; u < VV; ++u) {
            const int e = lane + u * 64, o = e / (NDV * 2), d = e % (NDV * 2) * 8;
            const int key = min(k0 + o, last);
            const size_t row = (key >= k0 + 16 ? b1 : b0) + (key & mask);
            vreg[u] = (uint4){0, 0, 0, 0};
            if (d < a.vdim)
                vreg[u] = *reinterpret_cast<const uint4*>(vp + row * a.G * a.vdim + d);
        }
    };
    bf16* vt = v_lds[wave];
    int k0 = key_lo + wave * 32;
    if (k0 < key_hi) load_tile(k0);
    for (; k0 < key_hi; k0 += 128) {
        f32x4 s[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            s[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < NDQ; ++c) s[u] = mfma16(as_frag(kreg[u * NDQ + c]), qf[c], s[u]);
        }
#pragma unroll
        for (int u = 0; u < VV; ++u) {
            const int e = lane + u * 64;
            *reinterpret_cast<uint4*>(vt + e / (NDV * 2) * LDV + e % (NDV * 2) * 8) = vreg[u];
        }
        if (k0 + 128 < key_hi) load_tile(k0 + 128);
        float p[2][4], mx = PA_NEG;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[u][r] = k0 + u * 16 + g * 4 + r < key_hi ? ce.score(s[u][r]) : PA_NEG;
                mx = fmaxf(mx, p[u][r]);
            }
        if (ONLINE) {
            mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE_SIZE));
            mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE_SIZE));
            const float m_new = fmaxf(m, mx), f = __builtin_amdgcn_exp2f(m - m_new);
            m = m_new;
            l *= f;
#pragma unroll
            for (int j = 0; j < NDV; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) acc[j][r] *= f;
        }
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[u][r] = __builtin_amdgcn_exp2f(p[u][r] - m);
                l += p[u][r];
            }
        const bf16x8 pf = weights_frag(p[0], p[1]);
        const bf16* r0 = vt + (g * 4 + (r16 >> 2)) * LDV + (r16 & 3) * 4;
#pragma unroll
        for (int j = 0; j < NDV; ++j)
            acc[j] = mfma16(tr_pair(r0 + j * 16, r0 + 16 * LDV + j * 16), pf, acc[j]);
    }
    // the waves' shares: acc as [vdim][16 heads] in each wave's tile
    l += __shfl_xor(l, 16, WAVE_SIZE);
    l += __shfl_xor(l, 32, WAVE_SIZE);
    if (g == 0) {
        m_lds[wave][r16] = m;
        l_lds[wave][r16] = l;
    }
    float* sh = reinterpret_cast<float*>(vt);
#pragma unroll
    for (int j = 0; j < NDV; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) sh[(j * 16 + g * 4 + r) * 16 + r16] = acc[j][r];
    __syncthreads();
    for (int e = tid; e < 16 * a.vdim; e += PA_THREADS) {
        const int c = e / a.vdim, d = e % a.vdim;
        if (h0 + c >= per) break;
        const int hh = g_kv * per + h0 + c;
        float M = fmaxf(fmaxf(m_lds[0][c], m_lds[1][c]), fmaxf(m_lds[2][c], m_lds[3][c]));
        const float sk = a.sink[hh] * LOG2E;
        if (nsplit == 1) M = fmaxf(M, sk);
        float L = nsplit == 1 ? __builtin_amdgcn_exp2f(sk - M) : 0.f, o = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float f = __builtin_amdgcn_exp2f(m_lds[w][c] - M);
            L = fmaf(l_lds[w][c], f, L);
            o = fmaf(reinterpret_cast<const float*>(v_lds[w])[d * 16 + c], f, o);
        }
        if (nsplit == 1) {
            const float z = ldf((const bf16*)a.gate + t * a.ld_gate + hh);
            stf((bf16*)a.out + t * a.ld_out + (size_t)hh * a.vdim + d,
                o * gate_of(z, a.out_scale) / L);
        } else {
            const size_t pb = ((size_t)blockIdx.x * a.H + hh) * nsplit + split;
            part_acc[pb * a.vdim + d] = o;
            if (d == 0) {
                part_ml[pb * 2] = M;
                part_ml[pb * 2 + 1] = L;
            }
        }
    }
}

// one workgroup per (row, head)
__global__ void paged_combine_kernel(
    PagedArgs a, int nsplit, const float* __restrict__ part_acc,
    const float* __restrict__ part_ml) {
    const size_t i = blockIdx.x / a.H, t = a.rows ? a.rows[i] : i;
    const int h = blockIdx.x % a.H;
    const float* ml = part_ml + (size_t)blockIdx.x * nsplit * 2;
    const float sk = a.sink[h] * LOG2E;
    float M = sk;
    for (int s = 0; s < nsplit; ++s) M = fmaxf(M, ml[2 * s]);
    float L = __builtin_amdgcn_exp2f(sk - M);
    for (int s = 0; s < nsplit; ++s)
        L = fmaf(ml[2 * s + 1], __builtin_amdgcn_exp2f(ml[2 * s] - M), L);
    const float f = gate_of(ldf((const bf16*)a.gate + t * a.ld_gate + h), a.out_scale) / L;
    for (int d = threadIdx.x; d < a.vdim; d += blockDim.x) {
        float o = 0.f;
        for (int s = 0; s < nsplit; ++s)
            o = fmaf(part_acc[((size_t)blockIdx.x * nsplit + s) * a.vdim + d],
                     __builtin_amdgcn_exp2f(ml[2 * s] - M), o);
        stf((bf16*)a.out + t * a.ld_out + (size_t)h * a.vdim + d, o * f);
    }
}

// ---------------------------------------------------------------------------
// Tiles: one workgroup per (64*MR rows of a segment, head), 16*MR rows a
// wave; tiles of 64 keys, loaded to registers a tile ahead and staged in LDS.
// The head varies fastest over the grid, so the heads that share keys run
// together.
// ---------------------------------------------------------------------------
template <int NDQ, int NDV, int MR, bool ONLINE>
__launch_bounds__(PA_THREADS)
__global__ void paged_tiles_kernel(
    PagedArgs a, int page_shift, const int* __restrict__ cu,
    const int* __restrict__ tile_seg, const int* __restrict__ tile_off) {
    constexpr int LDQ = NDQ * 32 + 8, LDV = NDV * 16 + 8;
    constexpr int KV = NDQ, VV = NDV / 2;
    __shared__ __align__(16) bf16 k_lds[64 * LDQ], v_lds[64 * LDV];
    const int h = blockIdx.x % a.H, tile = blockIdx.x / a.H;
    const int seg = tile_seg[tile], off = tile_off[tile];
    const int q0 = cu[seg], nq = cu[seg + 1] - q0;
    const int ctx = (int)a.positions[q0];  // position of the segment's first row
    const int* bt = a.tables + (size_t)seg * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const int g_kv = h / (a.H / a.G);
    const bf16 *kp = (const bf16*)a.k + (size_t)g_kv * a.dim;
    const bf16 *vp = (const bf16*)a.v + (size_t)g_kv * a.vdim;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const int wrow0 = off + wave * 16 * MR;
    const CapExp ce(a.scale, a.cap);

    bf16x8 qf[MR][NDQ];
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        const int row = min(wrow0 + i * 16 + r16, nq - 1);
        const bf16* qr = (const bf16*)a.q + (size_t)(q0 + row) * a.ldq + (size_t)h * a.dim;
#pragma unroll
        for (int c = 0; c < NDQ; ++c) {
            uint4 x = {0, 0, 0, 0};
            if (c * 32 + g * 8 < a.dim) x = *reinterpret_cast<const uint4*>(qr + c * 32 + g * 8);
            qf[i][c] = as_frag(x);
        }
    }
    const float sk = a.sink[h] * LOG2E;
    float m[MR], l[MR];
    f32x4 acc[MR][NDV];
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        m[i] = ONLINE ? sk : fmaxf(a.cap * LOG2E, sk);
        l[i] = g == 0 ? __builtin_amdgcn_exp2f(sk - m[i]) : 0.f;  // the sink, once a row
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
    const int key_end = ctx + min(nq, off + 64 * MR);  // keys any row here sees
    uint4 kreg[KV], vreg[VV];
    auto load_tile = [&](int k0) {
        auto row_of = [&](int key) {
            key = min(key, key_end - 1);
            return ((size_t)bt[key >> page_shift] << page_shift) + (key & mask);
        };
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * 256, d = e % (NDQ * 4) * 8;
            kreg[c] = (uint4){0, 0, 0, 0};
            if (d < a.dim)
                kreg[c] = *reinterpret_cast<const uint4*>(
                    kp + row_of(k0 + e / (NDQ * 4)) * a.G * a.dim + d);
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * 256, d = e % (NDV * 2) * 8;
            vreg[c] = (uint4){0, 0, 0, 0};
            if (d < a.vdim)
                vreg[c] = *reinterpret_cast<const uint4*>(
                    vp + row_of(k0 + e / (NDV * 2)) * a.G * a.vdim + d);
        }
    };
    load_tile(0);
    for (int k0 = 0; k0 < key_end; k0 += 64) {
        __syncthreads();
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * 256;
            *reinterpret_cast<uint4*>(k_lds + e / (NDQ * 4) * LDQ + e % (NDQ * 4) * 8) = kreg[c];
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * 256;
            *reinterpret_cast<uint4*>(v_lds + e / (NDV * 2) * LDV + e % (NDV * 2) * 8) = vreg[c];
        }
        __syncthreads();
        if (k0 + 64 < key_end) load_tile(k0 + 64);
        if (k0 > ctx + wrow0 + 16 * MR - 1) continue;  // all masked for this wave
        f32x4 s[MR][4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
#pragma unroll
            for (int i = 0; i < MR; ++i) s[i][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                const bf16x8 kf = *reinterpret_cast<const bf16x8*>(
                    k_lds + (u * 16 + r16) * LDQ + c * 32 + g * 8);
#pragma unroll
                for (int i = 0; i < MR; ++i) s[i][u] = mfma16(kf, qf[i][c], s[i][u]);
            }
        }
        const bool edge = k0 + 63 > ctx + wrow0;  // some row does not see all keys
        bf16x8 pf[MR][2];
#pragma unroll
        for (int i = 0; i < MR; ++i) {
            const int pos = ctx + wrow0 + i * 16 + r16;
            float p[4][4], mx = PA_NEG;
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    p[u][r] = ce.score(s[i][u][r]);
                    if (edge && k0 + u * 16 + g * 4 + r > pos) p[u][r] = PA_NEG;
                    mx = fmaxf(mx, p[u][r]);
                }
            if (ONLINE) {
                mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE_SIZE));
                mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE_SIZE));
                const float m_new = fmaxf(m[i], mx), f = __builtin_amdgcn_exp2f(m[i] - m_new);
                m[i] = m_new;
                l[i] *= f;
#pragma unroll
                for (int j = 0; j < NDV; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r) acc[i][j][r] *= f;
            }
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    p[u][r] = __builtin_amdgcn_exp2f(p[u][r] - m[i]);
                    l[i] += p[u][r];
                }
            pf[i][0] = weights_frag(p[0], p[1]);
            pf[i][1] = weights_frag(p[2], p[3]);
        }
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            const bf16* r0 = v_lds + (c * 32 + g * 4 + (r16 >> 2)) * LDV + (r16 & 3) * 4;
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16x8 vf = tr_pair(r0 + j * 16, r0 + 16 * LDV + j * 16);
#pragma unroll
                for (int i = 0; i < MR; ++i) acc[i][j] = mfma16(vf, pf[i][c], acc[i][j]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        float L = l[i];
        L += __shfl_xor(L, 16, WAVE_SIZE);
        L += __shfl_xor(L, 32, WAVE_SIZE);
        const int row = wrow0 + i * 16 + r16;
        if (row >= nq) continue;
        const size_t t = q0 + row;
        const float f = gate_of(ldf((const bf16*)a.gate + t * a.ld_gate + h), a.out_scale) / L;
        bf16* o = (bf16*)a.out + t * a.ld_out + (size_t)h * a.vdim;
#pragma unroll
        for (int j = 0; j < NDV; ++j) {
            const int d = j * 16 + g * 4;  // vdim is a multiple of 8
            if (d < a.vdim)
                *reinterpret_cast<uint2*>(o + d) = make_uint2(
                    cvt_pk_bf16(acc[i][j][0] * f, acc[i][j][1] * f),
                    cvt_pk_bf16(acc[i][j][2] * f, acc[i][j][3] * f));
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
template <typename T>
static hipError_t paged_any(const PagedArgs& a, int nrows, hipStream_t stream) {
    const size_t lds = (a.dim + PA_THREADS) * sizeof(float);
    if (lds > 48 * 1024) return hipErrorInvalidValue;
    const dim3 grid(nrows, a.H);
    if (a.vdim <= 256) paged_any_kernel<T, 1><<<grid, PA_THREADS, lds, stream>>>(a);
    else if (a.vdim <= 1024) paged_any_kernel<T, 4><<<grid, PA_THREADS, lds, stream>>>(a);
    else return hipErrorInvalidValue;
    HIP_CHECK_LAST();
    return hipSuccess;
}

// sizes of the MFMA forms: multiples of 8 up to 256, power-of-two pages of at
// least 16 tokens
static bool paged_mfma_ok(const PagedArgs& a) {
    return a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 && a.vdim <= 256 &&
           a.block_size >= 16 && (a.block_size & (a.block_size - 1)) == 0;
}
#define PAGED_SIZES(GO)                               \
    if (a.dim <= 64 && a.vdim <= 64) GO(2, 4)         \
    else if (a.dim <= 128 && a.vdim <= 128) GO(4, 8)  \
    else GO(8, 16)

static PagedArgs paged_args(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* sink, const void* gate, int64_t ld_gate, float scale, float cap,
    float out_scale, const int64_t* positions, const int* row_seg, const int* tables,
    const int* rows, int max_blocks, int block_size, int H, int G, int dim, int vdim) {
    return PagedArgs{out, ld_out, q, ldq, k, v, sink, gate, ld_gate, scale, cap, out_scale,
                     positions, row_seg, tables, rows, max_blocks, block_size, H, G, dim, vdim};
}

// nsplit 0: the any-size form
extern "C" hipError_t launch_paged_rows(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* sink, const void* gate, int64_t ld_gate, float scale, float cap,
    float out_scale, const int64_t* positions, const int* row_seg, const int* tables,
    const int* rows, int max_blocks, int block_size, int H, int G, int dim, int vdim, int nrows,
    int nsplit, float* part_acc, float* part_ml, int f32, hipStream_t stream) {
    if (nrows <= 0) return hipSuccess;
    const PagedArgs a =
        paged_args(out, ld_out, q, ldq, k, v, sink, gate, ld_gate, scale, cap, out_scale,
                   positions, row_seg, tables, rows, max_blocks, block_size, H, G, dim, vdim);
    if (nsplit == 0) return f32 ? paged_any<float>(a, nrows, stream) : paged_any<bf16>(a, nrows, stream);
    if (f32 || !paged_mfma_ok(a) || (nsplit > 1 && (!part_acc || !part_ml)))
        return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size);
    const dim3 grid(nrows, G * ceil_div_i(H / G, 16), nsplit);
#define GO(A, B)                                                                         \
    {                                                                                    \
        if (cap > 30.f)                                                                  \
            paged_rows_kernel<A, B, true><<<grid, PA_THREADS, 0, stream>>>(              \
                a, shift, nsplit, part_acc, part_ml);                                    \
        else                                                                             \
            paged_rows_kernel<A, B, false><<<grid, PA_THREADS, 0, stream>>>(             \
                a, shift, nsplit, part_acc, part_ml);                                    \
    }
    PAGED_SIZES(GO)
#undef GO
    HIP_CHECK_LAST();
    if (nsplit > 1) {
        const int th = vdim <= 64 ? 64 : 128;
        paged_combine_kernel<<<nrows * H, th, 0, stream>>>(
            a, nsplit, part_acc, part_ml);
        HIP_CHECK_LAST();
    }
    return hipSuccess;
}

extern "C" hipError_t launch_paged_tiles(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    const float* sink, const void* gate, int64_t ld_gate, float scale, float cap,
    float out_scale, const int64_t* positions, const int* tables, int max_blocks,
    int block_size, int H, int G, int dim, int vdim, const int* cu, const int* tile_seg,
    const int* tile_off, int ntiles, int tile_rows, hipStream_t stream) {
    if (ntiles <= 0) return hipSuccess;
    const PagedArgs a =
        paged_args(out, ld_out, q, ldq, k, v, sink, gate, ld_gate, scale, cap, out_scale,
                   positions, nullptr, tables, nullptr, max_blocks, block_size, H, G, dim, vdim);
    if (!paged_mfma_ok(a) || (tile_rows != 64 && tile_rows != 128)) return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size);
#define GO2(A, B, M)                                                                     \
    {                                                                                    \
        if (cap > 30.f)                                                                  \
            paged_tiles_kernel<A, B, M, true><<<ntiles * H, PA_THREADS, 0, stream>>>(    \
                a, shift, cu, tile_seg, tile_off);                                       \
        else                                                                             \
            paged_tiles_kernel<A, B, M, false><<<ntiles * H, PA_THREADS, 0, stream>>>(   \
                a, shift, cu, tile_seg, tile_off);                                       \
    }
#define GO(A, B)                                                                         \
    {                                                                                    \
        if (tile_rows == 128) GO2(A, B, 2)                                               \
        else GO2(A, B, 1)                                                                \
    }
    PAGED_SIZES(GO)
#undef GO
#undef GO2
    HIP_CHECK_LAST();
    return hipSuccess;
}
