// Latent attention for gfx950: softmax attention with a sink over cached
// latent rows [c (rank) | rotated key part | zero pad].
//
// Folded form: queries are already in the latent space, one cached row is
// key and value of every head. Unfolded form: per-head keys and values.

#include "lds_dma.h"
#include "mfma.h"

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

// ---------------------------------------------------------------------------
// Folded form on MFMA (bf16). One workgroup: one row, 16*HT heads, one split
// of the row's keys, 4*HT waves, tiles of 64 keys. Cached rows stream through
// two LDS buffers by global_load_lds (a tile in flight behind the one in
// use); 16-byte chunks are XOR-swizzled by row, on the source address, so
// that row-wise and transposing reads both spread over the banks.
//   scores: wave (ht, kq) takes 16 heads x 16 keys;
//   sums: a wave takes its share of the latent dimensions for all heads.
// One split writes the output (softmax started from the sink); several write
// partials that latent_combine_kernel merges with the sink. Splits divide
// the row's own key count, so a launch of fixed shape (captured graphs)
// balances at every context length.
// ---------------------------------------------------------------------------
#define LF_KT 64
#define LF_PAGES 512  // page ids held in LDS (a tile has at most 64)
#define LA_NEG (-1e30f)

// NKC: 32-wide chunks that cover a cached row (even); RT: 16-wide tiles that
// cover the rank (a multiple of 4, at most 2*NKC)
template <int NKC, int RT, int HT>
__launch_bounds__(256 * HT)
__global__ void latent_folded_mfma_kernel(
    bf16* __restrict__ out, float* __restrict__ part_acc, float* __restrict__ part_ml,
    const bf16* __restrict__ q, const bf16* __restrict__ latent,
    const float* __restrict__ sink, float scale, const int64_t* __restrict__ positions,
    const int* __restrict__ row_seg, const int* __restrict__ tables, int max_blocks,
    int page_shift, int H, int rank, int row_w, int nsplit) {
    constexpr int WAVES = 4 * HT;
    constexpr int RC = NKC * 4;                   // 16-byte chunks per LDS row
    constexpr int TILE = LF_KT * RC * 8;          // elements per buffer
    constexpr int NI = RC / WAVES;                // transfers per wave and tile
    constexpr int NT = (RT + WAVES - 1) / WAVES;  // rank tiles per wave
    __shared__ __align__(16) bf16 k_lds[2 * TILE];
    __shared__ bf16 p_lds[16 * HT][LF_KT + 8];
    __shared__ float mx_lds[2][4][16 * HT];
    __shared__ float l_lds[4][16 * HT];
    __shared__ int page_lds[LF_PAGES];
    const size_t t = blockIdx.x;
    const int h0 = blockIdx.y * 16 * HT, split = blockIdx.z;
    const int n = (int)positions[t] + 1;
    const int span = (n + nsplit * LF_KT - 1) / (nsplit * LF_KT) * LF_KT;
    const int key_lo = split * span, key_hi = min(n, key_lo + span);
    const int* bt = tables + (size_t)row_seg[t] * max_blocks;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int ht = wave >> 2, kq = wave & 3;
    const int r16 = lane & 15, g = lane >> 4;

    // page ids from the page of key k0 on
    int page0 = 0;
    auto load_pages = [&](int k0) {
        page0 = k0 >> page_shift;
        const int pages = ((key_hi - 1) >> page_shift) + 1 - page0;
        for (int i = tid; i < min(pages, LF_PAGES); i += 64 * WAVES) page_lds[i] = bt[page0 + i];
        __syncthreads();
    };
    // LDS chunk e of a tile holds chunk (e % RC) ^ swizzle(row) of row e / RC.
    // Past the last key: any row, its weight is 0; past the row's end: any
    // column, the queries are 0 there.
    auto stage = [&](int k0, int buf) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int e0 = (wave * NI + i) * 64, e = e0 + lane;
            const int row = e / RC, c = (e % RC) ^ ((row >> 1) & 7);
            const int key = min(k0 + row, key_hi - 1);
            const uint32_t at =
                ((uint32_t)page_lds[(key >> page_shift) - page0] << page_shift) +
                (key & ((1 << page_shift) - 1));
            dma16(latent + (size_t)at * row_w + (c * 8 < row_w ? c * 8 : 0),
                  k_lds + buf * TILE + e0 * 8);
        }
    };
    if (key_lo < key_hi) {
        load_pages(key_lo);
        stage(key_lo, 0);
    }

    bf16x8 qf[NKC];
    {
        const bf16* qr = q + (t * H + min(h0 + ht * 16 + r16, H - 1)) * row_w;
#pragma unroll
        for (int c = 0; c < NKC; ++c) {
            const bool in = c * 32 + g * 8 < row_w;
            uint4 v = *reinterpret_cast<const uint4*>(qr + (in ? c * 32 + g * 8 : 0));
            if (!in) v = (uint4){0, 0, 0, 0};
            qf[c] = as_frag(v);
        }
    }
    float m[HT][4], l[4];
    f32x4 acc[HT][NT];
#pragma unroll
    for (int i = 0; i < HT; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
            m[i][r] = nsplit == 1 ? sink[min(h0 + i * 16 + g * 4 + r, H - 1)] : LA_NEG;
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) l[r] = nsplit == 1 && kq == 0 && r16 == 0 ? 1.f : 0.f;

    dma_barrier();
    int buf = 0;
#pragma unroll 1
    for (int k0 = key_lo; k0 < key_hi; k0 += LF_KT, buf ^= 1) {
        if (k0 + LF_KT < key_hi) {
            if (((min(k0 + 2 * LF_KT, key_hi) - 1) >> page_shift) - page0 >= LF_PAGES)
                load_pages(k0 + LF_KT);
            stage(k0 + LF_KT, buf ^ 1);
        }
        const bf16* kt = k_lds + buf * TILE;
        f32x4 s = (f32x4){0.f, 0.f, 0.f, 0.f};
        {
            const int row = kq * 16 + r16, sw = (row >> 1) & 7;
            const bf16* even = kt + (row * RC + (g ^ sw)) * 8;
            const bf16* odd = kt + (row * RC + ((4 + g) ^ sw)) * 8;
#pragma unroll
            for (int c = 0; c < NKC; ++c)
                s = mfma16(qf[c], *reinterpret_cast<const bf16x8*>(
                                      (c & 1 ? odd : even) + (c >> 1) * 64), s);
        }
        const bool in = k0 + kq * 16 + r16 < key_hi;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            s[r] = in ? s[r] * scale : LA_NEG;
            const float v = row16_max(s[r]);
            if (r16 == 0) mx_lds[buf][kq][ht * 16 + g * 4 + r] = v;
        }
        lds_barrier();
#pragma unroll
        for (int i = 0; i < HT; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = i * 16 + g * 4 + r;
                const float m_new = fmaxf(
                    m[i][r], fmaxf(fmaxf(mx_lds[buf][0][row], mx_lds[buf][1][row]),
                                   fmaxf(mx_lds[buf][2][row], mx_lds[buf][3][row])));
                const float f = __expf(m[i][r] - m_new);
                m[i][r] = m_new;
                if (i == ht) {
                    const float p = in ? __expf(s[r] - m_new) : 0.f;
                    l[r] = l[r] * f + p;
                    p_lds[row][kq * 16 + r16] = f2bf(p);
                }
#pragma unroll
                for (int j = 0; j < NT; ++j) acc[i][j][r] *= f;
            }
        lds_barrier();
#pragma unroll
        for (int c = 0; c < LF_KT / 32; ++c) {
            bf16x8 pf[HT];
#pragma unroll
            for (int i = 0; i < HT; ++i)
                pf[i] = *reinterpret_cast<const bf16x8*>(
                    &p_lds[i * 16 + r16][c * 32 + g * 8]);
            // transposing reads of rows k, k+4 (see tr_frag), swizzled
            const int row = c * 32 + g * 8 + (r16 >> 2);
            const int sw0 = (row >> 1) & 7, sw1 = ((row + 4) >> 1) & 7;
            const bf16* r0 = kt + row * RC * 8 + (r16 & 1) * 4;
#pragma unroll
            for (int j = 0; j < NT; ++j) {
                // the last wave's tiles may lie past RT: repeat one, unused
                const int tile = NT * WAVES == RT ? wave * NT + j : min(wave * NT + j, RT - 1);
                const int ch = tile * 2 + ((r16 >> 1) & 1);
                const bf16x8 vf =
                    tr_pair(r0 + (ch ^ sw0) * 8, r0 + 4 * RC * 8 + (ch ^ sw1) * 8);
#pragma unroll
                for (int i = 0; i < HT; ++i) acc[i][j] = mfma16(pf[i], vf, acc[i][j]);
            }
        }
        dma_barrier();
    }
    // the waves' shares of the denominator
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const float v = row16_sum(l[r]);
        if (r16 == 0) l_lds[kq][ht * 16 + g * 4 + r] = v;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < HT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = i * 16 + g * 4 + r, h = h0 + row;
            if (h >= H) continue;
            const float lt = l_lds[0][row] + l_lds[1][row] + l_lds[2][row] + l_lds[3][row];
            const size_t th = t * H + h, pb = th * nsplit + split;
            const float inv = 1.f / lt;
#pragma unroll
            for (int j = 0; j < NT; ++j) {
                const int d = (wave * NT + j) * 16 + r16;
                if (d >= rank) continue;
                if (nsplit == 1) stf(out + th * rank + d, acc[i][j][r] * inv);
                else part_acc[pb * rank + d] = acc[i][j][r];
            }
            if (nsplit > 1 && wave == 0 && r16 == 0) {
                part_ml[pb * 2] = m[i][r];
                part_ml[pb * 2 + 1] = lt;
            }
        }
}

// one workgroup per (row, head); a thread owns 4 latent dimensions when the
// rank allows
__global__ void latent_combine_kernel(
    bf16* __restrict__ out, const float* __restrict__ part_acc,
    const float* __restrict__ part_ml, const float* __restrict__ sink, int H, int rank,
    int nsplit) {
    const size_t th = blockIdx.x;
    const float sk = sink[th % H];
    const float2* ml = reinterpret_cast<const float2*>(part_ml) + th * nsplit;
    float M = sk;
    for (int s = 0; s < nsplit; ++s) M = fmaxf(M, ml[s].x);
    float den = __expf(sk - M);
    for (int s = 0; s < nsplit; ++s) den += ml[s].y * __expf(ml[s].x - M);
    const float inv = 1.f / den;
    const float* pa = part_acc + th * nsplit * rank;
    if (rank % 4 == 0) {
        for (int d = threadIdx.x * 4; d < rank; d += blockDim.x * 4) {
            float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int s = 0; s < nsplit; ++s) {
                const float w = __expf(ml[s].x - M) * inv;
                const float4 v = *reinterpret_cast<const float4*>(pa + (size_t)s * rank + d);
                a.x = fmaf(v.x, w, a.x);
                a.y = fmaf(v.y, w, a.y);
                a.z = fmaf(v.z, w, a.z);
                a.w = fmaf(v.w, w, a.w);
            }
            *reinterpret_cast<uint2*>(out + th * rank + d) =
                make_uint2(pack2(a.x, a.y), pack2(a.z, a.w));
        }
        return;
    }
    for (int d = threadIdx.x; d < rank; d += blockDim.x) {
        float a = 0.f;
        for (int s = 0; s < nsplit; ++s)
            a += pa[(size_t)s * rank + d] * __expf(ml[s].x - M);
        stf(out + th * rank + d, a * inv);
    }
}

template <int NKC, int RT>
static void folded_go(
    bf16* out, float* part_acc, float* part_ml, const bf16* q, const bf16* latent,
    const float* sink, float scale, const int64_t* positions, const int* row_seg,
    const int* tables, int rows, int H, int rank, int row_w, int page_shift, int max_blocks,
    int nsplit, hipStream_t stream) {
    if (H > 16)
        latent_folded_mfma_kernel<NKC, RT, 2>
            <<<dim3(rows, ceil_div_i(H, 32), nsplit), 512, 0, stream>>>(
                out, part_acc, part_ml, q, latent, sink, scale, positions, row_seg, tables,
                max_blocks, page_shift, H, rank, row_w, nsplit);
    else
        latent_folded_mfma_kernel<NKC, RT, 1><<<dim3(rows, 1, nsplit), 256, 0, stream>>>(
            out, part_acc, part_ml, q, latent, sink, scale, positions, row_seg, tables,
            max_blocks, page_shift, H, rank, row_w, nsplit);
}

extern "C" hipError_t launch_latent_folded_mfma(
    void* out, float* part_acc, float* part_ml, const void* q, const void* latent,
    const float* sink, float scale, const int64_t* positions, const int* row_seg,
    const int* tables, int rows, int H, int rank, int row_w, int block_size, int max_blocks,
    int nsplit, hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (block_size & (block_size - 1)) return hipErrorInvalidValue;
    const int page_shift = __builtin_ctz(block_size);
    if (row_w % 8 || row_w > 576 || rank > row_w || (nsplit > 1 && (!part_acc || !part_ml)))
        return hipErrorInvalidValue;
#define GO(NKC, RT)                                                                       \
    folded_go<NKC, RT>((bf16*)out, part_acc, part_ml, (const bf16*)q,                     \
                       (const bf16*)latent, sink, scale, positions, row_seg, tables, rows, \
                       H, rank, row_w, page_shift, max_blocks, nsplit, stream)
    if (row_w <= 128) GO(4, 8);
    else if (row_w <= 192) { if (rank <= 128) GO(6, 8); else GO(6, 12); }
    else if (row_w <= 320) { if (rank <= 256) GO(10, 16); else GO(10, 20); }
    else { if (rank <= 512) GO(18, 32); else GO(18, 36); }
#undef GO
    HIP_CHECK_LAST();
    if (nsplit > 1) {
        latent_combine_kernel<<<rows * H, 128, 0, stream>>>(
            (bf16*)out, part_acc, part_ml, sink, H, rank, nsplit);
        HIP_CHECK_LAST();
    }
    return hipSuccess;
}

// ---------------------------------------------------------------------------
// Unfolded form (bf16): flash attention over per-head keys [unrotated |
// shared rotated part] and values. Query rows of a segment are its last
// cu_q[s+1]-cu_q[s] positions, its keys all cu_k[s+1]-cu_k[s]. One workgroup:
// 64*MR query rows of one head, 16*MR a wave; keys in tiles of 64, loaded to
// registers a tile ahead and staged in LDS (values are read transposed). The
// head varies fastest over the grid, so a head's keys stay in one XCD's L2.
// ---------------------------------------------------------------------------
template <int NDQ, int NDV, int MR>  // 32-chunks of a query, 16-tiles of a value
__launch_bounds__(256)
__global__ void latent_unfolded_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ q, const bf16* __restrict__ kv,
    const bf16* __restrict__ lat, int64_t lat_row, const float* __restrict__ sink, float scale,
    const int* __restrict__ cu_q, const int* __restrict__ cu_k,
    const int* __restrict__ tile_seg, const int* __restrict__ tile_off, int H, int dim,
    int rot, int vdim, int rank) {
    constexpr int LDQ = NDQ * 32 + 8, LDV = NDV * 16 + 8, LDP = 64 + 8;
    __shared__ bf16 k_lds[64][LDQ];
    __shared__ bf16 v_lds[64][LDV];
    __shared__ bf16 p_lds[4][16 * MR][LDP];
    const int h = blockIdx.x % H, tile = blockIdx.x / H;
    const int seg = tile_seg[tile], off = tile_off[tile];
    const int q0 = cu_q[seg], nq = cu_q[seg + 1] - q0;
    const int kbase = cu_k[seg], nk = cu_k[seg + 1] - kbase;
    const int ctx = nk - nq;  // position of the segment's first query row
    const int dq = dim + rot;
    const size_t ldkv = (size_t)H * (dim + vdim);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const int wrow0 = off + wave * 16 * MR;

    bf16x8 qf[MR][NDQ];
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        const bf16* qr = q + ((size_t)(q0 + min(wrow0 + i * 16 + r16, nq - 1)) * H + h) * dq;
#pragma unroll
        for (int c = 0; c < NDQ; ++c) {
            uint4 v = {0, 0, 0, 0};
            if (c * 32 + g * 8 < dq) v = *reinterpret_cast<const uint4*>(qr + c * 32 + g * 8);
            qf[i][c] = as_frag(v);
        }
    }
    float m[MR][4], l[MR][4];
    f32x4 acc[MR][NDV];
    const float sk = sink[h];
#pragma unroll
    for (int i = 0; i < MR; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            m[i][r] = sk;
            l[i][r] = r16 == 0 ? 1.f : 0.f;  // the sink, once per row
        }
#pragma unroll
        for (int j = 0; j < NDV; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
    constexpr int KV = (64 * NDQ * 4) / 256, VV = (64 * NDV * 2) / 256;
    uint4 kreg[KV], vreg[VV];
    auto load_tile = [&](int k0) {
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * 256, key = k0 + e / (NDQ * 4), d = e % (NDQ * 4) * 8;
            kreg[c] = (uint4){0, 0, 0, 0};
            if (key < nk && d < dq) {
                const bf16* src = d < dim
                    ? kv + (size_t)(kbase + key) * ldkv + (size_t)h * dim + d
                    : lat + (size_t)(kbase + key) * lat_row + rank + d - dim;
                kreg[c] = *reinterpret_cast<const uint4*>(src);
            }
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * 256, key = k0 + e / (NDV * 2), d = e % (NDV * 2) * 8;
            vreg[c] = (uint4){0, 0, 0, 0};
            if (key < nk && d < vdim)
                vreg[c] = *reinterpret_cast<const uint4*>(
                    kv + (size_t)(kbase + key) * ldkv + (size_t)H * dim + (size_t)h * vdim + d);
        }
    };
    const int key_end = ctx + min(nq, off + 64 * MR);  // keys any row here sees
    load_tile(0);
    for (int k0 = 0; k0 < key_end; k0 += 64) {
        __syncthreads();
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * 256;
            *reinterpret_cast<uint4*>(&k_lds[e / (NDQ * 4)][e % (NDQ * 4) * 8]) = kreg[c];
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * 256;
            *reinterpret_cast<uint4*>(&v_lds[e / (NDV * 2)][e % (NDV * 2) * 8]) = vreg[c];
        }
        __syncthreads();
        if (k0 + 64 < key_end) load_tile(k0 + 64);
        if (k0 > ctx + wrow0 + 16 * MR - 1) continue;  // all masked for this wave
        f32x4 s[MR][4];
#pragma unroll
        for (int i = 0; i < MR; ++i)
#pragma unroll
            for (int u = 0; u < 4; ++u) s[i][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                const bf16x8 kf =
                    *reinterpret_cast<const bf16x8*>(&k_lds[u * 16 + r16][c * 32 + g * 8]);
#pragma unroll
                for (int i = 0; i < MR; ++i) s[i][u] = mfma16(qf[i][c], kf, s[i][u]);
            }
        const bool edge = k0 + 63 > ctx + wrow0;  // some row does not see all keys
#pragma unroll
        for (int i = 0; i < MR; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int pos = ctx + wrow0 + i * 16 + g * 4 + r;
                float mx = LA_NEG;
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    float v = s[i][u][r] * scale;
                    if (edge && k0 + u * 16 + r16 > pos) v = LA_NEG;
                    s[i][u][r] = v;
                    mx = fmaxf(mx, v);
                }
                const float m_new = fmaxf(m[i][r], row16_max(mx));
                const float f = __expf(m[i][r] - m_new);
                m[i][r] = m_new;
                float sum = 0.f;
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    const float p = __expf(s[i][u][r] - m_new);
                    sum += p;
                    p_lds[wave][i * 16 + g * 4 + r][u * 16 + r16] = f2bf(p);
                }
                l[i][r] = l[i][r] * f + sum;
#pragma unroll
                for (int j = 0; j < NDV; ++j) acc[i][j][r] *= f;
            }
        // a wave reads back its own weights: no barrier
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            bf16x8 pf[MR];
#pragma unroll
            for (int i = 0; i < MR; ++i)
                pf[i] = *reinterpret_cast<const bf16x8*>(
                    &p_lds[wave][i * 16 + r16][c * 32 + g * 8]);
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16x8 vf = tr_frag(&v_lds[0][0], LDV, c * 32, j * 16);
#pragma unroll
                for (int i = 0; i < MR; ++i) acc[i][j] = mfma16(pf[i], vf, acc[i][j]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < MR; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float inv = 1.f / row16_sum(l[i][r]);
            const int row = wrow0 + i * 16 + g * 4 + r;
            if (row >= nq) continue;
            bf16* o = out + ((size_t)(q0 + row) * H + h) * vdim;
#pragma unroll
            for (int j = 0; j < NDV; ++j)
                if (j * 16 + r16 < vdim) stf(o + j * 16 + r16, acc[i][j][r] * inv);
        }
}

template <int NDQ, int NDV>
static void unfolded_go(
    bf16* out, const bf16* q, const bf16* kv, const bf16* lat, int64_t lat_row,
    const float* sink, float scale, const int* cu_q, const int* cu_k, const int* tile_seg,
    const int* tile_off, int ntiles, int tile_rows, int H, int dim, int rot, int vdim,
    int rank, hipStream_t stream) {
    if (tile_rows == 128)
        latent_unfolded_kernel<NDQ, NDV, 2><<<ntiles * H, 256, 0, stream>>>(
            out, q, kv, lat, lat_row, sink, scale, cu_q, cu_k, tile_seg, tile_off, H, dim,
            rot, vdim, rank);
    else
        latent_unfolded_kernel<NDQ, NDV, 1><<<ntiles * H, 256, 0, stream>>>(
            out, q, kv, lat, lat_row, sink, scale, cu_q, cu_k, tile_seg, tile_off, H, dim,
            rot, vdim, rank);
}

extern "C" hipError_t launch_latent_unfolded(
    void* out, const void* q, const void* kv, const void* lat, int64_t lat_row,
    const float* sink, float scale, const int* cu_q, const int* cu_k, const int* tile_seg,
    const int* tile_off, int ntiles, int tile_rows, int H, int dim, int rot, int vdim,
    int rank, hipStream_t stream) {
    if (ntiles <= 0) return hipSuccess;
    if (dim % 8 || rot % 8 || vdim % 8 || rank % 8 || lat_row % 8 ||
        (tile_rows != 64 && tile_rows != 128))
        return hipErrorInvalidValue;
    const int dq = dim + rot;
#define GO(A, B)                                                                         \
    unfolded_go<A, B>((bf16*)out, (const bf16*)q, (const bf16*)kv, (const bf16*)lat,     \
                      lat_row, sink, scale, cu_q, cu_k, tile_seg, tile_off, ntiles,      \
                      tile_rows, H, dim, rot, vdim, rank, stream)
    if (dq <= 64 && vdim <= 64) GO(2, 4);
    else if (dq <= 96 && vdim <= 64) GO(3, 4);
    else if (dq <= 128 && vdim <= 128) GO(4, 8);
    else if (dq <= 192 && vdim <= 128) GO(6, 8);
    else if (dq <= 256 && vdim <= 256) GO(8, 16);
    else return hipErrorInvalidValue;
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}
