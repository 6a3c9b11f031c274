// Grouped-query softmax attention over cache pages for gfx950, in a window
// with kept first tokens, plain or differential. A row at position p sees the
// keys j <= p with p - j < window or j < keep_first. A page holds block_size
// tokens, a token's row the keys (or values) of all G key heads; query head h
// reads key head h/(H/G).
//
// With two maps a head has two queries and a key head two keys, next to each
// other, over the same values: with a1 and a2 the maps' outputs it gives
// o / sqrt(mean(o^2) + eps) * gain of o = a1 - lam a2.
//
// Three forms of one function, as in attention_paged.hip: any size, rows
// (decoding and short portions: one query row a workgroup) and tiles (prompts:
// 64 or 128 query rows of a head a workgroup). The MFMA forms compute
// S^T = K Q^T and O^T = V^T P^T: a lane keeps one query column, so its softmax
// state is one scalar, and with the key order
//   k slot (g, j): key 4g+j for j < 4, 16+4g+(j-4) above (g = lane/16)
// two 16-key score fragments are the P^T operand as they stand. Keys outside
// the window and the kept ones are never read: the kept tokens' tiles come
// first, then the window's.

#include "mfma.h"

#define WA_THREADS 256
#define WA_NEG (-1e30f)
#define LOG2E 1.4426950408889634f

struct WindowArgs {
    void* out;
    int64_t ld_out;                // row stride; heads are vdim apart
    const void* q;
    int64_t ldq;
    const void *k, *v;             // pages
    float scale, lam, gain, eps;
    const int64_t* positions;
    const int *row_seg, *tables;
    const int* rows;               // nullable: which rows of the batch
    int max_blocks, block_size, H, G, dim, vdim, window, keep;
};

// the tiles of `size` keys that rows at positions first..last see together
struct KeyTiles {
    int kept, start, count;
    __device__ __forceinline__ KeyTiles(int first, int last, int window, int keep, int size) {
        const int lo = max(0, first - window + 1);
        kept = (min(keep, lo) + size - 1) / size;
        start = max(kept * size, lo / size * size);
        count = kept + max(0, (last + size - start) / size);
    }
    __device__ __forceinline__ int key(int i, int size) const {
        return i < kept ? i * size : start + (i - kept) * size;
    }
};

__device__ __forceinline__ bool seen(int key, int pos, int window, int keep) {
    return key <= pos && (pos - key < window || key < keep);
}

// ---------------------------------------------------------------------------
// Any size: one workgroup per (row, head), a key a thread for the scores, a
// value dimension a thread for the sums, the maps one after the other.
// ---------------------------------------------------------------------------
template <typename T, int ND, int MAPS>
__launch_bounds__(WA_THREADS)
__global__ void window_any_kernel(WindowArgs a) {
    extern __shared__ float lds[];  // [dim] query, [256] weights
    float* qs = lds;
    float* ps = lds + a.dim;
    __shared__ float red[8];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int h = blockIdx.y, g = h / (a.H / a.G), bs = a.block_size;
    const int pos = (int)a.positions[t];
    const int lo = max(0, pos - a.window + 1), kept = min(a.keep, lo), n = kept + pos + 1 - lo;
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const T *kp = (const T*)a.k, *vp = (const T*)a.v;
    auto slot_of = [&](int i) {
        const int key = i < kept ? i : lo + i - kept;
        return (size_t)bt[key / bs] * bs + key % bs;
    };
    float o[MAPS][ND];
#pragma unroll
    for (int map = 0; map < MAPS; ++map) {
        __syncthreads();
        for (int i = tid; i < a.dim; i += WA_THREADS)
            qs[i] = ldf((const T*)a.q + t * a.ldq + ((size_t)h * MAPS + map) * a.dim + i);
        float m = -INFINITY, l = 0.f;
#pragma unroll
        for (int d = 0; d < ND; ++d) o[map][d] = 0.f;
        for (int k0 = 0; k0 < n; k0 += WA_THREADS) {
            __syncthreads();
            float s = -INFINITY;
            if (k0 + tid < n) {
                const T* kr = kp + ((slot_of(k0 + tid) * a.G + g) * MAPS + map) * a.dim;
                s = 0.f;
                for (int i = 0; i < a.dim; ++i) s = fmaf(qs[i], ldf(kr + i), s);
                s *= a.scale;
            }
            float v = wave_reduce_max(s);
            if (lane == 0) red[wave] = v;
            __syncthreads();
            const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
            const float p = k0 + tid < n ? expf(s - m_new) : 0.f;
            ps[tid] = p;
            v = wave_reduce_sum(p);
            if (lane == 0) red[4 + wave] = v;
            __syncthreads();
            const float f = expf(m - m_new);
            l = l * f + red[4] + red[5] + red[6] + red[7];
            m = m_new;
#pragma unroll
            for (int d = 0; d < ND; ++d) o[map][d] *= f;
            const int here = min(WA_THREADS, n - k0);
            for (int j = 0; j < here; ++j) {
                const T* vr = vp + (slot_of(k0 + j) * a.G + g) * a.vdim;
                const float pj = ps[j];
#pragma unroll
                for (int d = 0; d < ND; ++d) {
                    const int i = tid + d * WA_THREADS;
                    if (i < a.vdim) o[map][d] = fmaf(pj, ldf(vr + i), o[map][d]);
                }
            }
        }
#pragma unroll
        for (int d = 0; d < ND; ++d) o[map][d] /= l;
    }
    float f = 1.f;
    if (MAPS == 2) {
        float ss = 0.f;
#pragma unroll
        for (int d = 0; d < ND; ++d) {
            o[0][d] -= a.lam * o[MAPS - 1][d];
            if (tid + d * WA_THREADS < a.vdim) ss += o[0][d] * o[0][d];
        }
        ss = wave_reduce_sum(ss);
        __syncthreads();
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        f = a.gain / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.vdim + a.eps);
    }
#pragma unroll
    for (int d = 0; d < ND; ++d) {
        const int i = tid + d * WA_THREADS;
        if (i < a.vdim) stf((T*)a.out + t * a.ld_out + (size_t)h * a.vdim + i, o[0][d] * f);
    }
}

__device__ __forceinline__ bf16x8 weights_frag(const float* lo, const float* hi) {
    uint4 v;
    v.x = cvt_pk_bf16(lo[0], lo[1]);
    v.y = cvt_pk_bf16(lo[2], lo[3]);
    v.z = cvt_pk_bf16(hi[0], hi[1]);
    v.w = cvt_pk_bf16(hi[2], hi[3]);
    return as_frag(v);
}

// ---------------------------------------------------------------------------
// Rows: one workgroup per (row, 16 query columns of a key head, split of the
// keys); a column is a head, or a head's map (2 head + map). A column's query
// is zero outside its own map's part of the key row, so all columns share the
// product with whole key rows of KD = maps * dim values. The 4 waves take
// tiles of 32 keys in turn, each with its own softmax state, without a
// barrier: keys go from global memory into the fragments, values through the
// wave's LDS tile (read back transposed), both loaded a tile ahead. The waves'
// shares meet in LDS at the end; several splits leave partials for
// window_combine_kernel.
// ---------------------------------------------------------------------------
template <int NDQ, int NDV, int MAPS>
__launch_bounds__(WA_THREADS)
__global__ void window_rows_kernel(
    WindowArgs a, int page_shift, int nsplit, float* part_acc, float* part_ml) {
    constexpr int LDV = NDV * 16 + 8, TILE = 32 * LDV, LDO = NDV * 16 + 4;
    constexpr int KV = 2 * NDQ, VV = NDV;  // 16-byte loads a lane and tile
    static_assert(16 * LDO * 4 <= TILE * 2, "a wave's share fits its tile");
    __shared__ __align__(16) bf16 v_lds[4][TILE];
    __shared__ float m_lds[4][16], l_lds[4][16];
    const size_t t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    const int per = a.H / a.G, cols = per * MAPS, nct = (cols + 15) / 16;
    const int g_kv = blockIdx.y / nct, c0 = blockIdx.y % nct * 16, split = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pos = (int)a.positions[t], KD = a.dim * MAPS;
    const KeyTiles kt(pos, pos, a.window, a.keep, 32);
    const int span = (kt.count + nsplit * 4 - 1) / (nsplit * 4) * 4;
    const int tile_lo = split * span, tile_hi = min(kt.count, tile_lo + span);
    const int* bt = a.tables + (size_t)a.row_seg[t] * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const bf16 *kp = (const bf16*)a.k + (size_t)g_kv * KD;
    const bf16 *vp = (const bf16*)a.v + (size_t)g_kv * a.vdim;
    const float c2 = a.scale * LOG2E;

    bf16x8 qf[NDQ];
    {
        const int col = min(c0 + r16, cols - 1), map = col % MAPS;
        const bf16* qr = (const bf16*)a.q + t * a.ldq + ((size_t)g_kv * cols + col) * a.dim;
#pragma unroll
        for (int c = 0; c < NDQ; ++c) {
            const int d = c * 32 + g * 8 - map * a.dim;
            uint4 x = {0, 0, 0, 0};
            if (d >= 0 && d < a.dim) x = *reinterpret_cast<const uint4*>(qr + d);
            qf[c] = as_frag(x);
        }
    }
    float m = WA_NEG, l = 0.f;
    f32x4 acc[NDV];
#pragma unroll
    for (int j = 0; j < NDV; ++j) acc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};

    uint4 kreg[KV], vreg[VV];
    // rows of the keys k0 .. k0+31 in the pages; past the last any row
    auto load_tile = [&](int k0) {
        const size_t b0 = (size_t)bt[k0 >> page_shift] << page_shift;
        const size_t b1 = (size_t)bt[min(k0 + 16, pos) >> page_shift] << page_shift;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int key = min(k0 + u * 16 + r16, pos);
            const size_t row = (u && k0 + 16 <= pos ? b1 : b0) + (key & mask);
            const bf16* p = kp + row * a.G * KD;
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                kreg[u * NDQ + c] = (uint4){0, 0, 0, 0};
                if (c * 32 + g * 8 < KD)
                    kreg[u * NDQ + c] = *reinterpret_cast<const uint4*>(p + c * 32 + g * 8);
            }
        }
#pragma unroll
        for (int u = 0; u < VV; ++u) {
            const int e = lane + u * 64, o = e / (NDV * 2), d = e % (NDV * 2) * 8;
            const int key = min(k0 + o, pos);
            const size_t row = (key >= k0 + 16 ? b1 : b0) + (key & mask);
            vreg[u] = (uint4){0, 0, 0, 0};
            if (d < a.vdim)
                vreg[u] = *reinterpret_cast<const uint4*>(vp + row * a.G * a.vdim + d);
        }
    };
    bf16* vt = v_lds[wave];
    int tile = tile_lo + wave;
    if (tile < tile_hi) load_tile(kt.key(tile, 32));
    for (; tile < tile_hi; tile += 4) {
        const int k0 = kt.key(tile, 32);
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
        if (tile + 4 < tile_hi) load_tile(kt.key(tile + 4, 32));
        float p[2][4], mx = WA_NEG;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[u][r] = seen(k0 + u * 16 + g * 4 + r, pos, a.window, a.keep) ? s[u][r] * c2
                                                                              : WA_NEG;
                mx = fmaxf(mx, p[u][r]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE_SIZE));
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE_SIZE));
        const float m_new = fmaxf(m, mx), f = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        l *= f;
#pragma unroll
        for (int j = 0; j < NDV; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[j][r] *= f;
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
    // the waves' shares: acc as [16 columns][vdim] in each wave's tile
    l += __shfl_xor(l, 16, WAVE_SIZE);
    l += __shfl_xor(l, 32, WAVE_SIZE);
    if (g == 0) {
        m_lds[wave][r16] = m;
        l_lds[wave][r16] = l;
    }
    float* sh = reinterpret_cast<float*>(vt);
#pragma unroll
    for (int j = 0; j < NDV; ++j)
        *reinterpret_cast<f32x4*>(sh + r16 * LDO + j * 16 + g * 4) = acc[j];
    __syncthreads();
    // a wave per head; a lane takes every 64th value
    constexpr int NL = (NDV * 16 + 63) / 64;
    for (int hd = wave; hd < 16 / MAPS; hd += 4) {
        if (c0 + hd * MAPS >= cols) break;
        const int hh = g_kv * per + c0 / MAPS + hd;
        float o[MAPS][NL], ss = 0.f;
#pragma unroll
        for (int map = 0; map < MAPS; ++map) {
            const int c = hd * MAPS + map;
            const float M = fmaxf(fmaxf(m_lds[0][c], m_lds[1][c]), fmaxf(m_lds[2][c], m_lds[3][c]));
            float L = 0.f, w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                w[i] = __builtin_amdgcn_exp2f(m_lds[i][c] - M);
                L = fmaf(l_lds[i][c], w[i], L);
            }
            const size_t pb = (((size_t)blockIdx.x * a.H + hh) * MAPS + map) * nsplit + split;
#pragma unroll
            for (int e = 0; e < NL; ++e) {
                const int d = lane + e * 64;
                float v = 0.f;
                if (d < NDV * 16) {
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        v = fmaf(reinterpret_cast<const float*>(v_lds[i])[c * LDO + d], w[i], v);
                }
                if (nsplit > 1) {
                    if (d < a.vdim) part_acc[pb * a.vdim + d] = v;
                } else {
                    o[map][e] = v / L;
                }
            }
            if (nsplit > 1 && lane == 0) {
                part_ml[pb * 2] = M;
                part_ml[pb * 2 + 1] = L;
            }
        }
        if (nsplit > 1) continue;
        float f = 1.f;
        if (MAPS == 2) {
#pragma unroll
            for (int e = 0; e < NL; ++e) {
                o[0][e] -= a.lam * o[MAPS - 1][e];
                ss += o[0][e] * o[0][e];  // (values past vdim are 0)
            }
            f = a.gain / sqrtf(wave_reduce_sum(ss) / (float)a.vdim + a.eps);
        }
#pragma unroll
        for (int e = 0; e < NL; ++e) {
            const int d = lane + e * 64;
            if (d < a.vdim)
                stf((bf16*)a.out + t * a.ld_out + (size_t)hh * a.vdim + d, o[0][e] * f);
        }
    }
}

// a wave per (row, head)
template <int MAPS>
__launch_bounds__(WA_THREADS)
__global__ void window_combine_kernel(
    WindowArgs a, int nrows, int nsplit, const float* __restrict__ part_acc,
    const float* __restrict__ part_ml) {
    const size_t item = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= (size_t)nrows * a.H) return;
    const size_t i = item / a.H, t = a.rows ? a.rows[i] : i;
    const int h = item % a.H, lane = threadIdx.x & 63;
    float o[MAPS][4], ss = 0.f;
#pragma unroll
    for (int map = 0; map < MAPS; ++map) {
        const size_t pb = (item * MAPS + map) * nsplit;
        const float* ml = part_ml + pb * 2;
        float M = WA_NEG, L = 0.f;
        for (int s = 0; s < nsplit; ++s) M = fmaxf(M, ml[2 * s]);
#pragma unroll
        for (int e = 0; e < 4; ++e) o[map][e] = 0.f;
        for (int s = 0; s < nsplit; ++s) {
            const float w = __builtin_amdgcn_exp2f(ml[2 * s] - M);
            L = fmaf(ml[2 * s + 1], w, L);
            const float* pa = part_acc + (pb + s) * a.vdim;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (lane + e * 64 < a.vdim) o[map][e] = fmaf(pa[lane + e * 64], w, o[map][e]);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) o[map][e] /= L;
    }
    float f = 1.f;
    if (MAPS == 2) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            o[0][e] -= a.lam * o[MAPS - 1][e];
            ss += o[0][e] * o[0][e];
        }
        f = a.gain / sqrtf(wave_reduce_sum(ss) / (float)a.vdim + a.eps);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (lane + e * 64 < a.vdim)
            stf((bf16*)a.out + t * a.ld_out + (size_t)h * a.vdim + lane + e * 64, o[0][e] * f);
}

// ---------------------------------------------------------------------------
// Tiles: one workgroup per (16*MR*NW rows of a segment, head), 16*MR rows a
// wave; tiles of 64 keys, loaded to registers a tile ahead and staged in LDS.
// Both maps of a head run together: they share the values' fragments.
// NDQ: 32-wide slices of a map's key dims.
// ---------------------------------------------------------------------------
template <int NDQ, int NDV, int MR, int NW, int MAPS>
__launch_bounds__(NW * 64)
__global__ void window_tiles_kernel(
    WindowArgs a, int page_shift, const int* __restrict__ cu,
    const int* __restrict__ tile_seg, const int* __restrict__ tile_off) {
    // a key row in LDS: the maps' parts next to each other, zeros after them
    constexpr int LQ = NDQ * 32 * MAPS, LDQ = LQ + 8, LDV = NDV * 16 + 8, NT = NW * 64;
    constexpr int KV = 64 * LQ / 8 / NT, VV = 64 * NDV * 2 / NT;
    __shared__ __align__(16) bf16 k_lds[64 * LDQ], v_lds[64 * LDV];
    const int h = blockIdx.x % a.H, tile = blockIdx.x / a.H;
    const int seg = tile_seg[tile], off = tile_off[tile];
    const int q0 = cu[seg], nq = cu[seg + 1] - q0;
    const int ctx = (int)a.positions[q0];  // position of the segment's first row
    const int* bt = a.tables + (size_t)seg * a.max_blocks;
    const int mask = (1 << page_shift) - 1;
    const int g_kv = h / (a.H / a.G), KD = a.dim * MAPS;
    const bf16 *kp = (const bf16*)a.k + (size_t)g_kv * KD;
    const bf16 *vp = (const bf16*)a.v + (size_t)g_kv * a.vdim;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const int wrow0 = off + wave * 16 * MR;
    const float c2 = a.scale * LOG2E;

    bf16x8 qf[MR][MAPS][NDQ];
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        const int row = min(wrow0 + i * 16 + r16, nq - 1);
        const bf16* qr = (const bf16*)a.q + (size_t)(q0 + row) * a.ldq + (size_t)h * KD;
#pragma unroll
        for (int map = 0; map < MAPS; ++map)
#pragma unroll
            for (int c = 0; c < NDQ; ++c) {
                const int d = c * 32 + g * 8;
                uint4 x = {0, 0, 0, 0};
                if (d < a.dim) x = *reinterpret_cast<const uint4*>(qr + map * a.dim + d);
                qf[i][map][c] = as_frag(x);
            }
    }
    float m[MR][MAPS], l[MR][MAPS];
    f32x4 acc[MR][MAPS][NDV];
#pragma unroll
    for (int i = 0; i < MR; ++i)
#pragma unroll
        for (int map = 0; map < MAPS; ++map) {
            m[i][map] = WA_NEG;
            l[i][map] = 0.f;
#pragma unroll
            for (int j = 0; j < NDV; ++j) acc[i][map][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        }
    const int pos_last = ctx + min(nq, off + 16 * MR * NW) - 1;  // of the workgroup's rows
    const KeyTiles kt(ctx + off, pos_last, a.window, a.keep, 64);
    uint4 kreg[KV], vreg[VV];
    int page[4];  // of the tile that is loaded next, per 16 keys: looked up a tile ahead
    auto look_up = [&](int it) {
        const int k0 = kt.key(min(it, kt.count - 1), 64);
#pragma unroll
        for (int u = 0; u < 4; ++u) page[u] = bt[min(k0 + u * 16, pos_last) >> page_shift];
    };
    auto load_tile = [&](int k0) {
        auto row_of = [&](int o) {  // past the last key: any row
            const int key = min(k0 + o, pos_last), u = (key - k0) >> 4;
            const int p = u == 0 ? page[0] : u == 1 ? page[1] : u == 2 ? page[2] : page[3];
            return ((size_t)p << page_shift) + (key & mask);
        };
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * NT, d = e % (LQ / 8) * 8;
            kreg[c] = (uint4){0, 0, 0, 0};
            if (d < KD)
                kreg[c] = *reinterpret_cast<const uint4*>(
                    kp + row_of(e / (LQ / 8)) * a.G * KD + d);
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * NT, d = e % (NDV * 2) * 8;
            vreg[c] = (uint4){0, 0, 0, 0};
            if (d < a.vdim)
                vreg[c] = *reinterpret_cast<const uint4*>(
                    vp + row_of(e / (NDV * 2)) * a.G * a.vdim + d);
        }
    };
    const int wp0 = ctx + wrow0, wp1 = wp0 + 16 * MR - 1;  // this wave's positions
    look_up(0);
    load_tile(kt.key(0, 64));
    look_up(1);
    for (int it = 0; it < kt.count; ++it) {
        const int k0 = kt.key(it, 64);
        __syncthreads();
#pragma unroll
        for (int c = 0; c < KV; ++c) {
            const int e = tid + c * NT;
            *reinterpret_cast<uint4*>(k_lds + e / (LQ / 8) * LDQ + e % (LQ / 8) * 8) = kreg[c];
        }
#pragma unroll
        for (int c = 0; c < VV; ++c) {
            const int e = tid + c * NT;
            *reinterpret_cast<uint4*>(v_lds + e / (NDV * 2) * LDV + e % (NDV * 2) * 8) = vreg[c];
        }
        __syncthreads();
        if (it + 1 < kt.count) {
            load_tile(kt.key(it + 1, 64));
            look_up(it + 2);
        }
        // no row of this wave sees a key of the tile
        if (k0 > wp1 || (wp0 - (k0 + 63) >= a.window && k0 >= a.keep)) continue;
        const bool edge =  // some row does not see all keys
            k0 + 63 > wp0 || (wp1 - k0 >= a.window && k0 + 63 >= a.keep);
        bf16x8 pf[MR][MAPS][2];
#pragma unroll
        for (int map = 0; map < MAPS; ++map) {
            f32x4 s[MR][4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
#pragma unroll
                for (int i = 0; i < MR; ++i) s[i][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int c = 0; c < NDQ; ++c) {
                    const bf16x8 kf = *reinterpret_cast<const bf16x8*>(
                        k_lds + (u * 16 + r16) * LDQ + map * a.dim + c * 32 + g * 8);
#pragma unroll
                    for (int i = 0; i < MR; ++i) s[i][u] = mfma16(kf, qf[i][map][c], s[i][u]);
                }
            }
#pragma unroll
            for (int i = 0; i < MR; ++i) {
                const int pos = wp0 + i * 16 + r16;
                float p[4][4], mx = WA_NEG;
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        p[u][r] = s[i][u][r] * c2;
                        if (edge && !seen(k0 + u * 16 + g * 4 + r, pos, a.window, a.keep))
                            p[u][r] = WA_NEG;
                        mx = fmaxf(mx, p[u][r]);
                    }
                mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE_SIZE));
                mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE_SIZE));
                // (what a row sums up before its first seen key is scaled by 0)
                const float m_new = fmaxf(m[i][map], mx);
                const float f = __builtin_amdgcn_exp2f(m[i][map] - m_new);
                if (__any(f != 1.f)) {
                    m[i][map] = m_new;
                    l[i][map] *= f;
#pragma unroll
                    for (int j = 0; j < NDV; ++j)
#pragma unroll
                        for (int r = 0; r < 4; ++r) acc[i][map][j][r] *= f;
                }
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        p[u][r] = __builtin_amdgcn_exp2f(p[u][r] - m[i][map]);
                        l[i][map] += p[u][r];
                    }
                pf[i][map][0] = weights_frag(p[0], p[1]);
                pf[i][map][1] = weights_frag(p[2], p[3]);
            }
        }
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            const bf16* r0 = v_lds + (c * 32 + g * 4 + (r16 >> 2)) * LDV + (r16 & 3) * 4;
#pragma unroll
            for (int j = 0; j < NDV; ++j) {
                const bf16x8 vf = tr_pair(r0 + j * 16, r0 + 16 * LDV + j * 16);
#pragma unroll
                for (int i = 0; i < MR; ++i)
#pragma unroll
                    for (int map = 0; map < MAPS; ++map)
                        acc[i][map][j] = mfma16(vf, pf[i][map][c], acc[i][map][j]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < MR; ++i) {
        float inv[MAPS];
#pragma unroll
        for (int map = 0; map < MAPS; ++map) {
            float L = l[i][map];
            L += __shfl_xor(L, 16, WAVE_SIZE);
            L += __shfl_xor(L, 32, WAVE_SIZE);
            inv[map] = 1.f / L;
        }
        float f = inv[0];
        if (MAPS == 2) {
            const float f2 = a.lam * inv[MAPS - 1];
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < NDV; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float o = acc[i][0][j][r] * inv[0] - acc[i][MAPS - 1][j][r] * f2;
                    acc[i][0][j][r] = o;
                    ss += o * o;  // (values past vdim are 0)
                }
            ss += __shfl_xor(ss, 16, WAVE_SIZE);
            ss += __shfl_xor(ss, 32, WAVE_SIZE);
            f = a.gain / sqrtf(ss / (float)a.vdim + a.eps);
        }
        const int row = wrow0 + i * 16 + r16;
        if (row >= nq) continue;
        bf16* o = (bf16*)a.out + (size_t)(q0 + row) * a.ld_out + (size_t)h * a.vdim;
#pragma unroll
        for (int j = 0; j < NDV; ++j) {
            const int d = j * 16 + g * 4;  // vdim is a multiple of 8
            if (d < a.vdim)
                *reinterpret_cast<uint2*>(o + d) = make_uint2(
                    cvt_pk_bf16(acc[i][0][j][0] * f, acc[i][0][j][1] * f),
                    cvt_pk_bf16(acc[i][0][j][2] * f, acc[i][0][j][3] * f));
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
template <typename T, int MAPS>
static hipError_t window_any(const WindowArgs& a, int nrows, hipStream_t stream) {
    const size_t lds = (a.dim + WA_THREADS) * sizeof(float);
    if (lds > 48 * 1024) return hipErrorInvalidValue;
    const dim3 grid(nrows, a.H);
    if (a.vdim <= 256) window_any_kernel<T, 1, MAPS><<<grid, WA_THREADS, lds, stream>>>(a);
    else if (a.vdim <= 1024) window_any_kernel<T, 4, MAPS><<<grid, WA_THREADS, lds, stream>>>(a);
    else return hipErrorInvalidValue;
    HIP_CHECK_LAST();
    return hipSuccess;
}

// sizes of the MFMA forms: multiples of 8 up to 256 (a key row: its maps
// together), power-of-two pages of at least 16 tokens
static bool window_mfma_ok(const WindowArgs& a, int maps) {
    return a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim * maps <= 256 && a.vdim <= 256 &&
           a.block_size >= 16 && (a.block_size & (a.block_size - 1)) == 0;
}

static WindowArgs window_args(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    float scale, int window, int keep, float lam, float gain, float eps,
    const int64_t* positions, const int* row_seg, const int* tables, const int* rows,
    int max_blocks, int block_size, int H, int G, int dim, int vdim) {
    return WindowArgs{out, ld_out, q, ldq, k, v, scale, lam, gain, eps, positions, row_seg,
                      tables, rows, max_blocks, block_size, H, G, dim, vdim, window, keep};
}

// nsplit 0: the any-size form
extern "C" hipError_t launch_window_rows(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    int maps, float scale, int window, int keep, float lam, float gain, float eps,
    const int64_t* positions, const int* row_seg, const int* tables, const int* rows,
    int max_blocks, int block_size, int H, int G, int dim, int vdim, int nrows, int nsplit,
    float* part_acc, float* part_ml, int f32, hipStream_t stream) {
    if (nrows <= 0) return hipSuccess;
    if (maps < 1 || maps > 2 || window < 1 || keep < 0) return hipErrorInvalidValue;
    const WindowArgs a =
        window_args(out, ld_out, q, ldq, k, v, scale, window, keep, lam, gain, eps, positions,
                    row_seg, tables, rows, max_blocks, block_size, H, G, dim, vdim);
    if (nsplit == 0) {
        if (maps == 2)
            return f32 ? window_any<float, 2>(a, nrows, stream) : window_any<bf16, 2>(a, nrows, stream);
        return f32 ? window_any<float, 1>(a, nrows, stream) : window_any<bf16, 1>(a, nrows, stream);
    }
    if (f32 || !window_mfma_ok(a, maps) || (nsplit > 1 && (!part_acc || !part_ml)))
        return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size), kd = dim * maps;
    const dim3 grid(nrows, G * ceil_div_i(H / G * maps, 16), nsplit);
#define GO(A, B)                                                                         \
    {                                                                                    \
        if (maps == 2)                                                                   \
            window_rows_kernel<A, B, 2><<<grid, WA_THREADS, 0, stream>>>(                \
                a, shift, nsplit, part_acc, part_ml);                                    \
        else                                                                             \
            window_rows_kernel<A, B, 1><<<grid, WA_THREADS, 0, stream>>>(                \
                a, shift, nsplit, part_acc, part_ml);                                    \
    }
    if (kd <= 64 && vdim <= 64) GO(2, 4)
    else if (kd <= 128 && vdim <= 64) GO(4, 4)
    else if (kd <= 128 && vdim <= 128) GO(4, 8)
    else GO(8, 16)
#undef GO
    HIP_CHECK_LAST();
    if (nsplit > 1) {
        const int blocks = ceil_div_i(nrows * H, 4);
        if (maps == 2)
            window_combine_kernel<2><<<blocks, WA_THREADS, 0, stream>>>(
                a, nrows, nsplit, part_acc, part_ml);
        else
            window_combine_kernel<1><<<blocks, WA_THREADS, 0, stream>>>(
                a, nrows, nsplit, part_acc, part_ml);
        HIP_CHECK_LAST();
    }
    return hipSuccess;
}

extern "C" hipError_t launch_window_tiles(
    void* out, int64_t ld_out, const void* q, int64_t ldq, const void* k, const void* v,
    int maps, float scale, int window, int keep, float lam, float gain, float eps,
    const int64_t* positions, const int* tables, int max_blocks, int block_size, int H, int G,
    int dim, int vdim, const int* cu, const int* tile_seg, const int* tile_off, int ntiles,
    int tile_rows, hipStream_t stream) {
    if (ntiles <= 0) return hipSuccess;
    if (maps < 1 || maps > 2 || window < 1 || keep < 0) return hipErrorInvalidValue;
    const WindowArgs a =
        window_args(out, ld_out, q, ldq, k, v, scale, window, keep, lam, gain, eps, positions,
                    nullptr, tables, nullptr, max_blocks, block_size, H, G, dim, vdim);
    if (!window_mfma_ok(a, maps) || (tile_rows != 64 && tile_rows != 128))
        return hipErrorInvalidValue;
    const int shift = __builtin_ctz(block_size);
#define GO3(A, B, M, N, P)                                                               \
    window_tiles_kernel<A, B, M, N, P><<<ntiles * H, N * 64, 0, stream>>>(               \
        a, shift, cu, tile_seg, tile_off)
#define GO(A, B, P)                                                                      \
    {                                                                                    \
        if (tile_rows == 64) GO3(A, B, 1, 4, P);                                         \
        else GO3(A, B, 1, 8, P);                                                         \
    }
    if (maps == 2) {
        if (dim <= 32 && vdim <= 64) GO(1, 4, 2)
        else if (dim <= 64 && vdim <= 64) GO(2, 4, 2)
        else if (dim <= 64 && vdim <= 128) GO(2, 8, 2)
        else if (dim <= 128 && vdim <= 128) GO(4, 8, 2)
        else GO(4, 16, 2)
    } else {
        if (dim <= 64 && vdim <= 64) GO(2, 4, 1)
        else if (dim <= 128 && vdim <= 128) GO(4, 8, 1)
        else GO(8, 16, 1)
    }
#undef GO
#undef GO3
    HIP_CHECK_LAST();
    return hipSuccess;
}
