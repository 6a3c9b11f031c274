// Mixture-of-experts feed-forward for gfx950: top-k routing, the rows grouped
// by expert on the device (no host round trip: the launches' shapes depend on
// token and expert counts only, so captured graphs hold), and the experts'
// two products over the groups,
//
//   act[r] = glu(W_gate[e] h[token(r)], W_up[e] h[token(r)]),  out[r] = W_down[e] act[r]
//
// with the clamped GLU (rows.h) or silu(gate) * up.
//
// A group fills whole tiles of tile_rows rows; row_token is -1 in the rest.
// The weighted sum over a token's experts is part of the stream kernel.
//
// Weights of the MFMA forms lie in fragments, [N/16][K/32][64 lanes][8]: one
// wave load of 1 KiB is an operand in lane order. N is padded to 256, K to
// 64 with zeros; gate and up rows alternate in blocks of 16.

#include "lds_dma.h"
#include "mfma.h"
#include "rows.h"

#define MAX_EXPERTS 1024

// ---------------------------------------------------------------------------
// One wave a token: the top logits (ties: the lower index) and scale times the
// softmax over them.
// ---------------------------------------------------------------------------
template <int PER>  // logits a lane
__launch_bounds__(256)
__global__ void route_topk_kernel(
    int* __restrict__ ids, float* __restrict__ weights, const float* __restrict__ z,
    const float* __restrict__ bias, float scale, int T, int E, int top) {
    const int lane = threadIdx.x & 63;
    const size_t t = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= T) return;
    float v[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int e = i * 64 + lane;
        v[i] = e < E ? z[t * E + e] + (bias != nullptr ? bias[e] : 0.f) : -INFINITY;
    }
    float mine = -INFINITY, first = 0.f;
    int my_id = 0;
    for (int k = 0; k < top; ++k) {
        float best = -INFINITY;
        int at = 1 << 30;
#pragma unroll
        for (int i = 0; i < PER; ++i)
            if (v[i] > best) {
                best = v[i];
                at = i * 64 + lane;
            }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) {
            const float b2 = __shfl_xor(best, off, WAVE_SIZE);
            const int a2 = __shfl_xor(at, off, WAVE_SIZE);
            if (b2 > best || (b2 == best && a2 < at)) {
                best = b2;
                at = a2;
            }
        }
        at = min(at, E - 1);  // (a row without a finite logit)
        if (k == 0) first = best;
        if (lane == k) {
            mine = best;
            my_id = at;
        }
#pragma unroll
        for (int i = 0; i < PER; ++i)
            if (i * 64 + lane == at) v[i] = -INFINITY;
    }
    const float p = lane < top ? expf(mine - first) : 0.f;
    const float sum = wave_reduce_sum(p);
    if (lane < top) {
        ids[t * top + lane] = my_id;
        weights[t * top + lane] = p / sum * scale;
    }
}

// ---------------------------------------------------------------------------
// Rows by expert, in one workgroup: slot[i] is where (token, choice) i went.
// The order within a group is arbitrary; no value depends on it. tile_info,
// [4 * max_tiles + 1]: per tile its expert (-1: none), the expert's first tile,
// how many the expert has, and the tile's rows; then the number of tiles.
// ---------------------------------------------------------------------------
__launch_bounds__(1024)
__global__ void route_plan_kernel(
    int* __restrict__ slot, int* __restrict__ row_token, int* __restrict__ tile_info,
    const int* __restrict__ ids, int n, int top, int E, int tile_rows, int max_tiles) {
    __shared__ int count[MAX_EXPERTS], end[MAX_EXPERTS], cursor[MAX_EXPERTS];
    const int tid = threadIdx.x;
    count[tid] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    const int tiles = tid < E ? (count[tid] + tile_rows - 1) / tile_rows : 0;
    end[tid] = tiles;
    __syncthreads();
    for (int off = 1; off < 1024; off <<= 1) {  // inclusive sums
        const int v = tid >= off ? end[tid - off] : 0;
        __syncthreads();
        end[tid] += v;
        __syncthreads();
    }
    const int first = end[tid] - tiles;
    cursor[tid] = first * tile_rows;
    for (int i = first; i < end[tid]; ++i) {
        tile_info[4 * i] = tid;
        tile_info[4 * i + 1] = first;
        tile_info[4 * i + 2] = tiles;
        tile_info[4 * i + 3] = min(tile_rows, count[tid] - (i - first) * tile_rows);
    }
    if (tid == 0) tile_info[4 * max_tiles] = end[1023];
    for (int r = first * tile_rows + count[tid]; r < end[tid] * tile_rows; ++r) row_token[r] = -1;
    for (int i = end[1023] + tid; i < max_tiles; i += 1024) tile_info[4 * i] = -1;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) {
        const int r = atomicAdd(&cursor[ids[i]], 1);
        slot[i] = r;
        row_token[r] = i / top;
    }
}

struct ExpertArgs {
    void* out;               // [rows, ld_out]
    const void* x;           // GLU: [tokens, ldx], rows by row_token; else [rows, ldx]
    const void* w;
    const int *row_token, *tile_info;
    int max_tiles;
    int64_t ldx, ld_out;
    int N, K;                // output width (GLU: of act), input width
    int silu;                // the GLU: silu(gate) * up, or clamped at limit
    float limit;
};

template <typename T>
__device__ __forceinline__ float expert_glu(float g, float u, const ExpertArgs& a) {
    return a.silu ? silu_glu<T>(g, u) : clamped_glu<T>(g, u, a.limit);
}

// ---------------------------------------------------------------------------
// Any size: tiles of 16 rows x 16 outputs, weights [E, N (GLU: 2N), K]
// ---------------------------------------------------------------------------
template <typename T, bool GLU>
__launch_bounds__(256)
__global__ void expert_any_kernel(ExpertArgs a) {
    __shared__ float x_lds[16][33], w_lds[GLU ? 2 : 1][16][33];
    const int tile = blockIdx.x, n0 = blockIdx.y * 16, e = a.tile_info[4 * tile];
    if (e < 0) return;
    const int tid = threadIdx.x, row = tid >> 4, col = tid & 15;
    const T* w = (const T*)a.w + (size_t)e * (GLU ? 2 : 1) * a.N * a.K;
    float acc = 0.f, up = 0.f;
    for (int k0 = 0; k0 < a.K; k0 += 32) {
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int i = tid + u * 256, r = i >> 5, k = k0 + (i & 31);
            int src = tile * 16 + r;
            if (GLU) src = max(a.row_token[src], 0);
            const bool in = k < a.K;
            x_lds[r][i & 31] = in ? ldf((const T*)a.x + (size_t)src * a.ldx + k) : 0.f;
            const int n = n0 + r;
            w_lds[0][r][i & 31] = in && n < a.N ? ldf(w + (size_t)n * a.K + k) : 0.f;
            if (GLU)
                w_lds[GLU ? 1 : 0][r][i & 31] =
                    in && n < a.N ? ldf(w + (size_t)(a.N + n) * a.K + k) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 32; ++k) {
            acc = fmaf(x_lds[row][k], w_lds[0][col][k], acc);
            if (GLU) up = fmaf(x_lds[row][k], w_lds[GLU ? 1 : 0][col][k], up);
        }
    }
    if (n0 + col < a.N) {
        if (GLU) acc = expert_glu<T>(acc, up, a);
        stf((T*)a.out + (size_t)(tile * 16 + row) * a.ld_out + n0 + col, acc);
    }
}

__device__ __forceinline__ void store4(bf16* p, const f32x4& v) {
    *reinterpret_cast<uint2*>(p) = make_uint2(cvt_pk_bf16(v[0], v[1]), cvt_pk_bf16(v[2], v[3]));
}
__device__ __forceinline__ f32x4 glu4(const f32x4& g, const f32x4& u, const ExpertArgs& a) {
    f32x4 o;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = expert_glu<bf16>(g[r], u[r], a);
    return o;
}

// ---------------------------------------------------------------------------
// Few rows an expert (decoding): weights stream once. One workgroup: a tile
// of 16*MF rows, 4 weight fragments (64 outputs, GLU: 32); the 4 waves share
// the steps of K and meet in LDS. C fragments hold [output][row].
// ---------------------------------------------------------------------------
template <int MF, bool GLU>
__launch_bounds__(256)
__global__ void expert_stream_kernel(ExpertArgs a, int nfrags, int ksteps) {
    __shared__ f32x4 red[4][MF * 4][64];
    const int tile = blockIdx.y, e = a.tile_info[4 * tile];
    if (e < 0) return;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4, nf0 = blockIdx.x * 4;
    const uint4* w = (const uint4*)a.w + ((size_t)e * nfrags + nf0) * ksteps * 64 + lane;
    const bf16* xr[MF];
#pragma unroll
    for (int i = 0; i < MF; ++i) {
        int src = tile * 16 * MF + i * 16 + r16;
        if (GLU) src = max(a.row_token[src], 0);
        xr[i] = (const bf16*)a.x + (size_t)src * a.ldx;
    }
    f32x4 acc[MF][4];
#pragma unroll
    for (int i = 0; i < MF; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = wave; s < ksteps; s += 4) {
        const int k = s * 32 + g * 8;
        uint4 wf[4], xf[MF];
#pragma unroll
        for (int j = 0; j < 4; ++j) wf[j] = w[((size_t)j * ksteps + s) * 64];
#pragma unroll
        for (int i = 0; i < MF; ++i)  // past K the weights are 0
            xf[i] = *reinterpret_cast<const uint4*>(xr[i] + (k < a.K ? k : 0));
#pragma unroll
        for (int i = 0; i < MF; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i][j] = mfma16(as_frag(wf[j]), as_frag(xf[i]), acc[i][j]);
    }
#pragma unroll
    for (int i = 0; i < MF; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) red[wave][i * 4 + j][lane] = acc[i][j];
    __syncthreads();
    auto sum = [&](int f) {
        f32x4 v = red[0][f][lane];
#pragma unroll
        for (int u = 1; u < 4; ++u) {
            const f32x4 o = red[u][f][lane];
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] += o[r];
        }
        return v;
    };
    if (GLU) {
        for (int it = wave; it < 2 * MF; it += 4) {
            const int i = it >> 1, pair = it & 1;
            const int row = tile * 16 * MF + i * 16 + r16;
            const int n = (nf0 / 2 + pair) * 16 + g * 4;
            const f32x4 v = glu4(sum(i * 4 + pair * 2), sum(i * 4 + pair * 2 + 1), a);
            if (n < a.N) store4((bf16*)a.out + (size_t)row * a.ld_out + n, v);
        }
    } else {
        for (int it = wave; it < 4 * MF; it += 4) {
            const int i = it >> 2, j = it & 3;
            const int row = tile * 16 * MF + i * 16 + r16, n = (nf0 + j) * 16 + g * 4;
            const f32x4 v = sum(i * 4 + j);
            if (n < a.N) store4((bf16*)a.out + (size_t)row * a.ld_out + n, v);
        }
    }
}

// ---------------------------------------------------------------------------
// Many rows an expert (prompts): 256 rows x 16 weight fragments a workgroup,
// 8 waves of 64 rows x 128 outputs; waves without rows only help to bring the
// weights, and since two waves share a SIMD, one of each half, a half-empty
// tile takes half the time. K runs in steps of 64 through two LDS buffers
// filled by global-to-LDS transfers a step ahead. Weights come as fragments;
// rows in pieces of 8 rows x 128 bytes (whole cache lines), their 16-byte
// chunks XOR-swizzled by row on the source address, so that fragment reads
// spread over the banks.
// ---------------------------------------------------------------------------
template <bool GLU>
__launch_bounds__(512)
__global__ void expert_tile_kernel(ExpertArgs a, int nfrags, int ksteps, int ntn) {
    // [buffer][32 pieces of rows | 16 weight fragments x 2][1 KiB]
    __shared__ __align__(16) bf16 lds[2][64][512];
    // each XCD (8, round robin) takes a contiguous part of the tiles there are;
    // within an expert its row tiles vary fastest, so that what runs together
    // shares rows and weights in the XCD's L2
    const int total = a.tile_info[4 * a.max_tiles] * ntn, per = (total + 7) / 8;
    const int b = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || b >= total) return;
    const int4 info = reinterpret_cast<const int4*>(a.tile_info)[b / ntn];
    const int in_e = b - info.y * ntn;
    const int tile = info.y + in_e % info.z, nf0 = in_e / info.z * 16;
    const int rows = reinterpret_cast<const int4*>(a.tile_info)[tile].w;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r16 = lane & 15, g = lane >> 4;
    const bf16* w =
        (const bf16*)a.w + ((size_t)info.x * nfrags + nf0 + wave * 2) * ksteps * 512 + lane * 8;
    const size_t wstep = (size_t)ksteps * 512;
    const bool works = (wave >> 1) * 64 < rows;  // this wave's 64 rows count
    const bf16* xr[4];  // it brings 32 of them: lane = row lane/8 of a piece
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        int src = tile * 256 + wave * 32 + i * 8 + (lane >> 3);
        if (GLU) src = max(a.row_token[src], 0);
        xr[i] = (const bf16*)a.x + (size_t)src * a.ldx;
    }
    const int chunk = ((lane & 7) ^ (lane >> 3)) * 8;
    auto stage = [&](int s, int buf) {  // steps s and s+1 of 32
        const int k = s * 32 + chunk, kk = k < a.K ? k : 0;  // past K the weights are 0
        if (works) {
#pragma unroll
            for (int i = 0; i < 4; ++i) dma16(xr[i] + kk, lds[buf][wave * 4 + i]);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int u = 0; u < 2; ++u)
                dma16(w + i * wstep + (size_t)(s + u) * 512, lds[buf][32 + (wave * 2 + i) * 2 + u]);
    };
    f32x4 acc[8][4];  // [weight fragment][row fragment]
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[j][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int wm = (wave >> 1) * 4, wn = (wave & 1) * 8;
    const int piece = r16 >> 3, at = (r16 & 7) * 64;  // of a 16-row fragment
    stage(0, 0);
    dma_barrier();
    int buf = 0;
    for (int s = 0; s < ksteps; s += 2, buf ^= 1) {
        if (s + 2 < ksteps) stage(s + 2, buf ^ 1);
        if (works) {
            __builtin_amdgcn_s_setprio(1);  // before the waves that still issue transfers
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int slot = ((u * 4 + g) ^ (r16 & 7)) * 8;
                bf16x8 xf[4];
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    xf[i] = *reinterpret_cast<const bf16x8*>(
                        &lds[buf][(wm + i) * 2 + piece][at + slot]);
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const bf16x8 wf = *reinterpret_cast<const bf16x8*>(
                        &lds[buf][32 + (wn + j) * 2 + u][lane * 8]);
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc[j][i] = mfma16(wf, xf[i], acc[j][i]);
                }
            }
            __builtin_amdgcn_s_setprio(0);
        }
        dma_barrier();
    }
    if (!works) return;
    const int f0 = nf0 + wn;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = tile * 256 + (wm + i) * 16 + r16;
        bf16* o = (bf16*)a.out + (size_t)row * a.ld_out;
        if (GLU) {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int n = (f0 / 2 + j) * 16 + g * 4;
                if (n < a.N) store4(o + n, glu4(acc[2 * j][i], acc[2 * j + 1][i], a));
            }
        } else {
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int n = (f0 + j) * 16 + g * 4;
                if (n < a.N) store4(o + n, acc[j][i]);
            }
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
extern "C" hipError_t launch_route_topk(
    int* ids, float* weights, const float* z, const float* bias, float scale, int T, int E,
    int top, hipStream_t stream) {
    if (T <= 0) return hipSuccess;
    if (E > MAX_EXPERTS || top > 64 || top > E || top < 1) return hipErrorInvalidValue;
    const int grid = ceil_div_i(T, 4);
#define GO(PER) \
    route_topk_kernel<PER><<<grid, 256, 0, stream>>>(ids, weights, z, bias, scale, T, E, top)
    if (E <= 64) GO(1);
    else if (E <= 256) GO(4);
    else GO(16);
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}

extern "C" hipError_t launch_route_plan(
    int* slot, int* row_token, int* tile_info, const int* ids, int n, int top, int E,
    int tile_rows, int max_tiles, hipStream_t stream) {
    if (n <= 0) return hipSuccess;
    if (E > MAX_EXPERTS) return hipErrorInvalidValue;
    route_plan_kernel<<<1, 1024, 0, stream>>>(
        slot, row_token, tile_info, ids, n, top, E, tile_rows, max_tiles);
    HIP_CHECK_LAST();
    return hipSuccess;
}

// glu: 0 none, 1 clamped, 2 silu; frag: weights in fragments (bf16), else dense
// [E, N or 2N, K] and tiles of 16 rows
extern "C" hipError_t launch_expert_product(
    void* out, int64_t ld_out, const void* x, int64_t ldx, const void* w, const int* row_token,
    const int* tile_info, int N, int K, int glu, float limit, int frag, int nfrags,
    int ksteps, int tile_rows, int max_tiles, int f32, hipStream_t stream) {
    if (max_tiles <= 0) return hipSuccess;
    const ExpertArgs a = {out, x, w, row_token, tile_info, max_tiles, ldx, ld_out, N, K,
                          glu == 2, limit};
    if (!frag) {
        if (tile_rows != 16) return hipErrorInvalidValue;
        const dim3 grid(max_tiles, ceil_div_i(N, 16));
        if (f32) {
            if (glu) expert_any_kernel<float, true><<<grid, 256, 0, stream>>>(a);
            else {
                expert_any_kernel<float, false><<<grid, 256, 0, stream>>>(a);
            }
        } else {
            if (glu) expert_any_kernel<bf16, true><<<grid, 256, 0, stream>>>(a);
            else {
                expert_any_kernel<bf16, false><<<grid, 256, 0, stream>>>(a);
            }
        }
        HIP_CHECK_LAST();
        return hipSuccess;
    }
    if (f32 || nfrags % 16 || ksteps % 2 || N % 8 || K % 8 || ldx % 8 || ld_out % 8 ||
        ksteps * 32 < K || nfrags * 16 < (glu ? 2 : 1) * N)
        return hipErrorInvalidValue;
    if (tile_rows == 256) {
        const int ntn = nfrags / 16, grid = ceil_div_i(max_tiles * ntn, 8) * 8;
        if (glu) expert_tile_kernel<true><<<grid, 512, 0, stream>>>(a, nfrags, ksteps, ntn);
        else {
            expert_tile_kernel<false><<<grid, 512, 0, stream>>>(a, nfrags, ksteps, ntn);
        }
        HIP_CHECK_LAST();
        return hipSuccess;
    }
    const dim3 grid(nfrags / 4, max_tiles);
#define GO(MF)                                                                            \
    {                                                                                     \
        if (glu) expert_stream_kernel<MF, true><<<grid, 256, 0, stream>>>(a, nfrags, ksteps); \
        else {                                                                           \
            expert_stream_kernel<MF, false><<<grid, 256, 0, stream>>>(a, nfrags, ksteps);\
        }                                                                                \
    }
    if (tile_rows == 16) GO(1)
    else if (tile_rows == 32) GO(2)
    else if (tile_rows == 64) GO(4)
    else return hipErrorInvalidValue;
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}
