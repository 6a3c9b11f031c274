// Linear recurrences for gfx950, token by token: Mamba-2 (SSD), mLSTM and
// fixed decays (lightning attention) over the segments of a flat batch, state
// in fp32.
//
// A state matrix is kept transposed, [value dim][key dim], key dim dense: 16
// lanes share a value row and hold its key dims as float4s, so state traffic
// is coalesced and a read-out is a 4-step shuffle. One workgroup: one
// segment, one head, 64 value rows (16 lane groups x 4 rows); state stays in
// registers over the segment's tokens. Bandwidth bound at one token.

#include "mfma.h"
#include "recurrence.h"

#define SCAN_ROWS 64  // value rows per workgroup

// ---------------------------------------------------------------------------
// SCAN_SSD:   S <- exp(-e^A dt) S + dt x B^T, y = S C + D x
// SCAN_MLSTM: S, n with log gates i, f and running maximum m;
//             y = S q / (max(|n.q|, e^-m) + 1e-6)
// SCAN_FIXED: S <- decay S + silu(v) silu(k)^T, y = S silu(q)
// Every 64-row tile of S keeps its own copy of n and m (they are read by
// every tile and written at the end).
// ---------------------------------------------------------------------------
enum { SCAN_SSD, SCAN_MLSTM, SCAN_FIXED };

struct ScanArgs {
    void* y;              // [T, H*dv]
    const void* q;        // SSD: C        rows of stride ldq, head stride via group
    const void* k;        // SSD: B
    const void* v;        // SSD: x
    int64_t ldq, ldk, ldv;
    const float* gates;   // SSD: raw dt [T, H]; mLSTM: raw i | f [T, 2H]
    const float* bias;    // SSD: dt_bias [H]; mLSTM: [2H]
    const float* A_log;   // SSD [H]; fixed: the decays
    const float* D;       // SSD [H]
    float cap, qscale;
    int H, per_group, dk, dv;
    float* S;             // [slots, H, dv, dk]
    float* n;             // [slots, tiles, H, dk]
    float* m;             // [slots, tiles, H]
    const int64_t* positions;
    const int* cu;
    const int* slots;
    const int* seg_list;  // nullable: the segments to run
};

__device__ __forceinline__ float scan_silu(float z) { return z / (1.f + expf(-z)); }

template <typename T, int E4, int KIND>
__launch_bounds__(256)
__global__ void scan_kernel(ScanArgs a) {
    constexpr bool MLSTM = KIND == SCAN_MLSTM;
    const int seg = a.seg_list ? a.seg_list[blockIdx.z] : blockIdx.z;
    const int h = blockIdx.y, tile = blockIdx.x, tiles = gridDim.x;
    const int slot = a.slots[seg];
    const int r0 = a.cu[seg], r1 = a.cu[seg + 1];
    const int l16 = threadIdx.x & 15, grp = threadIdx.x >> 4;
    const int row0 = tile * SCAN_ROWS + grp * 4;
    const int dk = a.dk, dv = a.dv, H = a.H;
    T* y = (T*)a.y;
    if (slot < 0) {  // padding row
        for (int t = r0; t < r1; ++t)
            if (l16 < 4 && row0 + l16 < dv)
                stf(y + (size_t)t * H * dv + (size_t)h * dv + row0 + l16, 0.f);
        return;
    }
    const int hk = h / a.per_group;
    const bool fresh = a.positions[r0] == 0;
    const bool vec = (dk & 3) == 0;
    float* Sp = a.S + ((size_t)slot * H + h) * dv * dk;
    float* np = MLSTM ? a.n + (((size_t)slot * tiles + tile) * H + h) * dk : nullptr;
    float* mp = MLSTM ? a.m + ((size_t)slot * tiles + tile) * H + h : nullptr;
    float S[4][E4][4], nv[E4][4];
    float m = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        if (!fresh && row0 + r < dv) {
            load_state<E4, true>(Sp + (size_t)(row0 + r) * dk, l16, dk, vec, S[r]);
        } else {
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) S[r][e][j] = 0.f;
        }
    }
    if (MLSTM) {
        if (!fresh) {
            load_state<E4>(np, l16, dk, vec, nv);
            m = *mp;
        } else {
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) nv[e][j] = 0.f;
        }
    }
    for (int t = r0; t < r1; ++t) {
        float k[E4][4], q[E4][4], v[4], keep, add;
        load_dims<T, E4>((const T*)a.k + (size_t)t * a.ldk + (size_t)hk * dk, l16, dk, k);
        load_dims<T, E4>((const T*)a.q + (size_t)t * a.ldq + (size_t)hk * dk, l16, dk, q);
        const T* vp = (const T*)a.v + (size_t)t * a.ldv + (size_t)h * dv;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = row0 + r < dv ? ldf(vp + row0 + r) : 0.f;
        if (KIND == SCAN_FIXED) {
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    k[e][j] = scan_silu(k[e][j]);
                    q[e][j] = scan_silu(q[e][j]);
                }
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = scan_silu(v[r]);
            keep = a.A_log[h];
            add = 1.f;
        } else if (MLSTM) {
            const float* g = a.gates + (size_t)t * 2 * H;
            const float i = soft_cap_f(g[h] + a.bias[h], a.cap);
            const float f = log_sigmoid_f(soft_cap_f(g[H + h] + a.bias[H + h], a.cap));
            const float m_new = fmaxf(f + m, i);
            keep = expf(f + m - m_new);
            add = expf(i - m_new);
            m = m_new;
        } else {
            const float dt = softplus_f(a.gates[(size_t)t * H + h] + a.bias[h]);
            keep = expf(-expf(a.A_log[h]) * dt);
            add = dt;
        }
        float den = 1.f;
        if (MLSTM) {
            float nq = 0.f;
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    q[e][j] *= a.qscale;
                    nv[e][j] = keep * nv[e][j] + add * k[e][j];
                    nq = fmaf(nv[e][j], q[e][j], nq);
                }
            den = fmaxf(fabsf(row16_sum(nq)), expf(-m)) + 1e-6f;
        }
        float o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float av = add * v[r];
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    S[r][e][j] = fmaf(av, k[e][j], keep * S[r][e][j]);
                    s = fmaf(S[r][e][j], q[e][j], s);
                }
            o[r] = row16_sum(s);
        }
        const float dh = KIND == SCAN_SSD ? a.D[h] : 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (l16 == r && row0 + r < dv)
                stf(y + (size_t)t * H * dv + (size_t)h * dv + row0 + r,
                    MLSTM ? o[r] / den : o[r] + dh * v[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
        if (row0 + r < dv)
            store_state<E4>(Sp + (size_t)(row0 + r) * dk, l16, dk, vec, S[r]);
    if (MLSTM && grp == 0) {
        store_state<E4>(np, l16, dk, vec, nv);
        if (l16 == 0) *mp = m;
    }
}

template <typename T, int KIND>
static hipError_t scan_go(const ScanArgs& a, int nseg, hipStream_t stream) {
    const dim3 grid(ceil_div_i(a.dv, SCAN_ROWS), a.H, nseg);  // neighbours share a state
    if (a.dk <= 64) scan_kernel<T, 1, KIND><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 128) scan_kernel<T, 2, KIND><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 256) scan_kernel<T, 4, KIND><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 512) scan_kernel<T, 8, KIND><<<grid, 256, 0, stream>>>(a);
    else return hipErrorInvalidValue;
    HIP_CHECK_LAST();
    return hipSuccess;
}

extern "C" hipError_t launch_ssd_scan(
    void* y, const void* xbc, int64_t ld, const float* dt, const float* dt_bias,
    const float* A_log, const float* D, int H, int P, int N, int G, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* seg_list,
    int nseg, int f32, hipStream_t stream) {
    if (nseg <= 0) return hipSuccess;
    const size_t es = f32 ? 4 : 2;
    ScanArgs a = {};
    a.y = y;
    a.v = xbc;
    a.k = (const char*)xbc + (size_t)H * P * es;
    a.q = (const char*)xbc + ((size_t)H * P + (size_t)G * N) * es;
    a.ldq = a.ldk = a.ldv = ld;
    a.gates = dt; a.bias = dt_bias; a.A_log = A_log; a.D = D;
    a.H = H; a.per_group = H / G; a.dk = N; a.dv = P;
    a.S = S; a.positions = positions; a.cu = cu; a.slots = slots; a.seg_list = seg_list;
    return f32 ? scan_go<float, SCAN_SSD>(a, nseg, stream) : scan_go<bf16, SCAN_SSD>(a, nseg, stream);
}

extern "C" hipError_t launch_mlstm_scan(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* gates, const float* bias, float cap, float qscale, int H,
    int dk, int dv, float* S, float* n, float* m, const int64_t* positions, const int* cu,
    const int* slots, const int* seg_list, int nseg, int f32, hipStream_t stream) {
    if (nseg <= 0) return hipSuccess;
    ScanArgs a = {};
    a.y = y; a.q = q; a.k = k; a.v = v; a.ldq = ldq; a.ldk = ldk; a.ldv = ldv;
    a.gates = gates; a.bias = bias; a.cap = cap; a.qscale = qscale;
    a.H = H; a.per_group = 1; a.dk = dk; a.dv = dv;
    a.S = S; a.n = n; a.m = m;
    a.positions = positions; a.cu = cu; a.slots = slots; a.seg_list = seg_list;
    return f32 ? scan_go<float, SCAN_MLSTM>(a, nseg, stream) : scan_go<bf16, SCAN_MLSTM>(a, nseg, stream);
}

extern "C" hipError_t launch_fixed_scan(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* decay, int H, int dk, int dv, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* seg_list, int nseg,
    int f32, hipStream_t stream) {
    if (nseg <= 0) return hipSuccess;
    ScanArgs a = {};
    a.y = y; a.q = q; a.k = k; a.v = v; a.ldq = ldq; a.ldk = ldk; a.ldv = ldv;
    a.A_log = decay; a.H = H; a.per_group = 1; a.dk = dk; a.dv = dv; a.S = S;
    a.positions = positions; a.cu = cu; a.slots = slots; a.seg_list = seg_list;
    return f32 ? scan_go<float, SCAN_FIXED>(a, nseg, stream) : scan_go<bf16, SCAN_FIXED>(a, nseg, stream);
}
