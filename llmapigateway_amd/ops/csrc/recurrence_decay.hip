// Linear recurrences with a decay per key channel for gfx950 (gated linear
// attention, WKV): per head, with q, k in dk and v in dv dimensions,
//
//   GLA:  S_t = diag(w_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t
//   WKV:  o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t,  then S_t as above
//
// The log decays log w come from a low-rank product (decay_logs). The state
// is fp32, transposed [slots, H, dv, dk] as in recurrence.hip. Token by
// token (decoding, short portions, fp32, any size) or in chunks of 64 rows
// on MFMA. With F the chunk's inclusive sums of log w and E_t = F_t (GLA) or
// F_(t-1) (WKV), all exponents below are <= 0:
//
//   o_t   = (q_t e^(E_t))^T S_in + sum_{s<t} P[t,s] v_s + d_t v_t
//   P[t,s] = sum_i q_t[i] k_s[i] e^(E_t[i] - F_s[i]),  d_t = q_t.(u k_t), u = 1 for GLA
//   S_out = diag(e^(F_L)) S_in + sum_s (k_s e^(F_L - F_s)) v_s^T
//
// P between two 16-row blocks factors through the sum R before the later one:
// (q e^(E_t-R)).(k e^(R-F_s)); inside a block it is taken row by row.

#include "lds_dma.h"
#include "mfma.h"
#include "recurrence.h"

#define CH 64  // rows per chunk
#define LDT (CH + 8)

// ---------------------------------------------------------------------------
// log decays from z = act(a) W2^T + bias
//   LOG_EXP:      act = tanh, log w = -e^z            (w = exp(-exp(z)))
//   LOG_SIGMOID:  act = id,   log w = log sigmoid(z) * c,   c = 1 / tau
//   LOG_SOFTPLUS: act = id,   log w = -softplus(z) * c,     c = rate[channel]
// ---------------------------------------------------------------------------
enum { LOG_SIGMOID, LOG_EXP, LOG_SOFTPLUS };

template <int KIND>
__device__ __forceinline__ float log_decay(float z, float c) {
    // e^-80 is as good as 0, and sums of 64 of them keep their precision
    if (KIND == LOG_EXP) return fmaxf(-expf(z), -80.f);
    return fmaxf(log_sigmoid_f(KIND == LOG_SOFTPLUS ? -z : z) * c, -80.f);
}

// the same for bf16 steps, whose z has bf16 rounding in it: hardware exponential
// and logarithm, log(1 + x) by its series where x is small
template <int KIND>
__device__ __forceinline__ float log_decay_fast(float z, float c) {
    if (KIND == LOG_EXP) return fmaxf(-__expf(z), -80.f);
    if (KIND == LOG_SOFTPLUS) z = -z;
    const float x = __expf(-fabsf(z));
    const float l = x < 0.02f ? x * (1.f + x * (-0.5f + x * (1.f / 3.f))) : __logf(1.f + x);
    return fmaxf((fminf(z, 0.f) - l) * c, -80.f);
}

#define DL_ROWS 8
template <typename T, int KIND>
__launch_bounds__(256)
__global__ void decay_logs_any_kernel(
    float* __restrict__ out, const T* __restrict__ a, int64_t lda, const T* __restrict__ w2,
    const float* __restrict__ bias, const float* __restrict__ rate, float inv_tau, int rows,
    int N, int R) {
    extern __shared__ float act[];  // [DL_ROWS][R]
    const int t0 = blockIdx.x * DL_ROWS, n = blockIdx.y * 256 + threadIdx.x;
    for (int e = threadIdx.x; e < DL_ROWS * R; e += 256) {
        const int t = t0 + e / R;
        const float v = t < rows ? ldf(a + (size_t)t * lda + e % R) : 0.f;
        act[e] = KIND == LOG_EXP ? tanhf(v) : v;
    }
    __syncthreads();
    if (n >= N) return;
    float z[DL_ROWS];
#pragma unroll
    for (int i = 0; i < DL_ROWS; ++i) z[i] = bias[n];
    for (int r = 0; r < R; ++r) {
        const float w = ldf(w2 + (size_t)n * R + r);
#pragma unroll
        for (int i = 0; i < DL_ROWS; ++i) z[i] = fmaf(act[i * R + r], w, z[i]);
    }
#pragma unroll
    for (int i = 0; i < DL_ROWS; ++i)
        if (t0 + i < rows)
            out[(size_t)(t0 + i) * N + n] =
                log_decay<KIND>(z[i], KIND == LOG_SOFTPLUS ? rate[n] : inv_tau);
}

// MFMA form: a wave takes 16 rows x 64 channels; C fragments hold [channel][row]
template <int KIND>
__launch_bounds__(256)
__global__ void decay_logs_mfma_kernel(
    float* __restrict__ out, const bf16* __restrict__ a, int64_t lda,
    const bf16* __restrict__ w2, const float* __restrict__ bias,
    const float* __restrict__ rate, float inv_tau, int rows, int N, int R) {
    constexpr bool EXP = KIND == LOG_EXP;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
    const int t = (blockIdx.y * 4 + wave) * 16 + r16, n0 = blockIdx.x * 64;
    if ((blockIdx.y * 4 + wave) * 16 >= rows) return;
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    // 128 of the rank at a time, all loads ahead of the products; past an end
    // any row, or rank 0 against zeros
    const bf16* ar = a + (size_t)min(t, rows - 1) * lda;
    const bf16* wr[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) wr[j] = w2 + (size_t)min(n0 + j * 16 + r16, N - 1) * R;
    for (int r0 = 0; r0 < R; r0 += 128) {
        uint4 x[4], w[4][4];
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            const int r = r0 + s * 32 + g * 8, rr = r < R ? r : 0;
            x[s] = *reinterpret_cast<const uint4*>(ar + rr);
#pragma unroll
            for (int j = 0; j < 4; ++j) w[s][j] = *reinterpret_cast<const uint4*>(wr[j] + rr);
            if (r >= R) x[s] = (uint4){0, 0, 0, 0};
        }
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            float f[8];
            bf16x8 hi, lo;
            unpack8(x[s], f);
            if (EXP) {
#pragma unroll
                for (int i = 0; i < 8; ++i) f[i] = tanh_fast(f[i]);
            }
            split_frag(f, hi, lo);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                acc[j] = mfma16(as_frag(w[s][j]), hi, acc[j]);
                if (EXP) acc[j] = mfma16(as_frag(w[s][j]), lo, acc[j]);
            }
        }
    }
    if (t >= rows) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int n = n0 + j * 16 + g * 4;
        if (n >= N) continue;  // N is a multiple of 4
        const float4 b = *reinterpret_cast<const float4*>(bias + n);
        float4 c = make_float4(inv_tau, inv_tau, inv_tau, inv_tau);
        if (KIND == LOG_SOFTPLUS) c = *reinterpret_cast<const float4*>(rate + n);
        *reinterpret_cast<float4*>(out + (size_t)t * N + n) = make_float4(
            log_decay_fast<KIND>(acc[j][0] + b.x, c.x), log_decay_fast<KIND>(acc[j][1] + b.y, c.y),
            log_decay_fast<KIND>(acc[j][2] + b.z, c.z), log_decay_fast<KIND>(acc[j][3] + b.w, c.w));
    }
}

// ---------------------------------------------------------------------------
// Token by token: a workgroup holds 64 value rows of a head's state in
// registers over a segment's tokens; 16 lanes share 4 value rows, a lane
// holds key dims 64e + 4*l16 + j.
// ---------------------------------------------------------------------------
struct DecayArgs {
    void* y;              // [T, H*dv]
    const void *q, *k, *v;
    int64_t ldq, ldk, ldv;
    float* logw;          // [T, H*dk]
    const float* u;       // WKV: [H, dk]
    float qscale;
    int T, H, dk, dv;
    float* S;             // [slots, H, dv, dk]
    const int64_t* positions;
    const int *cu, *slots;
    const int* seg_list;  // scan: nullable
    // chunks
    const int *segs, *first, *chunk_seg, *chunk_off;
    uint16_t *s_hi, *s_lo;  // [chunks, H, dv, dk]
};

template <typename T, int E4, bool WKV>
__launch_bounds__(256)
__global__ void decay_scan_kernel(DecayArgs a) {
    const int seg = a.seg_list ? a.seg_list[blockIdx.z] : blockIdx.z;
    const int h = blockIdx.y, slot = a.slots[seg];
    const int r0 = a.cu[seg], r1 = a.cu[seg + 1];
    const int l16 = threadIdx.x & 15, grp = threadIdx.x >> 4;
    const int row0 = blockIdx.x * 64 + grp * 4;
    const int dk = a.dk, dv = a.dv, H = a.H;
    T* y = (T*)a.y + (size_t)h * dv;
    if (slot < 0) {  // padding row
        for (int t = r0; t < r1; ++t)
            if (l16 < 4 && row0 + l16 < dv) stf(y + (size_t)t * H * dv + row0 + l16, 0.f);
        return;
    }
    const bool fresh = a.positions[r0] == 0, vec = (dk & 3) == 0;
    float* Sp = a.S + ((size_t)slot * H + h) * dv * dk;
    float S[4][E4][4], u[E4][4];
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
    if (WKV) load_state<E4>(a.u + (size_t)h * dk, l16, dk, false, u);
    for (int t = r0; t < r1; ++t) {
        float k[E4][4], q[E4][4], w[E4][4], v[4], o[4];
        load_dims<T, E4>((const T*)a.k + (size_t)t * a.ldk + (size_t)h * dk, l16, dk, k);
        load_dims<T, E4>((const T*)a.q + (size_t)t * a.ldq + (size_t)h * dk, l16, dk, q);
        load_state<E4>(a.logw + ((size_t)t * H + h) * dk, l16, dk, vec, w);
        const T* vp = (const T*)a.v + (size_t)t * a.ldv + (size_t)h * dv;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = row0 + r < dv ? ldf(vp + row0 + r) : 0.f;
        float bonus = 0.f;
#pragma unroll
        for (int e = 0; e < E4; ++e)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                q[e][j] *= a.qscale;
                w[e][j] = expf(w[e][j]);
                if (WKV) bonus = fmaf(q[e][j] * u[e][j], k[e][j], bonus);
            }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float s = WKV ? bonus * v[r] : 0.f;
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float next = fmaf(v[r], k[e][j], w[e][j] * S[r][e][j]);
                    s = fmaf(WKV ? S[r][e][j] : next, q[e][j], s);
                    S[r][e][j] = next;
                }
            o[r] = row16_sum(s);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (l16 == r && row0 + r < dv) stf(y + (size_t)t * H * dv + row0 + r, o[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
        if (row0 + r < dv) store_state<E4>(Sp + (size_t)(row0 + r) * dk, l16, dk, vec, S[r]);
}

// ---------------------------------------------------------------------------
// Chunked form. logw becomes F in place, per chunk.
// ---------------------------------------------------------------------------
__launch_bounds__(256)
__global__ void decay_sums_kernel(DecayArgs a) {
    const int c = blockIdx.x, N = a.H * a.dk, i = blockIdx.y * 256 + threadIdx.x;
    if (i >= N) return;
    const int seg = a.chunk_seg[c], r0 = a.cu[seg] + a.chunk_off[c];
    const int n = min(CH, a.cu[seg + 1] - r0);
    float* p = a.logw + (size_t)r0 * N + i;
    float sum = 0.f;
    for (int s0 = 0; s0 < n; s0 += 8) {
        float f[8];
#pragma unroll
        for (int s = 0; s < 8; ++s) f[s] = s0 + s < n ? p[(size_t)(s0 + s) * N] : 0.f;
#pragma unroll
        for (int s = 0; s < 8; ++s) {
            sum += f[s];
            if (s0 + s < n) p[(size_t)(s0 + s) * N] = sum;
        }
    }
}

// grid (segments, H, dv tiles * dk tiles of 64): walks a segment's chunks and
// leaves the state before each. C fragments hold S[dk][dv]: wave = 16 key
// dims, lane = 4 consecutive key dims of one value dim per dv tile.
__launch_bounds__(256)
__global__ void decay_state_kernel(DecayArgs a) {
    __shared__ bf16 k_hi[CH][LDT], k_lo[CH][LDT], v_lds[CH][LDT];
    const int seg = a.segs[blockIdx.x], h = blockIdx.y;
    const int dk = a.dk, dv = a.dv, H = a.H, N = H * dk;
    const int nkt = (dk + 63) / 64, vt = blockIdx.z / nkt, kt = blockIdx.z % nkt;
    const int slot = a.slots[seg], row_lo = a.cu[seg], row_hi = a.cu[seg + 1];
    const int c_lo = a.first[blockIdx.x], c_hi = a.first[blockIdx.x + 1];
    const bool fresh = a.positions[row_lo] == 0;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const int kd = kt * 64 + wave * 16 + g * 4;  // first of this lane's key dims
    const bf16 *kp = (const bf16*)a.k + (size_t)h * dk, *vp = (const bf16*)a.v + (size_t)h * dv;
    const float* Fp = a.logw + (size_t)h * dk;
    f32x4 S[4];
    float* Sp = a.S + ((size_t)slot * H + h) * dv * dk;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int vd = vt * 64 + j * 16 + r16;
        S[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (!fresh && vd < dv && kd < dk)
            S[j] = *reinterpret_cast<const f32x4*>(Sp + (size_t)vd * dk + kd);
    }
    const int d8 = tid % 8 * 8, kcol = kt * 64 + d8;
    struct Rows {  // a chunk's operands on their way to LDS
        uint4 k[2], v[2];
        float F[2][8], Fl[8];
        f32x4 keep;
    };
    auto load_rows = [&](Rows& x, int r0) {
        const int last = min(r0 + CH, row_hi) - 1;
        x.keep = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (kd < dk) x.keep = *reinterpret_cast<const f32x4*>(Fp + (size_t)last * N + kd);
        if (kcol < dk) load8f(Fp + (size_t)last * N + kcol, x.Fl);
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int r = r0 + tid / 8 + u * 32;
            x.k[u] = x.v[u] = (uint4){0, 0, 0, 0};
            if (r < row_hi) {
                if (kcol < dk) {
                    x.k[u] = *reinterpret_cast<const uint4*>(kp + (size_t)r * a.ldk + kcol);
                    load8f(Fp + (size_t)r * N + kcol, x.F[u]);
                }
                if (vt * 64 + d8 < dv)
                    x.v[u] = *reinterpret_cast<const uint4*>(vp + (size_t)r * a.ldv + vt * 64 + d8);
            }
        }
    };
    // one chunk; its register set then takes the chunk after the next
    auto run_chunk = [&](Rows& x, int c) {
        const int r0 = row_lo + (c - c_lo) * CH;
        const size_t base = ((size_t)c * H + h) * dv;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int vd = vt * 64 + j * 16 + r16;
            if (vd < dv && kd < dk) {
                uint32_t hi[2], lo[2];
#pragma unroll
                for (int r = 0; r < 2; ++r) {
                    hi[r] = cvt_pk_bf16(S[j][2 * r], S[j][2 * r + 1]);
                    float p, q;
                    unpack2(hi[r], p, q);
                    lo[r] = cvt_pk_bf16(S[j][2 * r] - p, S[j][2 * r + 1] - q);
                }
                const size_t at = (base + vd) * dk + kd;
                *reinterpret_cast<uint2*>(a.s_hi + at) = make_uint2(hi[0], hi[1]);
                *reinterpret_cast<uint2*>(a.s_lo + at) = make_uint2(lo[0], lo[1]);
            }
        }
        // barriers that leave the loads of later chunks under way
        lds_barrier();  // the previous chunk's tiles have been read
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int s = tid / 8 + u * 32;
            float f[8];
            bf16x8 hi, lo;
            unpack8(x.k[u], f);
            if (r0 + s < row_hi && kcol < dk) {
#pragma unroll
                for (int i = 0; i < 8; ++i) f[i] *= __expf(x.Fl[i] - x.F[u][i]);
            }
            split_frag(f, hi, lo);
            *reinterpret_cast<bf16x8*>(&k_hi[s][d8]) = hi;
            *reinterpret_cast<bf16x8*>(&k_lo[s][d8]) = lo;
            *reinterpret_cast<uint4*>(&v_lds[s][d8]) = x.v[u];
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float f = __expf(x.keep[r]);
#pragma unroll
            for (int j = 0; j < 4; ++j) S[j][r] *= f;
        }
        if (c + 2 < c_hi) load_rows(x, r0 + 2 * CH);
        lds_barrier();
#pragma unroll
        for (int s0 = 0; s0 < CH; s0 += 32) {
            const bf16x8 ah = tr_frag(&k_hi[0][0], LDT, s0, wave * 16);
            const bf16x8 al = tr_frag(&k_lo[0][0], LDT, s0, wave * 16);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const bf16x8 vf = tr_frag(&v_lds[0][0], LDT, s0, j * 16);
                S[j] = mfma16(ah, vf, S[j]);
                S[j] = mfma16(al, vf, S[j]);
            }
        }
    };
    Rows even, odd;
    load_rows(even, row_lo);
    if (c_lo + 1 < c_hi) load_rows(odd, row_lo + CH);
    for (int c = c_lo; c < c_hi; c += 2) {
        run_chunk(even, c);
        if (c + 1 < c_hi) run_chunk(odd, c + 1);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int vd = vt * 64 + j * 16 + r16;
        if (vd < dv && kd < dk) *reinterpret_cast<f32x4*>(Sp + (size_t)vd * dk + kd) = S[j];
    }
}

// ---------------------------------------------------------------------------
// grid (chunks, H, dv / (64*NB)). First a wave takes 16 query rows: q e^E and
// the rows of P, to LDS; then 16*NB value dims: C fragments hold [dv][row].
// NC: 32-wide slices of the key dims.
// ---------------------------------------------------------------------------
template <int NC, int NB, bool WKV>
__launch_bounds__(256)
__global__ void decay_out_kernel(DecayArgs a) {
    constexpr int LDK = NC * 32 + 8, LDV = NB * 64 + 8;
    __shared__ __align__(16) bf16 q_lds[2][CH * LDK];
    __shared__ __align__(16) bf16 p_lds[2][CH * LDT];
    __shared__ __align__(16) bf16 v_lds[32 * LDV];  // half of the chunk's rows
    const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * NB * 64;
    const int dk = a.dk, dv = a.dv, H = a.H, N = H * dk;
    const int seg = a.chunk_seg[c], r0 = a.cu[seg] + a.chunk_off[c];
    const int n = min(CH, a.cu[seg + 1] - r0);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const bf16 *kp = (const bf16*)a.k + (size_t)r0 * a.ldk + (size_t)h * dk;
    const bf16 *vp = (const bf16*)a.v + (size_t)r0 * a.ldv + (size_t)h * dv;
    const float* Fp = a.logw + (size_t)r0 * N + (size_t)h * dk;
    uint4 v_late[NB];  // the other half
#pragma unroll
    for (int u = 0; u < NB; ++u) {
        const int e = tid + u * 256, s = e / (NB * 8), d = e % (NB * 8) * 8;
        uint4 x = {0, 0, 0, 0};
        v_late[u] = x;
        if (v0 + d < dv) {
            if (s < n) x = *reinterpret_cast<const uint4*>(vp + (size_t)s * a.ldv + v0 + d);
            if (s + 32 < n)
                v_late[u] = *reinterpret_cast<const uint4*>(vp + (size_t)(s + 32) * a.ldv + v0 + d);
        }
        *reinterpret_cast<uint4*>(v_lds + s * LDV + d) = x;
    }
    {
        const int b0 = wave * 16, t = min(b0 + r16, n - 1);  // this lane's row
        const bf16* qr = (const bf16*)a.q + (size_t)(r0 + t) * a.ldq + (size_t)h * dk;
        float* w_own = reinterpret_cast<float*>(&p_lds[0][b0 * LDT]);  // until P goes there
        f32x4 P[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) P[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        for (int cc = 0; cc < NC; ++cc) {
            const int d = cc * 32 + g * 8;
            const bool in = d < dk;
            const int dd = in ? d : 0;
            uint4 qraw = *reinterpret_cast<const uint4*>(qr + dd);
            if (!in) qraw = (uint4){0, 0, 0, 0};
            float q[8], E[8], R[8], f[8];
            bf16x8 qh, ql;
            unpack8(qraw, q);
            const int te = WKV ? t - 1 : t;
            if (te >= 0) {
                load8f(Fp + (size_t)te * N + dd, E);
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) E[i] = 0.f;
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) f[i] = q[i] * __expf(E[i]);
            split_frag(f, qh, ql);
            *reinterpret_cast<bf16x8*>(&q_lds[0][(b0 + r16) * LDK + d]) = qh;
            *reinterpret_cast<bf16x8*>(&q_lds[1][(b0 + r16) * LDK + d]) = ql;
            if (b0 >= n) continue;  // (uniform in the wave) no rows here
            if (wave > 0) {  // earlier blocks, through the sums before this one
                load8f(Fp + (size_t)(b0 - 1) * N + dd, R);
#pragma unroll
                for (int i = 0; i < 8; ++i) f[i] = q[i] * __expf(E[i] - R[i]);
                split_frag(f, qh, ql);
                for (int j = 0; j < wave; ++j) {
                    const int s = j * 16 + r16;
                    float Fs[8], k[8];
                    bf16x8 kh, kl;
                    unpack8(*reinterpret_cast<const uint4*>(kp + (size_t)s * a.ldk + dd), k);
                    load8f(Fp + (size_t)s * N + dd, Fs);
#pragma unroll
                    for (int i = 0; i < 8; ++i) k[i] *= __expf(R[i] - Fs[i]);
                    split_frag(k, kh, kl);
                    f32x4 p = j == 0 ? P[0] : j == 1 ? P[1] : P[2];
                    p = mfma16(qh, kh, p);
                    p = mfma16(qh, kl, p);
                    p = mfma16(ql, kh, p);
                    if (j == 0) P[0] = p;
                    else if (j == 1) P[1] = p;
                    else P[2] = p;
                }
            }
            // this block: row tt of P is row tt of q against k_s w_(s+1) .. w_tt
            // (WKV: .. w_(tt-1), and u k_tt): the decayed keys are carried from
            // row to row, lane r16 holds key r16 (0 before its row is there)
            float k[8], u[8], kt[8];
            unpack8(*reinterpret_cast<const uint4*>(kp + (size_t)t * a.ldk + dd), k);
            if (WKV) load8f(a.u + (size_t)h * dk + dd, u);
            {
                float Fs[8], Fb[8];
                load8f(Fp + (size_t)t * N + dd, Fs);
                if (t > 0) {
                    load8f(Fp + (size_t)(t - 1) * N + dd, Fb);
                } else {
#pragma unroll
                    for (int i = 0; i < 8; ++i) Fb[i] = 0.f;
                }
#pragma unroll
                for (int i = 0; i < 8; ++i) Fs[i] = __expf(Fs[i] - Fb[i]);
                float* wp = w_own + r16 * 32 + g * 8;
                reinterpret_cast<float4*>(wp)[0] = make_float4(Fs[0], Fs[1], Fs[2], Fs[3]);
                reinterpret_cast<float4*>(wp)[1] = make_float4(Fs[4], Fs[5], Fs[6], Fs[7]);
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) kt[i] = 0.f;
            const int rows = min(16, n - b0);
#pragma unroll 4
            for (int tt = 0; tt < rows; ++tt) {
                float w[8];
                load8f(w_own + tt * 32 + g * 8, w);
                const bool mine = r16 == tt;
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const float next = mine ? k[i] : kt[i] * w[i];
                    f[i] = WKV ? (mine ? u[i] * k[i] : kt[i]) : next;
                    kt[i] = next;
                }
                bf16x8 kh, kl;
                split_frag(f, kh, kl);
                uint4 qm = qraw;
                if (!mine) qm = (uint4){0, 0, 0, 0};
                P[3] = mfma16(as_frag(qm), kh, P[3]);
                P[3] = mfma16(as_frag(qm), kl, P[3]);
            }
        }
        // rows of P: blocks before this wave's, its own, zeros after
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            f32x4 p = (f32x4){0.f, 0.f, 0.f, 0.f};
            if (j == wave) p = P[3];
            else if (j < wave) p = P[j];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                uint16_t hi, lo;
                split_bf16(p[r], hi, lo);
                const int at = (b0 + g * 4 + r) * LDT + j * 16 + r16;
                *reinterpret_cast<uint16_t*>(&p_lds[0][at]) = hi;
                *reinterpret_cast<uint16_t*>(&p_lds[1][at]) = lo;
            }
        }
    }
    __syncthreads();
    f32x4 o[4][NB];  // [row block][16 value dims]
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < NB; ++j) o[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int vw = wave * NB * 16;  // first of this wave's value dims
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        if (u) {
            __syncthreads();
#pragma unroll
            for (int k = 0; k < NB; ++k) {
                const int e = tid + k * 256;
                *reinterpret_cast<uint4*>(v_lds + e / (NB * 8) * LDV + e % (NB * 8) * 8) = v_late[k];
            }
            __syncthreads();
        }
        bf16x8 vf[NB];
#pragma unroll
        for (int j = 0; j < NB; ++j) vf[j] = tr_frag(v_lds, LDV, 0, vw + j * 16);
#pragma unroll
        for (int i = u * 2; i < 4; ++i) {
            const int at = (i * 16 + r16) * LDT + u * 32 + g * 8;
            const bf16x8 ph = *reinterpret_cast<const bf16x8*>(&p_lds[0][at]);
            const bf16x8 pl = *reinterpret_cast<const bf16x8*>(&p_lds[1][at]);
#pragma unroll
            for (int j = 0; j < NB; ++j) {
                o[i][j] = mfma16(vf[j], ph, o[i][j]);
                o[i][j] = mfma16(vf[j], pl, o[i][j]);
            }
        }
    }
    const size_t sbase = ((size_t)c * H + h) * dv;
    for (int cc = 0; cc < NC; ++cc) {
        const int d = cc * 32 + g * 8;
        bf16x8 sh[NB], sl[NB];
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int vd = v0 + vw + j * 16 + r16;
            uint4 x = {0, 0, 0, 0}, y = {0, 0, 0, 0};
            if (vd < dv && d < dk) {
                x = *reinterpret_cast<const uint4*>(a.s_hi + (sbase + vd) * dk + d);
                y = *reinterpret_cast<const uint4*>(a.s_lo + (sbase + vd) * dk + d);
            }
            sh[j] = as_frag(x);
            sl[j] = as_frag(y);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int at = (i * 16 + r16) * LDK + d;
            const bf16x8 qh = *reinterpret_cast<const bf16x8*>(&q_lds[0][at]);
            const bf16x8 ql = *reinterpret_cast<const bf16x8*>(&q_lds[1][at]);
#pragma unroll
            for (int j = 0; j < NB; ++j) {
                o[i][j] = mfma16(sh[j], qh, o[i][j]);
                o[i][j] = mfma16(sl[j], qh, o[i][j]);
                o[i][j] = mfma16(sh[j], ql, o[i][j]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = i * 16 + r16;
        if (t >= n) continue;
        bf16* yr = (bf16*)a.y + ((size_t)(r0 + t) * H + h) * dv;
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int vd = v0 + vw + j * 16 + g * 4;
            if (vd < dv)
                *reinterpret_cast<uint2*>(yr + vd) = make_uint2(
                    cvt_pk_bf16(o[i][j][0] * a.qscale, o[i][j][1] * a.qscale),
                    cvt_pk_bf16(o[i][j][2] * a.qscale, o[i][j][3] * a.qscale));
        }
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
// vec: bf16, R a multiple of 8, N of 4, rows aligned for 16-byte loads
extern "C" hipError_t launch_decay_logs(
    float* out, const void* a, int64_t lda, const void* w2, const float* bias,
    const float* rate, int kind, float inv_tau, int rows, int N, int R, int f32, int vec,
    hipStream_t stream) {
    if (rows <= 0) return hipSuccess;
    if (kind < LOG_SIGMOID || kind > LOG_SOFTPLUS || (kind == LOG_SOFTPLUS) != (rate != nullptr))
        return hipErrorInvalidValue;
    const bool mfma = !f32 && vec;
    const dim3 grid = mfma ? dim3(ceil_div_i(N, 64), ceil_div_i(rows, 64))
                           : dim3(ceil_div_i(rows, DL_ROWS), ceil_div_i(N, 256));
    const size_t lds = mfma ? 0 : (size_t)DL_ROWS * R * sizeof(float);
    if (lds > 48 * 1024) return hipErrorInvalidValue;
#define GO(K)                                                                            \
    {                                                                                    \
        if (mfma)                                                                        \
            decay_logs_mfma_kernel<K><<<grid, 256, 0, stream>>>(                         \
                out, (const bf16*)a, lda, (const bf16*)w2, bias, rate, inv_tau, rows, N, R); \
        else if (f32)                                                                    \
            decay_logs_any_kernel<float, K><<<grid, 256, lds, stream>>>(                 \
                out, (const float*)a, lda, (const float*)w2, bias, rate, inv_tau, rows, N, R); \
        else                                                                             \
            decay_logs_any_kernel<bf16, K><<<grid, 256, lds, stream>>>(                  \
                out, (const bf16*)a, lda, (const bf16*)w2, bias, rate, inv_tau, rows, N, R); \
    }
    if (kind == LOG_EXP) GO(LOG_EXP)
    else if (kind == LOG_SOFTPLUS) GO(LOG_SOFTPLUS)
    else GO(LOG_SIGMOID)
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}

// F in place: the sums of logw [T, N] within every chunk of 64 rows
extern "C" hipError_t launch_decay_sums(
    float* logw, int N, const int* cu, const int* chunk_seg, const int* chunk_off, int nchunks,
    hipStream_t stream) {
    if (nchunks <= 0) return hipSuccess;
    DecayArgs a = {};
    a.logw = logw; a.H = 1; a.dk = N;
    a.cu = cu; a.chunk_seg = chunk_seg; a.chunk_off = chunk_off;
    decay_sums_kernel<<<dim3(nchunks, ceil_div_i(N, 256)), 256, 0, stream>>>(a);
    HIP_CHECK_LAST();
    return hipSuccess;
}

template <typename T, bool WKV>
static hipError_t decay_scan_go(const DecayArgs& a, int nseg, hipStream_t stream) {
    const dim3 grid(ceil_div_i(a.dv, 64), a.H, nseg);  // neighbours share a state
    if (a.dk <= 64) decay_scan_kernel<T, 1, WKV><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 128) decay_scan_kernel<T, 2, WKV><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 256) decay_scan_kernel<T, 4, WKV><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 512) decay_scan_kernel<T, 8, WKV><<<grid, 256, 0, stream>>>(a);
    else return hipErrorInvalidValue;
    HIP_CHECK_LAST();
    return hipSuccess;
}

extern "C" hipError_t launch_decay_scan(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* logw, const float* u, float qscale, int T, int H, int dk, int dv,
    float* S, const int64_t* positions, const int* cu, const int* slots, const int* seg_list,
    int nseg, int f32, hipStream_t stream) {
    if (nseg <= 0) return hipSuccess;
    DecayArgs a = {y, q, k, v, ldq, ldk, ldv, const_cast<float*>(logw), u, qscale, T, H, dk, dv,
                   S, positions, cu, slots, seg_list};
    if (u)
        return f32 ? decay_scan_go<float, true>(a, nseg, stream)
                   : decay_scan_go<bf16, true>(a, nseg, stream);
    return f32 ? decay_scan_go<float, false>(a, nseg, stream)
               : decay_scan_go<bf16, false>(a, nseg, stream);
}

template <bool WKV>
static hipError_t decay_out_go(const DecayArgs& a, int nchunks, hipStream_t stream) {
#define GO(NC, NB)                                                                       \
    decay_out_kernel<NC, NB, WKV>                                                        \
        <<<dim3(nchunks, a.H, ceil_div_i(a.dv, NB * 64)), 256, 0, stream>>>(a)
    if (a.dk <= 64) { if (a.dv <= 64) GO(2, 1); else if (a.dv <= 128) GO(2, 2); else GO(2, 4); }
    else if (a.dk <= 128) { if (a.dv <= 128) GO(4, 2); else GO(4, 4); }
    else GO(8, 2);
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}

// bf16; dk (up to 256) and dv multiples of 8; scratch planes [2, chunks, H, dv, dk]
extern "C" hipError_t launch_decay_chunked(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, float* logw, const float* u, float qscale, int T, int H, int dk, int dv,
    float* S, const int64_t* positions, const int* cu, const int* slots, const int* segs,
    const int* first, const int* chunk_seg, const int* chunk_off, int nsegs, int nchunks,
    void* planes, hipStream_t stream) {
    if (nchunks <= 0) return hipSuccess;
    if (dk % 8 || dv % 8 || ldq % 8 || ldk % 8 || ldv % 8 || dk > 256) return hipErrorInvalidValue;
    DecayArgs a = {y, q, k, v, ldq, ldk, ldv, logw, u, qscale, T, H, dk, dv,
                   S, positions, cu, slots, nullptr, segs, first, chunk_seg, chunk_off};
    a.s_hi = (uint16_t*)planes;
    a.s_lo = a.s_hi + (size_t)nchunks * H * dv * dk;
    decay_sums_kernel<<<dim3(nchunks, ceil_div_i(H * dk, 256)), 256, 0, stream>>>(a);
    HIP_CHECK_LAST();
    decay_state_kernel<<<dim3(nsegs, H, ceil_div_i(dv, 64) * ceil_div_i(dk, 64)), 256, 0, stream>>>(a);
    HIP_CHECK_LAST();
    return u ? decay_out_go<true>(a, nchunks, stream) : decay_out_go<false>(a, nchunks, stream);
}
