// Gated delta rule with a decay per key channel for gfx950. Per head, with q, k
// in dk and v in dv dimensions, k and q divided by their lengths:
//
//   S <- diag(g_t) S,  u_t = beta_t (v_t - S^T k_t),  S <- S + k_t u_t^T,
//   o_t = S^T q_t
//
// log g comes from decay_logs, beta is the sigmoid of b. The state is fp32,
// transposed [slots, H, dv, dk] as in recurrence.hip. Token by token (decoding,
// short portions, fp32, any size) or in chunks of 64 rows on MFMA. With F the
// chunk's inclusive sums of log g, capitals for the chunk's rows, and
//
//   A[t,s] = sum_i k_t[i] k_s[i] e^(F_t[i] - F_s[i])   (s < t),  P likewise of q, k (s <= t)
//   U = (1 + diag(beta) A)^-1 diag(beta) (V - (K e^F) S_in) = U0 - W S_in
//   O = (Q e^F) S_in + P U
//   S_out = diag(e^(F_L)) S_in + (K e^(F_L - F))^T U
//
// U0, W, P, Q e^F and K e^(F_L-F) do not depend on the state: delta_intra_kernel
// makes them for all chunks at once and leaves them in the fragments that
// delta_state_kernel, which walks a segment's chunks, feeds to MFMA as they
// stand. fp32 operands go in as the sum of two bf16. A and P factor through the
// sums R in front of a 16-row block, (k e^(F_t-R)).(k e^(R-F_s)); where R - F_s
// is above 60 inside the block they are taken row by row instead.
//
// Operands whose k index runs over rows or dims that an accumulator holds use
// its order: k slot (g, j) is row 4g+j of one 16-row fragment for j < 4 and row
// 4g+j-4 of the next one above (g = lane/16), so a product's result is the next
// product's operand without crossing lanes.

#include "lds_dma.h"
#include "mfma.h"
#include "recurrence.h"

#define CH 64  // rows per chunk
#define LDT (CH + 8)
#define STAGE 4096      // bf16 values of a transfer stage: 8 fragments
#define RING 8          // stages in LDS, a power of two
#define MAX_SPREAD 60.f

struct DeltaArgs {
    void* y;              // [T, H*dv]
    const void *q, *k, *v, *b;
    int64_t ldq, ldk, ldv, ldb;
    float* logw;          // [T, H*dk]; chunks: F
    float qscale;
    int T, H, per, dk, dv;  // per: heads a query/key head
    float* S;             // [slots, H, dv, dk]
    const int64_t* positions;
    const int *cu, *slots;
    const int* seg_list;  // scan: nullable
    // chunks
    const int *segs, *first, *chunk_seg, *chunk_off;
    bf16* frags;          // [chunks, H, 3 NC + 2 stages]: W, Q, P, K
    float* u0;            // [chunks, H, dv tiles of 32, 2048]
};

// ---------------------------------------------------------------------------
// Token by token: a workgroup holds 64 value rows of a head's state in
// registers over a segment's tokens; 16 lanes share 4 value rows, a lane
// holds key dims 64e + 4*l16 + j.
// ---------------------------------------------------------------------------
template <typename T, int E4>
__launch_bounds__(256)
__global__ void delta_scan_kernel(DeltaArgs a) {
    const int seg = a.seg_list ? a.seg_list[blockIdx.z] : blockIdx.z;
    const int h = blockIdx.y, hk = h / a.per, slot = a.slots[seg];
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
    float S[4][E4][4];
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
    for (int t = r0; t < r1; ++t) {
        float k[E4][4], q[E4][4], w[E4][4], v[4], o[4];
        load_dims<T, E4>((const T*)a.k + (size_t)t * a.ldk + (size_t)hk * dk, l16, dk, k);
        load_dims<T, E4>((const T*)a.q + (size_t)t * a.ldq + (size_t)hk * dk, l16, dk, q);
        load_state<E4>(a.logw + ((size_t)t * H + h) * dk, l16, dk, vec, w);
        const T* vp = (const T*)a.v + (size_t)t * a.ldv + (size_t)h * dv;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = row0 + r < dv ? ldf(vp + row0 + r) : 0.f;
        const float beta = 1.f / (1.f + expf(-ldf((const T*)a.b + (size_t)t * a.ldb + h)));
        float kk = 0.f, qq = 0.f;
#pragma unroll
        for (int e = 0; e < E4; ++e)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                kk = fmaf(k[e][j], k[e][j], kk);
                qq = fmaf(q[e][j], q[e][j], qq);
                w[e][j] = expf(w[e][j]);
            }
        const float rk = 1.f / sqrtf(row16_sum(kk) + 1e-6f);
        const float rq = a.qscale / sqrtf(row16_sum(qq) + 1e-6f);
#pragma unroll
        for (int e = 0; e < E4; ++e)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                k[e][j] *= rk;
                q[e][j] *= rq;
            }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    S[r][e][j] *= w[e][j];
                    s = fmaf(S[r][e][j], k[e][j], s);
                }
            const float u = beta * (v[r] - row16_sum(s));
            s = 0.f;
#pragma unroll
            for (int e = 0; e < E4; ++e)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    S[r][e][j] = fmaf(u, k[e][j], S[r][e][j]);
                    s = fmaf(S[r][e][j], q[e][j], s);
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
// Chunks
// ---------------------------------------------------------------------------
__device__ __forceinline__ f32x4 zero4() { return (f32x4){0.f, 0.f, 0.f, 0.f}; }

// two accumulators as one operand
__device__ __forceinline__ void split_pair(const f32x4& a, const f32x4& b, bf16x8& hi, bf16x8& lo) {
    const float f[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
    split_frag(f, hi, lo);
}
// a b with both as hi + lo
__device__ __forceinline__ f32x4 mfma3(bf16x8 ah, bf16x8 al, bf16x8 bh, bf16x8 bl, f32x4 c) {
    c = mfma16(ah, bh, c);
    c = mfma16(ah, bl, c);
    return mfma16(al, bh, c);
}
__device__ __forceinline__ void store_frag(bf16* stage, int index, int lane, const bf16x8& f) {
    *reinterpret_cast<bf16x8*>(stage + index * 512 + lane * 8) = f;
}

// (1 + L)^-1 R for a block of 16 columns, L the chunk's strictly lower matrix in
// 16x16 blocks: T are the inverses of the diagonal blocks, A the negated blocks
// below them (rows 1, 2, 3 over blocks 0|1, row 3 over blocks 2|3)
struct Solver {
    bf16x8 ah[4], al[4], th[4], tl[4];
    // X_i as [row][column] in x; as [column][row] in xt if it is given
    __device__ __forceinline__ void operator()(const f32x4* R, f32x4* x, f32x4* xt) const {
        bf16x8 h01, l01, h2, l2;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            f32x4 acc = R[i];
            if (i > 0) acc = mfma3(ah[i - 1], al[i - 1], h01, l01, acc);
            if (i == 3) acc = mfma3(ah[3], al[3], h2, l2, acc);
            bf16x8 rh, rl;
            split_pair(acc, zero4(), rh, rl);
            x[i] = mfma3(th[i], tl[i], rh, rl, zero4());
            if (xt) xt[i] = mfma3(rh, rl, th[i], tl[i], zero4());
            if (i == 0) split_pair(x[0], zero4(), h01, l01);
            if (i == 1) split_pair(x[0], x[1], h01, l01);
            if (i == 2) split_pair(x[2], zero4(), h2, l2);
        }
    }
};

// grid (chunks, H). NC: 32-wide slices of the key dims.
template <int NC>
__launch_bounds__(256)
__global__ void delta_intra_kernel(DeltaArgs a) {
    __shared__ __align__(16) bf16 a_lds[2][CH * LDT], p_lds[2][CH * LDT];
    __shared__ __align__(16) float own[4][16 * 20];  // diagonal blocks of A, transposed
    __shared__ __align__(16) float w_lds[4][16 * 32];
    __shared__ uint4 t_lds[4][64];
    __shared__ float rk_lds[CH], b_lds[CH];
    const int c = blockIdx.x, h = blockIdx.y, hk = h / a.per;
    const int dk = a.dk, dv = a.dv, H = a.H, N = H * dk;
    const int seg = a.chunk_seg[c], r0 = a.cu[seg] + a.chunk_off[c];
    const int n = min(CH, a.cu[seg + 1] - r0);
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const bf16 *qp = (const bf16*)a.q + (size_t)r0 * a.ldq + (size_t)hk * dk;
    const bf16 *kp = (const bf16*)a.k + (size_t)r0 * a.ldk + (size_t)hk * dk;
    const bf16 *vp = (const bf16*)a.v + (size_t)r0 * a.ldv + (size_t)h * dv;
    const float* Fp = a.logw + (size_t)r0 * N + (size_t)h * dk;
    bf16* frags = a.frags + ((size_t)c * H + h) * (3 * NC + 2) * STAGE;
    bf16 *w_st = frags, *q_st = frags + NC * STAGE, *p_st = frags + 2 * NC * STAGE;
    bf16* k_st = p_st + 2 * STAGE;
    const int b0 = wave * 16, t_own = min(b0 + r16, n - 1);  // this lane's row

    // lengths and betas
    float rq;
    {
        float qq = 0.f, kk = 0.f;
#pragma unroll
        for (int cc = 0; cc < NC; ++cc) {
            const int d = cc * 32 + g * 8;
            if (d >= dk) continue;
            float f[8];
            unpack8(*reinterpret_cast<const uint4*>(qp + (size_t)t_own * a.ldq + d), f);
#pragma unroll
            for (int i = 0; i < 8; ++i) qq = fmaf(f[i], f[i], qq);
            unpack8(*reinterpret_cast<const uint4*>(kp + (size_t)t_own * a.ldk + d), f);
#pragma unroll
            for (int i = 0; i < 8; ++i) kk = fmaf(f[i], f[i], kk);
        }
        qq += __shfl_xor(qq, 16, WAVE_SIZE);
        qq += __shfl_xor(qq, 32, WAVE_SIZE);
        kk += __shfl_xor(kk, 16, WAVE_SIZE);
        kk += __shfl_xor(kk, 32, WAVE_SIZE);
        rq = a.qscale / sqrtf(qq + 1e-6f);
        if (g == 0) {
            const float z = ldf((const bf16*)a.b + (size_t)(r0 + t_own) * a.ldb + h);
            rk_lds[b0 + r16] = 1.f / sqrtf(kk + 1e-6f);
            b_lds[b0 + r16] = b0 + r16 < n ? 1.f / (1.f + expf(-z)) : 0.f;
        }
    }
    __syncthreads();

    // rows of A and P against the blocks up to this wave's
    f32x4 P[4], A[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) P[j] = A[j] = zero4();
    if (b0 < n) {
        bf16x8 qh[NC], ql[NC], kh[NC], kl[NC];
        float R[NC][8];
        uint32_t far = 0;  // slices of the key dims whose own block does not factor
#pragma unroll
        for (int cc = 0; cc < NC; ++cc) {
            const int d = cc * 32 + g * 8, dd = d < dk ? d : 0;
            uint4 q = *reinterpret_cast<const uint4*>(qp + (size_t)t_own * a.ldq + dd);
            uint4 k = *reinterpret_cast<const uint4*>(kp + (size_t)t_own * a.ldk + dd);
            if (d >= dk) q = k = (uint4){0, 0, 0, 0};
            float E[8], f[8], spread = 0.f;
            load8f(Fp + (size_t)t_own * N + dd, E);
            if (b0 > 0) {
                load8f(Fp + (size_t)(b0 - 1) * N + dd, R[cc]);
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) R[cc][i] = 0.f;
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                spread = fmaxf(spread, R[cc][i] - E[i]);
                E[i] = __expf(E[i] - R[cc][i]);
            }
            if (__any(spread > MAX_SPREAD)) far |= 1u << cc;
            unpack8(q, f);
#pragma unroll
            for (int i = 0; i < 8; ++i) f[i] *= E[i];
            split_frag(f, qh[cc], ql[cc]);
            unpack8(k, f);
#pragma unroll
            for (int i = 0; i < 8; ++i) f[i] *= E[i];
            split_frag(f, kh[cc], kl[cc]);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > wave) continue;
            const int s = min(j * 16 + r16, n - 1);
            uint4 k[NC];
            float Fs[NC][8];
#pragma unroll
            for (int cc = 0; cc < NC; ++cc) {
                const int d = cc * 32 + g * 8, dd = d < dk ? d : 0;
                k[cc] = *reinterpret_cast<const uint4*>(kp + (size_t)s * a.ldk + dd);
                load8f(Fp + (size_t)s * N + dd, Fs[cc]);
            }
#pragma unroll
            for (int cc = 0; cc < NC; ++cc) {
                float f[8];
                bf16x8 sh, sl;
                unpack8(k[cc], f);
#pragma unroll
                for (int i = 0; i < 8; ++i) f[i] *= __expf(R[cc][i] - Fs[cc][i]);
                split_frag(f, sh, sl);
                if (j == wave && (far >> cc & 1)) continue;
                P[j] = mfma3(qh[cc], ql[cc], sh, sl, P[j]);
                A[j] = mfma3(kh[cc], kl[cc], sh, sl, A[j]);
            }
        }
        // the other slices of the own block, row by row: row tt against k_s
        // g_(s+1) .. g_tt, the decayed keys carried from row to row; lane r16
        // holds key r16 (0 before its row is there)
        for (int cc = 0; cc < NC; ++cc) {
            if (!(far >> cc & 1)) continue;
            const int d = cc * 32 + g * 8, dd = d < dk ? d : 0;
            uint4 qraw = *reinterpret_cast<const uint4*>(qp + (size_t)t_own * a.ldq + dd);
            uint4 kraw = *reinterpret_cast<const uint4*>(kp + (size_t)t_own * a.ldk + dd);
            if (d >= dk) qraw = kraw = (uint4){0, 0, 0, 0};
            float k[8], kt[8];
            unpack8(kraw, k);
            {
                float Fs[8], Fb[8];
                load8f(Fp + (size_t)t_own * N + dd, Fs);
                if (t_own > 0) {
                    load8f(Fp + (size_t)(t_own - 1) * N + dd, Fb);
                } else {
#pragma unroll
                    for (int i = 0; i < 8; ++i) Fb[i] = 0.f;
                }
                float* wp = w_lds[wave] + r16 * 32 + g * 8;
#pragma unroll
                for (int i = 0; i < 8; ++i) wp[i] = __expf(Fs[i] - Fb[i]);
            }
            __builtin_amdgcn_wave_barrier();
#pragma unroll
            for (int i = 0; i < 8; ++i) kt[i] = 0.f;
            const int rows = min(16, n - b0);
            for (int tt = 0; tt < rows; ++tt) {
                float w[8];
                load8f(w_lds[wave] + tt * 32 + g * 8, w);
                const bool mine = r16 == tt;
#pragma unroll
                for (int i = 0; i < 8; ++i) kt[i] = mine ? k[i] : kt[i] * w[i];
                bf16x8 sh, sl;
                split_frag(kt, sh, sl);
                uint4 qm = qraw, km = kraw;
                if (!mine) qm = km = (uint4){0, 0, 0, 0};
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    if (j != wave) continue;
                    P[j] = mfma16(as_frag(qm), sh, P[j]);
                    P[j] = mfma16(as_frag(qm), sl, P[j]);
                    A[j] = mfma16(as_frag(km), sh, A[j]);
                    A[j] = mfma16(as_frag(km), sl, A[j]);
                }
            }
            __builtin_amdgcn_wave_barrier();
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int s = j * 16 + r16;
        const float rks = rk_lds[s];
        f32x4 diag;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = b0 + g * 4 + r;
            const float rqt = __shfl(rq, g * 4 + r, WAVE_SIZE);
            const float p = s <= t && t < n ? P[j][r] * rqt * rks : 0.f;
            const float x = s < t && t < n ? A[j][r] * rk_lds[t] * rks * b_lds[t] : 0.f;
            uint16_t hi, lo;
            split_bf16(p, hi, lo);
            *reinterpret_cast<uint16_t*>(&p_lds[0][t * LDT + s]) = hi;
            *reinterpret_cast<uint16_t*>(&p_lds[1][t * LDT + s]) = lo;
            split_bf16(j < wave ? -x : 0.f, hi, lo);
            *reinterpret_cast<uint16_t*>(&a_lds[0][t * LDT + s]) = hi;
            *reinterpret_cast<uint16_t*>(&a_lds[1][t * LDT + s]) = lo;
            diag[r] = x;
        }
        if (j == wave) *reinterpret_cast<f32x4*>(&own[wave][r16 * 20 + g * 4]) = diag;
    }
    __syncthreads();
    {  // row r16 of the inverse of 1 + this wave's diagonal block, from its end
        float T[16];
#pragma unroll
        for (int col = 15; col >= 0; --col) {
            float x = col == r16 ? 1.f : 0.f;
#pragma unroll
            for (int s4 = col / 4; s4 < 4; ++s4) {
                const f32x4 l = *reinterpret_cast<const f32x4*>(&own[wave][col * 20 + s4 * 4]);
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (s4 * 4 + j > col) x = fmaf(-T[s4 * 4 + j], l[j], x);
            }
            T[col] = x;
        }
        f32x4 mine;
#pragma unroll
        for (int j = 0; j < 4; ++j)
            mine[j] = g == 0 ? T[j] : g == 1 ? T[4 + j] : g == 2 ? T[8 + j] : T[12 + j];
        bf16x8 hi, lo;
        split_pair(mine, zero4(), hi, lo);
        const uint4 *hp = reinterpret_cast<const uint4*>(&hi), *lp = reinterpret_cast<const uint4*>(&lo);
        t_lds[wave][lane] = make_uint4(hp->x, hp->y, lp->x, lp->y);
    }
    __syncthreads();

    auto row_frag = [&](const bf16* m, int row, int col) {  // columns col+4g.., col+16+4g..
        const uint2 x = *reinterpret_cast<const uint2*>(m + row * LDT + col + 4 * g);
        const uint2 y = *reinterpret_cast<const uint2*>(m + row * LDT + col + 16 + 4 * g);
        const uint4 v = make_uint4(x.x, x.y, y.x, y.y);
        return as_frag(v);
    };
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
        if (ks == 1 && wave < 2) continue;  // nothing above the diagonal
#pragma unroll
        for (int pl = 0; pl < 2; ++pl)
            store_frag(p_st + ks * STAGE, (wave - 2 * ks) * 2 + pl, lane,
                       row_frag(p_lds[pl], b0 + r16, ks * 32));
    }
    for (int i = tid; i < NC * 32; i += 256)  // behind P's last fragments
        reinterpret_cast<float*>(p_st + STAGE + 2048)[i] =
            i < dk ? __expf(Fp[(size_t)(n - 1) * N + i]) : 0.f;
    for (int kk = 0; kk < NC; ++kk) {
        float f[8];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int d = kk * 32 + u * 16 + 4 * g;
            const bool in = d < dk && b0 + r16 < n;
            const int dd = in ? d : 0;
            const uint2 x = *reinterpret_cast<const uint2*>(qp + (size_t)t_own * a.ldq + dd);
            const f32x4 F = *reinterpret_cast<const f32x4*>(Fp + (size_t)t_own * N + dd);
            unpack2(x.x, f[u * 4], f[u * 4 + 1]);
            unpack2(x.y, f[u * 4 + 2], f[u * 4 + 3]);
#pragma unroll
            for (int j = 0; j < 4; ++j) f[u * 4 + j] = in ? f[u * 4 + j] * rq * __expf(F[j]) : 0.f;
        }
        bf16x8 hi, lo;
        split_frag(f, hi, lo);
        store_frag(q_st + kk * STAGE, wave * 2, lane, hi);
        store_frag(q_st + kk * STAGE, wave * 2 + 1, lane, lo);
    }

    Solver solve;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint4 t = t_lds[i][lane];
        const uint4 th = make_uint4(t.x, t.y, 0, 0), tl = make_uint4(t.z, t.w, 0, 0);
        solve.th[i] = as_frag(th);
        solve.tl[i] = as_frag(tl);
        const int row = min(i + 1, 3) * 16 + r16, col = i == 3 ? 32 : 0;
        solve.ah[i] = row_frag(a_lds[0], row, col);
        solve.al[i] = row_frag(a_lds[1], row, col);
    }
    for (int kk = wave; kk < NC; kk += 4) {
        f32x4 xt[2][4];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int d = kk * 32 + u * 16 + r16, dd = min(d, dk - 1);
            const bool in = d < dk;
            const float Fl = Fp[(size_t)(n - 1) * N + dd];
            f32x4 R[4], K[4], x[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = i * 16 + g * 4 + r, tt = min(t, n - 1);
                    R[i][r] = Fp[(size_t)tt * N + dd];
                    K[i][r] = ldf(kp + (size_t)tt * a.ldk + dd);
                }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = i * 16 + g * 4 + r;
                    const float F = R[i][r], k = in && t < n ? K[i][r] * rk_lds[t] : 0.f;
                    R[i][r] = k * b_lds[t] * __expf(F);
                    K[i][r] = k * __expf(Fl - F);
                }
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                bf16x8 hi, lo;
                split_pair(K[2 * ks], K[2 * ks + 1], hi, lo);
                store_frag(k_st + kk * STAGE, u * 4 + ks * 2, lane, hi);
                store_frag(k_st + kk * STAGE, u * 4 + ks * 2 + 1, lane, lo);
            }
            solve(R, x, xt[u]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            bf16x8 hi, lo;
            split_pair(-xt[0][i], -xt[1][i], hi, lo);
            store_frag(w_st + kk * STAGE, i * 2, lane, hi);
            store_frag(w_st + kk * STAGE, i * 2 + 1, lane, lo);
        }
    }
    const int nvg = (dv + 31) / 32;
    float* u0 = a.u0 + ((size_t)c * H + h) * nvg * 2048;
    for (int vt = wave; vt < 2 * nvg; vt += 4) {
        const int d = vt * 16 + r16, dd = min(d, dv - 1);
        f32x4 R[4], x[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                R[i][r] = ldf(vp + (size_t)min(i * 16 + g * 4 + r, n - 1) * a.ldv + dd);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r)  // (rows past the last have a beta of 0)
                R[i][r] = d < dv ? R[i][r] * b_lds[i * 16 + g * 4 + r] : 0.f;
        solve(R, x, nullptr);
#pragma unroll
        for (int i = 0; i < 4; ++i)
            *reinterpret_cast<f32x4*>(u0 + (size_t)vt * 1024 + i * 256 + lane * 4) = x[i];
    }
}

// ---------------------------------------------------------------------------
// grid (segments, H, dv tiles of 32): walks a segment's chunks; a wave holds 16
// columns of the state, [dk][16], in accumulators. What a chunk needs comes in
// stages of 8 KB through a ring in LDS, half of each by either wave, RING - 1
// stages ahead: U0, then W and Q per 32 key dims, P per 32 rows (the decays of
// the state behind it), K per 32 key dims.
// ---------------------------------------------------------------------------
template <int NC>
__launch_bounds__(128)
__global__ void delta_state_kernel(DeltaArgs a) {
    constexpr int NS = 3 * NC + 3;
    static_assert((NS + RING - 1) / NS < 3, "chunks that stages are sent for");
    __shared__ __align__(16) bf16 ring[RING][STAGE];
    const int seg = a.segs[blockIdx.x], h = blockIdx.y, vg = blockIdx.z, nvg = gridDim.z;
    const int dk = a.dk, dv = a.dv, H = a.H;
    const int slot = a.slots[seg], row_lo = a.cu[seg], row_hi = a.cu[seg + 1];
    const int c_lo = a.first[blockIdx.x], c_hi = a.first[blockIdx.x + 1];
    const bool fresh = a.positions[row_lo] == 0;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = vg * 32 + wave * 16;  // first of this wave's value dims
    f32x4 S[2 * NC];
    float* Sp = a.S + ((size_t)slot * H + h) * dv * dk + (size_t)(v0 + r16) * dk;
#pragma unroll
    for (int j = 0; j < 2 * NC; ++j) {
        const int d = j * 16 + g * 4;
        S[j] = zero4();
        if (!fresh && v0 + r16 < dv && d < dk) S[j] = *reinterpret_cast<const f32x4*>(Sp + d);
    }
    // Stages are numbered from the chunk that is being read; which one a
    // position in the code sends for is known there. Past the segment's last
    // chunk, that one again.
    const bf16* fr[3];
    const float* u0[3];
    auto point = [&](int c) {
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            const size_t ch = (size_t)min(c + i, c_hi - 1) * H + h;
            fr[i] = a.frags + ch * (3 * NC + 2) * STAGE;
            u0[i] = a.u0 + (ch * nvg + vg) * 2048;
        }
    };
    const uint32_t ring_at = lds_address(ring) + wave * 4096, lane_at = wave * 4096 + lane * 16;
    uint32_t to_slot = 0, in_slot = 0;
    auto send = [&](int stage) {
        const int q = stage / NS, r = stage % NS;
        const void* src = r == 0 ? (const void*)u0[q] : (const void*)(fr[q] + (r - 1) * STAGE);
        const uint32_t to = ring_at + to_slot * (STAGE * 2);
#pragma unroll
        for (int u = 0; u < 4; ++u) dma16(src, lane_at + u * 1024, to + u * 1024);
        to_slot = (to_slot + 1) % RING;
    };
    // the data of stage j, here for both waves; the stage before it has been read
    auto next = [&](int j) -> const bf16* {
        // the transfers of later stages may be under way
        asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(4 * (RING - 2)) : "memory");
        send(j + RING - 1);
        const bf16* p = ring[in_slot];
        in_slot = (in_slot + 1) % RING;
        return p;
    };
    // a stage's fragments, read while the products of the stage before run
    struct Stage {
        bf16x8 f[8];
    };
    auto read = [&](Stage& x, const bf16* st, int first, int count) {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < count)
                x.f[i] = *reinterpret_cast<const bf16x8*>(st + (first + i) * 512 + lane * 8);
    };
    // c[i] += (hi + lo of x.f[2i], x.f[2i+1]) (bh + bl), or with the operands
    // the other way round; the three products of a sum lie apart
    auto products = [&](f32x4* c, const Stage& x, int n_c, bf16x8 bh, bf16x8 bl, bool left) {
#pragma unroll
        for (int p = 0; p < 3; ++p)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (i >= n_c) continue;
                const bf16x8 m = x.f[2 * i + (p == 2)], b = p == 1 ? bl : bh;
                c[i] = left ? mfma16(m, b, c[i]) : mfma16(b, m, c[i]);
            }
    };
    point(c_lo);
#pragma unroll
    for (int i = 0; i < RING - 1; ++i) send(i);
    Stage now, ahead;
    read(ahead, next(0), wave * 4, 4);
    for (int c = c_lo; c < c_hi; ++c) {
        const int r0 = row_lo + (c - c_lo) * CH, n = min(CH, row_hi - r0);
        point(c);
        f32x4 U[4], o[4], keep[2 * NC];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            U[i] = *reinterpret_cast<const f32x4*>(&ahead.f[i]);
            o[i] = zero4();
        }
        read(ahead, next(1), 0, 8);
        bf16x8 sh[NC], sl[NC];
#pragma unroll
        for (int kk = 0; kk < NC; ++kk) split_pair(S[2 * kk], S[2 * kk + 1], sh[kk], sl[kk]);
#pragma unroll
        for (int kk = 0; kk < NC; ++kk) {  // W: [row][dv]
            now = ahead;
            read(ahead, next(2 + kk), 0, 8);
            products(U, now, 4, sh[kk], sl[kk], true);
        }
#pragma unroll
        for (int kk = 0; kk < NC; ++kk) {  // Q: [dv][row]
            now = ahead;
            read(ahead, next(2 + NC + kk), 0, 8);
            products(o, now, 4, sh[kk], sl[kk], false);
        }
        bf16x8 uh[2], ul[2];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) split_pair(U[2 * ks], U[2 * ks + 1], uh[ks], ul[ks]);
        now = ahead;
        {
            const bf16* st = next(2 + 2 * NC);
            read(ahead, st, 0, 4);
#pragma unroll
            for (int j = 0; j < 2 * NC; ++j)
                keep[j] = *reinterpret_cast<const f32x4*>(
                    reinterpret_cast<const float*>(st + 2048) + j * 16 + g * 4);
        }
        products(o, now, 4, uh[0], ul[0], false);
        now = ahead;
        read(ahead, next(3 + 2 * NC), 0, 8);
        products(o + 2, now, 2, uh[1], ul[1], false);
#pragma unroll
        for (int j = 0; j < 2 * NC; ++j) S[j] *= keep[j];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = i * 16 + r16, d = v0 + g * 4;
            if (t < n && d < dv)
                *reinterpret_cast<uint2*>((bf16*)a.y + ((size_t)(r0 + t) * H + h) * dv + d) =
                    make_uint2(cvt_pk_bf16(o[i][0], o[i][1]), cvt_pk_bf16(o[i][2], o[i][3]));
        }
#pragma unroll
        for (int kk = 0; kk < NC; ++kk) {
            now = ahead;
            if (kk + 1 < NC) read(ahead, next(4 + 2 * NC + kk), 0, 8);
            else read(ahead, next(NS), wave * 4, 4);  // the next chunk's U0
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                for (int p = 0; p < 3; ++p)
#pragma unroll
                    for (int u = 0; u < 2; ++u)
                        S[2 * kk + u] = mfma16(now.f[u * 4 + ks * 2 + (p == 2)],
                                               p == 1 ? ul[ks] : uh[ks], S[2 * kk + u]);
        }
    }
    dma_barrier();  // nothing is on its way to LDS when the workgroup ends
#pragma unroll
    for (int j = 0; j < 2 * NC; ++j) {
        const int d = j * 16 + g * 4;
        if (v0 + r16 < dv && d < dk) *reinterpret_cast<f32x4*>(Sp + d) = S[j];
    }
}

// ---------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------
template <typename T>
static hipError_t delta_scan_go(const DeltaArgs& a, int nseg, hipStream_t stream) {
    const dim3 grid(ceil_div_i(a.dv, 64), a.H, nseg);  // neighbours share a state
    if (a.dk <= 64) delta_scan_kernel<T, 1><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 128) delta_scan_kernel<T, 2><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 256) delta_scan_kernel<T, 4><<<grid, 256, 0, stream>>>(a);
    else if (a.dk <= 512) delta_scan_kernel<T, 8><<<grid, 256, 0, stream>>>(a);
    else return hipErrorInvalidValue;
    HIP_CHECK_LAST();
    return hipSuccess;
}

static DeltaArgs delta_args(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v, int64_t ldv,
    float* logw, const void* b, int64_t ldb, int T, int H, int G, int dk, int dv, float* S,
    const int64_t* positions, const int* cu, const int* slots) {
    DeltaArgs a = {};
    a.y = y; a.q = q; a.k = k; a.v = v; a.b = b;
    a.ldq = ldq; a.ldk = ldk; a.ldv = ldv; a.ldb = ldb;
    a.logw = logw; a.qscale = 1.f / sqrtf((float)dk);
    a.T = T; a.H = H; a.per = H / G; a.dk = dk; a.dv = dv; a.S = S;
    a.positions = positions; a.cu = cu; a.slots = slots;
    return a;
}

extern "C" hipError_t launch_delta_scan(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v, int64_t ldv,
    float* logw, const void* b, int64_t ldb, int T, int H, int G, int dk, int dv, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* seg_list, int nseg,
    int f32, hipStream_t stream) {
    if (nseg <= 0) return hipSuccess;
    DeltaArgs a = delta_args(y, q, ldq, k, ldk, v, ldv, logw, b, ldb, T, H, G, dk, dv, S,
                             positions, cu, slots);
    a.seg_list = seg_list;
    return f32 ? delta_scan_go<float>(a, nseg, stream) : delta_scan_go<bf16>(a, nseg, stream);
}

// slices of 32 key dims that the chunked kernels are built for
extern "C" int delta_slices(int dk) { return dk <= 32 ? 1 : dk <= 64 ? 2 : dk <= 128 ? 4 : 8; }

// bf16; dk (up to 256) and dv multiples of 8; logw holds F; scratch as in DeltaArgs
extern "C" hipError_t launch_delta_chunked(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v, int64_t ldv,
    float* logw, const void* b, int64_t ldb, int T, int H, int G, int dk, int dv, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* segs,
    const int* first, const int* chunk_seg, const int* chunk_off, int nsegs, int nchunks,
    void* frags, float* u0, hipStream_t stream) {
    if (nchunks <= 0) return hipSuccess;
    if (dk % 8 || dv % 8 || ldq % 8 || ldk % 8 || ldv % 8 || dk > 256) return hipErrorInvalidValue;
    DeltaArgs a = delta_args(y, q, ldq, k, ldk, v, ldv, logw, b, ldb, T, H, G, dk, dv, S,
                             positions, cu, slots);
    a.segs = segs; a.first = first; a.chunk_seg = chunk_seg; a.chunk_off = chunk_off;
    a.frags = (bf16*)frags;
    a.u0 = u0;
    const dim3 all(nchunks, H), walk(nsegs, H, ceil_div_i(dv, 32));
#define GO(NC)                                                                \
    {                                                                         \
        delta_intra_kernel<NC><<<all, 256, 0, stream>>>(a);                   \
        HIP_CHECK_LAST();                                                     \
        delta_state_kernel<NC><<<walk, 128, 0, stream>>>(a);                  \
    }
    switch (delta_slices(dk)) {
        case 1: GO(1) break;
        case 2: GO(2) break;
        case 4: GO(4) break;
        default: GO(8)
    }
#undef GO
    HIP_CHECK_LAST();
    return hipSuccess;
}
