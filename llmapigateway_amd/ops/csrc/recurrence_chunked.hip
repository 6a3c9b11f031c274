// Linear recurrences for gfx950 in chunks of 64 rows, on MFMA (bf16 data,
// fp32 state): the prompt form of recurrence.hip's scan. Fixed decays are the
// SSD form with dt = 1 and D = 0, on rows that silu has gone over already. With
// the chunk's inclusive sums F of the log decays,
//
//   SSD:   P[t,s] = (q_t.k_s) e^(F_t-F_s) dt_s
//          y_t    = sum_{s<=t} P[t,s] v_s + e^(F_t) S_in q_t + D v_t
//          S_out  = e^(F_L) S_in + sum_s e^(F_L-F_s) dt_s v_s k_s^T
//   mLSTM: b_s = i_s - F_s,  g_t = max(m_in, max_{s<=t} b_s),  m_t = F_t + g_t
//          P[t,s] = (q_t.k_s) e^(b_s-g_t),  inter factor e^(m_in-g_t), and the
//          normaliser n is S with v = 1.
//
// Three launches: chunk_gates (F and dt or b per row and head), state_pass
// (one workgroup walks a segment's chunks for a 64x64 tile of a head's state
// and leaves the state before every chunk), chunk_out (every chunk, head and
// value tile at once).
//
// fp32 operands of a product (weighted keys, state, P) go in as a sum of two
// bf16, so the products are as good as fp32 ones while q, k, v are exact.

#include "mfma.h"
#include "recurrence.h"

#define CH 64          // rows per chunk
#define LDT (CH + 8)   // LDS row stride of a 64-wide tile

struct ChunkArgs {
    bf16* y;                       // [T, H*dv]
    const bf16 *q, *k, *v;
    int64_t ldq, ldk, ldv;
    const float *gates, *bias, *A_log, *D;
    float cap, qscale;
    int T, H, per_group, dk, dv;
    float *S, *n, *m;              // caches (see recurrence.hip)
    const int64_t* positions;
    const int *cu, *slots, *segs, *first, *chunk_seg, *chunk_off;
    // scratch
    float *F, *b;                  // [H, T]
    uint16_t *s_hi, *s_lo;         // [chunks, H, dv, dk]
    float *n_in, *m_in;            // [chunks, H, dk], [chunks, H]
};

__device__ __forceinline__ float wave_scan_sum(float v, int lane) {
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float u = __shfl_up(v, off, WAVE_SIZE);
        if (lane >= off) v += u;
    }
    return v;
}
__device__ __forceinline__ float wave_scan_max(float v, int lane) {
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float u = __shfl_up(v, off, WAVE_SIZE);
        if (lane >= off) v = fmaxf(v, u);
    }
    return v;
}

// a wave per (chunk, head), a lane per row
template <bool MLSTM, bool FIXED = false>
__global__ void chunk_gates_kernel(ChunkArgs a) {
    const int c = blockIdx.x, lane = threadIdx.x & 63;
    const int h = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (h >= a.H) return;
    const int seg = a.chunk_seg[c], r0 = a.cu[seg] + a.chunk_off[c];
    const int n = min(CH, a.cu[seg + 1] - r0), H = a.H;
    float decay = 0.f, in = 0.f;
    if (lane < n) {
        const size_t t = r0 + lane;
        if (FIXED) {
            // e^-80 is as good as 0, and sums of 64 of them keep their precision
            decay = fmaxf(logf(a.A_log[h]), -80.f);
            in = 1.f;
        } else if (MLSTM) {
            const float* g = a.gates + t * 2 * H;
            in = soft_cap_f(g[h] + a.bias[h], a.cap);
            decay = log_sigmoid_f(soft_cap_f(g[H + h] + a.bias[H + h], a.cap));
        } else {
            in = softplus_f(a.gates[t * H + h] + a.bias[h]);
            decay = -expf(a.A_log[h]) * in;
        }
    }
    const float F = wave_scan_sum(decay, lane);
    if (lane < n) {
        a.F[(size_t)h * a.T + r0 + lane] = F;
        a.b[(size_t)h * a.T + r0 + lane] = MLSTM ? in - F : in;
    }
}

// ---------------------------------------------------------------------------
// grid (segments, H, dv tiles * dk tiles); C fragments hold S[dk][dv]: wave =
// 16 key dims, lane = 4 consecutive key dims of one value dim per dv tile.
// ---------------------------------------------------------------------------
template <bool MLSTM>
__launch_bounds__(256)
__global__ void state_pass_kernel(ChunkArgs a) {
    __shared__ bf16 k_hi[CH][LDT], k_lo[CH][LDT], v_lds[CH][LDT];
    __shared__ float w_lds[CH];
    const int seg = a.segs[blockIdx.x], h = blockIdx.y;
    const int dk = a.dk, dv = a.dv, H = a.H, hk = h / a.per_group;
    const int nkt = (dk + 63) / 64, vt = blockIdx.z / nkt, kt = blockIdx.z % nkt;
    const int slot = a.slots[seg], row_lo = a.cu[seg], row_hi = a.cu[seg + 1];
    const int c_lo = a.first[blockIdx.x], c_hi = a.first[blockIdx.x + 1];
    const bool fresh = a.positions[row_lo] == 0;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const int kd = kt * 64 + wave * 16 + g * 4;  // first of this lane's key dims
    const int tiles = (dv + 63) / 64;

    f32x4 S[4], nv = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = 0.f;
    float* Sp = a.S + ((size_t)slot * H + h) * dv * dk;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int vd = vt * 64 + j * 16 + r16;
        S[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (!fresh && vd < dv && kd < dk)
            S[j] = *reinterpret_cast<const f32x4*>(Sp + (size_t)vd * dk + kd);
    }
    if (MLSTM && !fresh) {
        m = a.m[((size_t)slot * tiles + vt) * H + h];
        if (vt == 0 && kd < dk)
            nv = *reinterpret_cast<const f32x4*>(a.n + ((size_t)slot * tiles * H + h) * dk + kd);
    }

    uint4 kreg[2], vreg[2];
    float F_last, F_row, b_row;  // of the chunk that is loaded, a row per lane
    auto load_rows = [&](int r0) {
        const size_t at = (size_t)h * a.T + r0;
        const int last = min(CH, row_hi - r0) - 1;
        F_last = a.F[at + last];
        F_row = a.F[at + min(lane, last)];
        b_row = a.b[at + min(lane, last)];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int e = tid + u * 256, r = r0 + e / 8, d = e % 8 * 8;
            kreg[u] = vreg[u] = (uint4){0, 0, 0, 0};
            if (r < row_hi) {
                if (kt * 64 + d < dk)
                    kreg[u] = *reinterpret_cast<const uint4*>(
                        a.k + (size_t)r * a.ldk + (size_t)hk * dk + kt * 64 + d);
                if (vt * 64 + d < dv)
                    vreg[u] = *reinterpret_cast<const uint4*>(
                        a.v + (size_t)r * a.ldv + (size_t)h * dv + vt * 64 + d);
            }
        }
    };
    load_rows(row_lo);
    for (int c = c_lo; c < c_hi; ++c) {
        const int r0 = row_lo + (c - c_lo) * CH, n = min(CH, row_hi - r0);
        // the state before this chunk
        const size_t base = ((size_t)c * H + h) * dv;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int vd = vt * 64 + j * 16 + r16;
            if (vd < dv && kd < dk) {
                uint16_t hi[4], lo[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) split_bf16(S[j][r], hi[r], lo[r]);
                const size_t at = (base + vd) * dk + kd;
                *reinterpret_cast<uint2*>(a.s_hi + at) = make_uint2(
                    hi[0] | ((uint32_t)hi[1] << 16), hi[2] | ((uint32_t)hi[3] << 16));
                *reinterpret_cast<uint2*>(a.s_lo + at) = make_uint2(
                    lo[0] | ((uint32_t)lo[1] << 16), lo[2] | ((uint32_t)lo[3] << 16));
            }
        }
        if (MLSTM && vt == 0) {
            if (r16 == 0 && kd < dk)
                *reinterpret_cast<f32x4*>(a.n_in + ((size_t)c * H + h) * dk + kd) = nv;
            if (kt == 0 && tid == 0) a.m_in[(size_t)c * H + h] = m;
        }
        // weights of the chunk's rows at its end
        float keep, m_out = 0.f;
        {
            float w;
            if (MLSTM) {
                const float gl = fmaxf(m, wave_reduce_max(b_row));
                w = lane < n ? expf(b_row - gl) : 0.f;
                keep = expf(m - gl);
                m_out = F_last + gl;
            } else {
                w = lane < n ? expf(F_last - F_row) * b_row : 0.f;
                keep = expf(F_last);
            }
            __syncthreads();  // the previous chunk's tiles have been read
            if (wave == 0) w_lds[lane] = w;
        }
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int e = tid + u * 256, s = e / 8, d = e % 8 * 8;
            const float w = w_lds[s];
            float f[8];
            unpack2(kreg[u].x, f[0], f[1]);
            unpack2(kreg[u].y, f[2], f[3]);
            unpack2(kreg[u].z, f[4], f[5]);
            unpack2(kreg[u].w, f[6], f[7]);
            uint4 hi, lo;
            uint32_t* hp = reinterpret_cast<uint32_t*>(&hi);
            uint32_t* lp = reinterpret_cast<uint32_t*>(&lo);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                uint16_t h0, l0, h1, l1;
                split_bf16(f[2 * i] * w, h0, l0);
                split_bf16(f[2 * i + 1] * w, h1, l1);
                hp[i] = h0 | ((uint32_t)h1 << 16);
                lp[i] = l0 | ((uint32_t)l1 << 16);
            }
            *reinterpret_cast<uint4*>(&k_hi[s][d]) = hi;
            *reinterpret_cast<uint4*>(&k_lo[s][d]) = lo;
            *reinterpret_cast<uint4*>(&v_lds[s][d]) = vreg[u];
        }
        __syncthreads();
        if (c + 1 < c_hi) load_rows(r0 + CH);
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[j][r] *= keep;
        if (MLSTM) {
#pragma unroll
            for (int r = 0; r < 4; ++r) nv[r] *= keep;
            m = m_out;
        }
        const short one = (short)0x3F80;
        const bf16x8 ones = (bf16x8){one, one, one, one, one, one, one, one};
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
            if (MLSTM) {
                nv = mfma16(ah, ones, nv);
                nv = mfma16(al, ones, nv);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int vd = vt * 64 + j * 16 + r16;
        if (vd < dv && kd < dk)
            *reinterpret_cast<f32x4*>(Sp + (size_t)vd * dk + kd) = S[j];
    }
    // n: every value tile's copy; m goes out with the last chunk's output (the
    // workgroups of other key tiles may still have to read it)
    if (MLSTM && vt == 0 && r16 == 0 && kd < dk)
        for (int c = 0; c < tiles; ++c)
            *reinterpret_cast<f32x4*>(a.n + (((size_t)slot * tiles + c) * H + h) * dk + kd) = nv;
}

// ---------------------------------------------------------------------------
// grid (chunks, H, dv / (16*NDT)); a wave owns 16 query rows
// ---------------------------------------------------------------------------
template <bool MLSTM, int NDT>
__launch_bounds__(256)
__global__ void chunk_out_kernel(ChunkArgs a) {
    constexpr int DVT = NDT * 16, LDV = DVT + 8;
    // key-dim slices of the state (two planes) and of the keys; the weights
    // P take the state's place after the loop over slices
    constexpr int SP = DVT * LDT > 4 * 16 * LDT ? DVT * LDT : 4 * 16 * LDT;
    __shared__ bf16 s_lds[2][SP];
    __shared__ bf16 k_lds[CH][LDT];
    __shared__ bf16 v_lds[CH][LDV];
    __shared__ float F_lds[CH], b_lds[CH], g_lds[CH];
    const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * DVT;
    const int dk = a.dk, dv = a.dv, H = a.H, hk = h / a.per_group;
    const int seg = a.chunk_seg[c], r0 = a.cu[seg] + a.chunk_off[c];
    const int n = min(CH, a.cu[seg + 1] - r0);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int r16 = lane & 15, g = lane >> 4;
    const float m_in = MLSTM ? a.m_in[(size_t)c * H + h] : 0.f;
    if (wave == 0) {
        const size_t at = (size_t)h * a.T + r0 + min(lane, n - 1);
        const float F = a.F[at], b = a.b[at];
        F_lds[lane] = F;
        b_lds[lane] = b;
        if (MLSTM) {
            const float gt = fmaxf(m_in, wave_scan_max(b, lane));
            g_lds[lane] = gt;
            if (blockIdx.z == 0 && lane == 63 && a.chunk_off[c] + n == a.cu[seg + 1] - a.cu[seg]) {
                const int tiles = (dv + 63) / 64;
                for (int t = 0; t < tiles; ++t)
                    a.m[((size_t)a.slots[seg] * tiles + t) * H + h] = F + gt;
            }
        }
    }
#pragma unroll
    for (int u = 0; u < CH * DVT / 8 / 256; ++u) {
        const int e = tid + u * 256, s = e / (DVT / 8), d = e % (DVT / 8) * 8;
        uint4 x = {0, 0, 0, 0};
        if (s < n && v0 + d < dv)
            x = *reinterpret_cast<const uint4*>(
                a.v + (size_t)(r0 + s) * a.ldv + (size_t)h * dv + v0 + d);
        *reinterpret_cast<uint4*>(&v_lds[s][d]) = x;
    }

    f32x4 qk[4], o[NDT];
    float qn = 0.f;  // this lane's share of n_in . q of row r16
#pragma unroll
    for (int u = 0; u < 4; ++u) qk[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NDT; ++j) o[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const bf16* qr =
        a.q + (size_t)(r0 + min(wave * 16 + r16, n - 1)) * a.ldq + (size_t)hk * dk;
    const size_t sbase = ((size_t)c * H + h) * dv;
    for (int d0 = 0; d0 < dk; d0 += 64) {
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int e = tid + u * 256, s = e / 8, d = d0 + e % 8 * 8;
            uint4 x = {0, 0, 0, 0};
            if (s < n && d < dk)
                x = *reinterpret_cast<const uint4*>(
                    a.k + (size_t)(r0 + s) * a.ldk + (size_t)hk * dk + d);
            *reinterpret_cast<uint4*>(&k_lds[s][e % 8 * 8]) = x;
        }
#pragma unroll
        for (int u = 0; u < DVT * 8 / 256; ++u) {
            const int e = tid + u * 256, vd = e / 8, d = d0 + e % 8 * 8;
            uint4 x = {0, 0, 0, 0}, y = {0, 0, 0, 0};
            if (v0 + vd < dv && d < dk) {
                x = *reinterpret_cast<const uint4*>(a.s_hi + (sbase + v0 + vd) * dk + d);
                y = *reinterpret_cast<const uint4*>(a.s_lo + (sbase + v0 + vd) * dk + d);
            }
            *reinterpret_cast<uint4*>(&s_lds[0][vd * LDT + e % 8 * 8]) = x;
            *reinterpret_cast<uint4*>(&s_lds[1][vd * LDT + e % 8 * 8]) = y;
        }
        uint4 qv[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int d = d0 + u * 32 + g * 8;
            qv[u] = (uint4){0, 0, 0, 0};
            if (d < dk) qv[u] = *reinterpret_cast<const uint4*>(qr + d);
            if (MLSTM && d < dk) {
                const float* np = a.n_in + ((size_t)c * H + h) * dk + d;
                float f[8];
                unpack2(qv[u].x, f[0], f[1]);
                unpack2(qv[u].y, f[2], f[3]);
                unpack2(qv[u].z, f[4], f[5]);
                unpack2(qv[u].w, f[6], f[7]);
#pragma unroll
                for (int i = 0; i < 8; ++i) qn = fmaf(f[i], np[i], qn);
            }
        }
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const bf16x8 qf = as_frag(qv[u]);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                qk[j] = mfma16(qf, *reinterpret_cast<const bf16x8*>(
                                       &k_lds[j * 16 + r16][u * 32 + g * 8]), qk[j]);
#pragma unroll
            for (int j = 0; j < NDT; ++j) {
                const int at = (j * 16 + r16) * LDT + u * 32 + g * 8;
                o[j] = mfma16(qf, *reinterpret_cast<const bf16x8*>(&s_lds[0][at]), o[j]);
                o[j] = mfma16(qf, *reinterpret_cast<const bf16x8*>(&s_lds[1][at]), o[j]);
            }
        }
    }
    __syncthreads();  // the state slices are done: P takes their place
    bf16* p_hi = &s_lds[0][wave * 16 * LDT];
    bf16* p_lo = &s_lds[1][wave * 16 * LDT];
    if (MLSTM) {
        qn += __shfl_xor(qn, 16, WAVE_SIZE);
        qn += __shfl_xor(qn, 32, WAVE_SIZE);
    }
    float den[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int row = g * 4 + r, t = wave * 16 + row;
        const float Ft = F_lds[t], gt = MLSTM ? g_lds[t] : 0.f;
        const float inter = MLSTM ? expf(m_in - gt) * a.qscale : expf(Ft);
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int s = j * 16 + r16;
            float p = 0.f;
            if (s <= t && s < n)
                p = qk[j][r] * (MLSTM ? expf(b_lds[s] - gt) * a.qscale
                                      : expf(Ft - F_lds[s]) * b_lds[s]);
            sum += p;
            uint16_t hi, lo;
            split_bf16(p, hi, lo);
            *reinterpret_cast<uint16_t*>(p_hi + row * LDT + s) = hi;
            *reinterpret_cast<uint16_t*>(p_lo + row * LDT + s) = lo;
        }
        if (MLSTM) {
            const float nq = row16_sum(sum) + inter * __shfl(qn, row, WAVE_SIZE);
            den[r] = 1.f / (fmaxf(fabsf(nq), expf(-(Ft + gt))) + 1e-6f);
        } else {
            den[r] = 1.f;
        }
#pragma unroll
        for (int j = 0; j < NDT; ++j) o[j][r] *= inter;
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const bf16x8 ph = *reinterpret_cast<const bf16x8*>(p_hi + r16 * LDT + u * 32 + g * 8);
        const bf16x8 pl = *reinterpret_cast<const bf16x8*>(p_lo + r16 * LDT + u * 32 + g * 8);
#pragma unroll
        for (int j = 0; j < NDT; ++j) {
            const bf16x8 vf = tr_frag(&v_lds[0][0], LDV, u * 32, j * 16);
            o[j] = mfma16(ph, vf, o[j]);
            o[j] = mfma16(pl, vf, o[j]);
        }
    }
    const float skip = MLSTM || a.D == nullptr ? 0.f : a.D[h];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int t = wave * 16 + g * 4 + r;
        if (t >= n) continue;
        bf16* yr = a.y + ((size_t)(r0 + t) * H + h) * dv + v0;
#pragma unroll
        for (int j = 0; j < NDT; ++j) {
            const int d = j * 16 + r16;
            if (v0 + d < dv)
                stf(yr + d, MLSTM ? o[j][r] * den[r] : o[j][r] + skip * ldf(&v_lds[t][d]));
        }
    }
}

template <bool MLSTM, bool FIXED = false>
static hipError_t chunked_go(const ChunkArgs& a, int nsegs, int nchunks, hipStream_t stream) {
    if (nchunks <= 0) return hipSuccess;
    if (a.dk % 8 || a.dv % 8 || a.ldq % 8 || a.ldk % 8 || a.ldv % 8)
        return hipErrorInvalidValue;
    const int vt = ceil_div_i(a.dv, 64), kt = ceil_div_i(a.dk, 64);
    chunk_gates_kernel<MLSTM, FIXED><<<dim3(nchunks, ceil_div_i(a.H, 4)), 256, 0, stream>>>(a);
    HIP_CHECK_LAST();
    state_pass_kernel<MLSTM><<<dim3(nsegs, a.H, vt * kt), 256, 0, stream>>>(a);
    HIP_CHECK_LAST();
    if (a.dv <= 64)
        chunk_out_kernel<MLSTM, 4><<<dim3(nchunks, a.H, 1), 256, 0, stream>>>(a);
    else
        chunk_out_kernel<MLSTM, 8><<<dim3(nchunks, a.H, ceil_div_i(a.dv, 128)), 256, 0,
                                     stream>>>(a);
    HIP_CHECK_LAST();
    return hipSuccess;
}

// scratch: F and b [2, H, T] fp32, state planes [2, chunks, H, dv, dk] bf16,
// n_in [chunks, H, dk] and m_in [chunks, H] fp32 (mLSTM)
extern "C" hipError_t launch_ssd_chunked(
    void* y, const void* xbc, int64_t ld, const float* dt, const float* dt_bias,
    const float* A_log, const float* D, int T, int H, int P, int N, int G, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* segs,
    const int* first, const int* chunk_seg, const int* chunk_off, int nsegs, int nchunks,
    float* Fb, void* planes, hipStream_t stream) {
    ChunkArgs a = {};
    a.y = (bf16*)y;
    a.v = (const bf16*)xbc;
    a.k = a.v + (size_t)H * P;
    a.q = a.k + (size_t)G * N;
    a.ldq = a.ldk = a.ldv = ld;
    a.gates = dt; a.bias = dt_bias; a.A_log = A_log; a.D = D;
    a.T = T; a.H = H; a.per_group = H / G; a.dk = N; a.dv = P; a.S = S;
    a.positions = positions; a.cu = cu; a.slots = slots; a.segs = segs; a.first = first;
    a.chunk_seg = chunk_seg; a.chunk_off = chunk_off;
    a.F = Fb; a.b = Fb + (size_t)H * T;
    a.s_hi = (uint16_t*)planes;
    a.s_lo = a.s_hi + (size_t)nchunks * H * P * N;
    return chunked_go<false>(a, nsegs, nchunks, stream);
}

extern "C" hipError_t launch_mlstm_chunked(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* gates, const float* bias, float cap, float qscale, int T, int H,
    int dk, int dv, float* S, float* n, float* m, const int64_t* positions, const int* cu,
    const int* slots, const int* segs, const int* first, const int* chunk_seg,
    const int* chunk_off, int nsegs, int nchunks, float* Fb, void* planes, float* n_in,
    float* m_in, hipStream_t stream) {
    ChunkArgs a = {};
    a.y = (bf16*)y; a.q = (const bf16*)q; a.k = (const bf16*)k; a.v = (const bf16*)v;
    a.ldq = ldq; a.ldk = ldk; a.ldv = ldv;
    a.gates = gates; a.bias = bias; a.cap = cap; a.qscale = qscale;
    a.T = T; a.H = H; a.per_group = 1; a.dk = dk; a.dv = dv; a.S = S; a.n = n; a.m = m;
    a.positions = positions; a.cu = cu; a.slots = slots; a.segs = segs; a.first = first;
    a.chunk_seg = chunk_seg; a.chunk_off = chunk_off;
    a.F = Fb; a.b = Fb + (size_t)H * T;
    a.s_hi = (uint16_t*)planes;
    a.s_lo = a.s_hi + (size_t)nchunks * H * dv * dk;
    a.n_in = n_in; a.m_in = m_in;
    return chunked_go<true>(a, nsegs, nchunks, stream);
}

extern "C" hipError_t launch_fixed_chunked(
    void* y, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v,
    int64_t ldv, const float* decay, int T, int H, int dk, int dv, float* S,
    const int64_t* positions, const int* cu, const int* slots, const int* segs,
    const int* first, const int* chunk_seg, const int* chunk_off, int nsegs, int nchunks,
    float* Fb, void* planes, hipStream_t stream) {
    ChunkArgs a = {};
    a.y = (bf16*)y; a.q = (const bf16*)q; a.k = (const bf16*)k; a.v = (const bf16*)v;
    a.ldq = ldq; a.ldk = ldk; a.ldv = ldv;
    a.A_log = decay;
    a.T = T; a.H = H; a.per_group = 1; a.dk = dk; a.dv = dv; a.S = S;
    a.positions = positions; a.cu = cu; a.slots = slots; a.segs = segs; a.first = first;
    a.chunk_seg = chunk_seg; a.chunk_off = chunk_off;
    a.F = Fb; a.b = Fb + (size_t)H * T;
    a.s_hi = (uint16_t*)planes;
    a.s_lo = a.s_hi + (size_t)nchunks * H * dv * dk;
    return chunked_go<false, true>(a, nsegs, nchunks, stream);
}
