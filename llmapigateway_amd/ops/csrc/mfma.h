// bf16 MFMA fragments on gfx950 (v_mfma_f32_16x16x32_bf16):
//   A: lane l holds A[row = l&15][k = (l>>4)*8 + j], j = 0..7
//   B: lane l holds B[k = (l>>4)*8 + j][col = l&15]
//   C: lane l holds C[row = (l>>4)*4 + r][col = l&15], r = 0..3
#pragma once

#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(short)))) short bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(short)))) short bf16x4;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ bf16x8 as_frag(const uint4& v) {
    return *reinterpret_cast<const bf16x8*>(&v);
}

// sum / maximum over the 16 lanes of a fragment row, in every lane: DPP row
// rotations stay in the vector ALU (a shuffle goes through the LDS unit)
template <int N>
__device__ __forceinline__ float row16_ror(float v) {
    return __int_as_float(__builtin_amdgcn_update_dpp(
        0, __float_as_int(v), 0x120 + N, 0xF, 0xF, false));
}
__device__ __forceinline__ float row16_max(float v) {
    v = fmaxf(v, row16_ror<8>(v));
    v = fmaxf(v, row16_ror<4>(v));
    v = fmaxf(v, row16_ror<2>(v));
    return fmaxf(v, row16_ror<1>(v));
}
__device__ __forceinline__ float row16_sum(float v) {
    v += row16_ror<8>(v);
    v += row16_ror<4>(v);
    v += row16_ror<2>(v);
    return v + row16_ror<1>(v);
}

// ds_read_b64_tr_b16 twice: a 16-lane group's lanes address 4 rows of 16
// columns (lane i: row i/4, columns (i%4)*4..+3) and each gets one column
__device__ __forceinline__ bf16x8 tr_pair(const bf16* lo_rows, const bf16* hi_rows) {
    typedef __attribute__((address_space(3))) bf16x4* lds_ptr;
    const bf16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)lo_rows);
    const bf16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)hi_rows);
    return (bf16x8){lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
}

// Fragment whose k runs over the rows of a row-major LDS tile (a B operand
// stored [k][col], or an A operand stored [k][row]): rows k0..k0+31, columns
// c0..c0+15. Rows and c0 must keep 8-byte alignment.
__device__ __forceinline__ bf16x8 tr_frag(const bf16* tile, int stride, int k0, int c0) {
    const int lane = threadIdx.x & 63, g = lane >> 4, i = lane & 15;
    const bf16* p = tile + (k0 + g * 8 + (i >> 2)) * stride + c0 + (i & 3) * 4;
    return tr_pair(p, p + 4 * stride);
}

// two fp32 to packed bf16, one instruction (round to nearest even)
__device__ __forceinline__ uint32_t cvt_pk_bf16(float lo, float hi) {
    typedef __attribute__((__vector_size__(2 * sizeof(float)))) float f32x2;
    typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 b16x2;
    const b16x2 v = __builtin_convertvector((f32x2){lo, hi}, b16x2);
    return *reinterpret_cast<const uint32_t*>(&v);
}

// fp32 as a sum of two bf16 (16 mantissa bits): products of a fp32 operand
// with bf16 data keep fp32-like accuracy in two MFMAs
__device__ __forceinline__ void split_bf16(float v, uint16_t& hi, uint16_t& lo) {
    hi = f2bfbits(v);
    lo = f2bfbits(v - bfbits2f(hi));
}
// fp32 values as the sum of two bf16 fragments
__device__ __forceinline__ void split_frag(const float* f, bf16x8& hi, bf16x8& lo) {
    uint4 h, l;
    uint32_t* hp = reinterpret_cast<uint32_t*>(&h);
    uint32_t* lp = reinterpret_cast<uint32_t*>(&l);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        hp[i] = cvt_pk_bf16(f[2 * i], f[2 * i + 1]);
        float a, b;
        unpack2(hp[i], a, b);
        lp[i] = cvt_pk_bf16(f[2 * i] - a, f[2 * i + 1] - b);
    }
    hi = as_frag(h);
    lo = as_frag(l);
}
__device__ __forceinline__ void unpack8(const uint4& v, float* f) {
    unpack2(v.x, f[0], f[1]);
    unpack2(v.y, f[2], f[3]);
    unpack2(v.z, f[4], f[5]);
    unpack2(v.w, f[6], f[7]);
}
__device__ __forceinline__ void load8f(const float* p, float* f) {
    const float4 a = reinterpret_cast<const float4*>(p)[0];
    const float4 b = reinterpret_cast<const float4*>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
    f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
