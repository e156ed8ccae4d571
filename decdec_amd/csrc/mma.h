// 16 x 16 matrix-core tiles with a contraction of 32, in one shape for bf16 and for fp32 operands.
//
// A lane holds eight consecutive elements (along the contraction) of one row of A and of one column of B: row / column
// lane % 16, elements 8 (lane / 16) .. + 7.  bf16: one v_mfma_f32_16x16x32_bf16.  fp32: eight v_mfma_f32_16x16x4_f32, the
// i-th with element i of every lane -- the contraction index runs in another order, the same one for A and B.
// The result has row 4 (lane / 16) + v, column lane % 16 in register v.
#pragma once
#include "common.h"

namespace decdec {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <int DT> struct Frag;
template <> struct Frag<kBF16> { u32x4 v; };
template <> struct Frag<kFP32> { float v[8]; };

__device__ __forceinline__ void mma(const Frag<kBF16>& a, const Frag<kBF16>& b, f32x4& c) {
    bf16x8 x, y;
    __builtin_memcpy(&x, &a.v, 16);
    __builtin_memcpy(&y, &b.v, 16);
    c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, y, c, 0, 0, 0);
}
__device__ __forceinline__ void mma(const Frag<kFP32>& a, const Frag<kFP32>& b, f32x4& c) {
#pragma unroll
    for (int i = 0; i < 8; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[i], b.v[i], c, 0, 0, 0);
}

// eight consecutive elements (16-byte aligned)
__device__ __forceinline__ Frag<kBF16> frag_load(const uint16_t* p) {
    Frag<kBF16> f;
    f.v = *(const u32x4*)p;
    return f;
}
__device__ __forceinline__ Frag<kFP32> frag_load(const float* p) {
    Frag<kFP32> f;
    const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) { f.v[i] = a[i]; f.v[4 + i] = b[i]; }
    return f;
}
// eight elements a stride apart
__device__ __forceinline__ Frag<kFP32> frag_gather(const float* p, uint32_t stride) {
    Frag<kFP32> f;
#pragma unroll
    for (int i = 0; i < 8; ++i) f.v[i] = p[(size_t)i * stride];
    return f;
}
__device__ __forceinline__ Frag<kBF16> frag_gather(const uint16_t* p, uint32_t stride) {
    Frag<kBF16> f;
#pragma unroll
    for (int i = 0; i < 4; ++i)
        f.v[i] = (uint32_t)p[(size_t)(2 * i) * stride] | ((uint32_t)p[(size_t)(2 * i + 1) * stride] << 16);
    return f;
}
__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
    const bf16x2_t v = {(__bf16)a, (__bf16)b};
    uint32_t r;
    __builtin_memcpy(&r, &v, 4);
    return r;
}
// fp32 values as operands: exact for fp32; for bf16 the sum of a leading and a trailing part (16 significant bits)
__device__ __forceinline__ void frag_split(const float (&x)[8], Frag<kBF16>& hi, Frag<kBF16>& lo) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint32_t h = pack_bf16(x[2 * i], x[2 * i + 1]);
        hi.v[i] = h;
        lo.v[i] = pack_bf16(x[2 * i] - __uint_as_float(h << 16), x[2 * i + 1] - __uint_as_float(h & 0xFFFF0000u));
    }
}
__device__ __forceinline__ void frag_split(const float (&x)[8], Frag<kFP32>& hi, Frag<kFP32>&) {
#pragma unroll
    for (int i = 0; i < 8; ++i) hi.v[i] = x[i];
}

template <int DT> struct LaneOf { using t = uint16_t; };
template <> struct LaneOf<kFP32> { using t = float; };

// eight elements of a row as a fragment, zero past `valid`
template <int DT>
__device__ __forceinline__ Frag<DT> load8(const typename LaneOf<DT>::t* p, int valid, bool vec) {
    if (vec && valid >= 8) return frag_load(p);
    Frag<DT> f;
    if constexpr (DT == kFP32) {
#pragma unroll
        for (int i = 0; i < 8; ++i) f.v[i] = i < valid ? p[i] : 0.f;
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            f.v[i] = (uint32_t)(2 * i < valid ? p[2 * i] : 0) | ((uint32_t)(2 * i + 1 < valid ? p[2 * i + 1] : 0) << 16);
    }
    return f;
}
__device__ __forceinline__ void store8(uint16_t* p, const Frag<kBF16>& f) { *(u32x4*)p = f.v; }
__device__ __forceinline__ void store8(float* p, const Frag<kFP32>& f) {
#pragma unroll
    for (int i = 0; i < 8; i += 4) *(f32x4*)(p + i) = f32x4{f.v[i], f.v[i + 1], f.v[i + 2], f.v[i + 3]};
}
__device__ __forceinline__ void frag_values(const Frag<kBF16>& f, float (&x)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) { x[2 * i] = __uint_as_float(f.v[i] << 16); x[2 * i + 1] = __uint_as_float(f.v[i] & 0xFFFF0000u); }
}
__device__ __forceinline__ void frag_values(const Frag<kFP32>& f, float (&x)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = f.v[i];
}

__device__ __forceinline__ Frag<kBF16> frag_of(const float (&x)[8], const Frag<kBF16>&) {
    Frag<kBF16> f;
#pragma unroll
    for (int i = 0; i < 4; ++i) f.v[i] = pack_bf16(x[2 * i], x[2 * i + 1]);
    return f;
}
__device__ __forceinline__ Frag<kFP32> frag_of(const float (&x)[8], const Frag<kFP32>&) {
    Frag<kFP32> f;
#pragma unroll
    for (int i = 0; i < 8; ++i) f.v[i] = x[i];
    return f;
}

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + __expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// xIELU with the softplus of its two numbers already taken.  e^z - 1 - z by its series where the difference cancels.
__device__ __forceinline__ float xielu_f(float z, float sp, float sq) {
    const float n = fminf(z, 0.f);
    float s = 2.7557319e-7f;                               // 1 / 10!
    s = __builtin_fmaf(s, n, 2.7557319e-6f);
    s = __builtin_fmaf(s, n, 2.4801587e-5f);
    s = __builtin_fmaf(s, n, 1.9841270e-4f);
    s = __builtin_fmaf(s, n, 1.3888889e-3f);
    s = __builtin_fmaf(s, n, 8.3333333e-3f);
    s = __builtin_fmaf(s, n, 4.1666667e-2f);
    s = __builtin_fmaf(s, n, 1.6666667e-1f);
    s = __builtin_fmaf(s, n, 0.5f) * n * n;
    const float e = n > -0.7f ? s : __expf(n) - 1.f - n;
    return z > 0.f ? (sp * z + 0.5f) * z : (0.5f + sq) * e + 0.5f * z;
}

// GELU, tanh form: z (1 + tanh u) / 2 = z sigmoid(2 u)
__device__ __forceinline__ float gelu_tanh_f(float z) {
    return z * sigmoid_f(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

// Sum over a workgroup of `blockDim.x` (a multiple of 64) threads; red: at least 17 floats of LDS, free at the call.
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    __syncthreads();
    if (lane == 0) red[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (uint32_t w = 0; w < nw; ++w) t += red[w];
    return t;
}
// Two at once; red: 32 floats.
__device__ __forceinline__ void block_sum2(float& a, float& b, float* red) {
    a = wave_sum(a);
    b = wave_sum(b);
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    __syncthreads();
    if (lane == 0) { red[wave] = a; red[16 + wave] = b; }
    __syncthreads();
    a = b = 0.f;
    for (uint32_t w = 0; w < nw; ++w) { a += red[w]; b += red[16 + w]; }
}

}  // namespace decdec
