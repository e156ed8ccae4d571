// Row-wise pieces of decoders with a 32-bit residual stream: one-token GEMV with an activation on its first rows,
// embedding, gated residual + norm of the sublayer's output, residual + dynamic tanh, norm, activations, normed and gated
// read-out of a recurrence.
#include "mixers.h"
#include "mma.h"

namespace decdec {

// ---- one-token GEMV ---------------------------------------------------------------------------------------
// A wave owns ROWS rows; a lane requests 16 bytes of each per step, UN steps in flight.  VEC = false: element loads for
// row lengths that are not a multiple of 16 bytes.
template <int DT> struct Pack16;                       // the elements in 16 bytes
template <> struct Pack16<kBF16> { static constexpr int n = 8; };
template <> struct Pack16<kFP32> { static constexpr int n = 4; };

template <int DT>
__device__ __forceinline__ float dot16(const u32x4& w, const u32x4& x, float acc) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if constexpr (DT == kFP32) {
            acc = __builtin_fmaf(__uint_as_float(w[j]), __uint_as_float(x[j]), acc);
        } else {
            acc = __builtin_fmaf(__uint_as_float(w[j] << 16), __uint_as_float(x[j] << 16), acc);
            acc = __builtin_fmaf(__uint_as_float(w[j] & 0xFFFF0000u), __uint_as_float(x[j] & 0xFFFF0000u), acc);
        }
    }
    return acc;
}

template <int DT, int ROWS, bool VEC>
__global__ __launch_bounds__(256) void mix_gemv_kernel(const void* __restrict__ weight, const void* __restrict__ x,
                                                       void* __restrict__ out, const void* __restrict__ act,
                                                       const uint32_t act_rows, const int act_kind, const float scale,
                                                       const uint32_t N, const uint32_t K) {
    using E = Elem<DT>;
    constexpr uint32_t PE = Pack16<DT>::n, UN = ROWS >= 4 ? 2 : (ROWS == 2 ? 4 : 8);
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    const uint32_t row0 = (blockIdx.x * 4u + wave) * (uint32_t)ROWS;
    if (row0 >= N) return;
    float acc[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) acc[r] = 0.f;
    if constexpr (VEC) {
        const unsigned char* wr[ROWS];
#pragma unroll
        for (int r = 0; r < ROWS; ++r) {
            const uint32_t rr = row0 + r < N ? row0 + r : N - 1u;      // rows past the end re-read the last one; not stored
            wr[r] = (const unsigned char*)weight + (size_t)rr * K * E::bytes;
        }
        const uint32_t steps = (K + 64u * PE - 1u) / (64u * PE);
        for (uint32_t s = 0; s < steps; s += UN) {
            u32x4 wv[UN][ROWS], xv[UN];
#pragma unroll
            for (uint32_t u = 0; u < UN; ++u) {
                const uint32_t col = ((s + u) * 64u + lane) * PE;
                const bool ok = col < K;
                const size_t c = (size_t)(ok ? col : 0u) * E::bytes;
                xv[u] = *(const u32x4*)((const unsigned char*)x + c);
                if (!ok) xv[u] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
                for (int r = 0; r < ROWS; ++r) wv[u][r] = __builtin_nontemporal_load((const u32x4*)(wr[r] + c));
            }
#pragma unroll
            for (uint32_t u = 0; u < UN; ++u)
#pragma unroll
                for (int r = 0; r < ROWS; ++r) acc[r] = dot16<DT>(wv[u][r], xv[u], acc[r]);
        }
    } else {
        for (uint32_t c = lane; c < K; c += 64u) {
            const float xc = E::load(x, c);
#pragma unroll
            for (int r = 0; r < ROWS; ++r) {
                const uint32_t rr = row0 + r < N ? row0 + r : N - 1u;
                acc[r] = __builtin_fmaf(E::load(weight, (size_t)rr * K + c), xc, acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) acc[r] = wave_sum(acc[r]);
    if (lane < (uint32_t)ROWS && row0 + lane < N) {
        float v = acc[0];
#pragma unroll
        for (int r = 1; r < ROWS; ++r) v = lane == (uint32_t)r ? acc[r] : v;
        v *= scale;
        if (row0 + lane < act_rows)
            v = act_kind == DECDEC_ACT_GELU_TANH ? gelu_tanh_f(v) : xielu_f(v, softplus_f(E::load(act, 0)), softplus_f(E::load(act, 1)));
        E::store(out, row0 + lane, v);
    }
}

template <int DT, bool VEC>
static void gemv_rows(uint32_t N, uint32_t K, const void* w, const void* x, void* out, const void* act, uint32_t act_rows,
                      int act_kind, float scale, hipStream_t s) {
    if (N >= 16384u) hipLaunchKernelGGL((mix_gemv_kernel<DT, 4, VEC>), dim3((N + 15u) / 16u), dim3(256), 0, s, w, x, out, act, act_rows, act_kind, scale, N, K);
    else if (N >= 4096u) hipLaunchKernelGGL((mix_gemv_kernel<DT, 2, VEC>), dim3((N + 7u) / 8u), dim3(256), 0, s, w, x, out, act, act_rows, act_kind, scale, N, K);
    else hipLaunchKernelGGL((mix_gemv_kernel<DT, 1, VEC>), dim3((N + 3u) / 4u), dim3(256), 0, s, w, x, out, act, act_rows, act_kind, scale, N, K);
}

hipError_t launch_mix_gemv(int dt, const void* w, const void* x, void* out, const void* act, uint32_t act_rows, int act_kind,
                           float scale, uint32_t N, uint32_t K, hipStream_t s) {
    const bool al = ((uintptr_t)w % 16) == 0 && ((uintptr_t)x % 16) == 0;
    if (dt == kBF16) {
        if (al && K % 8u == 0) gemv_rows<kBF16, true>(N, K, w, x, out, act, act_rows, act_kind, scale, s);
        else gemv_rows<kBF16, false>(N, K, w, x, out, act, act_rows, act_kind, scale, s);
    } else if (dt == kFP32) {
        if (al && K % 4u == 0) gemv_rows<kFP32, true>(N, K, w, x, out, act, act_rows, act_kind, scale, s);
        else gemv_rows<kFP32, false>(N, K, w, x, out, act, act_rows, act_kind, scale, s);
    } else return hipErrorInvalidValue;
    return hipGetLastError();
}

// four neighbouring elements
template <int DT>
__device__ __forceinline__ void load4(const void* p, size_t i, float (&v)[4]) {
    if constexpr (DT == kFP32) {
        const u32x4 t = *(const u32x4*)((const float*)p + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = __uint_as_float(t[e]);
    } else {
        const u32x2 t = *(const u32x2*)((const uint16_t*)p + i);
        v[0] = __uint_as_float(t[0] << 16); v[1] = __uint_as_float(t[0] & 0xFFFF0000u);
        v[2] = __uint_as_float(t[1] << 16); v[3] = __uint_as_float(t[1] & 0xFFFF0000u);
    }
}
template <int DT>
__device__ __forceinline__ void store4(void* p, size_t i, const float (&v)[4]) {
    if constexpr (DT == kFP32) {
        u32x4 t;
#pragma unroll
        for (int e = 0; e < 4; ++e) t[e] = __float_as_uint(v[e]);
        *(u32x4*)((float*)p + i) = t;
    } else {
        u32x2 t;
        t[0] = pack_bf16(v[0], v[1]);
        t[1] = pack_bf16(v[2], v[3]);
        *(u32x2*)((uint16_t*)p + i) = t;
    }
}

// ---- embedding --------------------------------------------------------------------------------------------
template <int DT, bool VEC, bool NORM>
__global__ __launch_bounds__(1024) void mix_embed_kernel(const void* __restrict__ table, const long long* __restrict__ tokens,
                                                         float* __restrict__ x, void* __restrict__ xe, const decdec_tanh_norm norm,
                                                         uint32_t vocab, uint32_t dim) {
    using E = Elem<DT>;
    const float alpha = NORM ? E::load(norm.alpha, 0) : 0.f;
    const size_t r = blockIdx.x;
    long long t = tokens[r];
    if (t < 0 || t >= (long long)vocab) t = 0;
    if constexpr (VEC) {
        for (uint32_t i = 4u * threadIdx.x; i < dim; i += 4u * blockDim.x) {
            float v[4];
            load4<DT>(table, (size_t)t * dim + i, v);
            store4<kFP32>(x, r * dim + i, v);
            if constexpr (NORM) {
                float w[4], b[4];
                load4<DT>(norm.weight, i, w);
                load4<DT>(norm.bias, i, b);
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = __builtin_fmaf(tanhf(alpha * v[e]), w[e], b[e]);
            }
            if (xe != nullptr) store4<DT>(xe, r * dim + i, v);
        }
    } else {
        for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) {
            float v = E::load(table, (size_t)t * dim + i);
            x[r * dim + i] = v;
            if constexpr (NORM) v = __builtin_fmaf(tanhf(alpha * v), E::load(norm.weight, i), E::load(norm.bias, i));
            if (xe != nullptr) E::store(xe, r * dim + i, v);
        }
    }
}

template <int DT, bool NORM>
static hipError_t embed_dt(const void* table, const long long* tokens, float* x, void* xe, const decdec_tanh_norm& norm, uint32_t rows,
                           uint32_t vocab, uint32_t dim, hipStream_t s) {
    const uint32_t es = Elem<DT>::bytes;
    const bool vec = dim % 4u == 0 && (uintptr_t)x % 16u == 0 &&
                     ((uintptr_t)table | (uintptr_t)xe | (uintptr_t)norm.weight | (uintptr_t)norm.bias) % (4u * es) == 0;
    uint32_t threads = 64;
    while (threads < 1024u && threads < (vec ? dim / 4u : dim)) threads *= 2;
    if (vec) hipLaunchKernelGGL((mix_embed_kernel<DT, true, NORM>), dim3(rows), dim3(threads), 0, s, table, tokens, x, xe, norm, vocab, dim);
    else hipLaunchKernelGGL((mix_embed_kernel<DT, false, NORM>), dim3(rows), dim3(threads), 0, s, table, tokens, x, xe, norm, vocab, dim);
    return hipGetLastError();
}

hipError_t launch_mix_embed(int dt, const void* table, const long long* tokens, float* x, void* xe, const decdec_tanh_norm* norm,
                            uint32_t rows, uint32_t vocab, uint32_t dim, hipStream_t s) {
    const decdec_tanh_norm n = norm != nullptr ? *norm : decdec_tanh_norm{};
    if (dt == kBF16) return norm != nullptr ? embed_dt<kBF16, true>(table, tokens, x, xe, n, rows, vocab, dim, s)
                                            : embed_dt<kBF16, false>(table, tokens, x, xe, n, rows, vocab, dim, s);
    return norm != nullptr ? embed_dt<kFP32, true>(table, tokens, x, xe, n, rows, vocab, dim, s)
                           : embed_dt<kFP32, false>(table, tokens, x, xe, n, rows, vocab, dim, s);
}

// ---- residual with a dynamic tanh ahead of the next sublayer ------------------------------------------------
// Element by element, 1024 elements of a row per workgroup.  Y: there is something to add.
template <int DT, bool VEC, bool Y>
__global__ __launch_bounds__(256) void residual_tanh_kernel(float* __restrict__ x, const void* __restrict__ y, const decdec_tanh_norm norm,
                                                            void* __restrict__ out, const uint32_t dim) {
    using E = Elem<DT>;
    const size_t row = (size_t)blockIdx.x * dim;
    const uint32_t i0 = blockIdx.y * 1024u;
    if constexpr (VEC) {
        const uint32_t i = i0 + 4u * threadIdx.x;
        if (i >= dim) return;
        float xv[4], yv[4], w[4], b[4];
        load4<kFP32>(x, row + i, xv);
        if constexpr (Y) load4<DT>(y, row + i, yv);
        load4<DT>(norm.weight, i, w);
        load4<DT>(norm.bias, i, b);
        const float alpha = E::load(norm.alpha, 0);
        if constexpr (Y) {
#pragma unroll
            for (int e = 0; e < 4; ++e) xv[e] += yv[e];
            store4<kFP32>(x, row + i, xv);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) xv[e] = __builtin_fmaf(tanhf(alpha * xv[e]), w[e], b[e]);
        store4<DT>(out, row + i, xv);
    } else {
        const float alpha = E::load(norm.alpha, 0);
        for (uint32_t i = i0 + threadIdx.x; i < dim && i < i0 + 1024u; i += 256u) {
            float v = x[row + i];
            if constexpr (Y) { v += E::load(y, row + i); x[row + i] = v; }
            E::store(out, row + i, __builtin_fmaf(tanhf(alpha * v), E::load(norm.weight, i), E::load(norm.bias, i)));
        }
    }
}

template <int DT, bool Y>
static hipError_t residual_tanh_dt(float* x, const void* y, const decdec_tanh_norm& norm, void* out, uint32_t rows, uint32_t dim, hipStream_t s) {
    const uint32_t es = Elem<DT>::bytes;
    const bool vec = dim % 4u == 0 && (uintptr_t)x % 16u == 0 &&
                     ((uintptr_t)y | (uintptr_t)out | (uintptr_t)norm.weight | (uintptr_t)norm.bias) % (4u * es) == 0;
    const dim3 grid(rows, (dim + 1023u) / 1024u), block(256);
    if (vec) hipLaunchKernelGGL((residual_tanh_kernel<DT, true, Y>), grid, block, 0, s, x, y, norm, out, dim);
    else hipLaunchKernelGGL((residual_tanh_kernel<DT, false, Y>), grid, block, 0, s, x, y, norm, out, dim);
    return hipGetLastError();
}

hipError_t launch_mix_residual_tanh(int dt, float* x, const void* y, const decdec_tanh_norm& norm, void* out, uint32_t rows,
                                    uint32_t dim, hipStream_t s) {
    if (dt == kBF16) return y != nullptr ? residual_tanh_dt<kBF16, true>(x, y, norm, out, rows, dim, s) : residual_tanh_dt<kBF16, false>(x, y, norm, out, rows, dim, s);
    return y != nullptr ? residual_tanh_dt<kFP32, true>(x, y, norm, out, rows, dim, s) : residual_tanh_dt<kFP32, false>(x, y, norm, out, rows, dim, s);
}

// ---- gated residual with the norm on the sublayer's output -------------------------------------------------
// One workgroup per row.  Four neighbouring elements per thread and pass, everything a pass needs requested at once
// (VEC; element accesses otherwise).  The optional second norm (the model's last one) reads the row just written.
template <int DT, int PASSES>
__global__ __launch_bounds__(1024) void gated_residual_vec_kernel(float* __restrict__ x, const void* __restrict__ y,
                                                                  const void* __restrict__ gate, const uint32_t gate_ld,
                                                                  const void* __restrict__ bias, const void* __restrict__ weight,
                                                                  void* __restrict__ xe, const void* __restrict__ fw,
                                                                  void* __restrict__ fo, const uint32_t dim, const float eps) {
    __shared__ float red[17];
    const uint32_t tid = threadIdx.x;
    const size_t row = (size_t)blockIdx.x * dim, grow = (size_t)blockIdx.x * gate_ld;
    float xv[PASSES][4], yv[PASSES][4], wv[PASSES][4];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < PASSES; ++k) {
        const uint32_t i = 4u * (tid + (uint32_t)k * blockDim.x);
        const bool ok = i < dim;
        const uint32_t ic = ok ? i : 0u;                     // groups past the end re-read the first one; never used
        float gv[4], bv[4];
        load4<kFP32>(x, row + ic, xv[k]);
        load4<DT>(y, row + ic, yv[k]);
        load4<DT>(weight, ic, wv[k]);
        if (gate != nullptr) { load4<DT>(gate, grow + ic, gv); load4<DT>(bias, ic, bv); }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            if (gate != nullptr) yv[k][e] *= sigmoid_f(gv[e] + bv[e]);
            ss += ok ? yv[k][e] * yv[k][e] : 0.f;
        }
    }
    float r = 1.f / sqrtf(block_sum(ss, red) / (float)dim + eps);
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < PASSES; ++k) {
        const uint32_t i = 4u * (tid + (uint32_t)k * blockDim.x);
#pragma unroll
        for (int e = 0; e < 4; ++e) xv[k][e] += yv[k][e] * r * wv[k][e];
        if (i < dim) {
            store4<kFP32>(x, row + i, xv[k]);
            if (xe != nullptr) store4<DT>(xe, row + i, xv[k]);
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += xv[k][e] * xv[k][e];
        }
    }
    if (fo == nullptr) return;
    r = 1.f / sqrtf(block_sum(ss, red) / (float)dim + eps);
#pragma unroll
    for (int k = 0; k < PASSES; ++k) {
        const uint32_t i = 4u * (tid + (uint32_t)k * blockDim.x);
        if (i < dim) {
            float f[4];
            load4<DT>(fw, i, f);
#pragma unroll
            for (int e = 0; e < 4; ++e) f[e] *= xv[k][e] * r;
            store4<DT>(fo, row + i, f);
        }
    }
}

template <int DT>
__global__ __launch_bounds__(1024) void gated_residual_kernel(float* __restrict__ x, const void* __restrict__ y,
                                                              const void* __restrict__ gate, const uint32_t gate_ld,
                                                              const void* __restrict__ bias, const void* __restrict__ weight,
                                                              void* __restrict__ xe, const void* __restrict__ fw,
                                                              void* __restrict__ fo, const uint32_t dim, const float eps) {
    using E = Elem<DT>;
    __shared__ float red[17];
    const size_t row = (size_t)blockIdx.x * dim, grow = (size_t)blockIdx.x * gate_ld;
    auto gated = [&](uint32_t i) {
        const float v = E::load(y, row + i);
        return gate != nullptr ? v * sigmoid_f(E::load(gate, grow + i) + E::load(bias, i)) : v;
    };
    float ss = 0.f;
    for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) { const float v = gated(i); ss += v * v; }
    float r = 1.f / sqrtf(block_sum(ss, red) / (float)dim + eps);
    ss = 0.f;
    for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) {
        const float v = x[row + i] + gated(i) * r * E::load(weight, i);
        x[row + i] = v;
        if (xe != nullptr) E::store(xe, row + i, v);
        ss += v * v;
    }
    if (fo == nullptr) return;
    r = 1.f / sqrtf(block_sum(ss, red) / (float)dim + eps);
    for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) E::store(fo, row + i, x[row + i] * r * E::load(fw, i));
}

template <int DT>
static hipError_t gated_residual_dt(float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias,
                                    const void* weight, void* xe, const void* fw, void* fo, uint32_t rows, uint32_t dim,
                                    float eps, hipStream_t s) {
    uintptr_t al = (uintptr_t)x | (uintptr_t)y * (DT == kFP32 ? 1 : 2) | (uintptr_t)weight * (DT == kFP32 ? 1 : 2);
    for (const void* p : {gate, bias, (const void*)xe, fw, (const void*)fo}) al |= (uintptr_t)p * (DT == kFP32 ? 1 : 2);
    const bool vec = al % 16 == 0 && dim % 4u == 0 && gate_ld % 4u == 0 && dim <= 16384u;
    const uint32_t groups = (dim + 3u) / 4u;
    uint32_t threads = 64;
    while (threads < 1024u && threads < groups) threads *= 2;
    if (!vec) hipLaunchKernelGGL((gated_residual_kernel<DT>), dim3(rows), dim3(threads), 0, s, x, y, gate, gate_ld, bias, weight, xe, fw, fo, dim, eps);
    else if (groups <= threads) hipLaunchKernelGGL((gated_residual_vec_kernel<DT, 1>), dim3(rows), dim3(threads), 0, s, x, y, gate, gate_ld, bias, weight, xe, fw, fo, dim, eps);
    else if (groups <= 2 * threads) hipLaunchKernelGGL((gated_residual_vec_kernel<DT, 2>), dim3(rows), dim3(threads), 0, s, x, y, gate, gate_ld, bias, weight, xe, fw, fo, dim, eps);
    else hipLaunchKernelGGL((gated_residual_vec_kernel<DT, 4>), dim3(rows), dim3(threads), 0, s, x, y, gate, gate_ld, bias, weight, xe, fw, fo, dim, eps);
    return hipGetLastError();
}

hipError_t launch_mix_gated_residual(int dt, float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias,
                                     const void* weight, void* xe, const void* fw, void* fo, uint32_t rows, uint32_t dim,
                                     float eps, hipStream_t s) {
    if (dt == kBF16) return gated_residual_dt<kBF16>(x, y, gate, gate_ld, bias, weight, xe, fw, fo, rows, dim, eps, s);
    return gated_residual_dt<kFP32>(x, y, gate, gate_ld, bias, weight, xe, fw, fo, rows, dim, eps, s);
}

// ---- norm -------------------------------------------------------------------------------------------------
template <int DT>
__global__ __launch_bounds__(1024) void mix_rmsnorm_kernel(const float* __restrict__ x, const void* __restrict__ weight,
                                                           void* __restrict__ out, const uint32_t dim, const float eps) {
    using E = Elem<DT>;
    __shared__ float red[17];
    const size_t row = (size_t)blockIdx.x * dim;
    float ss = 0.f;
    for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) ss += x[row + i] * x[row + i];
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)dim + eps);
    for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) E::store(out, row + i, x[row + i] * r * E::load(weight, i));
}

hipError_t launch_mix_rmsnorm(int dt, const float* x, const void* weight, void* out, uint32_t rows, uint32_t dim, float eps,
                              hipStream_t s) {
    uint32_t threads = 64;
    while (threads < 1024u && threads < dim) threads *= 2;
    if (dt == kBF16) hipLaunchKernelGGL((mix_rmsnorm_kernel<kBF16>), dim3(rows), dim3(threads), 0, s, x, weight, out, dim, eps);
    else hipLaunchKernelGGL((mix_rmsnorm_kernel<kFP32>), dim3(rows), dim3(threads), 0, s, x, weight, out, dim, eps);
    return hipGetLastError();
}

// ---- activations ------------------------------------------------------------------------------------------
template <int DT, bool VEC, int ACT>
__global__ __launch_bounds__(256) void mix_activation_kernel(const void* in, const uint32_t ld,
                                                        const void* __restrict__ act, void* out, const uint32_t n) {
    using E = Elem<DT>;
    const float sp = ACT == DECDEC_ACT_XIELU ? softplus_f(E::load(act, 0)) : 0.f, sq = ACT == DECDEC_ACT_XIELU ? softplus_f(E::load(act, 1)) : 0.f;
    auto f = [&](float z) { return ACT == DECDEC_ACT_XIELU ? xielu_f(z, sp, sq) : gelu_tanh_f(z); };
    const size_t irow = (size_t)blockIdx.x * ld, orow = (size_t)blockIdx.x * n;
    if constexpr (VEC) {
        // four quads a workgroup's width apart, requested together
        for (uint32_t i0 = 4u * (blockIdx.y * 1024u + threadIdx.x); i0 < n; i0 += 4096u * gridDim.y) {
            float v[4][4];
#pragma unroll
            for (uint32_t k = 0; k < 4u; ++k) load4<DT>(in, irow + (i0 + 1024u * k < n ? i0 + 1024u * k : 0u), v[k]);
#pragma unroll
            for (uint32_t k = 0; k < 4u; ++k) {
#pragma unroll
                for (int e = 0; e < 4; ++e) v[k][e] = f(v[k][e]);
                if (i0 + 1024u * k < n) store4<DT>(out, orow + i0 + 1024u * k, v[k]);
            }
        }
    } else {
        for (uint32_t i = blockIdx.y * 256u + threadIdx.x; i < n; i += 256u * gridDim.y)
            E::store(out, orow + i, f(E::load(in, irow + i)));
    }
}

template <int DT, int ACT>
static hipError_t activation_dt(const void* in, uint32_t ld, const void* act, void* out, uint32_t rows, uint32_t n, hipStream_t s) {
    const uint32_t es = Elem<DT>::bytes;
    const bool vec = n % 4u == 0 && ld % 4u == 0 && (uintptr_t)in % (4 * es) == 0 && (uintptr_t)out % (4 * es) == 0;
    const uint32_t per = vec ? 4096u : 256u, gy = (n + per - 1u) / per;
    const dim3 grid(rows, gy < 16u ? gy : 16u), block(256);
    if (vec) hipLaunchKernelGGL((mix_activation_kernel<DT, true, ACT>), grid, block, 0, s, in, ld, act, out, n);
    else hipLaunchKernelGGL((mix_activation_kernel<DT, false, ACT>), grid, block, 0, s, in, ld, act, out, n);
    return hipGetLastError();
}

hipError_t launch_mix_activation(int dt, const void* in, uint32_t ld, const void* act, int kind, void* out, uint32_t rows,
                                 uint32_t n, hipStream_t s) {
    if (kind == DECDEC_ACT_GELU_TANH) return dt == kBF16 ? activation_dt<kBF16, DECDEC_ACT_GELU_TANH>(in, ld, act, out, rows, n, s)
                                                         : activation_dt<kFP32, DECDEC_ACT_GELU_TANH>(in, ld, act, out, rows, n, s);
    return dt == kBF16 ? activation_dt<kBF16, DECDEC_ACT_XIELU>(in, ld, act, out, rows, n, s)
                       : activation_dt<kFP32, DECDEC_ACT_XIELU>(in, ld, act, out, rows, n, s);
}

// ---- normed, gated read-out of a recurrence ----------------------------------------------------------------
// A workgroup per (row, group).
template <int DT>
__global__ __launch_bounds__(1024) void group_norm_gate_kernel(const float* __restrict__ o, const void* __restrict__ gate,
                                                               const uint32_t ld, const void* __restrict__ weight,
                                                               void* __restrict__ out, const uint32_t out_ld, const uint32_t n,
                                                               const float eps, const int kind, const float scale) {
    using E = Elem<DT>;
    __shared__ float red[17];
    const uint32_t r = blockIdx.x, g = blockIdx.y;
    const size_t base = (size_t)r * n * gridDim.y + (size_t)g * n, gbase = (size_t)r * ld + (size_t)g * n, obase = (size_t)r * out_ld + (size_t)g * n;
    float ss = 0.f;
    for (uint32_t i = threadIdx.x; i < n; i += blockDim.x) ss += o[base + i] * o[base + i];
    const float rs = scale / sqrtf(block_sum(ss, red) / (float)n + eps);
    for (uint32_t i = threadIdx.x; i < n; i += blockDim.x) {
        const float z = E::load(gate, gbase + i);
        const float gt = kind == DECDEC_GATE_SILU ? silu_f(z) : sigmoid_f(z);
        E::store(out, obase + i, o[base + i] * rs * E::load(weight, i) * gt);
    }
}

// Groups of at most 64 EP elements: a wave each, EP neighbouring elements per lane.  FULL: exactly 64 EP, aligned to EP.
template <int DT, int EP, bool FULL>
__global__ __launch_bounds__(256) void group_norm_gate_wave_kernel(const float* __restrict__ o, const void* __restrict__ gate,
                                                                   const uint32_t ld, const void* __restrict__ weight,
                                                                   void* __restrict__ out, const uint32_t out_ld, const uint32_t rows,
                                                                   const uint32_t groups, const uint32_t n, const float eps,
                                                                   const int kind, const float scale) {
    using E = Elem<DT>;
    const uint32_t lane = threadIdx.x & 63u, at = blockIdx.x * 4u + (threadIdx.x >> 6), r = at / groups, g = at - r * groups;
    if (r >= rows) return;
    const uint32_t i0 = lane * (uint32_t)EP;
    const size_t base = ((size_t)r * groups + g) * n, gbase = (size_t)r * ld + (size_t)g * n, obase = (size_t)r * out_ld + (size_t)g * n;
    float x[EP], z[EP], w[EP], ss = 0.f;
    if constexpr (FULL && EP == 4) {
        load4<kFP32>(o, base + i0, x);
        load4<DT>(gate, gbase + i0, z);
        load4<DT>(weight, i0, w);
        ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
    } else if constexpr (FULL && EP == 2) {
        const u32x2 t = *(const u32x2*)(o + base + i0);
        x[0] = __uint_as_float(t[0]);
        x[1] = __uint_as_float(t[1]);
        uint32_t a, b;
        E::load_raw2(gate, gbase + i0, a, b);
        z[0] = E::from_raw2_lo(a, b); z[1] = E::from_raw2_hi(a, b);
        E::load_raw2(weight, i0, a, b);
        w[0] = E::from_raw2_lo(a, b); w[1] = E::from_raw2_hi(a, b);
        ss = x[0] * x[0] + x[1] * x[1];
    } else
#pragma unroll
    for (int e = 0; e < EP; ++e) {
        const bool ok = FULL || i0 + e < n;
        const uint32_t i = ok ? i0 + e : 0u;
        x[e] = o[base + i];
        z[e] = E::load(gate, gbase + i);
        w[e] = E::load(weight, i);
        ss += ok ? x[e] * x[e] : 0.f;
    }
    const float rs = scale / sqrtf(wave_sum(ss) / (float)n + eps);
    if constexpr (FULL) {
#pragma unroll
        for (int e = 0; e < EP; ++e) x[e] *= rs * w[e] * (kind == DECDEC_GATE_SILU ? silu_f(z[e]) : sigmoid_f(z[e]));
        if constexpr (EP == 4) store4<DT>(out, obase + i0, x);
        else if constexpr (DT == kBF16) *(uint32_t*)((uint16_t*)out + obase + i0) = pack_bf16(x[0], x[1]);
        else *(u32x2*)((float*)out + obase + i0) = u32x2{__float_as_uint(x[0]), __float_as_uint(x[1])};
        return;
    }
#pragma unroll
    for (int e = 0; e < EP; ++e)
        if (FULL || i0 + e < n) E::store(out, obase + i0 + e, x[e] * rs * w[e] * (kind == DECDEC_GATE_SILU ? silu_f(z[e]) : sigmoid_f(z[e])));
}

// Longer groups: a workgroup each, four neighbouring elements per thread and pass.
template <int DT, int PASSES>
__global__ __launch_bounds__(1024) void group_norm_gate_vec_kernel(const float* __restrict__ o, const void* __restrict__ gate,
                                                                   const uint32_t ld, const void* __restrict__ weight,
                                                                   void* __restrict__ out, const uint32_t out_ld, const uint32_t n,
                                                                  const float eps, const int kind, const float scale) {
    __shared__ float red[17];
    const uint32_t tid = threadIdx.x;
    const size_t base = ((size_t)blockIdx.x * gridDim.y + blockIdx.y) * n, gbase = (size_t)blockIdx.x * ld + (size_t)blockIdx.y * n;
    const size_t obase = (size_t)blockIdx.x * out_ld + (size_t)blockIdx.y * n;
    float x[PASSES][4], z[PASSES][4], w[PASSES][4], ss = 0.f;
#pragma unroll
    for (int k = 0; k < PASSES; ++k) {
        const uint32_t i = 4u * (tid + (uint32_t)k * blockDim.x), ic = i < n ? i : 0u;
        load4<kFP32>(o, base + ic, x[k]);
        load4<DT>(gate, gbase + ic, z[k]);
        load4<DT>(weight, ic, w[k]);
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += i < n ? x[k][e] * x[k][e] : 0.f;
    }
    const float rs = scale / sqrtf(block_sum(ss, red) / (float)n + eps);
#pragma unroll
    for (int k = 0; k < PASSES; ++k) {
        const uint32_t i = 4u * (tid + (uint32_t)k * blockDim.x);
        if (i < n) {
#pragma unroll
            for (int e = 0; e < 4; ++e) x[k][e] *= rs * w[k][e] * (kind == DECDEC_GATE_SILU ? silu_f(z[k][e]) : sigmoid_f(z[k][e]));
            store4<DT>(out, obase + i, x[k]);
        }
    }
}

template <int DT>
static hipError_t group_norm_dt(const float* o, const void* gate, uint32_t ld, const void* weight, void* out, uint32_t out_ld,
                                uint32_t rows, uint32_t groups, uint32_t n, float eps, int kind, float scale, hipStream_t s) {
    const uint32_t es = Elem<DT>::bytes, waves = rows * groups;
    const dim3 wgrid((waves + 3u) / 4u), wblock(256);
    auto full = [&](uint32_t ep) {
        return n == 64u * ep && ld % ep == 0 && out_ld % ep == 0 && (uintptr_t)o % (4u * ep) == 0 && ((uintptr_t)gate | (uintptr_t)weight | (uintptr_t)out) % (es * ep) == 0;
    };
    if (full(2u)) hipLaunchKernelGGL((group_norm_gate_wave_kernel<DT, 2, true>), wgrid, wblock, 0, s, o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale);
    else if (n <= 128u) hipLaunchKernelGGL((group_norm_gate_wave_kernel<DT, 2, false>), wgrid, wblock, 0, s, o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale);
    else if (full(4u)) hipLaunchKernelGGL((group_norm_gate_wave_kernel<DT, 4, true>), wgrid, wblock, 0, s, o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale);
    else if (n <= 256u) hipLaunchKernelGGL((group_norm_gate_wave_kernel<DT, 4, false>), wgrid, wblock, 0, s, o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale);
    else {
        uint32_t threads = 64;
        const bool vec = n % 4u == 0 && ld % 4u == 0 && out_ld % 4u == 0 && n <= 16384u && (uintptr_t)o % 16u == 0 &&
                         ((uintptr_t)gate | (uintptr_t)weight | (uintptr_t)out) % (4u * es) == 0;
        const uint32_t want = vec ? (n + 3u) / 4u : n;
        while (threads < 1024u && threads < want) threads *= 2;
        const dim3 grid(rows, groups), block(threads);
        if (!vec) hipLaunchKernelGGL((group_norm_gate_kernel<DT>), grid, block, 0, s, o, gate, ld, weight, out, out_ld, n, eps, kind, scale);
        else if (want <= threads) hipLaunchKernelGGL((group_norm_gate_vec_kernel<DT, 1>), grid, block, 0, s, o, gate, ld, weight, out, out_ld, n, eps, kind, scale);
        else if (want <= 2u * threads) hipLaunchKernelGGL((group_norm_gate_vec_kernel<DT, 2>), grid, block, 0, s, o, gate, ld, weight, out, out_ld, n, eps, kind, scale);
        else hipLaunchKernelGGL((group_norm_gate_vec_kernel<DT, 4>), grid, block, 0, s, o, gate, ld, weight, out, out_ld, n, eps, kind, scale);
    }
    return hipGetLastError();
}

hipError_t launch_mix_group_norm_gate(int dt, const float* o, const void* gate, uint32_t ld, const void* weight, void* out,
                                      uint32_t out_ld, uint32_t rows, uint32_t groups, uint32_t n, float eps, int kind,
                                      float scale, hipStream_t s) {
    return dt == kBF16 ? group_norm_dt<kBF16>(o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale, s)
                       : group_norm_dt<kFP32>(o, gate, ld, weight, out, out_ld, rows, groups, n, eps, kind, scale, s);
}

}  // namespace decdec
