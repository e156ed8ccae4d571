// Latent attention: the keys and values of all heads are linear in one normed latent per token, which is what the cache
// holds, next to a rotated key part that the heads share.
//
// Many tokens: keys and values of the whole past are formed by two matrix products outside and attended by a tiled
// kernel.  One token: the up projections are absorbed -- a query is carried into the latent space (absorb kernel), all
// heads attend the same cache rows (step kernel, sequence split over workgroups), and the attended latents are carried
// to the values (merge kernel).  Scores, weights and sums are fp32; on bf16 storage a weight enters the value product as
// the sum of two bf16 numbers.
#include "mixers.h"
#include "mma.h"

namespace decdec {

template <int DT> __device__ __forceinline__ void store_elem(typename LaneOf<DT>::t* p, float v) { Elem<DT>::store(p, 0, v); }

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

// The new cache row of one token (a whole workgroup): normed latent, rotated shared key part.
template <int DT>
__device__ __forceinline__ void append_row(const decdec_latent& p, const void* proj, size_t row, long long pos, float* red) {
    using E = Elem<DT>;
    if (pos < 0 || pos >= (long long)p.max_seq) return;                    // uniform over the workgroup
    const uint32_t half = p.rot / 2u;
    const size_t src = row + p.off_c, dst = (size_t)pos * (p.rank + p.rot);
    float ss = 0.f;
    for (uint32_t i = threadIdx.x; i < p.rank; i += blockDim.x) { const float v = E::load(proj, src + i); ss += v * v; }
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)p.rank + p.eps);
    for (uint32_t i = threadIdx.x; i < p.rank; i += blockDim.x)
        E::store(p.cache, dst + i, E::load(proj, src + i) * r * E::load(p.norm, i));
    for (uint32_t i = threadIdx.x; i < half; i += blockDim.x) {
        const float u = E::load(proj, src + p.rank + 2u * i), v = E::load(proj, src + p.rank + 2u * i + 1u);
        const float c = p.cos_table[(size_t)pos * half + i], s = p.sin_table[(size_t)pos * half + i];
        E::store(p.cache, dst + p.rank + 2u * i, u * c - v * s);
        E::store(p.cache, dst + p.rank + 2u * i + 1u, v * c + u * s);
    }
}

template <int DT>
__global__ __launch_bounds__(256) void latent_append_kernel(const decdec_latent p, void* __restrict__ q_out) {
    using E = Elem<DT>;
    __shared__ float red[17];
    const uint32_t t = blockIdx.x, Dq = p.dim + p.rot, half = p.rot / 2u;
    const long long pos = *p.pos + (long long)t;
    const size_t row = (size_t)t * p.ld;
    append_row<DT>(p, p.proj, row, pos, red);
    const size_t trow = (size_t)(pos < 0 ? 0 : (pos < (long long)p.max_seq ? pos : (long long)p.max_seq - 1)) * half;
    const bool wide = p.dim % 8u == 0 && p.rot % 8u == 0 && p.ld % 8u == 0 && p.off_q % 8u == 0 && ((uintptr_t)p.proj | (uintptr_t)q_out) % 16u == 0;
    if (wide) {                                            // eight neighbouring elements: four pairs, or none to turn
        using T = typename LaneOf<DT>::t;
        const T* src = (const T*)p.proj + row + p.off_q;
        for (uint32_t i = threadIdx.x; i < p.heads * (Dq / 8u); i += 256u) {
            const uint32_t e = 8u * (i % (Dq / 8u));
            Frag<DT> f = frag_load(src + 8u * i);
            if (e >= p.dim) {
                float x[8];
                frag_values(f, x);
#pragma unroll
                for (uint32_t j = 0; j < 4u; ++j) {
                    const size_t at = trow + (e - p.dim) / 2u + j;
                    const float c = p.cos_table[at], s = p.sin_table[at], u = x[2 * j], v = x[2 * j + 1];
                    x[2 * j] = u * c - v * s;
                    x[2 * j + 1] = v * c + u * s;
                }
                f = frag_of(x, f);
            }
            store8((T*)q_out + (size_t)t * p.heads * Dq + 8u * i, f);
        }
        return;
    }
    for (uint32_t i = threadIdx.x; i < p.heads * (Dq / 2u); i += 256u) {
        const uint32_t h = i / (Dq / 2u), e = 2u * (i % (Dq / 2u));
        const size_t at = (size_t)t * p.heads * Dq + h * Dq + e;
        float u = E::load(p.proj, row + p.off_q + h * Dq + e), v = E::load(p.proj, row + p.off_q + h * Dq + e + 1u);
        if (e >= p.dim) {
            const uint32_t j = (e - p.dim) / 2u;
            const float c = p.cos_table[trow + j], s = p.sin_table[trow + j], u0 = u;
            u = u0 * c - v * s;
            v = v * c + u0 * s;
        }
        E::store(q_out, at, u);
        E::store(q_out, at + 1u, v);
    }
}

hipError_t launch_latent_append(int dt, const decdec_latent& p, void* q_out, uint32_t rows, hipStream_t s) {
    if (dt == kBF16) hipLaunchKernelGGL((latent_append_kernel<kBF16>), dim3(rows), dim3(256), 0, s, p, q_out);
    else hipLaunchKernelGGL((latent_append_kernel<kFP32>), dim3(rows), dim3(256), 0, s, p, q_out);
    return hipGetLastError();
}

// ---- many tokens ------------------------------------------------------------------------------------------
// Workgroups of four waves with 16 MT queries each, one per query block and head; the heads are dealt to the eight dies,
// so that the tiles of a head's keys and values are shared in one L2.  The transposed scores (keys x queries) leave a query in one
// lane column: its running maximum and sum are lane values, its weights are at once the right operand of the value
// product (out^T = V^T P^T), and nothing passes through LDS but the key and value tiles.  The contraction of that product
// visits keys 4 (lane / 16) + e of one 16-key tile, then of the next, in both operands.  The next tile is requested into
// registers while the present one is worked on.  Scores are kept in units of log 2.
constexpr uint32_t kKeys = 64;

template <int DT, int MT, int NK, int NV, bool VEC>
__global__ __launch_bounds__(256, DT == kFP32 ? 1 : 2) void latent_attention_kernel(const decdec_latent p, const void* __restrict__ q_in,
                                                               const void* __restrict__ k_in, const void* __restrict__ vt_in,
                                                               const uint32_t vt_ld, void* __restrict__ out,
                                                               const uint32_t start, const uint32_t rows, const uint32_t blocks) {
    using T = typename LaneOf<DT>::t;
    using E = Elem<DT>;
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, KL = 32u * NK + PAD, VL = kKeys + PAD;
    extern __shared__ __align__(16) unsigned char smem[];
    T* Kl = (T*)smem;                       // [kKeys][KL]
    T* Vl = Kl + kKeys * KL;                // [16 NV][VL]
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t turn = blockIdx.x >> 3, h = (blockIdx.x & 7u) + 8u * (turn / blocks);
    if (h >= p.heads) return;
    const uint32_t q0 = (blocks - 1u - turn % blocks) * (64u * MT);        // longest rows first
    const uint32_t Dq = p.dim + p.rot, D = p.dim, V = p.vdim, keys_total = start + rows;
    const T* q = (const T*)q_in;
    Frag<DT> qf[MT][NK];
    uint32_t qpos[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const uint32_t r = q0 + 16u * (MT * wave + (uint32_t)m) + l16, rc = r < rows ? r : rows - 1u;
        qpos[m] = start + rc;
#pragma unroll
        for (int s = 0; s < NK; ++s)
            qf[m][s] = load8<DT>(q + ((size_t)rc * p.heads + h) * Dq + 32u * s + 8u * lg, (int)Dq - (int)(32u * s + 8u * lg), VEC);
    }
    const float scale2 = p.scale * kLog2e;
    const float sink = p.sink != nullptr ? E::load(p.sink, h) * kLog2e : -__builtin_inff();
    float mx[MT], sum[MT];
    f32x4 o[MT][NV];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        mx[m] = sink;
        sum[m] = (p.sink != nullptr && lg == 0u) ? 1.f : 0.f;              // lane groups hold partial sums
#pragma unroll
        for (int n = 0; n < NV; ++n) o[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const uint32_t last = q0 + 64u * MT < rows ? q0 + 64u * MT : rows;     // one past the block's last query
    const uint32_t kend = start + last, wave_first = start + q0 + 16u * MT * wave, wave_last = wave_first + 16u * MT - 1u;
    const size_t kld = (size_t)p.heads * D, cld = p.rank + p.rot;
    const T* kb = (const T*)k_in + (size_t)h * D;
    const T* cb = (const T*)p.cache + p.rank;
    const T* vb = (const T*)vt_in + (size_t)h * V * vt_ld;
    // A key row is [unrotated part of the head | shared rotated part]; keys past the end repeat the last one and are never
    // weighted, value rows past vdim repeat the first one and are never stored.  A thread loads eight elements of every
    // slice of one key, and of every 32nd value row.
    Frag<DT> kr[VEC ? NK : 1], vr[VEC ? NV / 2 : 1];
    const uint32_t krow = tid >> 2, kcol = (tid & 3u) * 8u, vrow = tid >> 3, vcol = (tid & 7u) * 8u;
    auto request = [&](uint32_t k0) {
        const uint32_t key = k0 + krow < keys_total ? k0 + krow : keys_total - 1u;
        const T* un = kb + key * kld + kcol;
        const T* ro = cb + key * cld + kcol;
#pragma unroll
        for (int j = 0; j < NK; ++j) {
            const uint32_t c = 32u * j + kcol;
            kr[j] = frag_load(c < D ? un + 32u * j : (c < Dq ? ro + (32 * j - (int)D) : cb));
            if (c >= Dq) kr[j] = Frag<DT>{};
        }
        const T* vp = vb + k0 + vcol;
#pragma unroll
        for (int j = 0; j < NV / 2; ++j) vr[j] = frag_load(vp + (size_t)(vrow + 32u * j < V ? vrow + 32u * j : 0u) * vt_ld);
    };
    if constexpr (VEC) request(0u);
    for (uint32_t k0 = 0; k0 < kend; k0 += kKeys) {
        __syncthreads();
        if constexpr (VEC) {
#pragma unroll
            for (int j = 0; j < NK; ++j) store8(Kl + krow * KL + kcol + 32u * j, kr[j]);
#pragma unroll
            for (int j = 0; j < NV / 2; ++j) store8(Vl + (vrow + 32u * j) * VL + vcol, vr[j]);
        } else {
            for (uint32_t i = tid; i < kKeys * 32u * NK; i += 256u) {
                const uint32_t r = i / (32u * NK), c = i % (32u * NK), key = k0 + r < keys_total ? k0 + r : keys_total - 1u;
                Kl[r * KL + c] = c < D ? kb[key * kld + c] : (c < Dq ? cb[key * cld + c - D] : (T)0);
            }
            for (uint32_t i = tid; i < 16u * NV * kKeys; i += 256u) {
                const uint32_t d = i / kKeys, c = i % kKeys;
                Vl[d * VL + c] = d < V ? vb[(size_t)d * vt_ld + k0 + c] : (T)0;
            }
        }
        __syncthreads();
        if constexpr (VEC) { if (k0 + kKeys < kend) request(k0 + kKeys); }
        if (k0 > wave_last) continue;                                      // every key of the tile lies after the wave's queries
        f32x4 sc[MT][4];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int t = 0; t < 4; ++t) sc[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < NK; ++s)
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const Frag<DT> a = frag_load(Kl + (16u * t + l16) * KL + 32u * s + 8u * lg);
#pragma unroll
                for (int m = 0; m < MT; ++m) mma(a, qf[m][s], sc[m][t]);
            }
        const bool edge = k0 + kKeys > wave_first + 1u;                    // some key may lie after some query of the wave
        Frag<DT> hi[MT][2], lo[MT][2];
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            float best = mx[m];
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    float x = sc[m][t][v] * scale2;
                    if (edge && k0 + 16u * t + 4u * lg + (uint32_t)v > qpos[m]) x = -__builtin_inff();
                    sc[m][t][v] = x;
                    best = fmaxf(best, x);
                }
            best = fmaxf(best, __shfl_xor(best, 16, 64));
            best = fmaxf(best, __shfl_xor(best, 32, 64));
            if (__any(best > mx[m])) {
                const float corr = __builtin_amdgcn_exp2f(mx[m] - best);   // the first key is visible to every query: best is finite
                mx[m] = best;
                sum[m] *= corr;
#pragma unroll
                for (int n = 0; n < NV; ++n) o[m][n] *= corr;
            }
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                float w[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    w[e] = __builtin_amdgcn_exp2f(sc[m][2 * t + (e >> 2)][e & 3] - best);
                    sum[m] += w[e];
                }
                frag_split(w, hi[m][t], lo[m][t]);
            }
        }
#pragma unroll
        for (int n = 0; n < NV; ++n)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const T* vk = Vl + (16u * n + l16) * VL + 32u * t + 4u * lg;
                Frag<DT> a;
                if constexpr (DT == kFP32) {
                    const f32x4 x = *(const f32x4*)vk, y = *(const f32x4*)(vk + 16);
#pragma unroll
                    for (int e = 0; e < 4; ++e) { a.v[e] = x[e]; a.v[4 + e] = y[e]; }
                } else {
                    const u32x2 x = *(const u32x2*)vk, y = *(const u32x2*)(vk + 16);
                    a.v = u32x4{x[0], x[1], y[0], y[1]};
                }
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    mma(a, hi[m][t], o[m][n]);
                    if constexpr (DT != kFP32) mma(a, lo[m][t], o[m][n]);
                }
            }
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        float t = sum[m];
        t += __shfl_xor(t, 16, 64);
        t += __shfl_xor(t, 32, 64);
        const float r = 1.f / t;
        const uint32_t row = q0 + 16u * (MT * wave + (uint32_t)m) + l16;
        if (row < rows) {
#pragma unroll
            for (int n = 0; n < NV; ++n)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const uint32_t d = 16u * n + 4u * lg + (uint32_t)v;
                    if (d < V) E::store(out, ((size_t)row * p.heads + h) * V + d, o[m][n][v] * r);
                }
        }
    }
}

template <int DT, int MT, int NK, int NV, bool VEC = true>
static hipError_t attention_launch(const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld, void* out,
                                   uint32_t start, uint32_t rows, hipStream_t s) {
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u;
    constexpr size_t lds = (size_t)(kKeys * (32u * NK + PAD) + 16u * NV * (kKeys + PAD)) * Elem<DT>::bytes;
    static_assert(lds <= 160u * 1024u, "tiles must fit the LDS of a compute unit");
    if (hipError_t e = allow_lds<latent_attention_kernel<DT, MT, NK, NV, VEC>>(lds); e != hipSuccess) return e;
    const uint32_t blocks = (rows + 64u * MT - 1u) / (64u * MT);
    hipLaunchKernelGGL((latent_attention_kernel<DT, MT, NK, NV, VEC>), dim3(blocks * ((p.heads + 7u) / 8u * 8u)), dim3(256), lds, s,
                       p, q, k, vt, vt_ld, out, start, rows, blocks);
    return hipGetLastError();
}

template <int DT, int MT, int NK>
static hipError_t attention_nv(const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld, void* out,
                               uint32_t start, uint32_t rows, hipStream_t s) {
    if (p.vdim <= 64u) return attention_launch<DT, MT, NK, 4>(p, q, k, vt, vt_ld, out, start, rows, s);
    if (p.vdim <= 128u) return attention_launch<DT, MT, NK, 8>(p, q, k, vt, vt_ld, out, start, rows, s);
    return attention_launch<DT, 1, NK, 16>(p, q, k, vt, vt_ld, out, start, rows, s);
}

template <int DT, int MT>
static hipError_t attention_dt(const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld, void* out,
                               uint32_t start, uint32_t rows, hipStream_t s) {
    const uint32_t Dq = p.dim + p.rot;
    if (p.dim % 8u != 0 || p.rot % 8u != 0 || p.rank % 8u != 0) return attention_launch<DT, 1, 10, 16, false>(p, q, k, vt, vt_ld, out, start, rows, s);
    if (Dq <= 128u) return attention_nv<DT, MT, 4>(p, q, k, vt, vt_ld, out, start, rows, s);
    if (Dq <= 192u) return attention_nv<DT, MT, 6>(p, q, k, vt, vt_ld, out, start, rows, s);
    return attention_nv<DT, 1, 10>(p, q, k, vt, vt_ld, out, start, rows, s);
}

hipError_t launch_latent_attention(int dt, const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld,
                                   void* out, uint32_t start, uint32_t rows, hipStream_t s) {
    if (p.dim + p.rot > 320u || p.vdim > 256u) return hipErrorInvalidValue;
    if (dt == kBF16) return attention_dt<kBF16, 2>(p, q, k, vt, vt_ld, out, start, rows, s);
    return attention_dt<kFP32, 1>(p, q, k, vt, vt_ld, out, start, rows, s);
}

// ---- one token --------------------------------------------------------------------------------------------
// Queries in the latent space, scaled: qa fp32 [heads][rank + rot].  grid (heads + 1, rank / 64); the last x appends.
template <int DT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const decdec_latent p, float* __restrict__ qa) {
    using E = Elem<DT>;
    using T = typename LaneOf<DT>::t;
    __shared__ float red[17], q[512], part[32][68];
    const uint32_t tid = threadIdx.x, h = blockIdx.x, D = p.dim, half = p.rot / 2u, R = p.rank, Dq = D + p.rot;
    const long long pos = *p.pos;
    if (h == p.heads) {
        if (blockIdx.y == 0u) append_row<DT>(p, p.proj, 0, pos, red);
        return;
    }
    const uint32_t c0 = blockIdx.y * 64u, cg = tid & 7u, rg = tid >> 3, c = c0 + 8u * cg;
    const bool vec = R % 8u == 0;
    const T* uk = (const T*)p.uk + (size_t)h * D * R + c;
    const int valid = (int)R - (int)c;
    for (uint32_t i = tid; i < D; i += 256u) q[i] = E::load(p.proj, p.off_q + h * Dq + i);
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = 0.f;
#pragma unroll 4
    for (uint32_t d = rg; d < D; d += 32u) {
        float w[8];
        frag_values(load8<DT>(valid > 0 ? uk + (size_t)d * R : uk, valid > 0 ? valid : 0, vec), w);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = __builtin_fmaf(w[e], q[d], acc[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) part[rg][8u * cg + e] = acc[e];
    __syncthreads();
    float* dst = qa + (size_t)h * (R + p.rot);
    if (tid < 64u && c0 + tid < R) {
        float t = 0.f;
#pragma unroll
        for (int r = 0; r < 32; ++r) t += part[r][tid];
        dst[c0 + tid] = t * p.scale;
    }
    if (blockIdx.y == 0u) {
        const size_t trow = (size_t)(pos < 0 ? 0 : (pos < (long long)p.max_seq ? pos : (long long)p.max_seq - 1)) * half;
        for (uint32_t i = tid; i < half; i += 256u) {
            const size_t at = p.off_q + h * Dq + D + 2u * i;
            const float u = E::load(p.proj, at), v = E::load(p.proj, at + 1u), cs = p.cos_table[trow + i], sn = p.sin_table[trow + i];
            dst[R + 2u * i] = (u * cs - v * sn) * p.scale;
            dst[R + 2u * i + 1u] = (v * cs + u * sn) * p.scale;
        }
    }
}

struct StepSplit { uint32_t splits, span; };
// The splits in use for `len` keys and the keys each of them takes (a multiple of 64); max_splits workgroups at most.
__host__ __device__ inline StepSplit step_split(uint32_t len, uint32_t max_splits) {
    const uint32_t tiles = (len + 63u) / 64u, per = (tiles + max_splits - 1u) / max_splits;
    return {(tiles + per - 1u) / per, per * 64u};
}
static uint32_t step_max_splits(const decdec_latent& p) {
    const uint32_t groups = (p.heads + 15u) / 16u, want = 256u / groups, tiles = (p.max_seq + 63u) / 64u;
    const uint32_t n = want < 8u ? 8u : (want > 128u ? 128u : want);
    return n < tiles ? n : tiles;
}

// grid (splits, heads / 16), sixteen waves.  Scores transposed (keys x heads) as above: the 16-key blocks of the tile times
// shares of the contraction make sixteen wave tasks, summed through LDS; a wave then takes one head's softmax, a lane per
// key; the tile stays in LDS for the weighted sum over its keys, whose rows (latent components) are divided among the
// waves.  The next tile is requested into registers while the present one is worked on.
constexpr uint32_t kStepThreads = 1024;

template <int DT, int KT, int NR>
__global__ __launch_bounds__(kStepThreads) void latent_step_kernel(const decdec_latent p, const float* __restrict__ qa,
                                                                   float* __restrict__ parts, const uint32_t max_splits) {
    using T = typename LaneOf<DT>::t;
    constexpr uint32_t KB = KT / 16, SP = 16u / KB, NL = (KT * 80u + kStepThreads - 1u) / kStepThreads;   // rows of at most 640
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, QN = DT == kFP32 ? 1u : 2u;
    extern __shared__ __align__(16) unsigned char smem[];
    const uint32_t R = p.rank, W = R + p.rot, Wp = (W + 31u) & ~31u, KL = Wp + PAD, W8 = Wp / 8u;
    T* Kl = (T*)smem;                                    // [KT][KL]
    T* Ql = Kl + KT * KL;                                // [QN][16][KL]: leading and trailing parts
    __shared__ float Pl[SP][KT][17];
    __shared__ float mxs[16], sums[16], corrs[16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t h0 = blockIdx.y * 16u;
    const long long pos = *p.pos;
    if (pos < 0) return;
    const uint32_t len = pos + 1 < (long long)p.max_seq ? (uint32_t)pos + 1u : p.max_seq;
    const StepSplit sp = step_split(len, max_splits);
    if (blockIdx.x >= sp.splits) return;
    const uint32_t lo_key = blockIdx.x * sp.span, hi_key = lo_key + sp.span < len ? lo_key + sp.span : len;
    const bool vec = R % 8u == 0 && p.rot % 8u == 0;
    Frag<DT> kr[NL];
    // rows past the end repeat the last one; their weights are zero
    auto request = [&](uint32_t k0) {
#pragma unroll
        for (uint32_t j = 0; j < NL; ++j) {
            const uint32_t i = tid + kStepThreads * j, r = i / W8, c = (i - r * W8) * 8u, key = k0 + r < hi_key ? k0 + r : hi_key - 1u;
            const T* row = (const T*)p.cache + (size_t)key * W;
            if (vec) {
                kr[j] = frag_load(row + (c < W ? c : 0u));
                if (c >= W) kr[j] = Frag<DT>{};
            } else {
                kr[j] = load8<DT>(row + c, (int)W - (int)c, false);
            }
        }
    };
    request(lo_key);
    for (uint32_t i = tid; i < 16u * W8; i += kStepThreads) {
        const uint32_t r = i / W8, c = (i - r * W8) * 8u;
        float x[8];
#pragma unroll
        for (uint32_t e = 0; e < 8u; ++e) x[e] = 0.f;
        if (h0 + r < p.heads) {
            const float* src = qa + (size_t)(h0 + r) * W + c;
            if (vec && c + 8u <= W) {
                const f32x4 a = *(const f32x4*)src, b = *(const f32x4*)(src + 4);
#pragma unroll
                for (int e = 0; e < 4; ++e) { x[e] = a[e]; x[4 + e] = b[e]; }
            } else {
#pragma unroll
                for (uint32_t e = 0; e < 8u; ++e) x[e] = c + e < W ? src[e] : 0.f;
            }
        }
        Frag<DT> hi, lo;
        frag_split(x, hi, lo);
        store8(Ql + r * KL + c, hi);
        if constexpr (QN == 2u) store8(Ql + (16u + r) * KL + c, lo);
    }
    if (tid < 16u) { mxs[tid] = -__builtin_inff(); sums[tid] = 0.f; }
    f32x4 o[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (uint32_t k0 = lo_key; k0 < hi_key; k0 += KT) {
        __syncthreads();
#pragma unroll
        for (uint32_t j = 0; j < NL; ++j) {
            const uint32_t i = tid + kStepThreads * j, r = i / W8;
            if (r < (uint32_t)KT) store8(Kl + r * KL + (i - r * W8) * 8u, kr[j]);
        }
        __syncthreads();
        if (k0 + KT < hi_key) request(k0 + KT);
        {
            f32x4 sc = {0.f, 0.f, 0.f, 0.f};
            const uint32_t kb = wave % KB, part = wave / KB, slices = Wp / 32u;
            for (uint32_t s = part; s < slices; s += SP) {
                const Frag<DT> a = frag_load(Kl + (16u * kb + l16) * KL + 32u * s + 8u * lg);
#pragma unroll
                for (uint32_t n = 0; n < QN; ++n) mma(a, frag_load(Ql + (16u * n + l16) * KL + 32u * s + 8u * lg), sc);
            }
#pragma unroll
            for (int v = 0; v < 4; ++v) Pl[part][16u * kb + 4u * lg + v][l16] = sc[v];
        }
        __syncthreads();
        {
            float x = 0.f;
            const bool in = lane < (uint32_t)KT && k0 + lane < hi_key;
            if (in)
#pragma unroll
                for (uint32_t n = 0; n < SP; ++n) x += Pl[n][lane][wave];
            const float m0 = mxs[wave];
            float best = in ? fmaxf(x, m0) : m0;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) best = fmaxf(best, __shfl_xor(best, off, 64));
            const float w = in ? __expf(x - best) : 0.f;                   // the tile has at least one key: best is finite
            if (lane < (uint32_t)KT) Pl[0][lane][wave] = w;                // only this wave reads or writes the head's column
            const float t = wave_sum(w);
            if (lane == 0u) {
                const float corr = __expf(m0 - best);
                corrs[wave] = corr;
                sums[wave] = sums[wave] * corr + t;
                mxs[wave] = best;
            }
        }
        __syncthreads();
        const float corr = corrs[l16];
        Frag<DT> hi[KT / 32], lo[KT / 32];
#pragma unroll
        for (uint32_t j = 0; j < KT / 32; ++j) {
            float w[8];
#pragma unroll
            for (uint32_t e = 0; e < 8u; ++e) w[e] = Pl[0][32u * j + 8u * lg + e][l16];
            frag_split(w, hi[j], lo[j]);
        }
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const uint32_t tile = wave + 16u * (uint32_t)i;
            if (16u * tile < R) {
                o[i] *= corr;
#pragma unroll
                for (uint32_t j = 0; j < KT / 32; ++j) {
                    const Frag<DT> a = frag_gather(Kl + (32u * j + 8u * lg) * KL + 16u * tile + l16, KL);
                    mma(a, hi[j], o[i]);
                    if constexpr (QN == 2u) mma(a, lo[j], o[i]);
                }
            }
        }
    }
    // partial result of a head: [rank] sums, maximum, sum of weights
    if (h0 + l16 < p.heads) {
        float* dst = parts + ((size_t)blockIdx.x * p.heads + h0 + l16) * (R + 2u);
#pragma unroll
        for (int i = 0; i < NR; ++i)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const uint32_t r = 16u * (wave + 16u * (uint32_t)i) + 4u * lg + (uint32_t)v;
                if (r < R) dst[r] = o[i][v];
            }
        if (wave == 0u && lg == 0u) { dst[R] = mxs[l16]; dst[R + 1u] = sums[l16]; }
    }
}

// Merge of the splits and the values: grid (heads, vdim / 32), sixteen waves of two value rows each.  The value matrix'
// rows are requested first; they wait for nothing.
template <int DT>
__global__ __launch_bounds__(1024) void latent_merge_kernel(const decdec_latent p, const float* __restrict__ parts,
                                                            void* __restrict__ out, const uint32_t max_splits) {
    using E = Elem<DT>;
    using T = typename LaneOf<DT>::t;
    __shared__ float lat[1024], share[1024], ws[128];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, h = blockIdx.x, R = p.rank, V = p.vdim;
    const long long pos = *p.pos;
    if (pos < 0) return;
    const uint32_t len = pos + 1 < (long long)p.max_seq ? (uint32_t)pos + 1u : p.max_seq;
    const uint32_t n = step_split(len, max_splits).splits;               // at most 128
    const float* ph = parts + (size_t)h * (R + 2u);
    const size_t ps = (size_t)p.heads * (R + 2u);
    const bool vec = R % 8u == 0;
    Frag<DT> uv[2][2];
#pragma unroll
    for (uint32_t i = 0; i < 2u; ++i)
#pragma unroll
        for (uint32_t j = 0; j < 2u; ++j) {
            const uint32_t d = blockIdx.y * 32u + wave * 2u + i, c = lane * 8u + 512u * j;
            uv[i][j] = load8<DT>((const T*)p.uv + ((size_t)h * V + (d < V ? d : 0u)) * R + (c < R ? c : 0u), d < V ? (int)R - (int)c : 0, vec);
        }
    // the splits are summed in `groups` shares of the workgroup, Rp threads each
    const uint32_t Rp = (R + 63u) & ~63u, groups = 1024u / Rp, g = tid / Rp, r = tid - g * Rp;
    const bool mine = g < groups && r < R;
    if (wave == 0u) {
        const float sink = p.sink != nullptr ? E::load(p.sink, h) : -__builtin_inff();
        float m[2], l[2], M = sink;
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) {
            const uint32_t i = lane + 64u * e;
            m[e] = i < n ? ph[i * ps + R] : -__builtin_inff();
            l[e] = i < n ? ph[i * ps + R + 1u] : 0.f;
            M = fmaxf(M, m[e]);
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) M = fmaxf(M, __shfl_xor(M, off, 64));
#pragma unroll
        for (int e = 0; e < 2; ++e) m[e] = __expf(m[e] - M);               // exp(-inf) = 0 past the last split
        const float L = wave_sum(m[0] * l[0] + m[1] * l[1]) + (p.sink != nullptr ? __expf(sink - M) : 0.f);
        ws[lane] = m[0] / L;
        ws[lane + 64u] = m[1] / L;
    }
    __syncthreads();
    float t = 0.f;
    if (mine) {
        for (uint32_t s = g; s < n; s += 8u * groups) {
            float x[8];
#pragma unroll
            for (uint32_t e = 0; e < 8u; ++e) x[e] = s + e * groups < n ? ph[(s + e * groups) * ps + r] : 0.f;
#pragma unroll
            for (uint32_t e = 0; e < 8u; ++e) t = __builtin_fmaf(s + e * groups < n ? ws[s + e * groups] : 0.f, x[e], t);
        }
    }
    share[tid] = t;
    __syncthreads();
    {
        float a = 0.f;
        if (tid < R)
            for (uint32_t k = 0; k < groups; ++k) a += share[k * Rp + tid];
        lat[tid] = a;                                                      // zero past the rank
    }
    __syncthreads();
#pragma unroll
    for (uint32_t i = 0; i < 2u; ++i) {
        const uint32_t d = blockIdx.y * 32u + wave * 2u + i;
        float acc = 0.f;
#pragma unroll
        for (uint32_t j = 0; j < 2u; ++j) {
            float w[8];
            frag_values(uv[i][j], w);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = __builtin_fmaf(w[e], lat[lane * 8u + 512u * j + e], acc);
        }
        acc = wave_sum(acc);
        if (lane == 0u && d < V) E::store(out, (size_t)h * V + d, acc);
    }
}

size_t latent_step_workspace(const decdec_latent& p) {
    return ((size_t)p.heads * (p.rank + p.rot) + (size_t)step_max_splits(p) * p.heads * (p.rank + 2u)) * sizeof(float);
}

template <int DT, int KT, int NR>
static hipError_t step_launch(const decdec_latent& p, const float* qa, float* parts, dim3 grid, size_t lds, uint32_t splits, hipStream_t s) {
    if (hipError_t e = allow_lds<latent_step_kernel<DT, KT, NR>>(lds); e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_step_kernel<DT, KT, NR>), grid, dim3(kStepThreads), lds, s, p, qa, parts, splits);
    return hipGetLastError();
}

template <int DT, int KT>
static hipError_t step_dt(const decdec_latent& p, void* out, float* qa, float* parts, hipStream_t s) {
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, QN = DT == kFP32 ? 1u : 2u;
    const uint32_t splits = step_max_splits(p), Wp = (p.rank + p.rot + 31u) & ~31u, tiles = ((p.rank + 15u) / 16u + 15u) / 16u;
    const size_t lds = (size_t)(KT + QN * 16u) * (Wp + PAD) * Elem<DT>::bytes;
    if (lds > 140u * 1024u) return hipErrorInvalidValue;
    const dim3 grid(splits, (p.heads + 15u) / 16u), block(256);
    hipLaunchKernelGGL((latent_absorb_kernel<DT>), dim3(p.heads + 1u, (p.rank + 63u) / 64u), block, 0, s, p, qa);
    hipError_t e = tiles <= 1u ? step_launch<DT, KT, 1>(p, qa, parts, grid, lds, splits, s)
                 : tiles <= 3u ? step_launch<DT, KT, 3>(p, qa, parts, grid, lds, splits, s) : hipErrorInvalidValue;
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_merge_kernel<DT>), dim3(p.heads, (p.vdim + 31u) / 32u), dim3(1024), 0, s, p, parts, out, splits);
    return hipGetLastError();
}

hipError_t launch_latent_step(int dt, const decdec_latent& p, void* out, void* ws, hipStream_t s) {
    float* qa = (float*)ws;
    float* parts = qa + (size_t)p.heads * (p.rank + p.rot);
    if (dt == kBF16) return step_dt<kBF16, 64>(p, out, qa, parts, s);
    return step_dt<kFP32, 32>(p, out, qa, parts, s);
}

}  // namespace decdec
