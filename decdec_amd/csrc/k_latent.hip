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
// grid (query blocks, heads), four waves of 16 MT queries.  The transposed scores (keys x queries) leave a query in one
// lane column: its running maximum and sum are lane values, its weights are at once the right operand of the value
// product (out^T = V^T P^T), and nothing passes through LDS but the key and value tiles.  The contraction of that product
// visits keys 4 (lane / 16) + e of one 16-key tile, then of the next, in both operands.
constexpr uint32_t kKeys = 64;

template <int DT, int MT, int NK, int NV>
__global__ __launch_bounds__(256) void latent_attention_kernel(const decdec_latent p, const void* __restrict__ q_in,
                                                               const void* __restrict__ k_in, const void* __restrict__ vt_in,
                                                               const uint32_t vt_ld, void* __restrict__ out,
                                                               const uint32_t start, const uint32_t rows, const uint32_t keys_total) {
    using T = typename LaneOf<DT>::t;
    using E = Elem<DT>;
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, KL = 32u * NK + PAD, VL = kKeys + PAD;
    extern __shared__ __align__(16) unsigned char smem[];
    T* Kl = (T*)smem;                       // [kKeys][KL]
    T* Vl = Kl + kKeys * KL;                // [16 NV][VL]
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, Dq = p.dim + p.rot, D = p.dim, V = p.vdim;
    const uint32_t q0 = (gridDim.x - 1u - blockIdx.x) * (64u * MT);        // longest rows first
    const bool vec = D % 8u == 0 && p.rot % 8u == 0 && p.rank % 8u == 0 && (p.heads * D) % 8u == 0;
    const T* q = (const T*)q_in;
    Frag<DT> qf[MT][NK];
    uint32_t qpos[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const uint32_t r = q0 + 16u * (MT * wave + (uint32_t)m) + l16, rc = r < rows ? r : rows - 1u;
        qpos[m] = start + rc;
#pragma unroll
        for (int s = 0; s < NK; ++s)
            qf[m][s] = load8<DT>(q + ((size_t)rc * p.heads + h) * Dq + 32u * s + 8u * lg, (int)Dq - (int)(32u * s + 8u * lg), vec);
    }
    const float sink = p.sink != nullptr ? E::load(p.sink, h) : -__builtin_inff();
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
    const uint32_t kend = start + last;
    const T* kb = (const T*)k_in + (size_t)h * D;
    const T* cb = (const T*)p.cache + p.rank;
    const T* vb = (const T*)vt_in + (size_t)h * V * vt_ld;
    for (uint32_t k0 = 0; k0 < kend; k0 += kKeys) {
        __syncthreads();
        for (uint32_t i = tid; i < kKeys * 4u * NK; i += 256u) {
            const uint32_t r = i / (4u * NK), c = (i % (4u * NK)) * 8u, key = k0 + r;
            const bool in = key < keys_total;
            const T* rot = cb + (size_t)key * (p.rank + p.rot);
            Frag<DT> f;
            if (!in) f = load8<DT>(kb, 0, false);
            else if (vec) f = c < D ? load8<DT>(kb + (size_t)key * p.heads * D + c, 8, true) : load8<DT>(rot + (c - D), (int)Dq - (int)c, true);
            else if (c >= D) f = load8<DT>(rot + (c - D), (int)Dq - (int)c, false);
            else if (c + 8u <= D) f = load8<DT>(kb + (size_t)key * p.heads * D + c, 8, false);
            else {                                                         // the unrotated part ends inside
                T t[8];
#pragma unroll
                for (uint32_t e = 0; e < 8u; ++e)
                    t[e] = c + e < D ? kb[(size_t)key * p.heads * D + c + e] : (c + e < Dq ? rot[c + e - D] : (T)0);
                f = load8<DT>(t, 8, false);
            }
            store8(Kl + r * KL + c, f);
        }
        for (uint32_t i = tid; i < 16u * NV * (kKeys / 8u); i += 256u) {
            const uint32_t d = i / (kKeys / 8u), c = (i % (kKeys / 8u)) * 8u;
            store8(Vl + d * VL + c, load8<DT>(vb + (size_t)(d < V ? d : 0u) * vt_ld + k0 + c, d < V ? 8 : 0, true));
        }
        __syncthreads();
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
        const bool edge = k0 + kKeys > start + q0 + 16u * MT * wave + 1u;  // some key may lie after some query of the wave
        Frag<DT> hi[MT][2], lo[MT][2];
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            float best = mx[m];
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    float x = sc[m][t][v] * p.scale;
                    if (edge && k0 + 16u * t + 4u * lg + (uint32_t)v > qpos[m]) x = -__builtin_inff();
                    sc[m][t][v] = x;
                    best = fmaxf(best, x);
                }
            best = fmaxf(best, __shfl_xor(best, 16, 64));
            best = fmaxf(best, __shfl_xor(best, 32, 64));
            const float corr = __expf(mx[m] - best);                       // the first key is visible to every query: best is finite
            mx[m] = best;
            sum[m] *= corr;
#pragma unroll
            for (int n = 0; n < NV; ++n) o[m][n] *= corr;
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                float w[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    w[e] = __expf(sc[m][2 * t + (e >> 2)][e & 3] - best);
                    sum[m] += w[e];
                }
                frag_split(w, hi[m][t], lo[m][t]);
            }
        }
#pragma unroll
        for (int n = 0; n < NV; ++n)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const T* vr = Vl + (16u * n + l16) * VL + 32u * t + 4u * lg;
                Frag<DT> a;
                if constexpr (DT == kFP32) {
                    const f32x4 x = *(const f32x4*)vr, y = *(const f32x4*)(vr + 16);
#pragma unroll
                    for (int e = 0; e < 4; ++e) { a.v[e] = x[e]; a.v[4 + e] = y[e]; }
                } else {
                    const u32x2 x = *(const u32x2*)vr, y = *(const u32x2*)(vr + 16);
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

template <int DT, int MT, int NK, int NV>
static hipError_t attention_launch(const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld, void* out,
                                   uint32_t start, uint32_t rows, hipStream_t s) {
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u;
    constexpr size_t lds = (size_t)(kKeys * (32u * NK + PAD) + 16u * NV * (kKeys + PAD)) * Elem<DT>::bytes;
    static_assert(lds <= 160u * 1024u, "tiles must fit the LDS of a compute unit");
    if (hipError_t e = allow_lds<latent_attention_kernel<DT, MT, NK, NV>>(lds); e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_attention_kernel<DT, MT, NK, NV>), dim3((rows + 64u * MT - 1u) / (64u * MT), p.heads), dim3(256), lds, s,
                       p, q, k, vt, vt_ld, out, start, rows, start + rows);
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
    const uint32_t groups = (p.heads + 15u) / 16u, want = 128u / groups, tiles = (p.max_seq + 63u) / 64u;
    const uint32_t n = want < 8u ? 8u : (want > 64u ? 64u : want);
    return n < tiles ? n : tiles;
}

// grid (splits, heads / 16), four waves.  Scores transposed (keys x heads) as above, each wave 16 keys of the tile (and,
// where the tile has fewer than four 16-key blocks, a share of the contraction); the tile stays in LDS for the weighted
// sum over its keys, whose rows (latent components) are divided among the waves.
template <int DT, int KT, int NR>
__global__ __launch_bounds__(256) void latent_step_kernel(const decdec_latent p, const float* __restrict__ qa, float* __restrict__ parts,
                                                          const uint32_t max_splits) {
    using T = typename LaneOf<DT>::t;
    constexpr uint32_t KB = KT / 16, SP = 4u / KB;
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, QN = DT == kFP32 ? 1u : 2u;
    extern __shared__ __align__(16) unsigned char smem[];
    const uint32_t R = p.rank, W = R + p.rot, Wp = (W + 31u) & ~31u, KL = Wp + PAD;
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
    for (uint32_t i = tid; i < 16u * (Wp / 8u); i += 256u) {
        const uint32_t r = i / (Wp / 8u), c = (i % (Wp / 8u)) * 8u;
        float x[8];
#pragma unroll
        for (uint32_t e = 0; e < 8u; ++e) x[e] = (h0 + r < p.heads && c + e < W) ? qa[(size_t)(h0 + r) * W + c + e] : 0.f;
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
        for (uint32_t i = tid; i < KT * (Wp / 8u); i += 256u) {
            const uint32_t r = i / (Wp / 8u), c = (i % (Wp / 8u)) * 8u, key = k0 + r;
            const T* src = (const T*)p.cache + (size_t)key * W + c;
            store8(Kl + r * KL + c, load8<DT>(key < hi_key ? src : (const T*)p.cache, key < hi_key ? (int)W - (int)c : 0, vec));
        }
        __syncthreads();
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
            // 16 threads per head
            const uint32_t hd = tid >> 4, t = tid & 15u;
            float x[KB], best = mxs[hd];
            const float m0 = best;
#pragma unroll
            for (uint32_t j = 0; j < KB; ++j) {
                const uint32_t key = t + 16u * j;
                x[j] = 0.f;
#pragma unroll
                for (uint32_t n = 0; n < SP; ++n) x[j] += Pl[n][key][hd];
                if (k0 + key >= hi_key) x[j] = -__builtin_inff();
                best = fmaxf(best, x[j]);
            }
#pragma unroll
            for (int off = 1; off < 16; off <<= 1) best = fmaxf(best, __shfl_xor(best, off, 64));
            float sum = 0.f;
#pragma unroll
            for (uint32_t j = 0; j < KB; ++j) {
                x[j] = __expf(x[j] - best);                                // the tile has at least one key: best is finite
                sum += x[j];
                Pl[0][t + 16u * j][hd] = x[j];
            }
#pragma unroll
            for (int off = 1; off < 16; off <<= 1) sum += __shfl_xor(sum, off, 64);
            if (t == 0u) {
                const float corr = __expf(m0 - best);
                corrs[hd] = corr;
                sums[hd] = sums[hd] * corr + sum;
                mxs[hd] = best;
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
            const uint32_t tile = wave + 4u * (uint32_t)i;
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
                const uint32_t r = 16u * (wave + 4u * (uint32_t)i) + 4u * lg + (uint32_t)v;
                if (r < R) dst[r] = o[i][v];
            }
        if (wave == 0u && lg == 0u) { dst[R] = mxs[l16]; dst[R + 1u] = sums[l16]; }
    }
}

// Merge of the splits and the values: grid (heads, vdim / 32).
template <int DT>
__global__ __launch_bounds__(256) void latent_merge_kernel(const decdec_latent p, const float* __restrict__ parts,
                                                           void* __restrict__ out, const uint32_t max_splits) {
    using E = Elem<DT>;
    using T = typename LaneOf<DT>::t;
    extern __shared__ __align__(16) unsigned char smem[];
    float* lat = (float*)smem;                           // [rank rounded up to 8]
    __shared__ float ws[64];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, h = blockIdx.x, R = p.rank, V = p.vdim;
    const long long pos = *p.pos;
    if (pos < 0) return;
    const uint32_t len = pos + 1 < (long long)p.max_seq ? (uint32_t)pos + 1u : p.max_seq;
    const uint32_t n = step_split(len, max_splits).splits;               // at most 64
    const float* ph = parts + (size_t)h * (R + 2u);
    const size_t ps = (size_t)p.heads * (R + 2u);
    if (wave == 0u) {
        const float sink = p.sink != nullptr ? E::load(p.sink, h) : -__builtin_inff();
        const float m = lane < n ? ph[lane * ps + R] : -__builtin_inff();
        float M = fmaxf(m, sink);
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) M = fmaxf(M, __shfl_xor(M, off, 64));
        const float w = lane < n ? __expf(m - M) : 0.f;
        const float L = wave_sum(lane < n ? w * ph[lane * ps + R + 1u] : 0.f) + (p.sink != nullptr ? __expf(sink - M) : 0.f);
        ws[lane] = w / L;
    }
    __syncthreads();
    for (uint32_t r = tid; r < ((R + 7u) & ~7u); r += 256u) {
        float t = 0.f;
        if (r < R)
            for (uint32_t s = 0; s < n; ++s) t = __builtin_fmaf(ws[s], ph[s * ps + r], t);
        lat[r] = t;
    }
    __syncthreads();
    const bool vec = R % 8u == 0;
    for (uint32_t i = 0; i < 8u; ++i) {
        const uint32_t d = blockIdx.y * 32u + wave * 8u + i;
        if (d >= V) break;                                                 // uniform over the wave
        const T* uv = (const T*)p.uv + ((size_t)h * V + d) * R;
        float acc = 0.f;
        for (uint32_t c = lane * 8u; c < R; c += 512u) {
            float w[8];
            frag_values(load8<DT>(uv + c, (int)R - (int)c, vec), w);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = __builtin_fmaf(w[e], lat[c + e], acc);
        }
        acc = wave_sum(acc);
        if (lane == 0u) E::store(out, (size_t)h * V + d, acc);
    }
}

size_t latent_step_workspace(const decdec_latent& p) {
    return ((size_t)p.heads * (p.rank + p.rot) + (size_t)step_max_splits(p) * p.heads * (p.rank + 2u)) * sizeof(float);
}

template <int DT, int KT, int NR>
static hipError_t step_launch(const decdec_latent& p, const float* qa, float* parts, dim3 grid, size_t lds, uint32_t splits, hipStream_t s) {
    if (hipError_t e = allow_lds<latent_step_kernel<DT, KT, NR>>(lds); e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_step_kernel<DT, KT, NR>), grid, dim3(256), lds, s, p, qa, parts, splits);
    return hipGetLastError();
}

template <int DT, int KT>
static hipError_t step_dt(const decdec_latent& p, void* out, float* qa, float* parts, hipStream_t s) {
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, QN = DT == kFP32 ? 1u : 2u;
    const uint32_t splits = step_max_splits(p), Wp = (p.rank + p.rot + 31u) & ~31u, tiles = ((p.rank + 15u) / 16u + 3u) / 4u;
    const size_t lds = (size_t)(KT + QN * 16u) * (Wp + PAD) * Elem<DT>::bytes;
    if (lds > 140u * 1024u) return hipErrorInvalidValue;
    const dim3 grid(splits, (p.heads + 15u) / 16u), block(256);
    hipLaunchKernelGGL((latent_absorb_kernel<DT>), dim3(p.heads + 1u, (p.rank + 63u) / 64u), block, 0, s, p, qa);
    hipError_t e = tiles <= 2u ? step_launch<DT, KT, 2>(p, qa, parts, grid, lds, splits, s)
                 : tiles <= 8u ? step_launch<DT, KT, 8>(p, qa, parts, grid, lds, splits, s)
                 : tiles <= 16u ? step_launch<DT, KT, 16>(p, qa, parts, grid, lds, splits, s) : hipErrorInvalidValue;
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_merge_kernel<DT>), dim3(p.heads, (p.vdim + 31u) / 32u), block, ((size_t)p.rank + 8u) * 4u, s, p, parts, out, splits);
    return hipGetLastError();
}

hipError_t launch_latent_step(int dt, const decdec_latent& p, void* out, void* ws, hipStream_t s) {
    float* qa = (float*)ws;
    float* parts = qa + (size_t)p.heads * (p.rank + p.rot);
    if (dt == kBF16) return step_dt<kBF16, 64>(p, out, qa, parts, s);
    return step_dt<kFP32, 32>(p, out, qa, parts, s);
}

}  // namespace decdec
