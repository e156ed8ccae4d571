// Latent attention: the keys and values of all heads are linear in one normed latent per token, which is what the cache
// holds, next to a rotated key part that the heads share.
//
// Many tokens: keys and values of the whole past are formed by two matrix products outside and attended by a tiled
// kernel (k_attention.hip).  One token: the up projections are absorbed -- a query is carried into the latent space (absorb kernel), all
// heads attend the same cache rows (step kernel, sequence split over workgroups), and the attended latents are carried
// to the values (merge kernel).  Scores, weights and sums are fp32; on bf16 storage a weight enters the value product as
// the sum of two bf16 numbers.
#include "mixers.h"
#include "mma.h"

namespace decdec {

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
hipError_t launch_latent_attention(int dt, const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld,
                                   void* out, uint32_t start, uint32_t rows, hipStream_t s) {
    TileAttention a{};
    a.q = q; a.k = k; a.vt = vt; a.out = out; a.sink = p.sink;
    a.shared = (const char*)p.cache + (size_t)p.rank * (dt == kBF16 ? 2u : 4u);
    a.k_head = p.dim; a.k_row = (size_t)p.heads * p.dim;
    a.shared_row = p.rank + p.rot; a.vt_ld = vt_ld; a.out_ld = p.heads * p.vdim;
    a.heads = p.heads; a.share = 1; a.dim = p.dim; a.rot = p.rot; a.vdim = p.vdim;
    a.scale = p.scale; a.sink_score = -__builtin_inff(); a.out_scale = 1.f;
    return launch_tile_attention(dt, a, start, rows, s);
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
