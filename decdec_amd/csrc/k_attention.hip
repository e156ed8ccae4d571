// Causal softmax attention over cached keys and values, with an optional valueless score (sink) in the denominator and an
// optional gate per head on the read-out.
//
// Many tokens: one tiled kernel for keys of a head's own, or of a head's own part and a part that all heads share (latent
// attention).  Grouped attention: normed, partly rotated queries and keys; the cache holds the keys by head and the values
// transposed, which is how the products read them; one token takes two launches (shares of the sequence, then their merge).
// Scores, weights and sums are fp32; on bf16 storage a weight enters the value product as the sum of two bf16 numbers.
#include "mixers.h"
#include "mma.h"

namespace decdec {

// ---- many tokens ------------------------------------------------------------------------------------------
// Workgroups of four waves with 16 MT queries each, one per query block and head; neighbouring heads go to one die, so that
// the tiles of a head's keys and values (and of heads that share them) stay in one L2.  The transposed scores (keys x
// queries) leave a query in one lane column: its running maximum and sum are lane values, its weights are at once the right
// operand of the value product (out^T = V^T P^T), and nothing passes through LDS but the key and value tiles.  The
// contraction of that product visits keys 4 (lane / 16) + e of one 16-key tile, then of the next, in both operands.  The
// next tile is requested into registers while the present one is worked on.  Scores are kept in units of log 2.
constexpr uint32_t kKeys = 64;

template <int DT, int MT, int NK, int NV, bool VEC>
__global__ __launch_bounds__(256, DT == kFP32 ? 1 : 2) void tile_attention_kernel(const TileAttention p, const uint32_t start,
                                                                             const uint32_t rows, const uint32_t blocks) {
    using T = typename LaneOf<DT>::t;
    using E = Elem<DT>;
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, KL = 32u * NK + PAD, VL = kKeys + PAD;
    extern __shared__ __align__(16) unsigned char smem[];
    T* Kl = (T*)smem;                       // [kKeys][KL]
    T* Vl = Kl + kKeys * KL;                // [16 NV][VL]
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t turn = blockIdx.x >> 3, h = (blockIdx.x & 7u) * ((p.heads + 7u) / 8u) + turn / blocks;
    if (h >= p.heads) return;
    const uint32_t kvh = h / p.share;
    const uint32_t q0 = (blocks - 1u - turn % blocks) * (64u * MT);        // longest rows first
    const uint32_t Dq = p.dim + p.rot, D = p.dim, V = p.vdim, keys_total = start + rows;
    const T* q = (const T*)p.q;
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
    const float sink = (p.sink != nullptr ? E::load(p.sink, h) : p.sink_score) * kLog2e;      // minus infinity: none
    float mx[MT], sum[MT];
    f32x4 o[MT][NV];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        mx[m] = sink;
        sum[m] = (sink > -__builtin_inff() && lg == 0u) ? 1.f : 0.f;   // lane groups hold partial sums
#pragma unroll
        for (int n = 0; n < NV; ++n) o[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const uint32_t last = q0 + 64u * MT < rows ? q0 + 64u * MT : rows;     // one past the block's last query
    const uint32_t kend = start + last, wave_first = start + q0 + 16u * MT * wave, wave_last = wave_first + 16u * MT - 1u;
    const size_t kld = p.k_row, cld = p.shared_row, vt_ld = p.vt_ld;
    const T* kb = (const T*)p.k + kvh * p.k_head;
    const T* cb = (const T*)(p.shared != nullptr ? p.shared : p.k);
    const T* vb = (const T*)p.vt + (size_t)kvh * V * vt_ld;
    // A key row is [part of the head's own | part that the heads share]; keys past the end repeat the last one and are never
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
        for (int j = 0; j < NV / 2; ++j) vr[j] = frag_load(vp + (vrow + 32u * j < V ? vrow + 32u * j : 0u) * vt_ld);
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
                Vl[d * VL + c] = d < V ? vb[d * vt_ld + k0 + c] : (T)0;
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
        const uint32_t row = q0 + 16u * (MT * wave + (uint32_t)m) + l16;
        if (row < rows) {
            float r = p.out_scale / t;
            if (p.gate != nullptr) r *= sigmoid_f(E::load(p.gate, (size_t)row * p.gate_ld + h));
#pragma unroll
            for (int n = 0; n < NV; ++n)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const uint32_t d = 16u * n + 4u * lg + (uint32_t)v;
                    if (d < V) E::store(p.out, (size_t)row * p.out_ld + h * V + d, o[m][n][v] * r);
                }
        }
    }
}

template <int DT, int MT, int NK, int NV, bool VEC = true>
static hipError_t tile_launch(const TileAttention& p, uint32_t start, uint32_t rows, hipStream_t s) {
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u;
    constexpr size_t lds = (size_t)(kKeys * (32u * NK + PAD) + 16u * NV * (kKeys + PAD)) * Elem<DT>::bytes;
    static_assert(lds <= 160u * 1024u, "tiles must fit the LDS of a compute unit");
    if (hipError_t e = allow_lds<tile_attention_kernel<DT, MT, NK, NV, VEC>>(lds); e != hipSuccess) return e;
    const uint32_t blocks = (rows + 64u * MT - 1u) / (64u * MT);
    hipLaunchKernelGGL((tile_attention_kernel<DT, MT, NK, NV, VEC>), dim3(blocks * ((p.heads + 7u) / 8u * 8u)), dim3(256), lds, s,
                       p, start, rows, blocks);
    return hipGetLastError();
}

template <int DT, int MT, int NK>
static hipError_t tile_nv(const TileAttention& p, uint32_t start, uint32_t rows, hipStream_t s) {
    if (p.vdim <= 64u) return tile_launch<DT, MT, NK, 4>(p, start, rows, s);
    if (p.vdim <= 128u) return tile_launch<DT, MT, NK, 8>(p, start, rows, s);
    return tile_launch<DT, 1, NK, 16>(p, start, rows, s);
}

template <int DT, int MT>
static hipError_t tile_dt(const TileAttention& p, uint32_t start, uint32_t rows, hipStream_t s) {
    const uint32_t Dq = p.dim + p.rot;
    if (((p.dim | p.rot) % 8u | (p.k_row | p.k_head | p.shared_row | (uintptr_t)p.shared / Elem<DT>::bytes) % 8u) != 0)
        return tile_launch<DT, 1, 10, 16, false>(p, start, rows, s);
    if (Dq <= 128u) return tile_nv<DT, MT, 4>(p, start, rows, s);
    if (Dq <= 192u) return tile_nv<DT, MT, 6>(p, start, rows, s);
    return tile_nv<DT, 1, 10>(p, start, rows, s);
}

hipError_t launch_tile_attention(int dt, const TileAttention& p, uint32_t start, uint32_t rows, hipStream_t s) {
    if (p.dim + p.rot > 320u || p.vdim > 256u) return hipErrorInvalidValue;
    return dt == kBF16 ? tile_dt<kBF16, 2>(p, start, rows, s) : tile_dt<kFP32, 1>(p, start, rows, s);
}


// ---- grouped attention: queries, keys and values of new tokens ----------------------------------------------
// One head of one token by a wave: RMS norm over dim (weight may be null), then the pairs (2i, 2i + 1) of the first `rot`
// elements turned.  A lane takes elements 2 lane + 128 j and the next; dim is at most 320.
constexpr int kPairs = 3;

struct HeadRow { float x[kPairs][2], w[kPairs][2], c[kPairs], s[kPairs]; };
template <int DT>
__device__ __forceinline__ HeadRow head_fetch(const void* proj, size_t at, const void* weight, const decdec_grouped& p, size_t trow) {
    using E = Elem<DT>;
    const uint32_t lane = threadIdx.x & 63u, D = p.dim;
    HeadRow f;
#pragma unroll
    for (int j = 0; j < kPairs; ++j) {
        const uint32_t i0 = 2u * lane + 128u * (uint32_t)j;
        const bool turn = i0 < p.rot;
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) {
            const bool in = i0 + e < D;
            f.x[j][e] = in ? E::load(proj, at + i0 + e) : 0.f;
            f.w[j][e] = (weight != nullptr && in) ? E::load(weight, i0 + e) : 1.f;
        }
        f.c[j] = turn ? p.cos_table[trow + i0 / 2u] : 1.f;
        f.s[j] = turn ? p.sin_table[trow + i0 / 2u] : 0.f;
    }
    return f;
}
__device__ __forceinline__ void norm_rotate(const HeadRow& f, bool norm, const decdec_grouped& p, float (&x)[kPairs][2]) {
    float r = 1.f;
    if (norm) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < kPairs; ++j) ss += f.x[j][0] * f.x[j][0] + f.x[j][1] * f.x[j][1];
        r = 1.f / sqrtf(wave_sum(ss) / (float)p.dim + p.eps);
    }
#pragma unroll
    for (int j = 0; j < kPairs; ++j) {
        const float u = f.x[j][0] * r * f.w[j][0], v = f.x[j][1] * r * f.w[j][1];
        x[j][0] = u * f.c[j] - v * f.s[j];
        x[j][1] = v * f.c[j] + u * f.s[j];
    }
}

template <int DT>
__device__ __forceinline__ void store_pairs(void* dst, size_t at, uint32_t D, const float (&x)[kPairs][2]) {
    const uint32_t lane = threadIdx.x & 63u;
#pragma unroll
    for (int j = 0; j < kPairs; ++j) {
        const uint32_t i = 2u * lane + 128u * (uint32_t)j;
        if (i + 1u < D && (D & 1u) == 0u) {
            if constexpr (DT == kBF16) *(uint32_t*)((uint16_t*)dst + at + i) = pack_bf16(x[j][0], x[j][1]);
            else *(u32x2*)((float*)dst + at + i) = u32x2{__float_as_uint(x[j][0]), __float_as_uint(x[j][1])};
        } else {
            if (i < D) Elem<DT>::store(dst, at + i, x[j][0]);
            if (i + 1u < D) Elem<DT>::store(dst, at + i + 1u, x[j][1]);
        }
    }
}

// Queries to q_out [rows][heads][dim], keys to the cache: a wave per head of a token.
template <int DT>
__global__ __launch_bounds__(256) void grouped_append_kernel(const decdec_grouped p, void* __restrict__ q_out, const uint32_t rows) {
    const uint32_t at = blockIdx.x * 4u + (threadIdx.x >> 6), all = p.heads + p.kv_heads, t = at / all, j = at - t * all;
    if (t >= rows) return;
    const long long pos = *p.pos + (long long)t;
    if (pos < 0 || pos >= (long long)p.max_seq) return;
    const bool isq = j < p.heads;
    const uint32_t h = isq ? j : j - p.heads;
    const void* weight = isq ? p.q_norm : p.k_norm;
    float x[kPairs][2];
    norm_rotate(head_fetch<DT>(p.proj, (size_t)t * p.ld + (isq ? p.off_q : p.off_k) + h * p.dim, weight, p, (size_t)pos * (p.rot / 2u)),
                weight != nullptr, p, x);
    if (isq) store_pairs<DT>(q_out, ((size_t)t * p.heads + h) * p.dim, p.dim, x);
    else store_pairs<DT>(p.keys, ((size_t)h * p.max_seq + (size_t)pos) * p.dim, p.dim, x);
}

// The same for dim a multiple of 8 and rot of 8: gl lanes share a head, eight neighbouring elements each.
template <int DT>
__global__ __launch_bounds__(256) void grouped_append_vec_kernel(const decdec_grouped p, void* __restrict__ q_out, const uint32_t rows,
                                                                 const uint32_t gl) {
    using T = typename LaneOf<DT>::t;
    const uint32_t all = p.heads + p.kv_heads, D = p.dim, sub = threadIdx.x % gl, c = 8u * sub;
    const uint32_t at = blockIdx.x * (256u / gl) + threadIdx.x / gl, t = at / all, j = at - t * all;
    const long long pos = *p.pos + (long long)t;
    const bool ok = t < rows && pos >= 0 && pos < (long long)p.max_seq, live = ok && c < D, isq = j < p.heads;
    const uint32_t h = isq ? j : j - p.heads;
    const void* weight = isq ? p.q_norm : p.k_norm;
    const size_t trow = (size_t)(ok ? pos : 0) * (p.rot / 2u);
    float x[8], w[8], cs[4], sn[4], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) { x[e] = 0.f; w[e] = 1.f; }
    if (live) {
        frag_values(frag_load((const T*)p.proj + (size_t)t * p.ld + (isq ? p.off_q : p.off_k) + h * D + c), x);
        if (weight != nullptr) frag_values(frag_load((const T*)weight + c), w);
    }
    const bool turn = live && c < p.rot;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        cs[e] = turn ? p.cos_table[trow + c / 2u + e] : 1.f;
        sn[e] = turn ? p.sin_table[trow + c / 2u + e] : 0.f;
    }
    float r = 1.f;
    if (weight != nullptr) {
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
    }
    for (uint32_t off = 1; off < gl; off <<= 1) ss += __shfl_xor(ss, (int)off, 64);
    if (weight != nullptr) r = 1.f / sqrtf(ss / (float)D + p.eps);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const float u = x[2 * e] * r * w[2 * e], v = x[2 * e + 1] * r * w[2 * e + 1];
        x[2 * e] = u * cs[e] - v * sn[e];
        x[2 * e + 1] = v * cs[e] + u * sn[e];
    }
    if (!live) return;
    T* dst = isq ? (T*)q_out + ((size_t)t * p.heads + h) * D + c : (T*)p.keys + ((size_t)h * p.max_seq + (size_t)pos) * D + c;
    store8(dst, frag_of(x, Frag<DT>{}));
}

// Values, transposed, to the cache: grid (tokens / 64, channels / 64).
template <int DT>
__global__ __launch_bounds__(256) void grouped_values_kernel(const decdec_grouped p, const uint32_t rows) {
    using T = typename LaneOf<DT>::t;
    __shared__ T tile[64][65];
    const uint32_t t0 = blockIdx.x * 64u, c0 = blockIdx.y * 64u, chans = p.kv_heads * p.vdim, a = threadIdx.x & 63u, b = threadIdx.x >> 6;
    const long long pos = *p.pos + (long long)(t0 + a);
    for (uint32_t i = b; i < 64u; i += 4u)
        if (t0 + i < rows && c0 + a < chans) tile[i][a] = ((const T*)p.proj)[(size_t)(t0 + i) * p.ld + p.off_v + c0 + a];
    __syncthreads();
    if (t0 + a >= rows || pos < 0 || pos >= (long long)p.max_seq) return;
    for (uint32_t i = b; i < 64u && c0 + i < chans; i += 4u) ((T*)p.values)[(size_t)(c0 + i) * p.max_seq + (size_t)pos] = tile[a][i];
}

template <int DT>
static hipError_t grouped_append_dt(const decdec_grouped& p, void* q_out, uint32_t rows, hipStream_t s) {
    const uint32_t all = rows * (p.heads + p.kv_heads);
    uint32_t gl = 1;
    while (8u * gl < p.dim) gl *= 2;                        // at most 64: dim is at most 320
    const bool vec = (p.dim | p.rot | p.ld | p.off_q | p.off_k) % 8u == 0 &&
                     ((uintptr_t)p.proj | (uintptr_t)p.q_norm | (uintptr_t)p.k_norm) % 16u == 0;
    if (vec) hipLaunchKernelGGL((grouped_append_vec_kernel<DT>), dim3((all + 256u / gl - 1u) / (256u / gl)), dim3(256), 0, s, p, q_out, rows, gl);
    else hipLaunchKernelGGL((grouped_append_kernel<DT>), dim3((all + 3u) / 4u), dim3(256), 0, s, p, q_out, rows);
    hipLaunchKernelGGL((grouped_values_kernel<DT>), dim3((rows + 63u) / 64u, (p.kv_heads * p.vdim + 63u) / 64u), dim3(256), 0, s, p, rows);
    return hipGetLastError();
}

hipError_t launch_grouped_append(int dt, const decdec_grouped& p, void* q_out, uint32_t rows, hipStream_t s) {
    return dt == kBF16 ? grouped_append_dt<kBF16>(p, q_out, rows, s) : grouped_append_dt<kFP32>(p, q_out, rows, s);
}

hipError_t launch_grouped_attention(int dt, const decdec_grouped& p, const void* q, void* out, uint32_t start, uint32_t rows,
                                    hipStream_t s) {
    TileAttention a{};
    a.q = q; a.k = p.keys; a.vt = p.values; a.out = out;
    a.k_head = (size_t)p.max_seq * p.dim; a.k_row = p.dim;
    a.vt_ld = p.max_seq; a.out_ld = p.out_ld;
    a.heads = p.heads; a.share = p.heads / p.kv_heads; a.dim = p.dim; a.vdim = p.vdim;
    a.scale = p.scale; a.sink_score = p.sink; a.out_scale = p.out_scale;
    if (p.gated) { a.gate = (const char*)p.proj + (size_t)p.off_g * (dt == kBF16 ? 2u : 4u); a.gate_ld = p.ld; }
    return launch_tile_attention(dt, a, start, rows, s);
}

// ---- grouped attention, one token -----------------------------------------------------------------------------
// Shares of the earlier keys, `unit` (a workgroup's pass) at a time; max_splits workgroups at most, one at least (it holds
// the new token).
struct GroupedSplit { uint32_t splits, span; };
__host__ __device__ inline GroupedSplit grouped_split(uint32_t keys, uint32_t unit, uint32_t max_splits) {
    const uint32_t tiles = (keys + unit - 1u) / unit, per = tiles == 0u ? 1u : (tiles + max_splits - 1u) / max_splits;
    return {tiles == 0u ? 1u : (tiles + per - 1u) / per, per * unit};
}
constexpr uint32_t kGroupedSplits = 128;

static bool grouped_small(const decdec_grouped& p) { return p.dim <= 128u && p.vdim <= 128u; }
static uint32_t grouped_unit(int dt, const decdec_grouped& p) { return dt == kBF16 && grouped_small(p) ? 256u : 128u; }
static uint32_t grouped_max_splits(int dt, const decdec_grouped& p) {
    const uint32_t groups = p.kv_heads * ((p.heads / p.kv_heads + 15u) / 16u), unit = grouped_unit(dt, p);
    const uint32_t want = 512u / groups, tiles = (p.max_seq + unit - 1u) / unit;
    const uint32_t n = want < 8u ? 8u : (want > kGroupedSplits ? kGroupedSplits : want);
    return n < tiles ? n : tiles;
}

// grid (splits, kv_heads, heads that share a key / 16), four waves, 16 KB keys a wave and pass.  Scores transposed (keys x
// heads): a wave's keys and values come from memory straight into the operands of its products.  Wave 0 of split 0 starts
// from the new token (which it also appends), every other wave from nothing; the waves are merged through LDS.
template <int DT, int KB, int NK, int NV>
__global__ __launch_bounds__(256, 1) void grouped_step_kernel(const decdec_grouped p, float* __restrict__ parts, const uint32_t max_splits) {
    using T = typename LaneOf<DT>::t;
    using E = Elem<DT>;
    constexpr uint32_t PAD = DT == kFP32 ? 4u : 8u, QL = 32u * NK + PAD, OL = 16u * NV + 4u, UNIT = 64u * KB;
    extern __shared__ __align__(16) float ol[];             // [4][16][OL]
    __shared__ __align__(16) T Ql[16][QL];
    __shared__ T knew[32 * NK], vnew[256];
    __shared__ float mxs[4][16], sums[4][16], snew[16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t kvh = blockIdx.y, share = p.heads / p.kv_heads, g0 = blockIdx.z * 16u, D = p.dim, V = p.vdim;
    const uint32_t h0 = kvh * share + g0, nh = share - g0 < 16u ? share - g0 : 16u;
    const long long pos = *p.pos;
    if (pos < 0 || pos >= (long long)p.max_seq) return;
    const GroupedSplit sp = grouped_split((uint32_t)pos, UNIT, max_splits);
    if (blockIdx.x >= sp.splits) return;
    const uint32_t lo = blockIdx.x * sp.span, hi = lo + sp.span < (uint32_t)pos ? lo + sp.span : (uint32_t)pos;
    const bool vec = D % 8u == 0, first = blockIdx.x == 0u;
    const T* kb = (const T*)p.keys + (size_t)kvh * p.max_seq * D;
    const T* vb = (const T*)p.values + (size_t)kvh * V * p.max_seq;
    Frag<DT> kf[KB][NK], vf[NV][KB / 2];
    // keys past the last repeat it and value columns past it are finite: neither is weighted
    auto request = [&](uint32_t k0) {
#pragma unroll
        for (int b = 0; b < KB; ++b) {
            const uint32_t key = k0 + 16u * (uint32_t)b + l16 < hi ? k0 + 16u * (uint32_t)b + l16 : hi - 1u;
            const T* row = kb + (size_t)key * D;
#pragma unroll
            for (int s = 0; s < NK; ++s) {
                const uint32_t c = 32u * (uint32_t)s + 8u * lg;
                if (vec) {
                    kf[b][s] = frag_load(row + (c < D ? c : 0u));
                    if (c >= D) kf[b][s] = Frag<DT>{};
                } else {
                    kf[b][s] = load8<DT>(row + c, (int)D - (int)c, false);
                }
            }
        }
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const uint32_t d = 16u * (uint32_t)n + l16;
            const T* row = vb + (size_t)(d < V ? d : 0u) * p.max_seq + k0 + 4u * lg;
#pragma unroll
            for (int t = 0; t < KB / 2; ++t) {
                if constexpr (DT == kFP32) {
                    const f32x4 x = *(const f32x4*)(row + 32 * t), y = *(const f32x4*)(row + 32 * t + 16);
#pragma unroll
                    for (int e = 0; e < 4; ++e) { vf[n][t].v[e] = x[e]; vf[n][t].v[4 + e] = y[e]; }
                } else {
                    const u32x2 x = *(const u32x2*)(row + 32 * t), y = *(const u32x2*)(row + 32 * t + 16);
                    vf[n][t].v = u32x4{x[0], x[1], y[0], y[1]};
                }
            }
        }
    };
    // the wave's first query head and the new key ahead of the cache: memory answers in order
    const size_t trow = (size_t)pos * (p.rot / 2u);
    const HeadRow q0 = head_fetch<DT>(p.proj, p.off_q + (size_t)(h0 + (wave < nh ? wave : 0u)) * D, p.q_norm, p, trow);
    HeadRow kn{};
    T vn = (T)0;
    if (first) {
        if (wave == 3u) kn = head_fetch<DT>(p.proj, p.off_k + (size_t)kvh * D, p.k_norm, p, trow);
        if (tid < V) vn = ((const T*)p.proj)[p.off_v + kvh * V + tid];
    }
    uint32_t k0 = lo + wave * 16u * KB;
    if (k0 < hi) request(k0);
    for (uint32_t i = tid; i < 16u * 32u * NK; i += 256u) {                // zeros past dim and past the last head
        const uint32_t r = i / (32u * NK), c = i % (32u * NK);
        if (r >= nh || c >= D) Ql[r][c] = (T)0;
    }
    for (uint32_t j = wave; j < nh; j += 4u) {
        float x[kPairs][2];
        norm_rotate(j == wave ? q0 : head_fetch<DT>(p.proj, p.off_q + (size_t)(h0 + j) * D, p.q_norm, p, trow), p.q_norm != nullptr, p, x);
        store_pairs<DT>(&Ql[j][0], 0, D, x);
    }
    if (first && tid < V) {
        vnew[tid] = vn;
        if (blockIdx.z == 0u) ((T*)p.values)[(size_t)(kvh * V + tid) * p.max_seq + (size_t)pos] = vn;
    }
    if (first && wave == 3u) {
        float x[kPairs][2];
        norm_rotate(kn, p.k_norm != nullptr, p, x);
        store_pairs<DT>(knew, 0, D, x);
        if (blockIdx.z == 0u) store_pairs<DT>(p.keys, ((size_t)kvh * p.max_seq + (size_t)pos) * D, D, x);
    }
    __syncthreads();
    const float scale2 = p.scale * kLog2e;
    float mx = -__builtin_inff(), sum = 0.f;
    f32x4 o[NV];
#pragma unroll
    for (int n = 0; n < NV; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (first) {
        const uint32_t r = tid >> 4, c = tid & 15u;
        float x = 0.f;
        for (uint32_t i = c; i < D; i += 16u) x = __builtin_fmaf(E::load(&Ql[r][0], i), E::load(knew, i), x);
#pragma unroll
        for (int off = 1; off < 16; off <<= 1) x += __shfl_xor(x, off, 64);
        if (c == 0u) snew[r] = x * scale2;
        __syncthreads();
        if (wave == 0u) {
            mx = snew[l16];
            sum = lg == 0u ? 1.f : 0.f;                                    // lane groups hold partial sums
#pragma unroll
            for (int n = 0; n < NV; ++n)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const uint32_t d = 16u * (uint32_t)n + 4u * lg + (uint32_t)v;
                    o[n][v] = d < V ? E::load(vnew, d) : 0.f;
                }
        }
    }
    Frag<DT> qf[NK];
#pragma unroll
    for (int s = 0; s < NK; ++s) qf[s] = frag_load(&Ql[l16][32u * s + 8u * lg]);
    for (; k0 < hi; k0 += UNIT) {
        f32x4 sc[KB];
#pragma unroll
        for (int b = 0; b < KB; ++b) {
            sc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < NK; ++s) mma(kf[b][s], qf[s], sc[b]);
        }
        float best = mx;
#pragma unroll
        for (int b = 0; b < KB; ++b)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const float x = k0 + 16u * (uint32_t)b + 4u * lg + (uint32_t)v < hi ? sc[b][v] * scale2 : -__builtin_inff();
                sc[b][v] = x;
                best = fmaxf(best, x);
            }
        best = fmaxf(best, __shfl_xor(best, 16, 64));
        best = fmaxf(best, __shfl_xor(best, 32, 64));                      // finite: the tile has a key
        const float corr = __builtin_amdgcn_exp2f(mx - best);
        mx = best;
        sum *= corr;
#pragma unroll
        for (int n = 0; n < NV; ++n) o[n] *= corr;
        Frag<DT> whi[KB / 2], wlo[KB / 2];
#pragma unroll
        for (int t = 0; t < KB / 2; ++t) {
            float w[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                w[e] = __builtin_amdgcn_exp2f(sc[2 * t + (e >> 2)][e & 3] - best);
                sum += w[e];
            }
            frag_split(w, whi[t], wlo[t]);
        }
#pragma unroll
        for (int n = 0; n < NV; ++n)
#pragma unroll
            for (int t = 0; t < KB / 2; ++t) {
                mma(vf[n][t], whi[t], o[n]);
                if constexpr (DT != kFP32) mma(vf[n][t], wlo[t], o[n]);
            }
        if (k0 + UNIT < hi) request(k0 + UNIT);
    }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (lg == 0u) { mxs[wave][l16] = mx; sums[wave][l16] = sum; }
#pragma unroll
    for (int n = 0; n < NV; ++n) *(f32x4*)&ol[(wave * 16u + l16) * OL + 16u * (uint32_t)n + 4u * lg] = o[n];
    __syncthreads();
    // partial result of a head: [vdim] sums, maximum, sum of weights; wave 0 has a key or the new token: M is finite
    for (uint32_t i = tid; i < nh * V; i += 256u) {
        const uint32_t h = i / V, d = i - h * V;
        const float M = fmaxf(fmaxf(mxs[0][h], mxs[1][h]), fmaxf(mxs[2][h], mxs[3][h]));
        float acc = 0.f, l = 0.f;
#pragma unroll
        for (uint32_t w = 0; w < 4u; ++w) {
            const float f = __builtin_amdgcn_exp2f(mxs[w][h] - M);
            acc = __builtin_fmaf(f, ol[(w * 16u + h) * OL + d], acc);
            l = __builtin_fmaf(f, sums[w][h], l);
        }
        float* dst = parts + ((size_t)blockIdx.x * p.heads + h0 + h) * (V + 2u);
        dst[d] = acc;
        if (d == 0u) { dst[V] = M; dst[V + 1u] = l; }
    }
}

// Merge of the splits, sink and gate: a workgroup per head; `groups` shares of the splits, Vp threads each.
template <int DT>
__global__ __launch_bounds__(1024) void grouped_merge_kernel(const decdec_grouped p, const float* __restrict__ parts, void* __restrict__ out,
                                                             const uint32_t unit, const uint32_t max_splits) {
    using E = Elem<DT>;
    __shared__ float share[1024], ws[kGroupedSplits];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, h = blockIdx.x, V = p.vdim;
    const long long pos = *p.pos;
    if (pos < 0 || pos >= (long long)p.max_seq) return;
    const uint32_t n = grouped_split((uint32_t)pos, unit, max_splits).splits;
    const float* ph = parts + (size_t)h * (V + 2u);
    const size_t ps = (size_t)p.heads * (V + 2u);
    const uint32_t Vp = (V + 63u) & ~63u, groups = 1024u / Vp, g = tid / Vp, d = tid - g * Vp;
    if (tid < 64u) {
        const float sink = p.sink * kLog2e;
        float m[2], l[2], M = sink;
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) {
            const uint32_t i = lane + 64u * e;
            m[e] = i < n ? ph[i * ps + V] : -__builtin_inff();
            l[e] = i < n ? ph[i * ps + V + 1u] : 0.f;
            M = fmaxf(M, m[e]);
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) M = fmaxf(M, __shfl_xor(M, off, 64));
#pragma unroll
        for (int e = 0; e < 2; ++e) m[e] = __builtin_amdgcn_exp2f(m[e] - M);
        const float L = wave_sum(m[0] * l[0] + m[1] * l[1]) + __builtin_amdgcn_exp2f(sink - M);
        const float r = p.out_scale * (p.gated ? sigmoid_f(E::load(p.proj, p.off_g + h)) : 1.f) / L;
        ws[lane] = m[0] * r;
        ws[lane + 64u] = m[1] * r;
    }
    __syncthreads();
    float t = 0.f;
    if (g < groups && d < V) {
        for (uint32_t s = g; s < n; s += 4u * groups) {
            float x[4];
#pragma unroll
            for (uint32_t e = 0; e < 4u; ++e) x[e] = s + e * groups < n ? ph[(s + e * groups) * ps + d] : 0.f;
#pragma unroll
            for (uint32_t e = 0; e < 4u; ++e) t = __builtin_fmaf(s + e * groups < n ? ws[s + e * groups] : 0.f, x[e], t);
        }
    }
    share[tid] = t;
    __syncthreads();
    if (tid < V) {
        float a = 0.f;
        for (uint32_t k = 0; k < groups; ++k) a += share[k * Vp + tid];
        E::store(out, h * V + tid, a);
    }
}

size_t grouped_step_workspace(const decdec_grouped& p) { return (size_t)kGroupedSplits * p.heads * (p.vdim + 2u) * sizeof(float); }

template <int DT, int KB, int NK, int NV>
static hipError_t grouped_step_launch(const decdec_grouped& p, float* parts, dim3 grid, uint32_t splits, hipStream_t s) {
    constexpr size_t lds = 4u * 16u * (16u * NV + 4u) * sizeof(float);
    if (hipError_t e = allow_lds<grouped_step_kernel<DT, KB, NK, NV>>(lds); e != hipSuccess) return e;
    hipLaunchKernelGGL((grouped_step_kernel<DT, KB, NK, NV>), grid, dim3(256), lds, s, p, parts, splits);
    return hipGetLastError();
}

template <int DT>
static hipError_t grouped_step_dt(const decdec_grouped& p, void* out, float* parts, hipStream_t s) {
    const uint32_t splits = grouped_max_splits(DT, p);
    const dim3 grid(splits, p.kv_heads, (p.heads / p.kv_heads + 15u) / 16u);
    const hipError_t e = grouped_small(p) ? grouped_step_launch<DT, DT == kBF16 ? 4 : 2, 4, 8>(p, parts, grid, splits, s)
                                          : grouped_step_launch<DT, 2, 10, 16>(p, parts, grid, splits, s);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((grouped_merge_kernel<DT>), dim3(p.heads), dim3(1024), 0, s, p, parts, out, grouped_unit(DT, p), splits);
    return hipGetLastError();
}

hipError_t launch_grouped_step(int dt, const decdec_grouped& p, void* out, void* ws, hipStream_t s) {
    return dt == kBF16 ? grouped_step_dt<kBF16>(p, out, (float*)ws, s) : grouped_step_dt<kFP32>(p, out, (float*)ws, s);
}

}  // namespace decdec
