// Linear recurrences with a 32-bit state per head: a decayed sum of outer products, and the gated delta rule.
//
// One token (decode): one kernel reads the state once, updates it in place and forms the read-out.
// Many tokens: chunks of 64.  With G_i the log-decay summed from the chunk's start to token i, S0 the state before the
// chunk and u_j the vector token j writes (its value in the plain form),
//     o_i = e^{G_i} q_i S0 + sum_{j <= i} e^{G_i - G_j} (q_i . k_j) u_j
//     S1  = e^{G_C} S0 + sum_j e^{G_C - G_j} k_j u_j^T
// and for the delta rule, with A_ij = beta_i e^{G_i - G_j} (k_i . k_j) below the diagonal,
//     (I + A) u = diag(beta) v - diag(beta e^G) k S0   =>   u = U - W S0.
// With a decay per key channel G is a vector and the exponentials stand inside the products over channels: q_i e^{G_i},
// k_j e^{G_C - G_j} and the scores sum_c q_ic k_jc e^{G_ic - G_jc} are formed once per chunk and head, the latter by blocks
// of 16 tokens so that no exponent is positive (channel_chunk_kernel); the rest is the same.
// Kernels: inputs (activation, convolution, unit norms, gates), U and W of every chunk (all chunks at once), states (one
// walk over the chunks per head and 16 state columns), read-out (all chunks at once).  All of it in fp32, the products on
// v_mfma_f32_16x16x4_f32.
#include "mixers.h"
#include "mma.h"

namespace decdec {

constexpr uint32_t C = kChunkRows;

template <int DT>
__device__ __forceinline__ float log_decay(const decdec_recurrence& p, const void* proj, size_t row, uint32_t h) {
    using E = Elem<DT>;
    return -expf(E::load(p.A_log, h)) * softplus_f(E::load(proj, row + p.off_a + h) + E::load(p.dt_bias, h));
}

// f(r, w[row0 + r] . x) for r < rows, by eight threads each; x: `rank` floats of LDS, zero up to the next multiple of 8.
template <int DT, typename F>
__device__ __forceinline__ void low_rank(const void* w, size_t row0, uint32_t rows, uint32_t rank, const float* x, F f) {
    using T = typename LaneOf<DT>::t;
    const uint32_t sub = threadIdx.x & 7u, step = blockDim.x >> 3;
    const bool vec = rank % 8u == 0 && (uintptr_t)w % 16u == 0;
    for (uint32_t r0 = 0; r0 < rows; r0 += step) {
        const uint32_t r = r0 + (threadIdx.x >> 3);
        const T* row = (const T*)w + (row0 + (r < rows ? r : 0u)) * rank;
        float acc = 0.f;
#pragma unroll 2
        for (uint32_t c = 8u * sub; c < rank; c += 64u) {
            float v[8];
            frag_values(load8<DT>(row + c, (int)rank - (int)c, vec), v);
#pragma unroll
            for (uint32_t e = 0; e < 8u; ++e) acc = __builtin_fmaf(v[e], x[c + e], acc);
        }
#pragma unroll
        for (int off = 1; off < 8; off <<= 1) acc += __shfl_xor(acc, off, 64);
        if (sub == 0u && r < rows) f(r, acc);
    }
}

// log-decay of one key channel, z the low-rank map's result
__device__ __forceinline__ float channel_log_decay(float rate, float sign, float z, float bias) { return -rate * softplus_f(sign * (z + bias)); }

// ---- one token --------------------------------------------------------------------------------------------
// grid (heads, column splits); a thread owns RPT rows (of `dim`) of one state column.  cw columns per workgroup.
template <int DT, bool DELTA, bool CHANNEL, int RPT>
__global__ __launch_bounds__(1024) void recurrence_step_kernel(const decdec_recurrence p, float* __restrict__ o_out,
                                                               void* __restrict__ out, const void* __restrict__ norm_weight,
                                                               const float eps, const int kind, const uint32_t cw) {
    using E = Elem<DT>;
    __shared__ float qs[512], ks[512], red[32], pa[1024], pb[1024];
    __shared__ float gs[CHANNEL ? 256 : 1], gl[CHANNEL ? 1024 : 1], la[CHANNEL ? kMaxRank + 8 : 1], lb[CHANNEL ? kMaxRank + 8 : 1];
    const uint32_t tid = threadIdx.x, h = blockIdx.x, kg = tid / cw, KG = blockDim.x / cw;
    const uint32_t D = p.dim, V = p.vdim, col = blockIdx.y * cw + tid % cw;
    const bool live = col < V;
    const long long pos = *p.pos;
    const bool fresh = pos <= 0;
    float* S = p.state + (size_t)h * D * V;
    float s[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t r = kg + (uint32_t)i * KG;
        s[i] = (r < D && live && !fresh) ? S[(size_t)r * V + col] : 0.f;
    }
    float v = 0.f, g = 0.f, beta = 1.f;
    if constexpr (CHANNEL) {
        const bool gate = p.g2 != nullptr && out != nullptr;
        for (uint32_t i = tid; i < p.rank_a + 8u; i += blockDim.x) la[i] = i < p.rank_a ? E::load(p.proj, p.off_a + i) : 0.f;
        if (gate)
            for (uint32_t i = tid; i < p.rank_g + 8u; i += blockDim.x) lb[i] = i < p.rank_g ? E::load(p.proj, p.off_g + i) : 0.f;
        __syncthreads();
        const float rate = p.rate[h];
        low_rank<DT>(p.a2, (size_t)h * D, D, p.rank_a, la, [&](uint32_t r, float z) {
            gs[r] = expf(channel_log_decay(rate, p.a_sign, z, p.a_bias[h * D + r]));
        });
        if (gate) low_rank<DT>(p.g2, (size_t)h * V, V, p.rank_g, lb, [&](uint32_t r, float z) { gl[r] = z; });
    }
    if constexpr (!DELTA && CHANNEL) {
        const float sc = 1.f / sqrtf((float)D);
        for (uint32_t i = tid; i < D; i += blockDim.x) {
            qs[i] = E::load(p.proj, p.off_q + h * D + i) * sc;
            ks[i] = E::load(p.proj, p.off_k + h * D + i);
        }
        if (live) v = E::load(p.proj, p.off_v + h * V + col);
    } else if constexpr (!DELTA) {
        for (uint32_t i = tid; i < D; i += blockDim.x) {
            qs[i] = silu_f(E::load(p.proj, p.off_q + h * D + i));
            ks[i] = silu_f(E::load(p.proj, p.off_k + h * D + i));
        }
        if (live) v = silu_f(E::load(p.proj, p.off_v + h * V + col));
        g = p.decay[(size_t)h * 65u + 1u];
    } else {
        const uint32_t share = p.heads / p.kv_heads, kvh = h / share, taps = p.taps;
        const uint32_t qk = p.kv_heads * D, chans = 2u * qk + p.heads * V;
        const bool keeper = h % share == 0u && blockIdx.y == 0u;
        const uint32_t slot = (uint32_t)(pos < 0 ? 0 : pos % (long long)taps);
        // channel c of the ring, whose projection is proj[src] and whose taps are w[wc * taps ..]
        auto conv = [&](uint32_t src, uint32_t c, const void* w, uint32_t wc, bool keep) {
            const float in = E::load(p.proj, src);
            float y = E::load(w, (size_t)wc * taps + taps - 1u) * in;
            for (uint32_t b0 = 1; b0 < taps; b0 += 4u) {                   // b tokens back, four requested together
                float wv[4], xv[4];
                bool ok[4];
#pragma unroll
                for (uint32_t e = 0; e < 4u; ++e) {
                    const uint32_t b = b0 + e;
                    ok[e] = b < taps && pos >= (long long)b;
                    const uint32_t bc = ok[e] ? b : 0u;
                    wv[e] = E::load(w, (size_t)wc * taps + taps - 1u - bc);
                    xv[e] = E::load(p.ring, (size_t)((slot + taps - bc) % taps) * chans + c);
                }
#pragma unroll
                for (uint32_t e = 0; e < 4u; ++e) y += ok[e] ? wv[e] * xv[e] : 0.f;
            }
            if (keep) ((typename LaneOf<DT>::t*)p.ring)[(size_t)slot * chans + c] = ((const typename LaneOf<DT>::t*)p.proj)[src];
            return silu_f(y);
        };
        float sq = 0.f, sk = 0.f;
        for (uint32_t i = tid; i < 2u * D; i += blockDim.x) {
            const bool isq = i < D;
            const uint32_t ch = kvh * D + (isq ? i : i - D);
            const float y = conv((isq ? p.off_q : p.off_k) + ch, (isq ? 0u : qk) + ch, isq ? p.conv_q : p.conv_k, ch, keeper);
            (isq ? qs : ks)[isq ? i : i - D] = y;
            sq += isq ? y * y : 0.f;
            sk += isq ? 0.f : y * y;
        }
        if (live) v = conv(p.off_v + h * V + col, 2u * qk + h * V + col, p.conv_v, h * V + col, kg == 0u);
        if constexpr (!CHANNEL) g = expf(log_decay<DT>(p, p.proj, 0, h));
        beta = sigmoid_f(E::load(p.proj, p.off_b + h));
        block_sum2(sq, sk, red);
        const float rq = 1.f / sqrtf(sq + 1e-6f) / sqrtf((float)D), rk = 1.f / sqrtf(sk + 1e-6f);
        for (uint32_t i = tid; i < D; i += blockDim.x) { qs[i] *= rq; ks[i] *= rk; }
    }
    __syncthreads();
    // a = k . gS, b = q . gS over this thread's rows; o = b + (q . k) u
    float a = 0.f, b = 0.f, qk = 0.f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t r = kg + (uint32_t)i * KG;
        const float kr = r < D ? ks[r] : 0.f, qr = r < D ? qs[r] : 0.f;
        s[i] *= CHANNEL ? (r < D ? gs[r] : 0.f) : g;
        a = __builtin_fmaf(kr, s[i], a);
        b = __builtin_fmaf(qr, s[i], b);
        qk = __builtin_fmaf(kr, qr, qk);
    }
    pa[tid] = DELTA ? a : qk;
    pb[tid] = b;
    __shared__ float pq[1024];
    if constexpr (DELTA) pq[tid] = qk;
    __syncthreads();
    a = 0.f; b = 0.f; qk = 0.f;
    for (uint32_t j = 0; j < KG; ++j) {
        const uint32_t at = j * cw + tid % cw;
        a += pa[at];
        b += pb[at];
        if constexpr (DELTA) qk += pq[at];
    }
    float u;
    if constexpr (DELTA) u = beta * (v - a); else { u = v; qk = a; }
    const float o = __builtin_fmaf(qk, u, b);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t r = kg + (uint32_t)i * KG;
        if (r < D && live) S[(size_t)r * V + col] = __builtin_fmaf(ks[r], u, s[i]);
    }
    if (out == nullptr) {
        if (kg == 0u && live) o_out[(size_t)h * V + col] = o;
        return;
    }
    const float ss = block_sum(kg == 0u && live ? o * o : 0.f, red);
    if (kg == 0u && live) {
        const float z = CHANNEL && p.g2 != nullptr ? gl[CHANNEL ? col : 0u] : E::load(p.proj, p.off_g + h * V + col);
        const float gt = p.out_scale * (kind == DECDEC_GATE_SILU ? silu_f(z) : sigmoid_f(z));
        E::store(out, (size_t)h * V + col, o / sqrtf(ss / (float)V + eps) * E::load(norm_weight, col) * gt);
    }
}

struct StepShape { uint32_t cw, threads, rpt; };
static StepShape step_shape(uint32_t D, uint32_t V, bool whole_head) {
    uint32_t cw = 32;
    if (whole_head) while (cw < V && cw < 1024u) cw *= 2;
    const uint32_t threads = whole_head ? 1024u : 512u, KG = threads / cw;
    return {cw, threads, (D + KG - 1u) / KG};
}

bool recurrence_step_fuses(uint32_t dim, uint32_t vdim) {
    const StepShape s = step_shape(dim, vdim, true);
    return s.cw >= vdim && s.rpt <= 32u;
}

template <int DT, bool DELTA, bool CHANNEL>
static hipError_t step_dt(const decdec_recurrence& p, float* o, void* out, const void* nw, float eps, int kind, hipStream_t s) {
    const StepShape sh = step_shape(p.dim, p.vdim, out != nullptr);
    const dim3 grid(p.heads, (p.vdim + sh.cw - 1u) / sh.cw), block(sh.threads);
    if (sh.rpt <= 4) hipLaunchKernelGGL((recurrence_step_kernel<DT, DELTA, CHANNEL, 4>), grid, block, 0, s, p, o, out, nw, eps, kind, sh.cw);
    else if (sh.rpt <= 16) hipLaunchKernelGGL((recurrence_step_kernel<DT, DELTA, CHANNEL, 16>), grid, block, 0, s, p, o, out, nw, eps, kind, sh.cw);
    else if (sh.rpt <= 32) hipLaunchKernelGGL((recurrence_step_kernel<DT, DELTA, CHANNEL, 32>), grid, block, 0, s, p, o, out, nw, eps, kind, sh.cw);
    else return hipErrorInvalidValue;
    return hipGetLastError();
}

template <int DT>
static hipError_t step_kind(const decdec_recurrence& p, float* o, void* out, const void* nw, float eps, int kind, hipStream_t s) {
    if (p.channel) return p.delta ? step_dt<DT, true, true>(p, o, out, nw, eps, kind, s) : step_dt<DT, false, true>(p, o, out, nw, eps, kind, s);
    return p.delta ? step_dt<DT, true, false>(p, o, out, nw, eps, kind, s) : step_dt<DT, false, false>(p, o, out, nw, eps, kind, s);
}

hipError_t launch_recurrence_step(int dt, const decdec_recurrence& p, float* o, void* out, const void* nw, float eps, int kind,
                                  hipStream_t s) {
    return dt == kBF16 ? step_kind<kBF16>(p, o, out, nw, eps, kind, s) : step_kind<kFP32>(p, o, out, nw, eps, kind, s);
}

// ---- many tokens ------------------------------------------------------------------------------------------
struct ChunkParams {
    const float* q;          // [rows][kv_heads][dim]
    const float* k;
    const float* v;          // [rows][heads][vdim]
    const float* lg;         // [rows][heads] log-decays (delta)
    const float* beta;       // [rows][heads] (delta)
    float* u;                // [rows][heads][vdim]: U, then the written vectors (delta; the values themselves otherwise)
    float* w;                // [rows][heads][dim] (delta)
    float* states;           // [chunks][heads][dim][vdim]
    float* qd;               // [rows][heads][dim] q e^G; the rest likewise: decays per channel
    float* kd;               // [rows][heads][dim] k e^{G_C - G}
    float* gend;             // [chunks][heads][dim] e^{G_C}
    float* scores;           // [chunks][heads][64][64]
    const float* a;          // [rows][heads][dim] before the softplus
    const float* a_bias;     // [heads][dim]
    const float* rate;       // [heads]
    float a_sign;
    const float* decay;      // [heads][65] (plain)
    float* state;
    float* o;
    const long long* pos;
    uint32_t rows, heads, kv_heads, dim, vdim;
};

template <int DT>
__global__ __launch_bounds__(256) void plain_inputs_kernel(const decdec_recurrence p, float* __restrict__ q, float* __restrict__ k,
                                                           float* __restrict__ v) {
    using E = Elem<DT>;
    const uint32_t t = blockIdx.x, nq = p.heads * p.dim, nv = p.heads * p.vdim;
    const size_t row = (size_t)t * p.ld;
    for (uint32_t i = threadIdx.x; i < nq; i += 256u) {
        q[(size_t)t * nq + i] = silu_f(E::load(p.proj, row + p.off_q + i));
        k[(size_t)t * nq + i] = silu_f(E::load(p.proj, row + p.off_k + i));
    }
    for (uint32_t i = threadIdx.x; i < nv; i += 256u) v[(size_t)t * nv + i] = silu_f(E::load(p.proj, row + p.off_v + i));
}

// four neighbouring elements
template <int DT>
__device__ __forceinline__ void quad(const void* p, size_t i, float (&v)[4]) {
    if constexpr (DT == kFP32) {
        const f32x4 t = *(const f32x4*)((const float*)p + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = t[e];
    } else {
        const u32x2 t = *(const u32x2*)((const uint16_t*)p + i);
        v[0] = __uint_as_float(t[0] << 16); v[1] = __uint_as_float(t[0] & 0xFFFF0000u);
        v[2] = __uint_as_float(t[1] << 16); v[3] = __uint_as_float(t[1] & 0xFFFF0000u);
    }
}

// The projections as they are, q scaled: grid (rows, shares of a row); VEC: four elements at a time.
template <int DT, bool VEC>
__global__ __launch_bounds__(256) void linear_inputs_kernel(const decdec_recurrence p, float* __restrict__ q, float* __restrict__ k,
                                                            float* __restrict__ v) {
    constexpr uint32_t N = VEC ? 4u : 1u;
    const uint32_t t = blockIdx.x, nq = p.heads * p.dim, nv = p.heads * p.vdim;
    const float sc = 1.f / sqrtf((float)p.dim);
    for (uint32_t i = N * (blockIdx.y * 256u + threadIdx.x); i < 2u * nq + nv; i += N * 256u * gridDim.y) {
        const bool isq = i < nq, isk = !isq && i < 2u * nq;
        const uint32_t c = isq ? i : (isk ? i - nq : i - 2u * nq);
        const size_t src = (size_t)t * p.ld + (isq ? p.off_q : (isk ? p.off_k : p.off_v)) + c;
        float* dst = (isq ? q : (isk ? k : v)) + (size_t)t * (isq || isk ? nq : nv) + c;
        const float f = isq ? sc : 1.f;
        if constexpr (VEC) {
            float x[4];
            quad<DT>(p.proj, src, x);
            *(f32x4*)dst = f32x4{x[0] * f, x[1] * f, x[2] * f, x[3] * f};
        } else {
            *dst = Elem<DT>::load(p.proj, src) * f;
        }
    }
}

template <int DT>
__global__ __launch_bounds__(256) void delta_inputs_kernel(const decdec_recurrence p, float* __restrict__ q, float* __restrict__ k,
                                                           float* __restrict__ v, float* __restrict__ lg, float* __restrict__ beta) {
    using E = Elem<DT>;
    const uint32_t t = blockIdx.x, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, D = p.dim, taps = p.taps;
    const uint32_t nqk = p.kv_heads * D, nv = p.heads * p.vdim, chans = 2u * nqk + nv;
    const long long pos0 = *p.pos;
    auto conv = [&](uint32_t off, uint32_t c, const void* w, uint32_t wc) {
        float y = 0.f;
        for (uint32_t b = 0; b < taps; ++b) {                              // b tokens back
            float in;
            if (b <= t) in = E::load(p.proj, (size_t)(t - b) * p.ld + off + wc);
            else if (pos0 + (long long)t >= (long long)b) in = E::load(p.ring, (size_t)((pos0 + t - b) % taps) * chans + c);
            else break;
            y = __builtin_fmaf(E::load(w, (size_t)wc * taps + taps - 1u - b), in, y);
        }
        return silu_f(y);
    };
    for (uint32_t j = wave; j < 2u * p.kv_heads; j += 4u) {
        const bool isq = j < p.kv_heads;
        const uint32_t ch0 = (isq ? j : j - p.kv_heads) * D;
        float y[8], ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint32_t i = lane + 64u * e;
            y[e] = i < D ? conv(isq ? p.off_q : p.off_k, (isq ? 0u : nqk) + ch0 + i, isq ? p.conv_q : p.conv_k, ch0 + i) : 0.f;
            ss += y[e] * y[e];
        }
        float r = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
        if (isq) r /= sqrtf((float)D);
        float* dst = (isq ? q : k) + (size_t)t * nqk + ch0;
#pragma unroll
        for (int e = 0; e < 8; ++e)
            if (lane + 64u * e < D) dst[lane + 64u * e] = y[e] * r;
    }
    for (uint32_t i = tid; i < nv; i += 256u) v[(size_t)t * nv + i] = conv(p.off_v, 2u * nqk + i, p.conv_v, i);
    for (uint32_t h = tid; h < p.heads; h += 256u) {
        if (!p.channel) lg[(size_t)t * p.heads + h] = log_decay<DT>(p, p.proj, (size_t)t * p.ld, h);
        beta[(size_t)t * p.heads + h] = sigmoid_f(E::load(p.proj, (size_t)t * p.ld + p.off_b + h));
    }
}

// The same for at most TAPS taps and widths that are multiples of four: a workgroup takes eight tokens and a group of query
// and key heads or 1024 value channels (grid.y counts the groups), a thread four neighbouring channels, whose inputs (and
// the taps before them) are all requested at once.
constexpr uint32_t kInputRows = 8;

template <int DT, int TAPS>
__global__ __launch_bounds__(256) void delta_inputs_quad_kernel(const decdec_recurrence p, float* __restrict__ q, float* __restrict__ k,
                                                                float* __restrict__ v, float* __restrict__ lg, float* __restrict__ beta,
                                                                const uint32_t rows, const uint32_t gl) {
    using E = Elem<DT>;
    constexpr int N = (int)kInputRows, B = TAPS - 1;
    const uint32_t tid = threadIdx.x, D = p.dim, taps = p.taps, t0 = blockIdx.x * kInputRows;
    const uint32_t nqk = p.kv_heads * D, nv = p.heads * p.vdim, chans = 2u * nqk + nv;
    const long long pos0 = *p.pos;
    // y[t] of channels off + wc .. + 3, ring channel c
    auto conv = [&](uint32_t off, uint32_t c, const void* w, uint32_t wc, float (&y)[N][4]) {
        float x[B + N][4], wt[TAPS][4];
#pragma unroll
        for (int i = 0; i < B + N; ++i) {
            const int t = (int)t0 + i - B;                                 // token of the portion, negative before it
            if (t >= 0) quad<DT>(p.proj, (size_t)((uint32_t)t < rows ? (uint32_t)t : rows - 1u) * p.ld + off + wc, x[i]);
            else if (pos0 + t >= 0 && -t < (int)taps) quad<DT>(p.ring, (size_t)((pos0 + t) % taps) * chans + c, x[i]);
            else x[i][0] = x[i][1] = x[i][2] = x[i][3] = 0.f;
        }
#pragma unroll
        for (int b = 0; b < TAPS; ++b)
#pragma unroll
            for (uint32_t e = 0; e < 4u; ++e)
                wt[b][e] = (uint32_t)b < taps ? E::load(w, (size_t)(wc + e) * taps + taps - 1u - (uint32_t)b) : 0.f;
#pragma unroll
        for (int t = 0; t < N; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                float a = 0.f;
#pragma unroll
                for (int b = 0; b < TAPS; ++b) a = __builtin_fmaf(wt[b][e], x[B + t - b][e], a);
                y[t][e] = silu_f(a);
            }
    };
    auto put = [&](float* dst, uint32_t t, uint32_t width, uint32_t c, const float (&y)[4], float r) {
        if (t0 + t < rows) *(f32x4*)(dst + (size_t)(t0 + t) * width + c) = f32x4{y[0] * r, y[1] * r, y[2] * r, y[3] * r};
    };
    const uint32_t per = 256u / gl, hgroups = (2u * p.kv_heads + per - 1u) / per;   // gl threads share a head
    if (blockIdx.y < hgroups) {
        const uint32_t j = blockIdx.y * per + tid / gl, c4 = (tid % gl) * 4u;
        const bool isq = j < p.kv_heads, live = j < 2u * p.kv_heads && c4 < D;
        const uint32_t ch = live ? (isq ? j : j - p.kv_heads) * D + c4 : 0u;
        float y[N][4];
        conv(isq || !live ? p.off_q : p.off_k, (isq || !live ? 0u : nqk) + ch, isq || !live ? p.conv_q : p.conv_k, ch, y);
#pragma unroll
        for (int t = 0; t < N; ++t) {
            float ss = live ? y[t][0] * y[t][0] + y[t][1] * y[t][1] + y[t][2] * y[t][2] + y[t][3] * y[t][3] : 0.f;
            for (uint32_t off = 1; off < gl; off <<= 1) ss += __shfl_xor(ss, (int)off, 64);
            float r = 1.f / sqrtf(ss + 1e-6f);
            if (isq) r /= sqrtf((float)D);
            if (live) put(isq ? q : k, (uint32_t)t, nqk, ch, y[t], r);
        }
    } else {
        const uint32_t c = 1024u * (blockIdx.y - hgroups) + 4u * tid;
        if (c < nv) {
            float y[N][4];
            conv(p.off_v, 2u * nqk + c, p.conv_v, c, y);
#pragma unroll
            for (int t = 0; t < N; ++t) put(v, (uint32_t)t, nv, c, y[t], 1.f);
        }
    }
    if (blockIdx.y + 1u == gridDim.y) {
        for (uint32_t i = tid; i < p.heads * kInputRows; i += 256u) {
            const uint32_t t = t0 + i / p.heads, h = i % p.heads;
            if (t < rows) {
                if (!p.channel) lg[(size_t)t * p.heads + h] = log_decay<DT>(p, p.proj, (size_t)t * p.ld, h);
                beta[(size_t)t * p.heads + h] = sigmoid_f(E::load(p.proj, (size_t)t * p.ld + p.off_b + h));
            }
        }
    }
}

// The last min(rows, taps) projections into the ring (after delta_inputs has read the old ones).
template <int DT>
__global__ __launch_bounds__(256) void ring_update_kernel(const decdec_recurrence p, const uint32_t rows) {
    using T = typename LaneOf<DT>::t;
    const uint32_t nqk = p.kv_heads * p.dim, nv = p.heads * p.vdim, chans = 2u * nqk + nv;
    const uint32_t c = blockIdx.x * 256u + threadIdx.x, t = rows - 1u - blockIdx.y;
    if (c >= chans) return;
    const uint32_t src = c < nqk ? p.off_q + c : (c < 2u * nqk ? p.off_k + c - nqk : p.off_v + c - 2u * nqk);
    const uint32_t slot = (uint32_t)((*p.pos + (long long)t) % p.taps);
    ((T*)p.ring)[(size_t)slot * chans + c] = ((const T*)p.proj)[(size_t)t * p.ld + src];
}

// Log-decays of a chunk summed up, in double: exponents are taken of differences, which must not lose what a long sum
// has swallowed.  One wave.
__device__ __forceinline__ void chunk_log_decay(const ChunkParams& p, uint32_t t0, uint32_t n, uint32_t h, double* G) {
    const uint32_t lane = threadIdx.x & 63u;
    double x = lane < n ? (double)p.lg[(size_t)(t0 + lane) * p.heads + h] : 0.0;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double y = __shfl_up(x, off, 64);
        if ((int)lane >= off) x += y;
    }
    G[lane] = x;
}

// eight floats of a row, zero past `valid`
__device__ __forceinline__ Frag<kFP32> row_frag(const float* p, int valid, bool vec) {
    Frag<kFP32> f;
    if (vec && valid >= 8) return frag_load(p);
#pragma unroll
    for (int i = 0; i < 8; ++i) f.v[i] = i < valid ? p[i] : 0.f;
    return f;
}

// 64 rows x 32 columns of an array of rows (stride ld), requested into registers and later put into LDS [64][36]; rows past
// n and columns past D are zero.
struct Slice { f32x4 x[2]; };
template <bool FULL>                                       // D is a multiple of 32
__device__ __forceinline__ Slice slice_fetch(const float* src, size_t ld, uint32_t n, uint32_t c0, uint32_t D, bool vec) {
    Slice s;
#pragma unroll
    for (uint32_t e = 0; e < 2; ++e) {
        const uint32_t i = threadIdx.x + 256u * e, r = i >> 3, c = c0 + (i & 7u) * 4u;
        const float* row = src + (size_t)(r < n ? r : 0u) * ld;
        if (FULL || vec) {                                 // D is a multiple of four
            s.x[e] = *(const f32x4*)(row + (FULL || c < D ? c : 0u));
            if (r >= n || (!FULL && c >= D)) s.x[e] = f32x4{0.f, 0.f, 0.f, 0.f};
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) s.x[e][j] = (r < n && c + (uint32_t)j < D) ? row[c + j] : 0.f;
        }
    }
    return s;
}
__device__ __forceinline__ void slice_put(const Slice& s, float (*dst)[36]) {
#pragma unroll
    for (uint32_t e = 0; e < 2; ++e) {
        const uint32_t i = threadIdx.x + 256u * e;
        *(f32x4*)&dst[i >> 3][(i & 7u) * 4u] = s.x[e];
    }
}

// (I + A) X = B of one chunk and head, X = [U | W], B = [beta v | wf times the rows at wsrc] (which may be W's own place).  A:
// strictly lower triangular, T: scratch for the inverses of the diagonal blocks; all in LDS, A written by the whole
// workgroup just before.
template <bool FULL>
__device__ __forceinline__ void chunk_solve(const ChunkParams& p, float (*A)[C + 4], float (*T)[20], const float* beta, const float* wf,
                                            const float* wsrc, const size_t wld, const uint32_t t0, const uint32_t n, const uint32_t h) {
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, D = p.dim, V = p.vdim;
    __syncthreads();
    // inverses of the four unit lower-triangular 16 x 16 blocks on the diagonal, a thread per column
    if (tid < C) {
        const uint32_t b = tid & ~15u, j = tid & 15u;
        float t[16];
#pragma unroll
        for (uint32_t i = 0; i < 16u; ++i) {
            float y = i == j ? 1.f : 0.f;
#pragma unroll
            for (uint32_t m = 0; m < i; ++m) y = __builtin_fmaf(-A[b + i][b + m], t[m], y);
            t[i] = y;
            T[b + i][j] = y;
        }
    }
    __syncthreads();
    // (I + A) X = B, block row by block row, a wave per 16 columns of B: an accumulator tile is at once the right
    // operand of the next product (row 4 (lane / 16) + v of the block in register v)
    const uint32_t l16 = lane & 15u, lg = lane >> 4;
    for (uint32_t c0 = 16u * wave; c0 < V + D; c0 += 64u) {
        const uint32_t c = c0 + l16;
        const bool isv = c < V, live = FULL || c < V + D;
        const float* src = isv ? p.v + ((size_t)t0 * p.heads + h) * V + c : wsrc + (live ? c - V : 0u);
        const size_t ld = isv ? (size_t)p.heads * V : wld;
        float* dst = isv ? p.u + ((size_t)t0 * p.heads + h) * V + c : p.w + ((size_t)t0 * p.heads + h) * D + (live ? c - V : 0u);
        const size_t dld = (size_t)p.heads * (isv ? V : D);
        f32x4 x[4];
#pragma unroll
        for (uint32_t b = 0; b < 4u; ++b)
#pragma unroll
            for (uint32_t v = 0; v < 4u; ++v) {
                const uint32_t i = 16u * b + 4u * lg + v;
                x[b][v] = live ? src[(size_t)(i < n ? i : 0u) * ld] : 0.f;
            }
#pragma unroll
        for (uint32_t b = 0; b < 4u; ++b)
#pragma unroll
            for (uint32_t v = 0; v < 4u; ++v) {
                const uint32_t i = 16u * b + 4u * lg + v;
                x[b][v] *= isv ? beta[i] : wf[i];                          // zero past the chunk's last token
            }
#pragma unroll
        for (uint32_t b = 0; b < 4u; ++b) {
#pragma unroll
            for (uint32_t m = 0; m < b; ++m) {
                const f32x4 a = *(const f32x4*)&A[16u * b + l16][16u * m + 4u * lg];
#pragma unroll
                for (uint32_t e = 0; e < 4u; ++e) x[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(-a[e], x[m][e], x[b], 0, 0, 0);
            }
            const f32x4 a = *(const f32x4*)&T[16u * b + l16][4u * lg];
            f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (uint32_t e = 0; e < 4u; ++e) y = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], x[b][e], y, 0, 0, 0);
            x[b] = y;
        }
#pragma unroll
        for (uint32_t b = 0; b < 4u; ++b)
#pragma unroll
            for (uint32_t v = 0; v < 4u; ++v) {
                const uint32_t i = 16u * b + 4u * lg + v;
                if (live && i < n) dst[(size_t)i * dld] = x[b][v];
            }
    }
}

// U and W of a chunk: grid (chunks, heads).
template <bool FULL>
__global__ __launch_bounds__(256) void delta_solve_kernel(const ChunkParams p) {
    __shared__ __align__(16) float Ks[C][36];
    __shared__ __align__(16) float A[C][C + 4];
    __shared__ __align__(16) float T[C][20];                // inverses of the diagonal blocks
    __shared__ double G[C];
    __shared__ float beta[C], bg[C];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, h = blockIdx.y, kvh = h / (p.heads / p.kv_heads);
    const uint32_t t0 = blockIdx.x * C, n = p.rows - t0 < C ? p.rows - t0 : C, D = p.dim;
    const float* k = p.k + ((size_t)t0 * p.kv_heads + kvh) * D;
    const size_t kld = (size_t)p.kv_heads * D;
    const bool vec = D % 4u == 0;
    if (wave == 0) {
        chunk_log_decay(p, t0, n, h, G);
        beta[lane] = lane < n ? p.beta[(size_t)(t0 + lane) * p.heads + h] : 0.f;
        bg[lane] = beta[lane] * expf((float)G[lane]);
    }
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    Slice ks = slice_fetch<FULL>(k, kld, n, 0u, D, vec);
    for (uint32_t c0 = 0; c0 < D; c0 += 32u) {
        __syncthreads();
        slice_put(ks, Ks);
        __syncthreads();
        if (c0 + 32u < D) ks = slice_fetch<FULL>(k, kld, n, c0 + 32u, D, vec);
        const Frag<kFP32> a = frag_load(&Ks[16u * wave + (lane & 15u)][8u * (lane >> 4)]);
#pragma unroll
        for (int j = 0; j < 4; ++j) mma(a, frag_load(&Ks[16u * j + (lane & 15u)][8u * (lane >> 4)]), acc[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const uint32_t r = 16u * wave + 4u * (lane >> 4) + (uint32_t)v, c = 16u * (uint32_t)j + (lane & 15u);
            A[r][c] = c < r ? beta[r] * acc[j][v] * expf((float)(G[r] - G[c])) : 0.f;
        }
    chunk_solve<FULL>(p, A, T, beta, bg, k, kld, t0, n, h);
}

// Decays per key channel: what the later kernels need of a chunk and head, and U and W for the delta rule: grid (chunks,
// heads).  Exponents are sums of log-decays (in units of log 2) from a block's start to a token, from a token to its block's
// end, and over whole blocks of 16 tokens, none of them positive.  Scores between different blocks are products of the
// scaled rows; inside a block the exponential of the difference of two tokens' sums is taken channel by channel.
template <bool DELTA, bool FULL>
__global__ __launch_bounds__(256) void channel_chunk_kernel(const ChunkParams p) {
    __shared__ __align__(16) float buf[5][C][36];
    __shared__ __align__(16) float Bt[4][36];               // sums over whole blocks
    __shared__ float beta[C];
    float (*Qs)[36] = buf[0], (*Ks)[36] = buf[1], (*Ls)[36] = buf[2], (*Ps)[36] = buf[3], (*Rs)[36] = buf[4];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, kvh = h / (p.heads / p.kv_heads), t0 = blockIdx.x * C, n = p.rows - t0 < C ? p.rows - t0 : C, D = p.dim;
    const size_t kld = (size_t)p.kv_heads * D, hld = (size_t)p.heads * D, hrow = ((size_t)t0 * p.heads + h) * D;
    const size_t chunk = (size_t)blockIdx.x * p.heads + h;
    const float* q = p.q + ((size_t)t0 * p.kv_heads + kvh) * D;
    const float* k = p.k + ((size_t)t0 * p.kv_heads + kvh) * D;
    const float rate2 = p.rate[h] * kLog2e;
    const bool vec = D % 4u == 0;
    if constexpr (DELTA) { if (wave == 0u) beta[lane] = lane < n ? p.beta[(size_t)(t0 + lane) * p.heads + h] : 0.f; }
    f32x4 pq[4], pk[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) pq[j] = pk[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    float dq[4] = {0.f, 0.f, 0.f, 0.f}, dk[4] = {0.f, 0.f, 0.f, 0.f};
    Slice qs = slice_fetch<FULL>(q, kld, n, 0u, D, vec), ks = slice_fetch<FULL>(k, kld, n, 0u, D, vec);
    Slice as = slice_fetch<FULL>(p.a + hrow, hld, n, 0u, D, vec);
    for (uint32_t c0 = 0; c0 < D; c0 += 32u) {
        __syncthreads();
        slice_put(qs, Qs);
        slice_put(ks, Ks);
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) {
            const uint32_t i = tid + 256u * e, r = i >> 3, c = (i & 7u) * 4u;
            f32x4 x;
#pragma unroll
            for (uint32_t j = 0; j < 4u; ++j) {
                const bool in = r < n && (FULL || c0 + c + j < D);
                // what 2^-64 is left of does not show in a sum; the bound keeps the differences after such a token sharp
                x[j] = in ? fmaxf(channel_log_decay(rate2, p.a_sign, as.x[e][j], p.a_bias[h * D + c0 + c + j]), -64.f) : 0.f;
            }
            *(f32x4*)&Ls[r][c] = x;
        }
        __syncthreads();
        if (c0 + 32u < D) {
            qs = slice_fetch<FULL>(q, kld, n, c0 + 32u, D, vec);
            ks = slice_fetch<FULL>(k, kld, n, c0 + 32u, D, vec);
            as = slice_fetch<FULL>(p.a + hrow, hld, n, c0 + 32u, D, vec);
        }
        {
            const uint32_t b = (tid >> 5) & 3u, c = tid & 31u;
            float x[16], run = 0.f;
#pragma unroll
            for (uint32_t i = 0; i < 16u; ++i) x[i] = Ls[16u * b + i][c];
            if (tid < 128u) {
#pragma unroll
                for (uint32_t i = 0; i < 16u; ++i) { run += x[i]; Ps[16u * b + i][c] = run; }
                Bt[b][c] = run;
            } else {
#pragma unroll
                for (int i = 15; i >= 0; --i) { Rs[16u * b + (uint32_t)i][c] = run; run += x[i]; }
            }
        }
        __syncthreads();
        // inside the wave's block: rows 4 lg + v, column l16
#pragma unroll 2
        for (uint32_t d = 0; d < 32u; d += 4u) {
            const f32x4 pj = *(const f32x4*)&Ps[16u * wave + l16][d], kj = *(const f32x4*)&Ks[16u * wave + l16][d];
#pragma unroll
            for (uint32_t v = 0; v < 4u; ++v) {
                const uint32_t r = 16u * wave + 4u * lg + v;
                const f32x4 pi = *(const f32x4*)&Ps[r][d], qi = *(const f32x4*)&Qs[r][d];
                f32x4 ki = kj;
                if constexpr (DELTA) ki = *(const f32x4*)&Ks[r][d];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float f = __builtin_amdgcn_exp2f(fminf(pi[e] - pj[e], 0.f)) * kj[e];
                    dq[v] = __builtin_fmaf(qi[e], f, dq[v]);
                    if constexpr (DELTA) dk[v] = __builtin_fmaf(ki[e], f, dk[v]);
                }
            }
        }
        // the wave's block against the earlier ones
        if (wave != 0u) {
            const uint32_t r = 16u * wave + l16;
            Frag<kFP32> qa = frag_load(&Qs[r][8u * lg]), ka = frag_load(&Ks[r][8u * lg]);
            const Frag<kFP32> pe = frag_load(&Ps[r][8u * lg]);
            float mid[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float f = __builtin_amdgcn_exp2f(pe.v[e]);
                qa.v[e] *= f;
                ka.v[e] *= f;
                mid[e] = 0.f;
            }
#pragma unroll
            for (int j = 2; j >= 0; --j) {
                if ((uint32_t)j < wave) {
                    Frag<kFP32> kb = frag_load(&Ks[16 * j + l16][8u * lg]);
                    const Frag<kFP32> re = frag_load(&Rs[16 * j + l16][8u * lg]), bt = frag_load(&Bt[j][8u * lg]);
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        kb.v[e] *= __builtin_amdgcn_exp2f(re.v[e] + mid[e]);
                        mid[e] += bt.v[e];
                    }
                    mma(qa, kb, pq[j]);
                    if constexpr (DELTA) mma(ka, kb, pk[j]);
                }
            }
        }
        // rows scaled to the chunk's start and end
        {
            const uint32_t r = tid >> 2, c = (tid & 3u) * 8u, b = r >> 4;
#pragma unroll
            for (uint32_t e = 0; e < 8u; e += 4u) {
                f32x4 pre = *(const f32x4*)&Ps[r][c + e], suf = *(const f32x4*)&Rs[r][c + e];
#pragma unroll
                for (uint32_t m = 0; m < 4u; ++m) {
                    const f32x4 t = *(const f32x4*)&Bt[m][c + e];
                    if (m < b) pre += t;
                    if (m > b) suf += t;
                }
                f32x4 x = *(const f32x4*)&Qs[r][c + e], y = *(const f32x4*)&Ks[r][c + e], z = y;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float f = __builtin_amdgcn_exp2f(pre[i]);
                    x[i] *= f;
                    z[i] *= f;
                    y[i] *= __builtin_amdgcn_exp2f(suf[i]);
                }
                if (r < n) {
                    const size_t at = hrow + (size_t)r * hld + c0 + c + e;
                    if (FULL || (vec && c0 + c + e < D)) {
                        *(f32x4*)(p.qd + at) = x;
                        *(f32x4*)(p.kd + at) = y;
                        if constexpr (DELTA) *(f32x4*)(p.w + at) = z;
                    } else if (!vec) {
#pragma unroll
                        for (uint32_t i = 0; i < 4u; ++i)
                            if (c0 + c + e + i < D) {
                                p.qd[at + i] = x[i];
                                p.kd[at + i] = y[i];
                                if constexpr (DELTA) p.w[at + i] = z[i];
                            }
                    }
                }
            }
        }
        if (tid < 32u && c0 + tid < D) p.gend[chunk * D + c0 + tid] = __builtin_amdgcn_exp2f(Bt[0][tid] + Bt[1][tid] + Bt[2][tid] + Bt[3][tid]);
    }
    float* out = p.scores + chunk * (C * C);
    __syncthreads();                                        // A takes the place of the slices
    float (*A)[C + 4] = (float (*)[C + 4])buf[0];
    float (*T)[20] = (float (*)[20])(&buf[0][0][0] + C * (C + 4));
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (uint32_t v = 0; v < 4u; ++v) {
            const uint32_t r = 16u * wave + 4u * lg + v, c = 16u * (uint32_t)j + l16;
            const bool before = (uint32_t)j < wave, own = (uint32_t)j == wave;
            out[r * C + c] = before ? pq[j][v] : (own && c <= r ? dq[v] : 0.f);
            if constexpr (DELTA) A[r][c] = beta[r] * (before ? pk[j][v] : (own && c < r ? dk[v] : 0.f));
        }
    if constexpr (DELTA) chunk_solve<FULL>(p, A, T, beta, beta, p.w + hrow, hld, t0, n, h);
}

// States: grid (heads, vdim / 16), one walk over the chunks.  Wave w owns the state's row tiles w, w + 4, ... (NT of them).
// What the next chunk needs from memory is requested as soon as this chunk's copy has been used.
// FULL: dim is 64 NT and vdim a multiple of 16.
template <bool DELTA, bool CHANNEL, int NT, bool FULL>
__global__ __launch_bounds__(256) void chunk_state_kernel(const ChunkParams p, const uint32_t chunks) {
    extern __shared__ __align__(16) float lds[];
    __shared__ double G[C];
    __shared__ __align__(16) float Vl[C][20];
    __shared__ float pw[C + 1];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.x, kvh = h / (p.heads / p.kv_heads), D = FULL ? 64u * NT : p.dim, V = p.vdim, v0 = blockIdx.y * 16u;
    const uint32_t Dp = (D + 31u) & ~31u, KL = Dp + 4u, tiles = Dp / 16u;
    float* Kl = lds;                        // [C][KL]
    float* Sl = lds + C * KL;               // [Dp][20]
    const bool fresh = *p.pos <= 0, vec = FULL || D % 4u == 0, vec8 = FULL || D % 8u == 0, col = FULL || v0 + l16 < V;
    float* S = p.state + (size_t)h * D * V + v0 + l16;
    if constexpr (!DELTA && !CHANNEL) { for (uint32_t i = tid; i <= C; i += 256u) pw[i] = p.decay[(size_t)h * 65u + i]; }
    f32x4 s[NT], gch[CHANNEL ? NT : 1];
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const uint32_t r = 16u * (wave + 4u * (uint32_t)i) + 4u * lg + (uint32_t)v;
            s[i][v] = ((FULL || (r < D && col)) && !fresh) ? S[(size_t)r * V] : 0.f;
        }
    const uint32_t kr = tid >> 2, kc = (tid & 3u) * 4u;                    // a thread's row of the keys, and columns kc + 16 j
    f32x4 kreg[4 * NT];
    Frag<kFP32> wreg[DELTA ? 2 * NT : 1];
    float ureg[4], lreg = 0.f;
    auto request_keys = [&](uint32_t t0) {
        const uint32_t n = p.rows - t0 < C ? p.rows - t0 : C;
        const size_t krow = (size_t)(t0 + (kr < n ? kr : 0u));
        const float* k = CHANNEL ? p.kd + (krow * p.heads + h) * D : p.k + (krow * p.kv_heads + kvh) * D;
#pragma unroll
        for (int j = 0; j < 4 * NT; ++j) {
            const uint32_t c = kc + 16u * (uint32_t)j;
            if (vec) {
                kreg[j] = *(const f32x4*)(k + (FULL || c < D ? c : 0u));
                if (kr >= n || (!FULL && c >= D)) kreg[j] = f32x4{0.f, 0.f, 0.f, 0.f};
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) kreg[j][e] = (kr < n && c + (uint32_t)e < D) ? k[c + e] : 0.f;
            }
        }
        if constexpr (CHANNEL) {
            const float* g = p.gend + ((size_t)(t0 / C) * p.heads + h) * D;
#pragma unroll
            for (int i = 0; i < NT; ++i)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const uint32_t r = 16u * (wave + 4u * (uint32_t)i) + 4u * lg + (uint32_t)v;
                    gch[i][v] = FULL || r < D ? g[r] : 0.f;
                }
        } else if constexpr (DELTA) lreg = (wave == 3u && lane < n) ? p.lg[(size_t)(t0 + lane) * p.heads + h] : 0.f;
    };
    auto request_writes = [&](uint32_t t0) {
        const uint32_t n = p.rows - t0 < C ? p.rows - t0 : C, ar = 16u * wave + l16;
        if constexpr (DELTA) {
            const float* w = p.w + ((size_t)(t0 + (ar < n ? ar : 0u)) * p.heads + h) * D;
#pragma unroll
            for (int j = 0; j < 2 * NT; ++j) {
                const uint32_t kk = 32u * (uint32_t)j + 8u * lg;
                wreg[j] = FULL ? frag_load(w + kk) : row_frag(w + kk, ar < n ? (int)D - (int)kk : 0, vec8);   // rows past n write nothing
            }
        }
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const uint32_t r = 16u * wave + 4u * lg + (uint32_t)v;
            const size_t at = ((size_t)(t0 + (r < n ? r : 0u)) * p.heads + h) * V + v0 + (col ? l16 : 0u);
            ureg[v] = DELTA ? p.u[at] : p.v[at];
        }
    };
    request_keys(0u);
    request_writes(0u);
    for (uint32_t ch = 0; ch < chunks; ++ch) {
        const uint32_t t0 = ch * C, n = p.rows - t0 < C ? p.rows - t0 : C;
        f32x4 gnow[CHANNEL ? NT : 1];
        if constexpr (CHANNEL) {
#pragma unroll
            for (int i = 0; i < NT; ++i) gnow[i] = gch[i];
        }
#pragma unroll
        for (int j = 0; j < 4 * NT; ++j)
            if (FULL || kc + 16u * (uint32_t)j < Dp) *(f32x4*)&Kl[kr * KL + kc + 16u * (uint32_t)j] = kreg[j];
        if constexpr (DELTA && !CHANNEL) {
            if (wave == 3u) {                                              // log-decays summed up, in double
                double x = (double)lreg;
#pragma unroll
                for (int off = 1; off < 64; off <<= 1) {
                    const double y = __shfl_up(x, off, 64);
                    if ((int)lane >= off) x += y;
                }
                G[lane] = x;
            }
        }
        float* st = p.states + ((size_t)ch * p.heads + h) * D * V + v0 + l16;
#pragma unroll
        for (int i = 0; i < NT; ++i)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const uint32_t r = 16u * (wave + 4u * (uint32_t)i) + 4u * lg + (uint32_t)v;
                if (FULL || r < Dp) Sl[r * 20u + l16] = s[i][v];
                if (FULL || (r < D && col)) st[(size_t)r * V] = s[i][v];
            }
        __syncthreads();
        if (ch + 1u < chunks) request_keys(t0 + C);
        const float gend = CHANNEL ? 1.f : (DELTA ? expf((float)G[C - 1]) : pw[n]);
        {
            // what the tokens write, 16 rows per wave
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
            if constexpr (DELTA) {
#pragma unroll
                for (int j = 0; j < 2 * NT; ++j)
                    if (FULL || 32u * (uint32_t)j < D) mma(wreg[j], frag_gather(Sl + (32u * (uint32_t)j + 8u * lg) * 20u + l16, 20u), acc);
            }
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const uint32_t r = 16u * wave + 4u * lg + (uint32_t)v;
                float x = 0.f;
                if (r < n && col) {
                    if constexpr (DELTA) {
                        x = ureg[v] - acc[v];
                        p.u[((size_t)(t0 + r) * p.heads + h) * V + v0 + l16] = x;
                        if constexpr (!CHANNEL) x *= expf((float)(G[C - 1] - G[r]));
                    } else if constexpr (CHANNEL) {
                        x = ureg[v];
                    } else {
                        x = ureg[v] * pw[n - 1u - r];
                    }
                }
                Vl[r][l16] = x;
            }
        }
        if (ch + 1u < chunks) request_writes(t0 + C);
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const uint32_t tile = wave + 4u * (uint32_t)i;
            if constexpr (CHANNEL) s[i] *= gnow[i]; else s[i] *= gend;
            if (FULL || tile < tiles) {
#pragma unroll
                for (uint32_t j0 = 0; j0 < C; j0 += 32u)
                    mma(frag_gather(Kl + (j0 + 8u * lg) * KL + 16u * tile + l16, KL), frag_gather(&Vl[j0 + 8u * lg][l16], 20u), s[i]);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const uint32_t r = 16u * (wave + 4u * (uint32_t)i) + 4u * lg + (uint32_t)v;
            if (FULL || (r < D && col)) S[(size_t)r * V] = s[i][v];
        }
}

// Read-out: grid (chunks, heads, vdim / 64).  FULL: dim is a multiple of 32 and vdim of 64.
template <bool DELTA, bool CHANNEL, bool FULL>
__global__ __launch_bounds__(256) void chunk_output_kernel(const ChunkParams p) {
    __shared__ __align__(16) float Qs[C][36];
    __shared__ __align__(16) float Ks[CHANNEL ? 1 : C][36];
    __shared__ __align__(16) float Ss[32][68];
    __shared__ __align__(16) float Ps[C][68];
    __shared__ __align__(16) float Vs[C][68];
    __shared__ double G[C];
    __shared__ float pw[C + 1];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, kvh = h / (p.heads / p.kv_heads), D = p.dim, V = p.vdim, v0 = blockIdx.z * 64u;
    const uint32_t t0 = blockIdx.x * C, n = p.rows - t0 < C ? p.rows - t0 : C;
    const bool vec = D % 4u == 0;
    const size_t kld = (size_t)(CHANNEL ? p.heads : p.kv_heads) * D;
    const float* q = CHANNEL ? p.qd + ((size_t)t0 * p.heads + h) * D : p.q + ((size_t)t0 * p.kv_heads + kvh) * D;
    const float* k = p.k + ((size_t)t0 * p.kv_heads + kvh) * D;
    const float* vv = (DELTA ? p.u : p.v) + ((size_t)t0 * p.heads + h) * V;
    const float* S = p.states + ((size_t)blockIdx.x * p.heads + h) * D * V;
    if constexpr (CHANNEL) {                                // the scores are there
        const float* sc = p.scores + ((size_t)blockIdx.x * p.heads + h) * (C * C);
#pragma unroll
        for (uint32_t e = 0; e < 4u; ++e) {
            const uint32_t i = tid + 256u * e;
            *(f32x4*)&Ps[i >> 4][(i & 15u) * 4u] = *(const f32x4*)(sc + 4u * i);
        }
    } else if constexpr (DELTA) { if (wave == 0) chunk_log_decay(p, t0, n, h, G); }
    else { for (uint32_t i = tid; i <= C; i += 256u) pw[i] = p.decay[(size_t)h * 65u + i]; }
    // four neighbouring columns of a 64-column array per thread and pass, 16 rows a pass
    const bool vecv = FULL || V % 4u == 0;
    const uint32_t vr = tid >> 4, vc = (tid & 15u) * 4u;
    auto value4 = [&](const float* row, bool in) {
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        if (vecv) {
            x = *(const f32x4*)(row + (FULL || v0 + vc < V ? v0 + vc : 0u));
            if (!in || (!FULL && v0 + vc >= V)) x = f32x4{0.f, 0.f, 0.f, 0.f};
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (in && v0 + vc + (uint32_t)e < V) x[e] = row[v0 + vc + e];
        }
        return x;
    };
    Slice qr = slice_fetch<FULL>(q, kld, n, 0u, D, vec), kr;
    if constexpr (!CHANNEL) kr = slice_fetch<FULL>(k, kld, n, 0u, D, vec);
    f32x4 sr[2], val[4];
    auto fetch_state = [&](uint32_t c0) {
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) {
            const uint32_t r = c0 + vr + 16u * e;
            sr[e] = value4(S + (size_t)(FULL || r < D ? r : 0u) * V, FULL || r < D);
        }
    };
    fetch_state(0u);
#pragma unroll
    for (uint32_t e = 0; e < 4u; ++e) {
        const uint32_t r = vr + 16u * e;
        val[e] = value4(vv + (size_t)(r < n ? r : 0u) * p.heads * V, r < n);
    }
#pragma unroll
    for (uint32_t e = 0; e < 4u; ++e) *(f32x4*)&Vs[vr + 16u * e][vc] = val[e];
    f32x4 pr[4], o[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) { pr[j] = f32x4{0.f, 0.f, 0.f, 0.f}; o[j] = f32x4{0.f, 0.f, 0.f, 0.f}; }
    for (uint32_t c0 = 0; c0 < D; c0 += 32u) {
        __syncthreads();
        slice_put(qr, Qs);
        if constexpr (!CHANNEL) slice_put(kr, Ks);
#pragma unroll
        for (uint32_t e = 0; e < 2u; ++e) *(f32x4*)&Ss[vr + 16u * e][vc] = sr[e];
        __syncthreads();
        if (c0 + 32u < D) {
            qr = slice_fetch<FULL>(q, kld, n, c0 + 32u, D, vec);
            if constexpr (!CHANNEL) kr = slice_fetch<FULL>(k, kld, n, c0 + 32u, D, vec);
            fetch_state(c0 + 32u);
        }
        const Frag<kFP32> a = frag_load(&Qs[16u * wave + l16][8u * lg]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if constexpr (!CHANNEL) { if ((uint32_t)j <= wave) mma(a, frag_load(&Ks[16u * j + l16][8u * lg]), pr[j]); }
            mma(a, frag_gather(&Ss[8u * lg][16u * j + l16], 68u), o[j]);
        }
    }
    __syncthreads();                               // decays are in LDS also where D is a single slice; Ps follows
    if constexpr (!CHANNEL)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
        const uint32_t r = 16u * wave + 4u * lg + (uint32_t)v;
        const float f0 = DELTA ? expf((float)G[r]) : pw[r + 1u];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const uint32_t c = 16u * (uint32_t)j + l16;
            float d = 0.f;
            if (c <= r) d = DELTA ? expf((float)(G[r] - G[c])) : pw[r - c];
            Ps[r][c] = pr[j][v] * d;
            o[j][v] *= f0;
        }
    }
    __syncthreads();
#pragma unroll
    for (uint32_t j0 = 0; j0 < C; j0 += 32u) {
        if (j0 > 16u * wave + 15u) break;
        const Frag<kFP32> a = frag_load(&Ps[16u * wave + l16][j0 + 8u * lg]);
#pragma unroll
        for (int j = 0; j < 4; ++j) mma(a, frag_gather(&Vs[j0 + 8u * lg][16u * j + l16], 68u), o[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const uint32_t r = 16u * wave + 4u * lg + (uint32_t)v, c = v0 + 16u * (uint32_t)j + l16;
            if (r < n && (FULL || c < V)) p.o[((size_t)(t0 + r) * p.heads + h) * V + c] = o[j][v];
        }
}

static size_t pad4(size_t n) { return (n + 3u) & ~(size_t)3u; }
static ChunkParams chunk_layout(const decdec_recurrence& p, uint32_t rows, float* base, size_t& floats) {
    ChunkParams c{};
    const size_t nq = pad4((size_t)rows * p.kv_heads * p.dim), nv = pad4((size_t)rows * p.heads * p.vdim), nh = pad4((size_t)rows * p.heads);
    const size_t chunks = (rows + C - 1u) / C;
    size_t at = 0;
    auto take = [&](size_t n) { float* r = base == nullptr ? nullptr : base + at; at += n; return r; };
    c.q = take(nq);
    c.k = take(nq);
    c.v = take(nv);
    const size_t nhd = pad4((size_t)rows * p.heads * p.dim);
    if (p.delta) {
        if (!p.channel) c.lg = take(nh);
        c.beta = take(nh);
        c.u = take(nv);
        c.w = take(nhd);
    }
    if (p.channel) {
        c.qd = take(nhd);
        c.kd = take(nhd);
        c.gend = take(pad4(chunks * p.heads * p.dim));
        c.scores = take(chunks * p.heads * C * C);
        c.a = p.a; c.a_bias = p.a_bias; c.rate = p.rate; c.a_sign = p.a_sign;
    }
    c.states = take(pad4(chunks * p.heads * p.dim * p.vdim));
    floats = at;
    c.decay = p.decay;
    c.state = p.state;
    c.pos = (const long long*)p.pos;
    c.rows = rows; c.heads = p.heads; c.kv_heads = p.kv_heads; c.dim = p.dim; c.vdim = p.vdim;
    return c;
}

size_t recurrence_workspace(const decdec_recurrence& p, uint32_t rows) {
    size_t n;
    chunk_layout(p, rows, nullptr, n);
    return n * sizeof(float);
}

template <bool DELTA, bool CHANNEL, int NT>
static hipError_t launch_state(const ChunkParams& c, uint32_t chunks, dim3 grid, size_t lds, hipStream_t s) {
    if (c.dim == 64u * NT && c.vdim % 16u == 0) {
        if (hipError_t e = allow_lds<chunk_state_kernel<DELTA, CHANNEL, NT, true>>(lds); e != hipSuccess) return e;
        hipLaunchKernelGGL((chunk_state_kernel<DELTA, CHANNEL, NT, true>), grid, dim3(256), lds, s, c, chunks);
    } else {
        if (hipError_t e = allow_lds<chunk_state_kernel<DELTA, CHANNEL, NT, false>>(lds); e != hipSuccess) return e;
        hipLaunchKernelGGL((chunk_state_kernel<DELTA, CHANNEL, NT, false>), grid, dim3(256), lds, s, c, chunks);
    }
    return hipGetLastError();
}

template <bool DELTA, bool CHANNEL>
static hipError_t launch_chunks(const ChunkParams& c, hipStream_t s) {
    const uint32_t chunks = (c.rows + C - 1u) / C, Dp = (c.dim + 31u) & ~31u, nt = (Dp / 16u + 3u) / 4u;
    const size_t lds = ((size_t)C * (Dp + 4u) + (size_t)Dp * 20u) * sizeof(float);
    const dim3 grid(c.heads, (c.vdim + 15u) / 16u), cgrid(chunks, c.heads), ogrid(chunks, c.heads, (c.vdim + 63u) / 64u), block(256);
    if constexpr (CHANNEL) {
        if (c.dim % 32u == 0 && c.vdim % 16u == 0) hipLaunchKernelGGL((channel_chunk_kernel<DELTA, true>), cgrid, block, 0, s, c);
        else hipLaunchKernelGGL((channel_chunk_kernel<DELTA, false>), cgrid, block, 0, s, c);
    } else if constexpr (DELTA) {
        if (c.dim % 32u == 0 && c.vdim % 16u == 0) hipLaunchKernelGGL(delta_solve_kernel<true>, cgrid, block, 0, s, c);
        else hipLaunchKernelGGL(delta_solve_kernel<false>, cgrid, block, 0, s, c);
    }
    const hipError_t e = nt == 1u ? launch_state<DELTA, CHANNEL, 1>(c, chunks, grid, lds, s)
                       : nt == 2u ? launch_state<DELTA, CHANNEL, 2>(c, chunks, grid, lds, s)
                       : nt <= 4u ? launch_state<DELTA, CHANNEL, 4>(c, chunks, grid, lds, s) : hipErrorInvalidValue;
    if (e != hipSuccess) return e;
    if (c.dim % 32u == 0 && c.vdim % 64u == 0) hipLaunchKernelGGL((chunk_output_kernel<DELTA, CHANNEL, true>), ogrid, block, 0, s, c);
    else hipLaunchKernelGGL((chunk_output_kernel<DELTA, CHANNEL, false>), ogrid, block, 0, s, c);
    return hipGetLastError();
}

template <int DT>
static hipError_t rows_dt(const decdec_recurrence& p, const ChunkParams& c, hipStream_t s) {
    const uint32_t es = Elem<DT>::bytes;
    if (!p.delta && p.channel) {
        const uint32_t all = p.heads * (2u * p.dim + p.vdim);
        const bool vec = ((p.heads * p.dim) | (p.heads * p.vdim) | p.ld | p.off_q | p.off_k | p.off_v) % 4u == 0 && (uintptr_t)p.proj % (4u * es) == 0;
        if (vec) hipLaunchKernelGGL((linear_inputs_kernel<DT, true>), dim3(c.rows, (all + 4095u) / 4096u), dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v);
        else hipLaunchKernelGGL((linear_inputs_kernel<DT, false>), dim3(c.rows, 1), dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v);
        return launch_chunks<false, true>(c, s);
    }
    if (!p.delta) {
        hipLaunchKernelGGL((plain_inputs_kernel<DT>), dim3(c.rows), dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v);
        return launch_chunks<false, false>(c, s);
    }
    uint32_t gl = 1;
    while (4u * gl < p.dim) gl *= 2;
    const bool quads = ((p.dim | p.ld | p.off_q | p.off_k | p.off_v | (p.heads * p.vdim)) & 3u) == 0 && p.taps <= 8u &&
                       (uintptr_t)p.proj % (4u * es) == 0 && (uintptr_t)p.ring % (4u * es) == 0;
    const dim3 wide((c.rows + kInputRows - 1u) / kInputRows,
                    (2u * p.kv_heads + 256u / gl - 1u) / (256u / gl) + (p.heads * p.vdim + 1023u) / 1024u);
    if (quads && p.taps <= 4u)
        hipLaunchKernelGGL((delta_inputs_quad_kernel<DT, 4>), wide, dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v, (float*)c.lg, (float*)c.beta, c.rows, gl);
    else if (quads)
        hipLaunchKernelGGL((delta_inputs_quad_kernel<DT, 8>), wide, dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v, (float*)c.lg, (float*)c.beta, c.rows, gl);
    else
        hipLaunchKernelGGL((delta_inputs_kernel<DT>), dim3(c.rows), dim3(256), 0, s, p, (float*)c.q, (float*)c.k, (float*)c.v, (float*)c.lg, (float*)c.beta);
    const uint32_t chans = 2u * p.kv_heads * p.dim + p.heads * p.vdim, keep = c.rows < p.taps ? c.rows : p.taps;
    hipLaunchKernelGGL((ring_update_kernel<DT>), dim3((chans + 255u) / 256u, keep), dim3(256), 0, s, p, c.rows);
    return p.channel ? launch_chunks<true, true>(c, s) : launch_chunks<true, false>(c, s);
}

hipError_t launch_recurrence_rows(int dt, const decdec_recurrence& p, float* o, void* ws, uint32_t rows, hipStream_t s) {
    size_t n;
    ChunkParams c = chunk_layout(p, rows, (float*)ws, n);
    c.o = o;
    return dt == kBF16 ? rows_dt<kBF16>(p, c, s) : rows_dt<kFP32>(p, c, s);
}

}  // namespace decdec
