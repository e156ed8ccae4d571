// C-ABI layer of libdecdec_mixers.so: argument validation in front of the mixer kernels.  Declarations:
// include/decdec_mixers.h.
#include <cstdarg>
#include <cstdio>
#include <string>

#include "mixers.h"

using namespace decdec;

namespace {

enum { kOk = 0, kInvalid = 1, kHipError = 2 };
thread_local std::string g_error;

int fail(int code, const char* fmt, ...) {
    char buf[512];
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(buf, sizeof(buf), fmt, ap);
    va_end(ap);
    g_error = buf;
    return code;
}

#define MX_HIP(expr)                                                                         \
    do {                                                                                     \
        hipError_t e_ = (expr);                                                              \
        if (e_ != hipSuccess) return fail(kHipError, "HIP error in %s: %s", #expr, hipGetErrorString(e_)); \
        return kOk;                                                                          \
    } while (0)
#define MX_CHECK(cond, ...)                              \
    do {                                                 \
        if (!(cond)) return fail(kInvalid, __VA_ARGS__); \
    } while (0)
#define MX_DTYPE(dtype) MX_CHECK((dtype) == kFP32 || (dtype) == kBF16, "dtype must be fp32 or bf16")

int check_recurrence(const decdec_recurrence* p) {
    MX_CHECK(p != nullptr && p->proj && p->state && p->pos, "null pointer argument");
    MX_CHECK(p->heads >= 1 && p->kv_heads >= 1 && p->heads % p->kv_heads == 0, "heads (%u) must be a multiple of kv_heads (%u)", p->heads, p->kv_heads);
    MX_CHECK(p->dim >= 1 && p->dim <= 256, "dim must be 1 .. 256, got %u", p->dim);
    MX_CHECK(p->vdim >= 1 && p->vdim <= 4096, "vdim must be 1 .. 4096, got %u", p->vdim);
    const uint32_t nqk = p->kv_heads * p->dim, nv = p->heads * p->vdim;
    MX_CHECK(p->off_q + nqk <= p->ld && p->off_k + nqk <= p->ld && p->off_v + nv <= p->ld, "projection offsets exceed the row");
    if (p->delta) {
        MX_CHECK(p->conv_q && p->conv_k && p->conv_v && p->ring && (p->channel || (p->A_log && p->dt_bias)), "null pointer argument");
        MX_CHECK(p->taps >= 1 && p->taps <= 64, "taps must be 1 .. 64, got %u", p->taps);
        MX_CHECK((p->channel || p->off_a + p->heads <= p->ld) && p->off_b + p->heads <= p->ld, "projection offsets exceed the row");
    } else {
        MX_CHECK((p->channel || p->decay != nullptr) && p->kv_heads == p->heads, "a plain recurrence needs decays and as many key as value heads");
    }
    if (p->channel) {
        MX_CHECK(p->rate && p->a_bias && (p->a_sign == 1.f || p->a_sign == -1.f), "decays per channel need rates, a bias and a sign");
        MX_CHECK(p->rank_a >= 1 && p->rank_a <= kMaxRank && p->off_a + p->rank_a <= p->ld, "the decay's rank must be 1 .. %u and fit the row", kMaxRank);
        MX_CHECK(p->g2 == nullptr || (p->rank_g >= 1 && p->rank_g <= kMaxRank && p->off_g + p->rank_g <= p->ld), "the gate's rank must be 1 .. %u and fit the row", kMaxRank);
    } else {
        MX_CHECK(p->g2 == nullptr, "a low-rank gate goes with decays per channel");
    }
    return kOk;
}

int check_latent(const decdec_latent* p) {
    MX_CHECK(p != nullptr && p->proj && p->norm && p->cache && p->pos && p->cos_table && p->sin_table, "null pointer argument");
    MX_CHECK(p->heads >= 1 && p->dim >= 2 && p->dim % 2 == 0 && p->rot >= 2 && p->rot % 2 == 0, "dim and rot must be even");
    MX_CHECK(p->dim + p->rot <= 320, "dim + rot must not exceed 320, got %u", p->dim + p->rot);
    MX_CHECK(p->vdim >= 1 && p->vdim <= 256, "vdim must be 1 .. 256, got %u", p->vdim);
    MX_CHECK(p->rank >= 1 && p->rank + p->rot <= 640, "rank + rot must not exceed 640, got %u", p->rank + p->rot);
    MX_CHECK(p->max_seq >= 1, "empty cache");
    MX_CHECK(p->off_q + p->heads * (p->dim + p->rot) <= p->ld && p->off_c + p->rank + p->rot <= p->ld, "projection offsets exceed the row");
    MX_CHECK(((uintptr_t)p->cache % 16) == 0, "cache must be 16-byte aligned");
    return kOk;
}

int check_grouped(const decdec_grouped* p) {
    MX_CHECK(p != nullptr && p->proj && p->keys && p->values && p->pos, "null pointer argument");
    MX_CHECK(p->heads >= 1 && p->kv_heads >= 1 && p->heads % p->kv_heads == 0, "heads (%u) must be a multiple of kv_heads (%u)", p->heads, p->kv_heads);
    MX_CHECK(p->heads <= 65535, "too many heads");
    MX_CHECK(p->dim >= 1 && p->dim <= 320, "dim must be 1 .. 320, got %u", p->dim);
    MX_CHECK(p->vdim >= 1 && p->vdim <= 256, "vdim must be 1 .. 256, got %u", p->vdim);
    MX_CHECK(p->rot % 2 == 0 && p->rot <= p->dim && (p->rot == 0 || (p->cos_table && p->sin_table)), "rot must be even, at most dim, and have tables");
    MX_CHECK(p->max_seq >= 64 && p->max_seq % 64 == 0, "the cache must hold a multiple of 64 positions");
    MX_CHECK(p->off_q + p->heads * p->dim <= p->ld && p->off_k + p->kv_heads * p->dim <= p->ld && p->off_v + p->kv_heads * p->vdim <= p->ld &&
             (!p->gated || p->off_g + p->heads <= p->ld), "projection offsets exceed the row");
    MX_CHECK(((uintptr_t)p->keys % 16) == 0 && ((uintptr_t)p->values % 16) == 0, "the cache must be 16-byte aligned");
    return kOk;
}

}  // namespace

extern "C" {

const char* decdec_mixers_last_error(void) { return g_error.c_str(); }

int decdec_mix_gemv(const void* weight, const void* x, void* out, const void* act, uint32_t act_rows, int act_kind, float scale,
                    int dtype, uint32_t N, uint32_t K, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(weight && x && out && N >= 1 && K >= 1, "null pointer or empty size");
    MX_CHECK(act_kind == DECDEC_ACT_XIELU || act_kind == DECDEC_ACT_GELU_TANH, "unknown activation");
    MX_CHECK(act_rows <= N && (act_rows == 0 || act_kind != DECDEC_ACT_XIELU || act != nullptr), "act_rows needs act and at most N rows");
    MX_HIP(launch_mix_gemv(dtype, weight, x, out, act, act_rows, act_kind, scale, N, K, (hipStream_t)stream));
}

int decdec_mix_embed(const void* table, const int64_t* tokens, float* x, void* x_e, const decdec_tanh_norm* norm, int dtype,
                     uint32_t rows, uint32_t vocab, uint32_t dim, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(table && tokens && x && vocab >= 1 && dim >= 1, "null pointer or empty size");
    MX_CHECK(norm == nullptr || (x_e && norm->alpha && norm->weight && norm->bias), "a norm needs its tensors and an output");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_embed(dtype, table, (const long long*)tokens, x, x_e, norm, rows, vocab, dim, (hipStream_t)stream));
}

int decdec_mix_residual_tanh(float* x, const void* y, const decdec_tanh_norm* norm, void* out, int dtype, uint32_t rows,
                             uint32_t dim, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(x && out && norm && norm->alpha && norm->weight && norm->bias && dim >= 1, "null pointer or empty size");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_residual_tanh(dtype, x, y, *norm, out, rows, dim, (hipStream_t)stream));
}

int decdec_mix_gated_residual(float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias, const void* weight,
                              void* x_e, const void* final_weight, void* final_out, int dtype, uint32_t rows, uint32_t dim,
                              float eps, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(x && y && weight && dim >= 1, "null pointer or empty size");
    MX_CHECK(gate == nullptr || (bias != nullptr && gate_ld >= dim), "a gate needs a bias and rows of at least dim elements");
    MX_CHECK((final_weight == nullptr) == (final_out == nullptr), "final_weight and final_out go together");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_gated_residual(dtype, x, y, gate, gate_ld, bias, weight, x_e, final_weight, final_out, rows, dim, eps, (hipStream_t)stream));
}

int decdec_mix_rmsnorm(const float* x, const void* weight, void* out, int dtype, uint32_t rows, uint32_t dim, float eps, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(x && weight && out && dim >= 1, "null pointer or empty size");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_rmsnorm(dtype, x, weight, out, rows, dim, eps, (hipStream_t)stream));
}

int decdec_mix_activation(const void* in, uint32_t ld, const void* act, int act_kind, void* out, int dtype, uint32_t rows, uint32_t n,
                          void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(act_kind == DECDEC_ACT_XIELU || act_kind == DECDEC_ACT_GELU_TANH, "unknown activation");
    MX_CHECK(in && (act || act_kind != DECDEC_ACT_XIELU) && out && n >= 1 && ld >= n, "null pointer or bad size");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_activation(dtype, in, ld, act, act_kind, out, rows, n, (hipStream_t)stream));
}

int decdec_mix_group_norm_gate(const float* o, const void* gate, uint32_t ld, const void* weight, void* out, uint32_t out_ld, int dtype,
                               uint32_t rows, uint32_t groups, uint32_t n, float eps, int gate_kind, float scale, void* stream) {
    MX_DTYPE(dtype);
    MX_CHECK(o && gate && weight && out && groups >= 1 && groups <= 65535 && n >= 1 && (uint64_t)ld >= (uint64_t)groups * n &&
             (uint64_t)out_ld >= (uint64_t)groups * n, "null pointer or bad size");
    MX_CHECK(gate_kind == DECDEC_GATE_SIGMOID || gate_kind == DECDEC_GATE_SILU, "unknown gate");
    if (rows == 0) return kOk;
    MX_HIP(launch_mix_group_norm_gate(dtype, o, gate, ld, weight, out, out_ld, rows, groups, n, eps, gate_kind, scale, (hipStream_t)stream));
}

int decdec_mix_recurrence_step_fuses(uint32_t dim, uint32_t vdim) { return recurrence_step_fuses(dim, vdim) ? 1 : 0; }

int decdec_mix_recurrence_step(const decdec_recurrence* p, float* o, void* out, const void* norm_weight, float eps, int gate_kind,
                               int dtype, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_recurrence(p)) return rc;
    MX_CHECK(o != nullptr || out != nullptr, "null pointer argument");
    if (out != nullptr) {
        MX_CHECK(norm_weight != nullptr && recurrence_step_fuses(p->dim, p->vdim), "the normed read-out needs a head per workgroup");
        MX_CHECK(p->g2 != nullptr || p->off_g + p->heads * p->vdim <= p->ld, "projection offsets exceed the row");
    }
    MX_CHECK(!p->channel || p->a2 != nullptr, "null pointer argument");
    MX_HIP(launch_recurrence_step(dtype, *p, o, out, norm_weight, eps, gate_kind, (hipStream_t)stream));
}

uint64_t decdec_mix_recurrence_workspace(const decdec_recurrence* p, uint32_t rows) { return (uint64_t)recurrence_workspace(*p, rows); }

int decdec_mix_recurrence_rows(const decdec_recurrence* p, float* o, void* workspace, uint64_t workspace_bytes, int dtype,
                               uint32_t rows, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_recurrence(p)) return rc;
    MX_CHECK(o && workspace && ((uintptr_t)workspace % 16) == 0, "null or unaligned pointer argument");
    MX_CHECK(workspace_bytes >= recurrence_workspace(*p, rows), "workspace too small");
    MX_CHECK(!p->channel || (p->a && ((uintptr_t)p->a % 16) == 0), "null or unaligned pointer argument");
    MX_CHECK(rows <= (1u << 20) && p->heads <= 65535, "too many rows or heads");
    if (rows == 0) return kOk;
    MX_HIP(launch_recurrence_rows(dtype, *p, o, workspace, rows, (hipStream_t)stream));
}

int decdec_mix_grouped_append(const decdec_grouped* p, void* q_out, int dtype, uint32_t rows, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_grouped(p)) return rc;
    MX_CHECK(q_out != nullptr && ((uintptr_t)q_out % 16) == 0, "null or unaligned pointer argument");
    MX_CHECK((uint64_t)rows * (p->heads + p->kv_heads) < (1ull << 32), "too many rows");
    if (rows == 0) return kOk;
    MX_HIP(launch_grouped_append(dtype, *p, q_out, rows, (hipStream_t)stream));
}

int decdec_mix_grouped_attention(const decdec_grouped* p, const void* q, void* out, int dtype, uint32_t start, uint32_t rows, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_grouped(p)) return rc;
    MX_CHECK(q && out && ((uintptr_t)q % 16) == 0, "null or unaligned pointer argument");
    MX_CHECK((uint64_t)start + rows <= p->max_seq, "%u + %u positions do not fit a cache of %u", start, rows, p->max_seq);
    MX_CHECK(p->out_ld >= p->heads * p->vdim, "out_ld too small");
    if (rows == 0) return kOk;
    MX_HIP(launch_grouped_attention(dtype, *p, q, out, start, rows, (hipStream_t)stream));
}

uint64_t decdec_mix_grouped_step_workspace(const decdec_grouped* p) { return (uint64_t)grouped_step_workspace(*p); }

int decdec_mix_grouped_step(const decdec_grouped* p, void* out, void* workspace, uint64_t workspace_bytes, int dtype, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_grouped(p)) return rc;
    MX_CHECK(out && workspace && p->kv_heads <= 65535, "null pointer argument or too many heads");
    MX_CHECK(workspace_bytes >= grouped_step_workspace(*p), "workspace too small");
    MX_HIP(launch_grouped_step(dtype, *p, out, workspace, (hipStream_t)stream));
}

int decdec_mix_latent_append(const decdec_latent* p, void* q_out, int dtype, uint32_t rows, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_latent(p)) return rc;
    MX_CHECK(q_out != nullptr, "null pointer argument");
    if (rows == 0) return kOk;
    MX_HIP(launch_latent_append(dtype, *p, q_out, rows, (hipStream_t)stream));
}

int decdec_mix_latent_attention(const decdec_latent* p, const void* q, const void* k, const void* vt, uint32_t vt_ld, void* out,
                                int dtype, uint32_t start, uint32_t rows, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_latent(p)) return rc;
    MX_CHECK(q && k && vt && out, "null pointer argument");
    MX_CHECK(((uintptr_t)q % 16) == 0 && ((uintptr_t)k % 16) == 0 && ((uintptr_t)vt % 16) == 0, "q, k and vt must be 16-byte aligned");
    MX_CHECK((uint64_t)start + rows <= p->max_seq, "%u + %u positions do not fit a cache of %u", start, rows, p->max_seq);
    MX_CHECK(vt_ld % 64 == 0 && vt_ld >= start + rows, "vt_ld must be a multiple of 64 and hold every key");
    MX_CHECK(p->heads <= 65535, "too many heads");
    if (rows == 0) return kOk;
    MX_HIP(launch_latent_attention(dtype, *p, q, k, vt, vt_ld, out, start, rows, (hipStream_t)stream));
}

uint64_t decdec_mix_latent_step_workspace(const decdec_latent* p) { return (uint64_t)latent_step_workspace(*p); }

int decdec_mix_latent_step(const decdec_latent* p, void* out, void* workspace, uint64_t workspace_bytes, int dtype, void* stream) {
    MX_DTYPE(dtype);
    if (int rc = check_latent(p)) return rc;
    MX_CHECK(out && workspace && p->uk && p->uv, "null pointer argument");
    MX_CHECK(((uintptr_t)p->uk % 16) == 0 && ((uintptr_t)p->uv % 16) == 0, "uk and uv must be 16-byte aligned");
    MX_CHECK(workspace_bytes >= latent_step_workspace(*p), "workspace too small");
    MX_HIP(launch_latent_step(dtype, *p, out, workspace, (hipStream_t)stream));
}

}  // extern "C"
