/* C ABI of libdecdec_mixers.so: the layers of decoders that are not a plain attention + gated-MLP stack -- decayed and
 * gated-delta linear recurrences, latent attention, gated residuals with a norm on the sublayer's output, xIELU.
 *
 * Conventions.  Every function enqueues on `stream` (a hipStream_t) and returns 0, or a non-zero status whose message
 * decdec_mixers_last_error() gives.  dtype: 0 = fp32, 2 = bf16 (the storage type of weights and activations, "E"
 * below); sums, norms, gates, attention scores and weights, recurrent states and the residual stream are fp32 in both.
 * `pos` points at one int64 in device memory: the position of the first token of the call, so that a captured decode
 * step can be replayed unchanged.  A call whose first position is 0 starts from an empty state whatever the state
 * memory holds.  Rows of projected inputs are read at offsets into one array of row stride `ld` (elements). */
#ifndef DECDEC_MIXERS_H
#define DECDEC_MIXERS_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum { DECDEC_GATE_SIGMOID = 0, DECDEC_GATE_SILU = 1 };

const char* decdec_mixers_last_error(void);

/* out[n] = W[n] . x for one token (W [N][K] row-major, x [K], out [N], all E; fp32 accumulation).  Rows below act_rows
 * pass xIELU with the two numbers act[0..1] (E, may be NULL when act_rows is 0). */
int decdec_mix_gemv(const void* weight, const void* x, void* out, const void* act, uint32_t act_rows, int dtype,
                    uint32_t N, uint32_t K, void* stream);
/* x[r] = table[tokens[r]] in fp32, and once more as E in x_e (may be NULL).  tokens outside the table read row 0. */
int decdec_mix_embed(const void* table, const int64_t* tokens, float* x, void* x_e, int dtype, uint32_t rows,
                     uint32_t vocab, uint32_t dim, void* stream);
/* Per row: x += rms_norm(y * sigmoid(gate + bias)) * weight; x_e (may be NULL) receives x as E.  gate may be NULL (no
 * gate; bias is not read then).  final_weight / final_out (both or neither): final_out = rms_norm(x) * final_weight. */
int decdec_mix_gated_residual(float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias,
                              const void* weight, void* x_e, const void* final_weight, void* final_out, int dtype,
                              uint32_t rows, uint32_t dim, float eps, void* stream);
/* out[r] = rms_norm(x[r]) * weight, fp32 in, E out. */
int decdec_mix_rmsnorm(const float* x, const void* weight, void* out, int dtype, uint32_t rows, uint32_t dim, float eps,
                       void* stream);
/* out[r][i] = xIELU(in[r * ld + i]), i < n, with softplus of act[0..1] as the two coefficients. */
int decdec_mix_xielu(const void* in, uint32_t ld, const void* act, void* out, int dtype, uint32_t rows, uint32_t n,
                     void* stream);
/* Read-out of a recurrence: per row, groups of n neighbouring elements are RMS-normed, multiplied by weight (indexed
 * by position in the group) and by the gate function of gate[r * ld + i].  o fp32 [rows][groups * n], out E. */
int decdec_mix_group_norm_gate(const float* o, const void* gate, uint32_t ld, const void* weight, void* out, int dtype,
                               uint32_t rows, uint32_t groups, uint32_t n, float eps, int gate_kind, void* stream);

/* One linear-recurrence layer.  State per head: dim x vdim fp32.
 *   delta = 0: S <- decay_h S + k v^T, o = S^T q with q, k, v = silu of the projections.
 *   delta = 1: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with q, k, v = silu of a short causal
 *              convolution of the projections, q and k unit vectors per head, q scaled by dim^-1/2,
 *              beta = sigmoid(b), g = exp(-exp(A_log) softplus(a + dt_bias)). */
typedef struct {
    const void* proj;            /* E [rows][ld] */
    uint32_t ld, off_q, off_k, off_v, off_g, off_a, off_b;
    uint32_t heads, kv_heads, dim, vdim, taps;
    uint32_t delta;
    const float* decay;          /* fp32 [heads][65]: decay^0 .. decay^64 (delta = 0) */
    const void* conv_q;          /* E [channels][taps] (delta = 1) */
    const void* conv_k;
    const void* conv_v;
    const void* A_log;           /* E [heads] */
    const void* dt_bias;
    void* ring;                  /* E [taps][2 kv_heads dim + heads vdim]: projections of the last tokens, slot = position % taps */
    float* state;                /* fp32 [heads][dim][vdim] */
    const int64_t* pos;
} decdec_recurrence;
/* One token.  Writes the read-out as fp32 to o [heads * vdim] (o may be NULL when out is given) or, with out != NULL,
 * normed per head, weighted and gated (gate function of proj[off_g + i]) as E: only where one workgroup holds a whole
 * head, see decdec_mix_recurrence_step_fuses. */
int decdec_mix_recurrence_step(const decdec_recurrence* p, float* o, void* out, const void* norm_weight, float eps,
                               int gate_kind, int dtype, void* stream);
int decdec_mix_recurrence_step_fuses(uint32_t dim, uint32_t vdim);
/* `rows` tokens in chunks of 64; o fp32 [rows][heads * vdim].  workspace: decdec_mix_recurrence_workspace bytes. */
uint64_t decdec_mix_recurrence_workspace(const decdec_recurrence* p, uint32_t rows);
int decdec_mix_recurrence_rows(const decdec_recurrence* p, float* o, void* workspace, uint64_t workspace_bytes, int dtype,
                               uint32_t rows, void* stream);

/* Latent attention.  cache E [max_seq][rank + rot]: the normed latent and the rotated shared key part of every token.
 * proj rows hold the queries ([heads][dim + rot]) at off_q and the down projection (rank + rot) at off_c. */
typedef struct {
    const void* proj;
    uint32_t ld, off_q, off_c;
    uint32_t heads, dim, rot, vdim, rank, max_seq;
    float eps, scale;
    const void* norm;            /* E [rank] */
    const void* uk;              /* E [heads * dim][rank] */
    const void* uv;              /* E [heads * vdim][rank] */
    const void* sink;            /* E [heads] or NULL */
    const float* cos_table;      /* fp32 [max_seq][rot / 2], magnitude included */
    const float* sin_table;
    void* cache;
    const int64_t* pos;
} decdec_latent;
/* Norms, rotates and appends `rows` tokens to the cache; q_out E [rows][heads][dim + rot] receives the rotated queries. */
int decdec_mix_latent_append(const decdec_latent* p, void* q_out, int dtype, uint32_t rows, void* stream);
/* Causal attention of `rows` queries (from `start`, known to the host) over start + rows keys: k E [keys][heads * dim]
 * unrotated keys, vt E [heads * vdim][vt_ld] transposed values, rotated parts from the cache; out E [rows][heads * vdim].
 * Both k and vt hold at least start + rows keys (vt rounded up to a multiple of 64). */
int decdec_mix_latent_attention(const decdec_latent* p, const void* q, const void* k, const void* vt, uint32_t vt_ld,
                                void* out, int dtype, uint32_t start, uint32_t rows, void* stream);
/* One token, the up projections absorbed: append, attend the latents directly, out E [heads * vdim]. */
uint64_t decdec_mix_latent_step_workspace(const decdec_latent* p);
int decdec_mix_latent_step(const decdec_latent* p, void* out, void* workspace, uint64_t workspace_bytes, int dtype,
                           void* stream);

#ifdef __cplusplus
}
#endif
#endif
