/* C ABI of libdecdec_mixers.so: the layers of decoders that are not a plain attention + gated-MLP stack -- decayed and
 * gated-delta linear recurrences with decays per head or per key channel, latent attention, grouped attention with a sink and
 * gated heads, gated residuals with a norm on the sublayer's output, residuals with a dynamic-tanh norm ahead of the next
 * sublayer, xIELU and GELU.
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
enum { DECDEC_ACT_XIELU = 0, DECDEC_ACT_GELU_TANH = 1 };

/* Dynamic tanh: tanh(alpha x) * weight + bias, alpha one E in device memory, weight and bias E [dim]. */
typedef struct {
    const void* alpha;
    const void* weight;
    const void* bias;
} decdec_tanh_norm;

const char* decdec_mixers_last_error(void);

/* out[n] = scale * W[n] . x for one token (W [N][K] row-major, x [K], out [N], all E; fp32 accumulation).  Rows below
 * act_rows pass the activation act_kind: xIELU with the two numbers act[0..1] (E), or the tanh form of GELU (act is not
 * read).  act may be NULL when act_rows is 0. */
int decdec_mix_gemv(const void* weight, const void* x, void* out, const void* act, uint32_t act_rows, int act_kind,
                    float scale, int dtype, uint32_t N, uint32_t K, void* stream);
/* x[r] = table[tokens[r]] in fp32, and once more as E in x_e (may be NULL), there through `norm` unless that is NULL.
 * tokens outside the table read row 0. */
int decdec_mix_embed(const void* table, const int64_t* tokens, float* x, void* x_e, const decdec_tanh_norm* norm, int dtype,
                     uint32_t rows, uint32_t vocab, uint32_t dim, void* stream);
/* Per row: x += y (E; may be NULL); out (E) = norm(x). */
int decdec_mix_residual_tanh(float* x, const void* y, const decdec_tanh_norm* norm, void* out, int dtype, uint32_t rows,
                             uint32_t dim, void* stream);
/* Per row: x += rms_norm(y * sigmoid(gate + bias)) * weight; x_e (may be NULL) receives x as E.  gate may be NULL (no
 * gate; bias is not read then).  final_weight / final_out (both or neither): final_out = rms_norm(x) * final_weight. */
int decdec_mix_gated_residual(float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias,
                              const void* weight, void* x_e, const void* final_weight, void* final_out, int dtype,
                              uint32_t rows, uint32_t dim, float eps, void* stream);
/* out[r] = rms_norm(x[r]) * weight, fp32 in, E out. */
int decdec_mix_rmsnorm(const float* x, const void* weight, void* out, int dtype, uint32_t rows, uint32_t dim, float eps,
                       void* stream);
/* out[r][i] = activation(in[r * ld + i]), i < n: xIELU with softplus of act[0..1] as the two coefficients, or the tanh
 * form of GELU (act is not read).  out may be `in` where ld is n. */
int decdec_mix_activation(const void* in, uint32_t ld, const void* act, int act_kind, void* out, int dtype, uint32_t rows,
                          uint32_t n, void* stream);
/* Read-out of a recurrence: per row, groups of n neighbouring elements are RMS-normed, multiplied by weight (indexed
 * by position in the group), by the gate function of gate[r * ld + i] and by scale.  o fp32 [rows][groups * n], out E, rows
 * out_ld apart. */
int decdec_mix_group_norm_gate(const float* o, const void* gate, uint32_t ld, const void* weight, void* out, uint32_t out_ld,
                               int dtype, uint32_t rows, uint32_t groups, uint32_t n, float eps, int gate_kind, float scale,
                               void* stream);

/* One linear-recurrence layer.  State per head: dim x vdim fp32.
 *   delta = 0: S <- decay_h S + k v^T, o = S^T q with q, k, v = silu of the projections.
 *   delta = 1: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with q, k, v = silu of a short causal
 *              convolution of the projections, q and k unit vectors per head, q scaled by dim^-1/2,
 *              beta = sigmoid(b), g = exp(-exp(A_log) softplus(a + dt_bias)).
 * channel = 1: the decays are one per head and key channel (a row of S) and come from a low-rank map of the projection a
 *              (rank_a elements at off_a): log g = -rate_h softplus(a_sign (A2 a + a_bias)).  With delta = 0, q, k and v are
 *              then the projections themselves, q scaled by dim^-1/2.  The read-out's gate may come from a low-rank map of
 *              rank_g elements at off_g (G2 != NULL). */
typedef struct {
    const void* proj;            /* E [rows][ld] */
    uint32_t ld, off_q, off_k, off_v, off_g, off_a, off_b;
    uint32_t heads, kv_heads, dim, vdim, taps;
    uint32_t delta, channel, rank_a, rank_g;
    float a_sign, out_scale;     /* out_scale: factor of the normed read-out of a one-token step */
    const float* decay;          /* fp32 [heads][65]: decay^0 .. decay^64 (delta = 0, channel = 0) */
    const void* conv_q;          /* E [channels][taps] (delta = 1) */
    const void* conv_k;
    const void* conv_v;
    const void* A_log;           /* E [heads] (delta = 1, channel = 0) */
    const void* dt_bias;
    const float* rate;           /* fp32 [heads] (channel = 1) */
    const float* a_bias;         /* fp32 [heads * dim] */
    const void* a2;              /* E [heads * dim][rank_a]: one-token steps apply it themselves */
    const void* g2;              /* E [heads * vdim][rank_g] or NULL */
    const float* a;              /* fp32 [rows][heads * dim]: a2 applied to the rows of several tokens */
    void* ring;                  /* E [taps][2 kv_heads dim + heads vdim]: projections of the last tokens, slot = position % taps */
    float* state;                /* fp32 [heads][dim][vdim] */
    const int64_t* pos;
} decdec_recurrence;
/* One token.  Writes the read-out as fp32 to o [heads * vdim] (o may be NULL when out is given) or, with out != NULL,
 * normed per head, weighted, gated (gate function of proj[off_g + i], or of G2's rows) and scaled as E: only where one workgroup holds a whole
 * head, see decdec_mix_recurrence_step_fuses. */
int decdec_mix_recurrence_step(const decdec_recurrence* p, float* o, void* out, const void* norm_weight, float eps,
                               int gate_kind, int dtype, void* stream);
int decdec_mix_recurrence_step_fuses(uint32_t dim, uint32_t vdim);
/* `rows` tokens in chunks of 64; o fp32 [rows][heads * vdim].  workspace: decdec_mix_recurrence_workspace bytes. */
uint64_t decdec_mix_recurrence_workspace(const decdec_recurrence* p, uint32_t rows);
int decdec_mix_recurrence_rows(const decdec_recurrence* p, float* o, void* workspace, uint64_t workspace_bytes, int dtype,
                               uint32_t rows, void* stream);

/* Grouped attention: heads / kv_heads query heads share a key / value head.  Queries and keys are RMS-normed per head over
 * dim (weights E [dim]; NULL: not normed), then the pairs (2i, 2i + 1) of their first `rot` elements are turned.  sink: a
 * valueless score in the softmax's denominator (minus infinity: none).  gated: the read-out of head h is multiplied by the
 * sigmoid of proj[off_g + h].  out_scale multiplies the read-out.  The cache holds keys by head and values transposed; the
 * key rows and value columns of positions to come are finite, and max_seq is a multiple of 64. */
typedef struct {
    const void* proj;
    uint32_t ld, off_q, off_k, off_v, off_g;
    uint32_t heads, kv_heads, dim, vdim, rot, max_seq, gated, out_ld;
    float eps, scale, sink, out_scale;
    const void* q_norm;
    const void* k_norm;
    const float* cos_table;      /* fp32 [max_seq][rot / 2] (may be NULL when rot is 0) */
    const float* sin_table;
    void* keys;                  /* E [kv_heads][max_seq][dim] */
    void* values;                /* E [kv_heads * vdim][max_seq] */
    const int64_t* pos;
} decdec_grouped;
/* Norms, rotates and appends `rows` tokens to the cache; q_out E [rows][heads][dim] receives the queries. */
int decdec_mix_grouped_append(const decdec_grouped* p, void* q_out, int dtype, uint32_t rows, void* stream);
/* Causal attention of `rows` queries (from `start`, known to the host) over start + rows cached keys; out E [rows][heads *
 * vdim], rows out_ld apart. */
int decdec_mix_grouped_attention(const decdec_grouped* p, const void* q, void* out, int dtype, uint32_t start, uint32_t rows,
                                 void* stream);
/* One token: append and attend, out E [heads * vdim]. */
uint64_t decdec_mix_grouped_step_workspace(const decdec_grouped* p);
int decdec_mix_grouped_step(const decdec_grouped* p, void* out, void* workspace, uint64_t workspace_bytes, int dtype,
                            void* stream);

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
