// Launch interface between the mixer kernels and their C ABI.
#pragma once
#include <hip/hip_runtime.h>
#include "../../include/decdec_mixers.h"
#include "common.h"

namespace decdec {

constexpr uint32_t kChunkRows = 64;        // tokens per chunk of a recurrence
constexpr uint32_t kMaxRank = 1024;        // of the low-rank maps of a recurrence

// Lets a kernel take more than 64 KB of dynamic LDS.
template <auto Kernel>
inline hipError_t allow_lds(size_t bytes) {
    static thread_local size_t allowed = 64 * 1024;
    if (bytes <= allowed) return hipSuccess;
    const hipError_t e = hipFuncSetAttribute((const void*)Kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    if (e == hipSuccess) allowed = bytes;
    return e;
}

// Operands of the tiled attention kernel, strides in elements.  A key row is `dim` elements of the (shared) head's own and
// `rot` elements all heads share.
struct TileAttention {
    const void* q;              // [rows][heads][dim + rot]
    const void* k;              // kv head k_head apart, key k_row apart
    const void* shared;         // key shared_row apart, or null (rot = 0)
    const void* vt;             // [kv heads * vdim][vt_ld]
    const void* sink;           // E [heads], or null: sink_score for all heads (minus infinity: no sink)
    const void* gate;           // rows gate_ld apart, one number per head, through a sigmoid; or null
    void* out;                  // rows out_ld apart, [heads][vdim]
    size_t k_head, k_row;
    uint32_t shared_row, vt_ld, gate_ld, out_ld, heads, share, dim, rot, vdim;
    float scale, sink_score, out_scale;
};

hipError_t launch_mix_gemv(int dt, const void* w, const void* x, void* out, const void* act, uint32_t act_rows, int act_kind,
                           float scale, uint32_t N, uint32_t K, hipStream_t s);
hipError_t launch_mix_embed(int dt, const void* table, const long long* tokens, float* x, void* xe, const decdec_tanh_norm* norm,
                            uint32_t rows, uint32_t vocab, uint32_t dim, hipStream_t s);
hipError_t launch_mix_residual_tanh(int dt, float* x, const void* y, const decdec_tanh_norm& norm, void* out, uint32_t rows,
                                    uint32_t dim, hipStream_t s);
hipError_t launch_mix_gated_residual(int dt, float* x, const void* y, const void* gate, uint32_t gate_ld, const void* bias,
                                     const void* weight, void* xe, const void* fw, void* fo, uint32_t rows, uint32_t dim,
                                     float eps, hipStream_t s);
hipError_t launch_mix_rmsnorm(int dt, const float* x, const void* weight, void* out, uint32_t rows, uint32_t dim, float eps,
                              hipStream_t s);
hipError_t launch_mix_activation(int dt, const void* in, uint32_t ld, const void* act, int kind, void* out, uint32_t rows,
                                 uint32_t n, hipStream_t s);
hipError_t launch_mix_group_norm_gate(int dt, const float* o, const void* gate, uint32_t ld, const void* weight, void* out,
                                      uint32_t out_ld, uint32_t rows, uint32_t groups, uint32_t n, float eps, int kind,
                                      float scale, hipStream_t s);
bool recurrence_step_fuses(uint32_t dim, uint32_t vdim);
hipError_t launch_recurrence_step(int dt, const decdec_recurrence& p, float* o, void* out, const void* nw, float eps, int kind,
                                  hipStream_t s);
size_t recurrence_workspace(const decdec_recurrence& p, uint32_t rows);
hipError_t launch_recurrence_rows(int dt, const decdec_recurrence& p, float* o, void* ws, uint32_t rows, hipStream_t s);
hipError_t launch_tile_attention(int dt, const TileAttention& p, uint32_t start, uint32_t rows, hipStream_t s);
hipError_t launch_grouped_append(int dt, const decdec_grouped& p, void* q_out, uint32_t rows, hipStream_t s);
hipError_t launch_grouped_attention(int dt, const decdec_grouped& p, const void* q, void* out, uint32_t start, uint32_t rows,
                                    hipStream_t s);
size_t grouped_step_workspace(const decdec_grouped& p);
hipError_t launch_grouped_step(int dt, const decdec_grouped& p, void* out, void* ws, hipStream_t s);
hipError_t launch_latent_append(int dt, const decdec_latent& p, void* q_out, uint32_t rows, hipStream_t s);
hipError_t launch_latent_attention(int dt, const decdec_latent& p, const void* q, const void* k, const void* vt, uint32_t vt_ld,
                                   void* out, uint32_t start, uint32_t rows, hipStream_t s);
size_t latent_step_workspace(const decdec_latent& p);
hipError_t launch_latent_step(int dt, const decdec_latent& p, void* out, void* ws, hipStream_t s);

}  // namespace decdec
