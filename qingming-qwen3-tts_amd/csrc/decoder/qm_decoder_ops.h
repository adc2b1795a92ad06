// qm_decoder_ops.h — launch parameters and launchers of the decoder language models' kernels, as the engine calls them.
// Every launcher checks its arguments on the host, enqueues on `stream` and returns a QM_* code.  `f32` chooses the
// activation type: 0 bf16, 1 fp32.
#pragma once

#include <hip/hip_runtime.h>

#include "../../../include/qm_attn.h"
#include "../../../include/qm_decoder.h"

namespace qm {

constexpr int kDecMaxWidth = 12288;       // columns of the residual stream (a block's threads hold a row)
constexpr int kDecMaxSplits = 64;         // key splits of one attention (a wave's lanes combine them)
constexpr int kDecMaxMerge = 4096;        // heads * key splits of one attention (their factors lie in LDS)
constexpr int kDecMaxHead = 256;          // channels of a head
constexpr int kAttentionMatrixRows = 16;  // rows from which bf16 attention goes to the matrix cores
constexpr int kChunkedRows = 16;          // rows from which a recurrence is computed in chunks (given scratch)
constexpr int kDecGroups = 3;             // linears in one launch
constexpr int kDotLdsMost = 159 * 1024;   // dynamic LDS of one block

// Linears of one launch.
struct DecLinearParams {
    qm_decoder_linear group[kDecGroups];
    int groups, rows;
};
using ResidualParams = qm_residual_norm;
using GatedNormParams = qm_gated_norm;
using AttentionPartials = qm_attention_partials;
using DecLinearGroup = qm_decoder_linear;
using ChunkAttentionParams = qm_chunk_attention;
using DecayAttentionParams = qm_decay_attention;
using DeltaParams = qm_general_delta;
using LatentRowsParams = qm_latent_rows;
using LatentAttentionParams = qm_latent_attention;
using ExpertParams = qm_experts;
constexpr int kLatentKeys = 64;           // keys per pass of the attention over latents; its splits are whole passes
constexpr int kLatentMaxRank = 1024;      // channels of a latent
constexpr int kLatentMaxRotary = 256;     // channels of the key part that heads share
constexpr int kExpertsMost = 1024;
constexpr int kDecayChunk = QM_DECAY_CHUNK;
constexpr int kDecayPowers = QM_DECAY_POWERS;

// float4s of a row that each of a block's 256 threads holds: the kernels' choices for a row of ld columns.
inline int row_vectors(int64_t ld) { return ld <= 1024 ? 1 : ld <= 2048 ? 2 : ld <= 4096 ? 4 : 12; }

// Whether the kernels take these arguments.
int32_t check_residual(const ResidualParams& prm);
int32_t check_attention(const ChunkAttentionParams& prm);
int32_t check_decay_attention(const DecayAttentionParams& prm);
int32_t launch_residual_norm(const ResidualParams& prm, int rows, int f32, hipStream_t stream);
int32_t launch_gated_norm(const GatedNormParams& prm, int rows, int f32, hipStream_t stream);
// Many rows of bf16 go to the matrix cores (linears of one launch in one grid, a gate/up pair in its own), few rows and
// fp32 to the streaming kernel.
int32_t launch_decoder_linears(const DecLinearParams& prm, int f32, hipStream_t stream);
// Rotation and cache write, then the attention.
int32_t launch_chunk_attention(const ChunkAttentionParams& prm, int f32, hipStream_t stream);
int32_t launch_chunk_attention_mfma(const ChunkAttentionParams& prm, hipStream_t stream);
int32_t launch_decay_attention(const DecayAttentionParams& prm, hipStream_t stream);
// Floats of scratch with which a pass of `rows` tokens is computed in chunks (0: it is not).
int64_t decay_scratch_floats(int rows, int heads, int dim, int vdim);
int64_t delta_scratch_floats(int rows, int heads, int dim);
bool delta_chunks_fit(const DeltaParams& prm);
int32_t launch_decay_chunks(const DecayAttentionParams& prm, hipStream_t stream);
int32_t launch_delta_chunks(const DeltaParams& prm, hipStream_t stream);
int32_t launch_general_delta(const DeltaParams& prm, hipStream_t stream);
int32_t launch_latent_rows(const LatentRowsParams& prm, int f32, hipStream_t stream);
// keep: what the step's token leaves in the cache, written by the launch that prepares the queries (NULL: it is there).
int32_t launch_latent_attention(const LatentAttentionParams& prm, const LatentRowsParams* keep, int f32, hipStream_t stream);
int32_t launch_latent_partials_mfma(const LatentAttentionParams& prm, hipStream_t stream);
bool latent_partials_fit_mfma(const LatentAttentionParams& prm);
int latent_q_stride(int kv_rank, int rot_dim);
int64_t expert_scratch_bytes(int rows, int experts, int top, int width_p, int ff_p, int f32);
int32_t launch_experts(const ExpertParams& prm, int f32, hipStream_t stream);

// ---- one token: a layer run in three launches -----------------------------------------------------------------------
// Residual sum and norm by every block for itself, then the linears that read it (row 0 of everything); the norm's output
// also goes to residual.h if that is given.
struct LayerInParams {
    ResidualParams residual;
    DecLinearParams linears;
};
// The output linears, each block preparing the input of its own: 0 as it is in memory, 1 the attention's key splits
// combined, 2 the gated norm, 3 a slice of fp32 values divided by its root mean square and weighted.
struct SliceNorm {
    const float* x;
    const float* weight;
    int n;
    float eps;
};
struct LayerOutParams {
    DecLinearParams linears;
    int input[kDecGroups];
    int chunk;                       // of the attention (input 1)
    AttentionPartials part;
    const int32_t* position_dev;
    GatedNormParams gated;           // (input 2)
    SliceNorm slice;                 // (input 3)
};
int32_t launch_layer_in(const LayerInParams& prm, int f32, hipStream_t stream);
// The attention (rotation and cache write included) beside the decayed linear attention, one token each.
int32_t launch_mixer_step(const ChunkAttentionParams& attention, const DecayAttentionParams& decay, int f32, hipStream_t stream);
int32_t launch_layer_out(const LayerOutParams& prm, int f32, hipStream_t stream);
// the id of the highest of `vocab` scores (lowest among equals)
int32_t launch_argmax(const float* scores, int vocab, int32_t* token, hipStream_t stream);
// step = the words below: the chosen token is put out and becomes the one to feed, the token that was fed the one before it,
// and the position moves on by `advance`
enum StepWord { kStepPosition, kStepBefore, kStepToken, kStepEmitted, kStepChosen, kStepWords };
int32_t launch_emit(int32_t* step, int32_t* out, int advance, hipStream_t stream);

}  // namespace qm
