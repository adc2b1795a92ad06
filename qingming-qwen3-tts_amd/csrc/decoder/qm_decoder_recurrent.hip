// qm_decoder_recurrent.hip — the decoder language models' recurrent mixers for gfx950: linear attention with a per-head
// decay and the generalized delta rule.  State and everything that enters it are fp32.
#include "../qm_host.h"
#include "qm_decoder_recurrent.h"

namespace qm {

template <int RD>
__global__ __launch_bounds__(kDecThreads) void decay_attention_kernel(DecayAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    decay_attention_block<RD>(prm, static_cast<int>(blockIdx.y), static_cast<int>(blockIdx.x), lds);
}

template <int RD>
__global__ __launch_bounds__(kDecThreads) void general_delta_kernel(DeltaParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    general_delta_block<RD>(prm, static_cast<int>(blockIdx.y), static_cast<int>(blockIdx.x), lds);
}

template <int RD>
__global__ __launch_bounds__(kDecThreads) void general_delta_step_kernel(DeltaParams prm) {
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) float lds[];
    general_delta_step<RD>(prm, static_cast<int>(blockIdx.y), static_cast<int>(blockIdx.x), lds);
}

template <int RD>
static int32_t decay_as(const DecayAttentionParams& prm, hipStream_t stream) {
    hipLaunchKernelGGL(decay_attention_kernel<RD>, dim3((prm.vdim + kRecColumns - 1) / kRecColumns, prm.heads), dim3(kDecThreads),
                       sizeof(float) * decay_lds_floats(RD), stream, prm);
    return launch_status();
}

int32_t check_decay_attention(const DecayAttentionParams& prm) {
    if (!prm.proj || !prm.powers || !prm.state || !prm.out) return QM_ERR_NULL;
    if (prm.rows < 0) return QM_ERR_ARGUMENT;
    if (prm.heads <= 0 || prm.heads > 65535 || prm.dim <= 0 || prm.vdim <= 0 || prm.dim > kDecMaxHead || prm.vdim > kDecMaxHead) return QM_ERR_GEOMETRY;
    if (prm.options & QM_DECAY_ROTARY) {
        if (prm.rot_dims < 0 || prm.rot_dims > prm.dim || prm.rot_dims % 2) return QM_ERR_GEOMETRY;
        if (prm.rot_dims > 0 && !prm.frequency) return QM_ERR_NULL;
        if (prm.position < 0) return QM_ERR_ARGUMENT;
    }
    return QM_OK;
}

int32_t launch_decay_attention(const DecayAttentionParams& prm, hipStream_t stream) {
    const int32_t rc = check_decay_attention(prm);
    if (rc != QM_OK || prm.rows == 0) return rc;
    if (prm.scratch && prm.rows >= kChunkedRows) return launch_decay_chunks(prm, stream);
    if (prm.dim <= 32) return decay_as<8>(prm, stream);
    if (prm.dim <= 64) return decay_as<16>(prm, stream);
    if (prm.dim <= 128) return decay_as<32>(prm, stream);
    return decay_as<64>(prm, stream);
}

template <int RD>
static int32_t delta_as(const DeltaParams& prm, hipStream_t stream) {
    const dim3 grid((prm.dim + kRecColumns - 1) / kRecColumns, prm.heads);
    if (prm.rows == 1) {
        hipLaunchKernelGGL(general_delta_step_kernel<RD>, grid, dim3(kDecThreads), sizeof(float) * delta_step_lds_floats(RD, prm.rank), stream, prm);
        return launch_status();
    }
    const int bytes = static_cast<int>(sizeof(float)) * delta_lds_floats(RD, prm.rank);
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(general_delta_kernel<RD>), kDotLdsMost, raised);
    if (rc != QM_OK) return rc;
    if (bytes > kDotLdsMost) return QM_ERR_GEOMETRY;
    hipLaunchKernelGGL(general_delta_kernel<RD>, grid, dim3(kDecThreads), bytes, stream, prm);
    return launch_status();
}

int32_t launch_general_delta(const DeltaParams& prm, hipStream_t stream) {
    if (!prm.proj || !prm.w2 || !prm.w0 || !prm.a_bias || !prm.state || !prm.out) return QM_ERR_NULL;
    if (prm.rows < 0) return QM_ERR_ARGUMENT;
    if (prm.heads <= 0 || prm.heads > 65535 || prm.dim <= 0 || prm.dim > kDecMaxHead || prm.rank <= 0 || prm.rank > 1024) return QM_ERR_GEOMETRY;
    if (prm.rows == 0) return QM_OK;
    if (prm.scratch && prm.rows >= kChunkedRows && delta_chunks_fit(prm)) return launch_delta_chunks(prm, stream);
    if (prm.dim <= 32) return delta_as<8>(prm, stream);
    if (prm.dim <= 64) return delta_as<16>(prm, stream);
    if (prm.dim <= 128) return delta_as<32>(prm, stream);
    return delta_as<64>(prm, stream);
}

}  // namespace qm
