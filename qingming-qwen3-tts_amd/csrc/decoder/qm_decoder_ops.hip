// qm_decoder_ops.hip — C ABI of the decoder language models' operators.
#include "../qm_host.h"
#include "qm_decoder_ops.h"

extern "C" int32_t qm_residual_norm_rows(const qm_residual_norm* op, int32_t rows, int32_t f32, void* hip_stream) {
    return op ? qm::launch_residual_norm(*op, rows, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int32_t qm_gated_norm_rows(const qm_gated_norm* op, int32_t rows, int32_t f32, void* hip_stream) {
    return op ? qm::launch_gated_norm(*op, rows, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int32_t qm_decoder_linear_rows(const qm_decoder_linear* linears, int32_t count, int32_t rows, int32_t f32, void* hip_stream) {
    if (!linears) return QM_ERR_NULL;
    if (count < 1 || count > qm::kDecGroups) return QM_ERR_ARGUMENT;
    qm::DecLinearParams prm = {};
    for (int i = 0; i < count; ++i) prm.group[i] = linears[i];
    prm.groups = count;
    prm.rows = rows;
    return qm::launch_decoder_linears(prm, f32, static_cast<hipStream_t>(hip_stream));
}
extern "C" int32_t qm_chunk_attention_rows(const qm_chunk_attention* op, int32_t f32, void* hip_stream) {
    return op ? qm::launch_chunk_attention(*op, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int32_t qm_decay_attention_rows(const qm_decay_attention* op, void* hip_stream) {
    return op ? qm::launch_decay_attention(*op, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int32_t qm_general_delta_rows(const qm_general_delta* op, void* hip_stream) {
    return op ? qm::launch_general_delta(*op, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int64_t qm_decay_attention_scratch_floats(int32_t rows, int32_t heads, int32_t dim, int32_t vdim) {
    return qm::decay_scratch_floats(rows, heads, dim, vdim);
}
extern "C" int64_t qm_general_delta_scratch_floats(int32_t rows, int32_t heads, int32_t dim) {
    return qm::delta_scratch_floats(rows, heads, dim);
}
