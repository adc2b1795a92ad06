// qm_decoder_norm.hip — row operators around the decoder language models' mixers: the residual sum with the norm that
// reads it, and the gated norm behind a recurrent mixer.  One block of 256 threads per row; a row is a few tens of KB, so
// both are bound by memory latency for few rows and by bandwidth for a prompt.
#include "qm_decoder_device.h"
#include "../qm_host.h"

namespace qm {

template <class T, int NV>
__global__ __launch_bounds__(kDecThreads) void residual_norm_kernel(ResidualParams prm) {
    __shared__ float sh_red[16];
    const int row = static_cast<int>(blockIdx.x);
    residual_norm_row<T, NV>(prm, row, sh_red, static_cast<T*>(prm.h) + row * prm.ld_h, true);
}

template <class T>
__global__ __launch_bounds__(kDecThreads) void gated_norm_kernel(GatedNormParams prm) {
    __shared__ float sh_red[4];
    const int64_t row = blockIdx.x;
    gated_norm_row<T>(prm, row, sh_red, static_cast<T*>(prm.out) + row * prm.ld_out);
}

int32_t check_residual(const ResidualParams& prm) {
    if (prm.width <= 0 || prm.ld_h < prm.width || prm.terms < 0 || prm.terms > 3) return QM_ERR_ARGUMENT;
    if (!prm.norm_w || (!prm.x_in && (!prm.embed || !prm.tokens))) return QM_ERR_NULL;
    if (prm.ld_h % 4 || prm.ld_h > kDecMaxWidth) return QM_ERR_GEOMETRY;
    if (!prm.x_in && prm.buckets > 0 && !prm.bigram) return QM_ERR_NULL;
    if (prm.buckets < 0 || (prm.buckets > 0 && (prm.mul_prev < 0 || prm.mul_cur < 0))) return QM_ERR_ARGUMENT;
    for (int i = 0; i < prm.terms; ++i) {
        if (!prm.term[i].y) return QM_ERR_NULL;
        if (prm.term[i].ld < prm.ld_h || prm.term[i].ld % 4) return QM_ERR_GEOMETRY;
    }
    return QM_OK;
}

template <class T>
static int32_t residual_as(const ResidualParams& prm, int rows, hipStream_t stream) {
    switch (row_vectors(prm.ld_h)) {
        case 1: hipLaunchKernelGGL((residual_norm_kernel<T, 1>), dim3(rows), dim3(kDecThreads), 0, stream, prm); break;
        case 2: hipLaunchKernelGGL((residual_norm_kernel<T, 2>), dim3(rows), dim3(kDecThreads), 0, stream, prm); break;
        case 4: hipLaunchKernelGGL((residual_norm_kernel<T, 4>), dim3(rows), dim3(kDecThreads), 0, stream, prm); break;
        default: hipLaunchKernelGGL((residual_norm_kernel<T, 12>), dim3(rows), dim3(kDecThreads), 0, stream, prm); break;
    }
    return launch_status();
}

int32_t launch_residual_norm(const ResidualParams& prm, int rows, int f32, hipStream_t stream) {
    const int32_t rc = check_residual(prm);
    if (rc != QM_OK) return rc;
    if (rows < 0) return QM_ERR_ARGUMENT;
    if (!prm.h) return QM_ERR_NULL;
    if (rows == 0) return QM_OK;
    return f32 ? residual_as<float>(prm, rows, stream) : residual_as<uint16_t>(prm, rows, stream);
}

int32_t launch_gated_norm(const GatedNormParams& prm, int rows, int f32, hipStream_t stream) {
    if (rows < 0 || prm.groups <= 0 || prm.size <= 0 || prm.ld_out < static_cast<int64_t>(prm.groups) * prm.size) return QM_ERR_ARGUMENT;
    if (!prm.o || !prm.gate || !prm.out) return QM_ERR_NULL;
    if (rows == 0) return QM_OK;
    if (f32) hipLaunchKernelGGL(gated_norm_kernel<float>, dim3(rows), dim3(kDecThreads), 0, stream, prm);
    else hipLaunchKernelGGL(gated_norm_kernel<uint16_t>, dim3(rows), dim3(kDecThreads), 0, stream, prm);
    return launch_status();
}

}  // namespace qm
