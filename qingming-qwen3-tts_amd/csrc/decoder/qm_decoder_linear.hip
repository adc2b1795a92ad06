// qm_decoder_linear.hip — linears of the decoder language models for few token rows (a decode step, a short portion of a
// prompt) and for the 32-bit mode: weight-streaming dot products; many bf16 rows are handed to the matrix-core kernel.
//
// Bound by HBM: every weight is read once per group of R rows.  A wave owns NR weight rows and streams them 16 bytes a
// lane, `kDotAhead` pieces of each row requested before the first is used; the input rows live in LDS as T.  Sums are fp32
// (packed bf16 dot products, or fmaf in the 32-bit mode), combined over the wave's lanes at the end.
#include <algorithm>

#include "qm_decoder_device.h"
#include "../qm_host.h"
#include "../qm_linear_rows_params.h"
#include "qm_decoder_dot.h"

namespace qm {

constexpr int kLinearRows = 4;                 // weight rows a wave streams at once

template <class T, int R>
__global__ __launch_bounds__(kDecThreads) void decoder_linear_kernel(DecLinearParams prm) {
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    T* xs = reinterpret_cast<T*>(smem);
    int tile = static_cast<int>(blockIdx.x);
    const DecLinearGroup& group = prm.group[dot_group<kLinearRows>(prm, tile)];
    const int row0 = static_cast<int>(blockIdx.y) * R;
    const int rows = min(R, prm.rows - row0);
    const int k = group.k;
    const DotRows<kLinearRows> d = dot_rows<kLinearRows>(group, tile);
    uint4 piece[kDotAhead][kLinearRows];
    dot_request<kLinearRows>(d, k, piece);
    constexpr int kVec = 16 / sizeof(T);
    for (int r = 0; r < R; ++r) {
        const int src = row0 + min(r, rows - 1);               // (a row past the end repeats the last one, never stored)
        const T* x = static_cast<const T*>(group.x) + src * group.ldx;
        for (int c = threadIdx.x * kVec; c < k; c += kDecThreads * kVec)
            *reinterpret_cast<uint4*>(xs + r * k + c) = *reinterpret_cast<const uint4*>(x + c);
    }
    __syncthreads();
    dot_finish<T, R, kLinearRows>(group, d, piece, xs, row0, rows);
}

template <class T, int R>
static int32_t launch_streaming(const DecLinearParams& prm, hipStream_t stream) {
    int k = 0;
    for (int g = 0; g < prm.groups; ++g) k = prm.group[g].k > k ? prm.group[g].k : k;
    const int tiles = dot_tiles_of<kLinearRows>(prm);
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(decoder_linear_kernel<T, R>), kDotLdsMost, raised);
    if (rc != QM_OK) return rc;
    hipLaunchKernelGGL((decoder_linear_kernel<T, R>), dim3(tiles, (prm.rows + R - 1) / R), dim3(kDecThreads), sizeof(T) * R * k, stream, prm);
    return launch_status();
}

template <class T>
static int32_t streaming(const DecLinearParams& prm, hipStream_t stream) {
    int k = 0;
    for (int g = 0; g < prm.groups; ++g) k = prm.group[g].k > k ? prm.group[g].k : k;
    const int64_t row_bytes = static_cast<int64_t>(k) * sizeof(T);
    if (row_bytes > kDotLds) return QM_ERR_GEOMETRY;
    if (prm.rows > 4 && 8 * row_bytes <= kDotLds) return launch_streaming<T, 8>(prm, stream);
    if (prm.rows > 2 && 4 * row_bytes <= kDotLds) return launch_streaming<T, 4>(prm, stream);
    if (prm.rows > 1 && 2 * row_bytes <= kDotLds) return launch_streaming<T, 2>(prm, stream);
    return launch_streaming<T, 1>(prm, stream);
}

// Rows from which the matrix cores take over: below, one 64-row tile is mostly empty and the weights' bytes decide.
constexpr int kDecMatrixRows = 16;

int32_t launch_decoder_linears(const DecLinearParams& prm, int f32, hipStream_t stream) {
    if (prm.rows < 0 || prm.groups < 1 || prm.groups > kDecGroups) return QM_ERR_ARGUMENT;
    for (int g = 0; g < prm.groups; ++g) {
        const DecLinearGroup& d = prm.group[g];
        if (!d.x || !d.w || (d.w_up ? !d.out : !d.out32)) return QM_ERR_NULL;
        if (d.n <= 0 || d.k <= 0 || d.n % 128 || d.k % 128 || d.ldx < d.k || d.ldo < d.n || d.ldx % 8 || d.ldo % 4) return QM_ERR_GEOMETRY;
    }
    if (prm.rows == 0) return QM_OK;
    if (f32) return streaming<float>(prm, stream);
    bool matrix = prm.rows >= kDecMatrixRows;
    for (int g = 0; g < prm.groups; ++g) matrix = matrix && prm.group[g].ldx == prm.group[g].k && prm.group[g].ldo == prm.group[g].n;
    if (!matrix) return streaming<uint16_t>(prm, stream);
    LinearRowsParams plain = {};
    int order[kDecGroups] = {0, 1, 2};         // long reductions first
    std::stable_sort(order, order + prm.groups, [&](int a, int b) { return prm.group[a].k > prm.group[b].k; });
    for (int i = 0; i < prm.groups; ++i) {
        const DecLinearGroup& d = prm.group[order[i]];
        if (d.w_up) {
            LinearRowsParams pair = {};
            pair.input = static_cast<const uint16_t*>(d.x);
            pair.weight[0] = d.w; pair.weight[1] = d.w_up;
            pair.output = static_cast<uint16_t*>(d.out);
            pair.rows = prm.rows; pair.columns = d.n; pair.reduction = d.k;
            pair.reduction_parts = 1; pair.groups = 1;
            const int32_t rc = launch_rows_mfma(pair, true, stream);
            if (rc != QM_OK) return rc;
            continue;
        }
        if (plain.groups == 0) {
            plain.input = static_cast<const uint16_t*>(d.x);
            plain.weight[0] = plain.weight[1] = d.w;
            plain.sums = d.out32;
            plain.rows = prm.rows; plain.columns = d.n; plain.reduction = d.k;
            plain.reduction_parts = 1;
        } else {
            const int at = plain.groups - 1;
            const int before = at == 0 ? 0 : plain.group_first_tile[at - 1];
            plain.group_first_tile[at] = before + (at == 0 ? plain.columns : plain.group_columns[at - 1]) / 128;
            plain.group_input[at] = static_cast<const uint16_t*>(d.x);
            plain.group_weight[at] = d.w;
            plain.group_sums[at] = d.out32;
            plain.group_columns[at] = d.n;
            plain.group_reduction[at] = d.k;
        }
        ++plain.groups;
    }
    plain.linear_by_linear = plain.groups > 1;
    return plain.groups ? launch_rows_mfma(plain, false, stream) : QM_OK;
}

}  // namespace qm
