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

// A linear of few columns (a router) over many bf16 rows: the large tiles of the matrix-core kernel would leave most CUs
// without a block and walk the whole reduction one step after the other.  Here a block takes 16 rows, its four waves every
// fourth 128 terms of the reduction (v_mfma_f32_16x16x32_bf16, operands straight from memory; the weights are few and stay in
// L2), and the four sums meet in LDS.  Bound by the latency of a wave's loads.
constexpr int kNarrowRows = 16;                        // token rows of a block
constexpr int kNarrowColumns = 64;                     // most columns
template <int TILES>
__global__ __launch_bounds__(kDecThreads) void narrow_linear_kernel(DecLinearGroup group, int rows) {
    __shared__ float sums[4][TILES * 16 * (kNarrowRows + 1)];
    typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, l16 = lane & 15;
    const int row0 = static_cast<int>(blockIdx.x) * kNarrowRows;
    const uint16_t* x = static_cast<const uint16_t*>(group.x) + min(row0 + l16, rows - 1) * group.ldx + 8 * g;
    const uint16_t* w[TILES];
#pragma unroll
    for (int t = 0; t < TILES; ++t) w[t] = group.w + static_cast<int64_t>(min(16 * t, group.n - 16) + l16) * group.k + 8 * g;
    f32x4_t acc[TILES] = {};
    for (int k = wave * 128; k < group.k; k += 512) {  // (all of 128 terms is asked for before the first is used)
        u32x4 b[4], a[4][TILES];
#pragma unroll
        for (int u = 0; u < 4; ++u) b[u] = *reinterpret_cast<const u32x4*>(x + k + 32 * u);
#pragma unroll
        for (int t = 0; t < TILES; ++t)
#pragma unroll
            for (int u = 0; u < 4; ++u) a[u][t] = *reinterpret_cast<const u32x4*>(w[t] + k + 32 * u);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int t = 0; t < TILES; ++t)
                acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a[u][t]), __builtin_bit_cast(bf16x8_t, b[u]), acc[t], 0, 0, 0);
    }
    // acc[t][r] is column 16 t + 4 g + r of row l16
#pragma unroll
    for (int t = 0; t < TILES; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) sums[wave][(16 * t + 4 * g + r) * (kNarrowRows + 1) + l16] = acc[t][r];
    __syncthreads();
    for (int i = threadIdx.x; i < kNarrowRows * TILES * 16; i += kDecThreads) {
        const int row = i / (TILES * 16), c = i % (TILES * 16), at = c * (kNarrowRows + 1) + row;
        if (row0 + row < rows && c < group.n)
            group.out32[static_cast<int64_t>(row0 + row) * group.ldo + c] = (sums[0][at] + sums[1][at]) + (sums[2][at] + sums[3][at]);
    }
}
template <int TILES>
static int32_t launch_narrow(const DecLinearParams& prm, hipStream_t stream) {
    hipLaunchKernelGGL(narrow_linear_kernel<TILES>, dim3((prm.rows + kNarrowRows - 1) / kNarrowRows), dim3(kDecThreads), 0, stream, prm.group[0], prm.rows);
    return launch_status();
}

// Rows from which the matrix cores take over: below, one 64-row tile is mostly empty and the weights' bytes decide.
constexpr int kDecMatrixRows = 16;

int32_t launch_decoder_linears(const DecLinearParams& prm, int f32, hipStream_t stream) {
    if (prm.rows < 0 || prm.groups < 1 || prm.groups > kDecGroups) return QM_ERR_ARGUMENT;
    for (int g = 0; g < prm.groups; ++g) {
        const DecLinearGroup& d = prm.group[g];
        if (!d.x || !d.w || (d.w_up ? !d.out : !d.out32)) return QM_ERR_NULL;
        if (d.n <= 0 || d.k <= 0 || d.n % (d.w_up ? 128 : 16) || d.k % 128 || d.ldx < d.k || d.ldo < d.n || d.ldx % 8 || d.ldo % 4) return QM_ERR_GEOMETRY;
    }
    if (prm.rows == 0) return QM_OK;
    if (f32) return streaming<float>(prm, stream);
    bool matrix = prm.rows >= kDecMatrixRows;
    if (matrix && prm.groups == 1 && prm.group[0].n <= kNarrowColumns && !prm.group[0].w_up)
        return prm.group[0].n <= 32 ? launch_narrow<2>(prm, stream) : launch_narrow<4>(prm, stream);
    for (int g = 0; g < prm.groups; ++g) matrix = matrix && prm.group[g].n % 128 == 0 && prm.group[g].ldx == prm.group[g].k && prm.group[g].ldo == prm.group[g].n;
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
