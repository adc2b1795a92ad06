// qm_decoder_experts.hip — mixture of experts for gfx950: each row's experts of the highest logits, weighted with the logits'
// sigmoid, their gated feed-forwards and the weighted sum.
//
// Few rows (and fp32) stream the chosen experts' weights as the other linears do; a one-token step's blocks find their expert
// from the logits themselves.  Many bf16 rows are copied expert by expert, each expert's rows from a multiple of the matrix-core
// linear's row tile on, and that linear takes every tile's weights from its expert.  Bound by HBM: the chosen experts' weights are
// read once per row (few rows) or once per row tile.
#include "../qm_host.h"
#include "../qm_linear_rows_params.h"
#include "qm_decoder_dot.h"

namespace qm {

constexpr int kExpertInRows = 4;               // weight rows per wave: gate/up
constexpr int kExpertOutRows = 2;              // down
constexpr int kRouteRows = kDecThreads / 64;   // rows per block of the router: a wave each
constexpr int kSortThreads = 1024;
constexpr int kExpertMatrixRows = 16;          // rows from which bf16 goes to the matrix cores
constexpr int kExpertLongTile = 256;           // rows per expert (on average) from which row tiles are 128 high, not 64

// What the kernels share in the scratch.
struct ExpertScratch {
    int32_t* id;               // [rows][top]
    float* weight;             // [rows][top]
    int32_t* place;            // [rows][top]: row among the sorted ones
    int32_t* tile_expert;      // [tiles], -1: none
    void* act;                 // [rows * top, or sorted rows][ff_p]
    uint16_t* x;               // [sorted rows][width_p]
    float* y;                  // [sorted rows][width_p]
    int tile_rows, tiles;
};

// How many of the `experts` logits come before logit e (lower numbers first among equals).
__device__ __forceinline__ int rank_of(const float* logits, int experts, int e) {
    const float own = logits[e];
    int rank = 0;
    for (int j = 0; j < experts; ++j) rank += logits[j] > own || (logits[j] == own && j < e);
    return rank;
}

__global__ __launch_bounds__(kDecThreads) void route_kernel(ExpertParams prm, ExpertScratch s) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int row = static_cast<int>(blockIdx.x) * kRouteRows + wave;
    float* logits = lds + wave * prm.experts;
    if (row < prm.rows)
        for (int e = lane; e < prm.experts; e += 64) logits[e] = prm.logits[row * prm.ld_logits + e];
    __syncthreads();
    if (row >= prm.rows) return;
    for (int e = lane; e < prm.experts; e += 64) {
        const int rank = rank_of(logits, prm.experts, e);
        if (rank >= prm.top) continue;
        s.id[row * prm.top + rank] = e;
        s.weight[row * prm.top + rank] = sigmoid_f32(logits[e]);
    }
}

// Gate/up of slot blockIdx.y's expert for row blockIdx.z.  ROUTE: the expert is found here, from the row's logits.
template <class T, bool ROUTE>
__global__ __launch_bounds__(kDecThreads) void expert_in_kernel(ExpertParams prm, ExpertScratch s) {
    request_arguments(prm, s);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    __shared__ int sh_expert;
    T* xs = reinterpret_cast<T*>(smem);                                        // [width_p]
    float* logits = reinterpret_cast<float*>(xs + prm.width_p);                // [experts]
    const int slot = static_cast<int>(blockIdx.y), row = static_cast<int>(blockIdx.z), tile = static_cast<int>(blockIdx.x);
    constexpr int kVec = 16 / sizeof(T);
    const T* x = static_cast<const T*>(prm.x) + static_cast<int64_t>(row) * prm.width_p;
    if (ROUTE)
        for (int e = threadIdx.x; e < prm.experts; e += kDecThreads) logits[e] = prm.logits[row * prm.ld_logits + e];
    for (int c = threadIdx.x * kVec; c < prm.width_p; c += kDecThreads * kVec)
        *reinterpret_cast<uint4*>(xs + c) = *reinterpret_cast<const uint4*>(x + c);
    __syncthreads();
    const int at = row * prm.top + slot;
    if (ROUTE) {
        for (int e = threadIdx.x; e < prm.experts; e += kDecThreads) {
            if (rank_of(logits, prm.experts, e) != slot) continue;
            sh_expert = e;
            if (tile == 0) {
                s.id[at] = e;
                s.weight[at] = sigmoid_f32(logits[e]);
            }
        }
        __syncthreads();
    }
    const int64_t expert = __builtin_amdgcn_readfirstlane(ROUTE ? sh_expert : s.id[at]);
    DecLinearGroup g = {};
    g.w = prm.gate + expert * prm.ff_p * prm.width_p;
    g.w_up = prm.up + expert * prm.ff_p * prm.width_p;
    g.out = static_cast<T*>(s.act) + static_cast<int64_t>(at) * prm.ff_p;
    g.ldo = g.n = prm.ff_p;
    g.k = prm.width_p;
    const DotRows<kExpertInRows> d = dot_rows<kExpertInRows>(g, tile);
    uint4 piece[kDotAhead][kExpertInRows];
    dot_request<kExpertInRows>(d, g.k, piece);
    dot_finish<T, 1, kExpertInRows>(g, d, piece, xs, 0, 1);
}

// Down of row blockIdx.y: the chosen experts' reductions one behind the other, each weighted.
template <class T>
__global__ __launch_bounds__(kDecThreads) void expert_out_kernel(ExpertParams prm, ExpertScratch s) {
    request_arguments(prm, s);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), row = static_cast<int>(blockIdx.y);
    const int total = prm.top * prm.ff_p;
    T* xs = reinterpret_cast<T*>(smem);                                        // [top][ff_p]
    int* sh_id = reinterpret_cast<int*>(xs + total);                           // [top]
    float* sh_weight = reinterpret_cast<float*>(sh_id + prm.top);              // [top]
    for (int i = threadIdx.x; i < prm.top; i += kDecThreads) {
        sh_id[i] = s.id[row * prm.top + i];
        sh_weight[i] = s.weight[row * prm.top + i];
    }
    __syncthreads();
    const int channel = (static_cast<int>(blockIdx.x) * 4 + wave) * kExpertOutRows;
    uint4 piece[kDotAhead][kExpertOutRows];
    auto request_one = [&](int at, uint4 (&to)[kExpertOutRows]) __attribute__((always_inline)) {
        const int from = at < total ? at : 0, slot = from / prm.ff_p;
        const uint16_t* w = prm.down + (static_cast<int64_t>(sh_id[slot]) * prm.width_p + channel) * prm.ff_p + (from - slot * prm.ff_p);
#pragma unroll
        for (int i = 0; i < kExpertOutRows; ++i) to[i] = *reinterpret_cast<const uint4*>(w + static_cast<int64_t>(i) * prm.ff_p);
    };
#pragma unroll
    for (int u = 0; u < kDotAhead; ++u) request_one(u * 512 + lane * 8, piece[u]);
    constexpr int kVec = 16 / sizeof(T);
    const T* act = static_cast<const T*>(s.act) + static_cast<int64_t>(row) * total;
    for (int c = threadIdx.x * kVec; c < total; c += kDecThreads * kVec) *reinterpret_cast<uint4*>(xs + c) = *reinterpret_cast<const uint4*>(act + c);
    __syncthreads();
    float acc[kExpertOutRows] = {};
    for (int k0 = 0; k0 < total; k0 += kDotAhead * 512) {
#pragma unroll
        for (int u = 0; u < kDotAhead; ++u) {
            const int at = k0 + u * 512 + lane * 8;
            if (at < total) {
                const float weight = sh_weight[at / prm.ff_p];
#pragma unroll
                for (int i = 0; i < kExpertOutRows; ++i) acc[i] = fmaf(weight, dot8(piece[u][i], xs + at, 0.0f), acc[i]);
            }
            if (k0 + kDotAhead * 512 < total) request_one(at + kDotAhead * 512, piece[u]);
        }
    }
#pragma unroll
    for (int i = 0; i < kExpertOutRows; ++i) {
        const float sum = wave_sum(acc[i]);
        if (lane == 0) prm.out32[static_cast<int64_t>(row) * prm.width_p + channel + i] = sum;
    }
}

// ---- many rows -----------------------------------------------------------------------------------------------------------
// Every assignment's place among the rows sorted by expert, and each row tile's expert: one block.
__global__ __launch_bounds__(kSortThreads) void expert_sort_kernel(ExpertParams prm, ExpertScratch s) {
    __shared__ int sh_count[kExpertsMost], sh_first[kExpertsMost];
    const int assignments = prm.rows * prm.top;
    for (int e = threadIdx.x; e < prm.experts; e += kSortThreads) sh_count[e] = 0;
    for (int t = threadIdx.x; t < s.tiles; t += kSortThreads) s.tile_expert[t] = -1;
    __syncthreads();
    for (int a = threadIdx.x; a < assignments; a += kSortThreads) s.place[a] = atomicAdd(&sh_count[s.id[a]], 1);
    __syncthreads();
    const int e = threadIdx.x;
    // (an inclusive sum of the experts' tiles, doubling the reach each time)
    const int own = e < prm.experts ? (sh_count[e] + s.tile_rows - 1) / s.tile_rows : 0;
    sh_first[e] = own;
    __syncthreads();
    for (int reach = 1; reach < prm.experts; reach *= 2) {
        const int before = e >= reach ? sh_first[e - reach] : 0;
        __syncthreads();
        sh_first[e] += before;
        __syncthreads();
    }
    const int first = sh_first[e] - own;
    __syncthreads();
    sh_first[e] = first * s.tile_rows;
    for (int t = 0; t < own; ++t) s.tile_expert[first + t] = e;
    __syncthreads();
    for (int a = threadIdx.x; a < assignments; a += kSortThreads) s.place[a] += sh_first[s.id[a]];
}

__global__ __launch_bounds__(kDecThreads) void expert_gather_kernel(ExpertParams prm, ExpertScratch s) {
    const int a = static_cast<int>(blockIdx.x);
    const uint16_t* x = static_cast<const uint16_t*>(prm.x) + static_cast<int64_t>(a / prm.top) * prm.width_p;
    uint16_t* to = s.x + static_cast<int64_t>(s.place[a]) * prm.width_p;
    for (int c = threadIdx.x * 8; c < prm.width_p; c += kDecThreads * 8) *reinterpret_cast<uint4*>(to + c) = *reinterpret_cast<const uint4*>(x + c);
}

__global__ __launch_bounds__(kDecThreads) void expert_combine_kernel(ExpertParams prm, ExpertScratch s) {
    const int row = static_cast<int>(blockIdx.x);
    for (int v = threadIdx.x; v < prm.width_p / 4; v += kDecThreads) {
        float4 sum = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
        for (int j0 = 0; j0 < prm.top; j0 += 4) {
            float4 y[4];
            float w[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int at = row * prm.top + min(j0 + j, prm.top - 1);
                y[j] = load4(s.y + static_cast<int64_t>(s.place[at]) * prm.width_p, v);
                w[j] = j0 + j < prm.top ? s.weight[at] : 0.0f;
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) sum = weighted(sum, w[j], y[j], make_float4(1.0f, 1.0f, 1.0f, 1.0f));
        }
        store4(prm.out32 + static_cast<int64_t>(row) * prm.width_p, v, sum.x, sum.y, sum.z, sum.w);
    }
}

static bool by_matrix(int rows, int f32) { return !f32 && rows >= kExpertMatrixRows; }

// The scratch's parts from `base` on; returns its bytes.
static int64_t lay_out(char* base, int rows, int experts, int top, int width_p, int ff_p, int f32, bool matrix, ExpertScratch& s) {
    const int64_t assignments = static_cast<int64_t>(rows) * top;
    int64_t at = 0;
    auto take = [&](int64_t bytes) {
        char* here = base + at;
        at += (bytes + 255) / 256 * 256;
        return here;
    };
    s.id = reinterpret_cast<int32_t*>(take(assignments * 4));
    s.weight = reinterpret_cast<float*>(take(assignments * 4));
    s.place = reinterpret_cast<int32_t*>(take(assignments * 4));
    s.tile_rows = assignments / experts >= kExpertLongTile ? 128 : 64;
    const int64_t full = assignments / s.tile_rows, used = assignments < experts ? assignments : experts;
    s.tiles = static_cast<int>(full + used);
    s.tile_expert = reinterpret_cast<int32_t*>(take(static_cast<int64_t>(s.tiles) * 4));
    const int64_t sorted = matrix ? static_cast<int64_t>(s.tiles) * s.tile_rows : 0;
    s.act = take((matrix ? sorted : assignments) * ff_p * (f32 ? 4 : 2));
    s.x = reinterpret_cast<uint16_t*>(take(sorted * width_p * 2));
    s.y = reinterpret_cast<float*>(take(sorted * width_p * 4));
    return at;
}

int64_t expert_scratch_bytes(int rows, int experts, int top, int width_p, int ff_p, int f32) {
    if (rows <= 0 || experts <= 0 || top <= 0 || width_p <= 0 || ff_p <= 0) return 0;
    ExpertScratch s;
    return lay_out(nullptr, rows, experts, top, width_p, ff_p, f32, by_matrix(rows, f32), s);      // (more rows never need less)
}

template <class T>
static int32_t stream_experts(const ExpertParams& prm, const ExpertScratch& s, hipStream_t stream) {
    const size_t in_lds = static_cast<size_t>(prm.width_p) * sizeof(T) + static_cast<size_t>(prm.experts) * sizeof(float);
    const size_t out_lds = static_cast<size_t>(prm.top) * prm.ff_p * sizeof(T) + static_cast<size_t>(prm.top) * 8;
    if (in_lds > static_cast<size_t>(kDotLdsMost) || out_lds > static_cast<size_t>(kDotLdsMost)) return QM_ERR_GEOMETRY;
    static std::atomic<bool> raised[3][kMaxDevices];
    int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(expert_in_kernel<T, true>), kDotLdsMost, raised[0]);
    if (rc == QM_OK) rc = ensure_dynamic_lds(reinterpret_cast<const void*>(expert_in_kernel<T, false>), kDotLdsMost, raised[1]);
    if (rc == QM_OK) rc = ensure_dynamic_lds(reinterpret_cast<const void*>(expert_out_kernel<T>), kDotLdsMost, raised[2]);
    if (rc != QM_OK) return rc;
    DecLinearGroup pair = {};
    pair.n = prm.ff_p;
    pair.w_up = prm.up;
    const dim3 in_grid(dot_tiles<kExpertInRows>(pair), prm.top, prm.rows), out_grid(prm.width_p / (4 * kExpertOutRows), prm.rows);
    if (prm.rows == 1) {
        hipLaunchKernelGGL((expert_in_kernel<T, true>), in_grid, dim3(kDecThreads), in_lds, stream, prm, s);
    } else {
        hipLaunchKernelGGL(route_kernel, dim3((prm.rows + kRouteRows - 1) / kRouteRows), dim3(kDecThreads), sizeof(float) * kRouteRows * prm.experts, stream,
                           prm, s);
        hipLaunchKernelGGL((expert_in_kernel<T, false>), in_grid, dim3(kDecThreads), in_lds, stream, prm, s);
    }
    hipLaunchKernelGGL(expert_out_kernel<T>, out_grid, dim3(kDecThreads), out_lds, stream, prm, s);
    return launch_status();
}

static int32_t matrix_experts(const ExpertParams& prm, const ExpertScratch& s, hipStream_t stream) {
    const int assignments = prm.rows * prm.top;
    hipLaunchKernelGGL(route_kernel, dim3((prm.rows + kRouteRows - 1) / kRouteRows), dim3(kDecThreads), sizeof(float) * kRouteRows * prm.experts, stream, prm,
                       s);
    hipLaunchKernelGGL(expert_sort_kernel, dim3(1), dim3(kSortThreads), 0, stream, prm, s);
    hipLaunchKernelGGL(expert_gather_kernel, dim3(assignments), dim3(kDecThreads), 0, stream, prm, s);
    int32_t rc = launch_status();
    if (rc != QM_OK) return rc;
    LinearRowsParams in = {};
    in.input = s.x;
    in.weight[0] = prm.gate;
    in.weight[1] = prm.up;
    in.output = static_cast<uint16_t*>(s.act);
    in.rows = s.tiles * s.tile_rows;
    in.columns = prm.ff_p;
    in.reduction = prm.width_p;
    in.reduction_parts = in.groups = 1;
    in.tile_matrix = s.tile_expert;
    in.tile_rows = s.tile_rows;
    rc = launch_rows_mfma(in, true, stream);
    if (rc != QM_OK) return rc;
    LinearRowsParams out = in;
    out.input = static_cast<const uint16_t*>(s.act);
    out.weight[0] = out.weight[1] = prm.down;
    out.output = nullptr;
    out.sums = s.y;
    out.columns = prm.width_p;
    out.reduction = prm.ff_p;
    rc = launch_rows_mfma(out, false, stream);
    if (rc != QM_OK) return rc;
    hipLaunchKernelGGL(expert_combine_kernel, dim3(prm.rows), dim3(kDecThreads), 0, stream, prm, s);
    return launch_status();
}

int32_t launch_experts(const ExpertParams& prm, int f32, hipStream_t stream) {
    if (prm.rows < 0 || prm.rows > 65535) return QM_ERR_ARGUMENT;
    if (!prm.x || !prm.logits || !prm.gate || !prm.up || !prm.down || !prm.out32 || !prm.scratch) return QM_ERR_NULL;
    if (prm.experts <= 0 || prm.experts > kExpertsMost || prm.top <= 0 || prm.top > prm.experts || prm.ld_logits < prm.experts) return QM_ERR_GEOMETRY;
    if (prm.width_p <= 0 || prm.ff_p <= 0 || prm.width_p % 128 || prm.ff_p % 128) return QM_ERR_GEOMETRY;
    if (prm.rows == 0) return QM_OK;
    const bool matrix = by_matrix(prm.rows, f32) && !(prm.options & QM_EXPERTS_ROWS);
    ExpertScratch s;
    if (lay_out(static_cast<char*>(prm.scratch), prm.rows, prm.experts, prm.top, prm.width_p, prm.ff_p, f32, matrix, s) > prm.scratch_bytes)
        return QM_ERR_WORKSPACE;
    if (matrix) return matrix_experts(prm, s, stream);
    return f32 ? stream_experts<float>(prm, s, stream) : stream_experts<uint16_t>(prm, s, stream);
}

}  // namespace qm

extern "C" int64_t qm_expert_scratch_bytes(int32_t rows, int32_t experts, int32_t top, int32_t width_p, int32_t ff_p, int32_t f32) {
    return qm::expert_scratch_bytes(rows, experts, top, width_p, ff_p, f32);
}
extern "C" int32_t qm_expert_rows(const qm_experts* op, int32_t f32, void* hip_stream) {
    return op ? qm::launch_experts(*op, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
