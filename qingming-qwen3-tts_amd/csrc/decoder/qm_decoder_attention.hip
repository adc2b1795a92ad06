// qm_decoder_attention.hip — softmax attention inside chunks of positions (position i sees j <= i with the same
// floor(. / chunk)), grouped query heads, over a ring cache of keys and values, for gfx950.
//
// Chunks count from position 0 of the sequence, so a query needs at most `chunk` keys, all of them in the cache however the
// prompt was cut.  Two kernels: few rows (decode) deal a chunk's keys to several blocks per key/value head and combine the
// partial results; many bf16 rows take the matrix-core kernel of qm_decoder_attention_mfma.hip.
#include "../qm_host.h"
#include "qm_decoder_attention.h"

namespace qm {

// Rotation of the rows' queries and keys, keys and values into the ring: one block per row.
template <class T>
__global__ __launch_bounds__(kDecThreads) void rope_cache_kernel(ChunkAttentionParams prm) {
    extern __shared__ float sh_turn[];         // [rot_dims / 2] cosines, then sines
    const int tid = threadIdx.x;
    const int row = static_cast<int>(blockIdx.x);
    const int position = position_of(prm.position_dev, prm.position) + row;
    const int half = prm.rot_dims >> 1;
    for (int i = tid; i < half; i += kDecThreads) rotary(position, prm.frequency[i], sh_turn[i], sh_turn[half + i]);
    __syncthreads();
    const float* proj = prm.proj + row * prm.ld_proj;
    auto channel = [&](const float* head, int c) {
        if (c >= prm.dim) return 0.0f;
        if (c >= prm.rot_dims) return head[c];
        const int pair = c < half ? c : c - half;
        const float u = head[pair], v = head[pair + half], cosine = sh_turn[pair], sine = sh_turn[half + pair];
        return c < half ? u * cosine - v * sine : v * cosine + u * sine;
    };
#pragma unroll 4
    for (int i = tid; i < prm.heads * prm.k_stride; i += kDecThreads) {
        const int h = i / prm.k_stride, c = i - h * prm.k_stride;
        static_cast<T*>(prm.q_rot)[static_cast<int64_t>(row) * prm.heads * prm.k_stride + i] = from_f32<T>(channel(proj + h * prm.dim, c));
    }
    const int64_t slot = position % prm.ring;
    for (int i = tid; i < prm.kv_heads * prm.k_stride; i += kDecThreads) {
        const int h = i / prm.k_stride, c = i - h * prm.k_stride;
        static_cast<T*>(prm.k_cache)[(static_cast<int64_t>(h) * prm.ring + slot) * prm.k_stride + c] =
            from_f32<T>(channel(proj + prm.k_column + h * prm.dim, c));
    }
    for (int i = tid; i < prm.kv_heads * prm.v_stride; i += kDecThreads) {
        const int h = i / prm.v_stride, c = i - h * prm.v_stride;
        static_cast<T*>(prm.v_cache)[(static_cast<int64_t>(h) * prm.ring + slot) * prm.v_stride + c] =
            from_f32<T>(c < prm.vdim ? proj[prm.v_column + h * prm.vdim + c] : 0.0f);
    }
}

template <class T, int GQ, int VC>
__global__ __launch_bounds__(kDecThreads) void chunk_attention_kernel(ChunkAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    chunk_attention_block<T, GQ, VC, false>(prm, static_cast<int>(blockIdx.x), static_cast<int>(blockIdx.y), static_cast<int>(blockIdx.z), lds);
}

template <class T>
__global__ __launch_bounds__(kDecThreads) void merge_attention_kernel(ChunkAttentionParams prm) {
    const int64_t row = blockIdx.x;
    const int position = position_of(prm.position_dev, prm.position) + static_cast<int>(row);
    merge_attention_row<T>(prm.part, row, attention_active_splits(position, prm.chunk, prm.part.keys_per_split),
                           static_cast<T*>(prm.out) + row * prm.ld_out, prm.ld_out);
}

int32_t check_attention(const ChunkAttentionParams& p) {
    if (p.rows < 0 || p.position < 0) return QM_ERR_ARGUMENT;
    if (!p.proj || !p.k_cache || !p.v_cache || !p.out || !p.part.ml || !p.part.acc || (p.rot_dims > 0 && !p.frequency)) return QM_ERR_NULL;
    if (p.heads <= 0 || p.kv_heads <= 0 || p.heads % p.kv_heads || p.dim <= 0 || p.vdim <= 0 || p.dim > kDecMaxHead || p.vdim > kDecMaxHead)
        return QM_ERR_GEOMETRY;
    if (p.k_stride != (p.dim + 7) / 8 * 8 || p.v_stride != (p.vdim + 7) / 8 * 8) return QM_ERR_GEOMETRY;
    if (p.rot_dims < 0 || p.rot_dims > p.dim || p.rot_dims % 2 || p.chunk <= 0 || p.ring <= 0) return QM_ERR_GEOMETRY;
    if (p.part.heads != p.heads || p.part.vdim != p.vdim || p.part.splits < 1 || p.part.splits > kDecMaxSplits) return QM_ERR_GEOMETRY;
    if (p.part.keys_per_split <= 0 || static_cast<int64_t>(p.part.keys_per_split) * p.part.splits < p.chunk) return QM_ERR_GEOMETRY;
    if (p.ld_out < static_cast<int64_t>(p.heads) * p.vdim || p.rows > 65535) return QM_ERR_GEOMETRY;
    return QM_OK;
}

int32_t launch_rope_cache(const ChunkAttentionParams& prm, int f32, hipStream_t stream) {
    const size_t lds = static_cast<size_t>(prm.rot_dims + 2) * sizeof(float);
    if (f32) hipLaunchKernelGGL(rope_cache_kernel<float>, dim3(prm.rows), dim3(kDecThreads), lds, stream, prm);
    else hipLaunchKernelGGL(rope_cache_kernel<uint16_t>, dim3(prm.rows), dim3(kDecThreads), lds, stream, prm);
    return launch_status();
}

template <class T, int GQ>
static int32_t launch_rows(const ChunkAttentionParams& prm, hipStream_t stream) {
    const dim3 grid(prm.part.splits, prm.kv_heads, prm.rows);
    const size_t lds = sizeof(float) * attention_lds_floats(GQ, prm.k_stride, prm.v_stride);
    if (prm.v_stride <= 128) hipLaunchKernelGGL((chunk_attention_kernel<T, GQ, 1>), grid, dim3(kDecThreads), lds, stream, prm);
    else hipLaunchKernelGGL((chunk_attention_kernel<T, GQ, 2>), grid, dim3(kDecThreads), lds, stream, prm);
    int32_t rc = launch_status();
    if (rc != QM_OK) return rc;
    hipLaunchKernelGGL(merge_attention_kernel<T>, dim3(prm.rows), dim3(kDecThreads), 0, stream, prm);
    return launch_status();
}

template <class T>
static int32_t attention_rows(const ChunkAttentionParams& prm, hipStream_t stream) {
    const int group = prm.heads / prm.kv_heads;
    return group == 1 ? launch_rows<T, 1>(prm, stream) : group == 2 ? launch_rows<T, 2>(prm, stream) : launch_rows<T, 4>(prm, stream);
}

int32_t launch_chunk_attention(const ChunkAttentionParams& prm, int f32, hipStream_t stream) {
    int32_t rc = check_attention(prm);
    if (rc != QM_OK || prm.rows == 0) return rc;
    if (!prm.q_rot) return QM_ERR_NULL;
    rc = launch_rope_cache(prm, f32, stream);
    if (rc != QM_OK) return rc;
    // (positions that only the device knows belong to one-token steps)
    if (!f32 && prm.rows >= kAttentionMatrixRows && !prm.position_dev && !(prm.options & QM_ATTENTION_ROWS)) return launch_chunk_attention_mfma(prm, stream);
    return f32 ? attention_rows<float>(prm, stream) : attention_rows<uint16_t>(prm, stream);
}

}  // namespace qm
