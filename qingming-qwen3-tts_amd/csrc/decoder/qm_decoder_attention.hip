// qm_decoder_attention.hip — softmax attention inside chunks of positions (position i sees j <= i with the same
// floor(. / chunk)), grouped query heads, over a ring cache of keys and values, for gfx950.
//
// Chunks count from position 0 of the sequence, so a query needs at most `chunk` keys, all of them in the cache however the
// prompt was cut.  Two kernels: few rows (decode) deal a chunk's keys to several blocks per key/value head and combine the
// partial results; many bf16 rows take the matrix-core kernel of qm_decoder_attention_mfma.hip.
#include "../qm_host.h"
#include "qm_decoder_attention.h"

namespace qm {

// Rotation of the rows' queries and keys, keys and values into the ring: one block per row.  The row's projections pass
// through LDS; a thread puts out eight channels at a time.
__device__ __forceinline__ void store8(uint16_t* to, const float (&v)[8]) {
    *reinterpret_cast<uint4*>(to) = make_uint4(pack_bf16_pair(v[0], v[1]), pack_bf16_pair(v[2], v[3]), pack_bf16_pair(v[4], v[5]), pack_bf16_pair(v[6], v[7]));
}
__device__ __forceinline__ void store8(float* to, const float (&v)[8]) {
    reinterpret_cast<float4*>(to)[0] = make_float4(v[0], v[1], v[2], v[3]);
    reinterpret_cast<float4*>(to)[1] = make_float4(v[4], v[5], v[6], v[7]);
}

template <class T>
__global__ __launch_bounds__(kDecThreads) void rope_cache_kernel(ChunkAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float sh_row[];             // q, k, v; cosines; sines
    const int tid = threadIdx.x;
    const int row = static_cast<int>(blockIdx.x);
    const int position = position_of(prm.position_dev, prm.position) + row;
    const int half = prm.rot_dims >> 1, q_n = prm.heads * prm.dim, k_n = prm.kv_heads * prm.dim, v_n = prm.kv_heads * prm.vdim;
    float* sh_cos = sh_row + q_n + k_n + v_n;
    float* sh_sin = sh_cos + half;
    const float* proj = prm.proj + row * prm.ld_proj;
#pragma unroll 4
    for (int i = tid; i < q_n; i += kDecThreads) sh_row[i] = proj[i];
#pragma unroll 4
    for (int i = tid; i < k_n; i += kDecThreads) sh_row[q_n + i] = proj[prm.k_column + i];
#pragma unroll 4
    for (int i = tid; i < v_n; i += kDecThreads) sh_row[q_n + k_n + i] = proj[prm.v_column + i];
    for (int i = tid; i < half; i += kDecThreads) rotary(position, prm.frequency[i], sh_cos[i], sh_sin[i]);
    __syncthreads();
    auto rotated = [&](const float* head, int c0, float (&v)[8]) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int c = c0 + e;
            const int pair = c < half ? c : c - half;
            const bool turns = c < prm.rot_dims;
            const float own = c < prm.dim ? head[c] : 0.0f;
            const float other = turns ? head[c < half ? c + half : pair] : 0.0f;
            const float cosine = turns ? sh_cos[pair] : 1.0f, sine = turns ? sh_sin[pair] : 0.0f;
            v[e] = c < half ? own * cosine - other * sine : own * cosine + other * sine;
        }
    };
    const int64_t slot = position % prm.ring;
    const int k_pieces = prm.k_stride >> 3, v_pieces = prm.v_stride >> 3;
    for (int i = tid; i < (prm.heads + prm.kv_heads) * k_pieces; i += kDecThreads) {
        const int h = i / k_pieces, c = (i - h * k_pieces) * 8;
        float v[8];
        rotated(sh_row + h * prm.dim, c, v);                                   // (the key heads follow the query heads)
        store8(h < prm.heads ? static_cast<T*>(prm.q_rot) + (static_cast<int64_t>(row) * prm.heads + h) * prm.k_stride + c
                             : static_cast<T*>(prm.k_cache) + (static_cast<int64_t>(h - prm.heads) * prm.ring + slot) * prm.k_stride + c, v);
    }
    for (int i = tid; i < prm.kv_heads * v_pieces; i += kDecThreads) {
        const int h = i / v_pieces, c = (i - h * v_pieces) * 8;
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = c + e < prm.vdim ? sh_row[q_n + k_n + h * prm.vdim + c + e] : 0.0f;
        store8(static_cast<T*>(prm.v_cache) + (static_cast<int64_t>(h) * prm.ring + slot) * prm.v_stride + c, v);
    }
}

template <class T, int GQ, int VC>
__global__ __launch_bounds__(kDecThreads) void chunk_attention_kernel(ChunkAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    chunk_attention_block<T, GQ, VC, false>(prm, static_cast<int>(blockIdx.x), static_cast<int>(blockIdx.y), static_cast<int>(blockIdx.z), lds);
}

template <class T>
__global__ __launch_bounds__(kDecThreads) void merge_attention_kernel(ChunkAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int64_t row = blockIdx.x;
    const int position = position_of(prm.position_dev, prm.position) + static_cast<int>(row);
    merge_attention_row<T>(prm.part, row, attention_active_splits(position, prm.chunk, prm.part.keys_per_split), lds,
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
    if (p.ld_out < static_cast<int64_t>(p.heads) * p.vdim || p.rows > 65535 || p.ld_out % 4) return QM_ERR_GEOMETRY;
    if (static_cast<int64_t>(p.heads) * p.part.splits > kDecMaxMerge) return QM_ERR_GEOMETRY;
    return QM_OK;
}

template <class T>
static int32_t rope_cache(const ChunkAttentionParams& prm, hipStream_t stream) {
    const size_t lds = sizeof(float) * (static_cast<size_t>(prm.heads + prm.kv_heads) * prm.dim + static_cast<size_t>(prm.kv_heads) * prm.vdim + prm.rot_dims);
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(rope_cache_kernel<T>), kDotLdsMost, raised);
    if (rc != QM_OK) return rc;
    if (lds > static_cast<size_t>(kDotLdsMost)) return QM_ERR_GEOMETRY;
    hipLaunchKernelGGL(rope_cache_kernel<T>, dim3(prm.rows), dim3(kDecThreads), lds, stream, prm);
    return launch_status();
}

template <class T, int GQ>
static int32_t launch_rows(const ChunkAttentionParams& prm, hipStream_t stream) {
    const dim3 grid(prm.part.splits, prm.kv_heads, prm.rows);
    const size_t lds = sizeof(float) * attention_lds_floats(GQ, prm.k_stride, prm.v_stride);
    if (prm.v_stride <= 128 && prm.k_stride <= 128) hipLaunchKernelGGL((chunk_attention_kernel<T, GQ, 1>), grid, dim3(kDecThreads), lds, stream, prm);
    else hipLaunchKernelGGL((chunk_attention_kernel<T, GQ, 2>), grid, dim3(kDecThreads), lds, stream, prm);
    int32_t rc = launch_status();
    if (rc != QM_OK) return rc;
    hipLaunchKernelGGL(merge_attention_kernel<T>, dim3(prm.rows), dim3(kDecThreads), sizeof(float) * prm.heads * prm.part.splits, stream, prm);
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
    rc = f32 ? rope_cache<float>(prm, stream) : rope_cache<uint16_t>(prm, stream);
    if (rc != QM_OK) return rc;
    // (positions that only the device knows belong to one-token steps)
    if (!f32 && prm.rows >= kAttentionMatrixRows && !prm.position_dev && !(prm.options & QM_ATTENTION_ROWS)) return launch_chunk_attention_mfma(prm, stream);
    return f32 ? attention_rows<float>(prm, stream) : attention_rows<uint16_t>(prm, stream);
}

}  // namespace qm
