// qm_decoder_latent.h — what the kernels of the attention over latents share.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

// A query that has gone through up_k lies in q_scratch as [latent part][rotated part], each padded with zeros: the latent part
// to the next of 64, 128, 256, 512 (a multiple of 512 beyond), the rotated part to a multiple of 64.
__host__ __device__ inline int latent_pad(int kv_rank) { return kv_rank <= 64 ? 64 : kv_rank <= 128 ? 128 : kv_rank <= 256 ? 256 : (kv_rank + 511) / 512 * 512; }
__host__ __device__ inline int latent_rotary_pad(int rot_dim) { return (rot_dim + 63) / 64 * 64; }

// Keys of one split when `keys` are dealt to at most `splits`.
__host__ __device__ inline int latent_keys_per_split(int keys, int splits) {
    const int each = (keys + splits - 1) / splits;
    return (each + kLatentKeys - 1) / kLatentKeys * kLatentKeys;
}

// Channel c of a vector whose channels 2i and 2i + 1 turn together.
__device__ __forceinline__ float turned_neighbour(const float* x, int c, const double* frequency, int position, float magnitude) {
    float cosine, sine;
    rotary(position, frequency[c >> 1], cosine, sine);
    const float u = x[c & ~1], v = x[c | 1];
    return magnitude * (c & 1 ? v * cosine + u * sine : u * cosine - v * sine);
}

// What one row leaves in the caches, by a block of 256 threads; sh_red: 4 floats of LDS.
template <class T>
__device__ __forceinline__ void latent_keep_row(const LatentRowsParams& prm, int row, float* sh_red) {
    const int position = position_of(prm.position_dev, prm.position) + row;
    const float* kv = prm.proj + row * prm.ld_proj + prm.kv_column;
    slice_norm_row<T>(kv, prm.kv_norm, prm.kv_rank, prm.ld_latent, prm.eps, sh_red, static_cast<T*>(prm.latent_cache) + position * prm.ld_latent);
    T* key = static_cast<T*>(prm.key_cache) + static_cast<int64_t>(position) * prm.key_stride;
    for (int c = threadIdx.x; c < prm.key_stride; c += kDecThreads)
        key[c] = from_f32<T>(c < prm.rot_dim ? turned_neighbour(kv + prm.kv_rank, c, prm.frequency, position, prm.magnitude) : 0.0f);
}

}  // namespace qm
