// qm_decoder_attention.h — one (row, key/value head, key split) of the chunked attention by a block of 256 threads.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

constexpr int kAttTile = 128;                  // keys per pass

// Eight consecutive values as they lie in memory, and as fp32.
template <class T> struct Raw8;
template <> struct Raw8<uint16_t> {
    uint4 w;
    __device__ __forceinline__ void load(const uint16_t* p) { w = *reinterpret_cast<const uint4*>(p); }
    __device__ __forceinline__ void widen(float (&v)[8]) const {
        v[0] = lo_bf16(w.x); v[1] = hi_bf16(w.x); v[2] = lo_bf16(w.y); v[3] = hi_bf16(w.y);
        v[4] = lo_bf16(w.z); v[5] = hi_bf16(w.z); v[6] = lo_bf16(w.w); v[7] = hi_bf16(w.w);
    }
};
template <> struct Raw8<float> {
    float4 a, b;
    __device__ __forceinline__ void load(const float* p) {
        a = reinterpret_cast<const float4*>(p)[0];
        b = reinterpret_cast<const float4*>(p)[1];
    }
    __device__ __forceinline__ void widen(float (&v)[8]) const {
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    }
};

// Channel c of a head as it enters the scores: channels i and i + rot_dims / 2 turn together, the rest pass, zeros behind.
__device__ __forceinline__ float rotated_channel(const float* head, int c, int dim, int rot_dims, const double* frequency, int position) {
    if (c >= dim) return 0.0f;
    if (c >= rot_dims) return head[c];
    const int half = rot_dims >> 1;
    const int pair = c < half ? c : c - half;
    float cosine, sine;
    rotary(position, frequency[pair], cosine, sine);
    const float u = head[pair], v = head[pair + half];
    return c < half ? u * cosine - v * sine : v * cosine + u * sine;
}

__host__ __device__ inline int attention_active_splits(int position, int chunk, int keys_per_split) {
    return position % chunk / keys_per_split + 1;
}

__host__ __device__ inline int attention_lds_floats(int gq, int k_stride, int v_stride) {
    const int scores = gq * k_stride + gq * kAttTile + 3 * gq;
    const int combine = 4 * gq * v_stride;
    return (scores > combine ? scores : combine) + 8;
}

// FUSED: q comes from the projections and is rotated here, and the block that holds the row's own key rotates and stores
// key and value first.  Otherwise q_rot and the cache are complete.  GQ query heads at a time; VC: pieces of 128 channels of a
// head.  Sixteen lanes hold a key (or a value) of 128 channels, a wave four of them, the block sixteen; a tile's eight keys
// and values of a lane are requested at once, before the first is used.
template <class T, int GQ, int VC, bool FUSED>
__device__ __forceinline__ void chunk_attention_block(const ChunkAttentionParams& prm, int split, int kv_head, int row, float* lds) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int sub = lane >> 4, l16 = lane & 15;
    const int position = position_of(prm.position_dev, prm.position) + row;
    const int in_chunk = position % prm.chunk;
    const int first = position - in_chunk;
    const int n = in_chunk + 1;
    const int begin = split * prm.part.keys_per_split;
    const int end = min(n, begin + prm.part.keys_per_split);
    if (begin >= end) return;
    const float* proj = prm.proj + row * prm.ld_proj;
    T* k_cache = static_cast<T*>(prm.k_cache) + static_cast<int64_t>(kv_head) * prm.ring * prm.k_stride;
    T* v_cache = static_cast<T*>(prm.v_cache) + static_cast<int64_t>(kv_head) * prm.ring * prm.v_stride;
    if (FUSED && end == n) {
        const int64_t slot = position % prm.ring;
        const float* k = proj + prm.k_column + kv_head * prm.dim;
        const float* v = proj + prm.v_column + kv_head * prm.vdim;
        for (int c = tid; c < prm.k_stride; c += kDecThreads)
            k_cache[slot * prm.k_stride + c] = from_f32<T>(rotated_channel(k, c, prm.dim, prm.rot_dims, prm.frequency, position));
        for (int c = tid; c < prm.v_stride; c += kDecThreads) v_cache[slot * prm.v_stride + c] = from_f32<T>(c < prm.vdim ? v[c] : 0.0f);
        __threadfence_block();
    }
    const int base_slot = first % prm.ring;
    auto slot_of = [&](int key) {
        const int s = base_slot + key;
        return static_cast<int64_t>(s >= prm.ring ? s - prm.ring : s);
    };
    const int group = prm.heads / prm.kv_heads;
    float* qs = lds;                           // [GQ][k_stride]
    float* sc = qs + GQ * prm.k_stride;        // [GQ][kAttTile]
    float* sh_m = sc + GQ * kAttTile;          // [GQ] running maximum, then sum, then rescaling factor
    float* sh_l = sh_m + GQ;
    float* sh_f = sh_l + GQ;
    for (int g0 = 0; g0 < group; g0 += GQ) {
        const int heads = min(GQ, group - g0);
        const int head0 = kv_head * group + g0;
        __syncthreads();
        for (int i = tid; i < GQ * prm.k_stride; i += kDecThreads) {
            const int g = i / prm.k_stride, c = i - g * prm.k_stride;
            float q = 0.0f;
            if (g < heads) {
                if (FUSED) q = to_f32(from_f32<T>(rotated_channel(proj + (head0 + g) * prm.dim, c, prm.dim, prm.rot_dims, prm.frequency, position)));
                else q = to_f32(static_cast<const T*>(prm.q_rot)[(static_cast<int64_t>(row) * prm.heads + head0 + g) * prm.k_stride + c]);
            }
            qs[i] = q;
        }
        if (tid < GQ) {
            sh_m[tid] = -INFINITY;
            sh_l[tid] = 0.0f;
        }
        float acc[GQ][VC][8];
#pragma unroll
        for (int g = 0; g < GQ; ++g)
#pragma unroll
            for (int x = 0; x < VC; ++x)
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[g][x][e] = 0.0f;
        __syncthreads();
        float q[GQ][VC][8];                    // (channels past the head: zeros, against whatever the clamped loads bring)
#pragma unroll
        for (int g = 0; g < GQ; ++g)
#pragma unroll
            for (int x = 0; x < VC; ++x)
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const int c = x * 128 + l16 * 8 + e;
                    q[g][x][e] = c < prm.k_stride ? qs[g * prm.k_stride + min(c, prm.k_stride - 1)] : 0.0f;
                }
        for (int tile = begin; tile < end; tile += kAttTile) {
            const int keys = min(kAttTile, end - tile);
            constexpr int kEach = kAttTile / 16;
            Raw8<T> k_raw[kEach][VC], v_raw[kEach][VC];
#pragma unroll
            for (int i = 0; i < kEach; ++i) {  // (keys past the last repeat it: not used)
                const int64_t slot = slot_of(tile + min(wave * 4 + sub + 16 * i, keys - 1));
#pragma unroll
                for (int x = 0; x < VC; ++x) k_raw[i][x].load(k_cache + slot * prm.k_stride + min(x * 128 + l16 * 8, prm.k_stride - 8));
            }
#pragma unroll
            for (int i = 0; i < kEach; ++i) {
                const int64_t slot = slot_of(tile + min(wave * 4 + sub + 16 * i, keys - 1));
#pragma unroll
                for (int x = 0; x < VC; ++x) v_raw[i][x].load(v_cache + slot * prm.v_stride + min(x * 128 + l16 * 8, prm.v_stride - 8));
            }
#pragma unroll
            for (int i = 0; i < kEach; ++i) {
                const int j = wave * 4 + sub + 16 * i;
                float s[GQ];
#pragma unroll
                for (int g = 0; g < GQ; ++g) s[g] = 0.0f;
#pragma unroll
                for (int x = 0; x < VC; ++x) {
                    float kv[8];
                    k_raw[i][x].widen(kv);
#pragma unroll
                    for (int g = 0; g < GQ; ++g)
#pragma unroll
                        for (int e = 0; e < 8; ++e) s[g] = fmaf(kv[e], q[g][x][e], s[g]);
                }
#pragma unroll
                for (int g = 0; g < GQ; ++g) {
                    s[g] = row16_allreduce_sum(s[g]);
                    if (l16 == 0) sc[g * kAttTile + j] = s[g] * prm.scale;
                }
            }
            __syncthreads();
            for (int g = wave; g < GQ; g += 4) {
                const float s0 = lane < keys ? sc[g * kAttTile + lane] : -INFINITY;
                const float s1 = lane + 64 < keys ? sc[g * kAttTile + lane + 64] : -INFINITY;
                const float before = sh_m[g];
                const float largest = fmaxf(before, wave_max(fmaxf(s0, s1)));
                const float p0 = lane < keys ? expf(s0 - largest) : 0.0f;
                const float p1 = lane + 64 < keys ? expf(s1 - largest) : 0.0f;
                sc[g * kAttTile + lane] = p0;
                sc[g * kAttTile + lane + 64] = p1;
                const float factor = expf(before - largest);
                const float sum = wave_sum(p0 + p1);
                if (lane == 0) {
                    sh_m[g] = largest;
                    sh_l[g] = sh_l[g] * factor + sum;
                    sh_f[g] = factor;
                }
            }
            __syncthreads();
#pragma unroll
            for (int g = 0; g < GQ; ++g) {
                const float f = sh_f[g];
#pragma unroll
                for (int x = 0; x < VC; ++x)
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[g][x][e] *= f;
            }
#pragma unroll
            for (int i = 0; i < kEach; ++i) {  // (weights past the last key are zero)
                const int j = wave * 4 + sub + 16 * i;
#pragma unroll
                for (int x = 0; x < VC; ++x) {
                    float vv[8];
                    v_raw[i][x].widen(vv);
#pragma unroll
                    for (int g = 0; g < GQ; ++g) {
                        const float p = sc[g * kAttTile + j];
#pragma unroll
                        for (int e = 0; e < 8; ++e) acc[g][x][e] = fmaf(p, vv[e], acc[g][x][e]);
                    }
                }
            }
            __syncthreads();
        }
        if (tid < heads) {
            const int64_t at = (static_cast<int64_t>(row) * prm.heads + head0 + tid) * prm.part.splits + split;
            prm.part.ml[at * 2] = sh_m[tid];
            prm.part.ml[at * 2 + 1] = sh_l[tid];
        }
        __syncthreads();
        float* combine = lds;                  // [4 waves][GQ][v_stride]
#pragma unroll
        for (int g = 0; g < GQ; ++g)
#pragma unroll
            for (int x = 0; x < VC; ++x)
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    float v = acc[g][x][e];
                    v += __shfl_xor(v, 16, 64);
                    v += __shfl_xor(v, 32, 64);
                    const int c = x * 128 + l16 * 8 + e;
                    if (sub == 0 && c < prm.v_stride) combine[(wave * GQ + g) * prm.v_stride + c] = v;
                }
        __syncthreads();
        for (int i = tid; i < heads * prm.vdim; i += kDecThreads) {
            const int g = i / prm.vdim, c = i - g * prm.vdim;
            const int64_t at = (static_cast<int64_t>(row) * prm.heads + head0 + g) * prm.part.splits + split;
            const int step = GQ * prm.v_stride, from = g * prm.v_stride + c;
            prm.part.acc[at * prm.vdim + c] = (combine[from] + combine[from + step]) + (combine[from + 2 * step] + combine[from + 3 * step]);
        }
    }
}

}  // namespace qm
