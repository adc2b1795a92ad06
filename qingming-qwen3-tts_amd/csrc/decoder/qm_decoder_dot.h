// qm_decoder_dot.h — the weight-streaming tile of the decoder language models' linears: a block of four waves, each with
// NR weight rows (half as many output channels of a gate/up pair), against R input rows in LDS.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

constexpr int kDotLds = 128 * 1024;            // input rows in LDS
constexpr int kDotAhead = 4;                   // pieces of each weight row under way at once

// Outputs of a block's tile with NR weight rows per wave, and the tiles of a linear.
template <int NR>
__host__ __device__ inline int dot_tile_outputs(const DecLinearGroup& g) { return 4 * (g.w_up ? NR / 2 : NR); }
template <int NR>
__host__ __device__ inline int dot_tiles(const DecLinearGroup& g) { return g.n / dot_tile_outputs<NR>(g); }

__device__ __forceinline__ float dot8(uint4 w, const uint16_t* x, float acc) {
    const uint4 v = *reinterpret_cast<const uint4*>(x);
    acc = dot2_bf16(w.x, v.x, acc);
    acc = dot2_bf16(w.y, v.y, acc);
    acc = dot2_bf16(w.z, v.z, acc);
    return dot2_bf16(w.w, v.w, acc);
}
__device__ __forceinline__ float dot8(uint4 w, const float* x, float acc) {
    const float4 a = *reinterpret_cast<const float4*>(x), b = *reinterpret_cast<const float4*>(x + 4);
    acc = fmaf(lo_bf16(w.x), a.x, acc); acc = fmaf(hi_bf16(w.x), a.y, acc);
    acc = fmaf(lo_bf16(w.y), a.z, acc); acc = fmaf(hi_bf16(w.y), a.w, acc);
    acc = fmaf(lo_bf16(w.z), b.x, acc); acc = fmaf(hi_bf16(w.z), b.y, acc);
    acc = fmaf(lo_bf16(w.w), b.z, acc); acc = fmaf(hi_bf16(w.w), b.w, acc);
    return acc;
}

// The weight rows of a wave in tile `tile` of the linear.
template <int NR>
struct DotRows {
    const uint16_t* row[NR];
    int channel;                               // first output of the wave
};
template <int NR>
__device__ __forceinline__ DotRows<NR> dot_rows(const DecLinearGroup& g, int tile) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    DotRows<NR> d;
    if (g.w_up) {
        d.channel = tile * dot_tile_outputs<NR>(g) + wave * (NR / 2);
#pragma unroll
        for (int i = 0; i < NR / 2; ++i) {
            d.row[2 * i] = g.w + static_cast<int64_t>(d.channel + i) * g.k;
            d.row[2 * i + 1] = g.w_up + static_cast<int64_t>(d.channel + i) * g.k;
        }
    } else {
        d.channel = tile * dot_tile_outputs<NR>(g) + wave * NR;
#pragma unroll
        for (int i = 0; i < NR; ++i) d.row[i] = g.w + static_cast<int64_t>(d.channel + i) * g.k;
    }
    return d;
}

template <int NR>
__device__ __forceinline__ void dot_request_one(const DotRows<NR>& d, int k, int at, uint4 (&piece)[NR]) {
    const int from = at < k ? at : 0;          // (past the end: not used; a load under a condition would stand behind a branch)
#pragma unroll
    for (int i = 0; i < NR; ++i) piece[i] = *reinterpret_cast<const uint4*>(d.row[i] + from);
}
// Requests the first pieces of a wave's weight rows; they may be asked for before the input rows are known.
template <int NR>
__device__ __forceinline__ void dot_request(const DotRows<NR>& d, int k, uint4 (&piece)[kDotAhead][NR]) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int u = 0; u < kDotAhead; ++u) dot_request_one<NR>(d, k, u * 512 + lane * 8, piece[u]);
}

// One tile: xs holds R input rows [R][k] in LDS, `piece` the first pieces.
template <class T, int R, int NR>
__device__ __forceinline__ void dot_finish(const DecLinearGroup& g, const DotRows<NR>& d, uint4 (&piece)[kDotAhead][NR], const T* xs, int row0,
                                           int rows) {
    const int lane = threadIdx.x & 63;
    const int k = g.k;
    float acc[NR][R];
#pragma unroll
    for (int i = 0; i < NR; ++i)
#pragma unroll
        for (int r = 0; r < R; ++r) acc[i][r] = 0.0f;
    for (int k0 = 0; k0 < k; k0 += kDotAhead * 512) {
#pragma unroll
        for (int u = 0; u < kDotAhead; ++u) {
            const int at = k0 + u * 512 + lane * 8;
            if (at < k) {
#pragma unroll
                for (int r = 0; r < R; ++r)
#pragma unroll
                    for (int i = 0; i < NR; ++i) acc[i][r] = dot8(piece[u][i], xs + r * k + at, acc[i][r]);
            }
            if (k0 + kDotAhead * 512 < k) dot_request_one<NR>(d, k, at + kDotAhead * 512, piece[u]);
        }
    }
#pragma unroll
    for (int i = 0; i < NR; ++i)
#pragma unroll
        for (int r = 0; r < R; ++r) acc[i][r] = wave_sum(acc[i][r]);
    if (lane != 0) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        if (r >= rows) break;
        const int64_t base = (row0 + r) * g.ldo + d.channel;
        if (g.w_up) {
#pragma unroll
            for (int i = 0; i < NR / 2; ++i)
                static_cast<T*>(g.out)[base + i] = from_f32<T>(silu_f32(acc[2 * i][r]) * acc[2 * i + 1][r]);
        } else {
#pragma unroll
            for (int i = 0; i < NR; ++i) g.out32[base + i] = acc[i][r];
        }
    }
}

// The linear and the tile in it that number `tile` of a launch means.
template <int NR>
__device__ __forceinline__ int dot_group(const DecLinearParams& prm, int& tile) {
    int g = 0;
    while (g + 1 < prm.groups && tile >= dot_tiles<NR>(prm.group[g])) tile -= dot_tiles<NR>(prm.group[g++]);
    return g;
}
template <int NR>
inline int dot_tiles_of(const DecLinearParams& prm) {
    int tiles = 0;
    for (int g = 0; g < prm.groups; ++g) tiles += dot_tiles<NR>(prm.group[g]);
    return tiles;
}

}  // namespace qm
