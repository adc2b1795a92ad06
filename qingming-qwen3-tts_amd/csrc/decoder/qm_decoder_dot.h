// qm_decoder_dot.h — the weight-streaming tile of the decoder language models' linears: a block of four waves, each with
// kDotRows weight rows (half as many output channels of a gate/up pair), against R input rows in LDS.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

constexpr int kDotRows = 4;                    // weight rows a wave streams at once
constexpr int kDotLds = 128 * 1024;            // input rows in LDS

__host__ __device__ inline int dot_tile_outputs(const DecLinearGroup& g) { return 4 * (g.w_up ? kDotRows / 2 : kDotRows); }
__host__ __device__ inline int dot_tiles(const DecLinearGroup& g) { return g.n / dot_tile_outputs(g); }

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

// The weight rows of a wave in tile `tile` of the group.
struct DotRows {
    const uint16_t* row[kDotRows];
    int channel;                               // first output of the wave
};
__device__ __forceinline__ DotRows dot_rows(const DecLinearGroup& g, int tile) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    DotRows d;
    if (g.w_up) {
        d.channel = tile * dot_tile_outputs(g) + wave * (kDotRows / 2);
#pragma unroll
        for (int i = 0; i < kDotRows / 2; ++i) {
            d.row[2 * i] = g.w + static_cast<int64_t>(d.channel + i) * g.k;
            d.row[2 * i + 1] = g.w_up + static_cast<int64_t>(d.channel + i) * g.k;
        }
    } else {
        d.channel = tile * dot_tile_outputs(g) + wave * kDotRows;
#pragma unroll
        for (int i = 0; i < kDotRows; ++i) d.row[i] = g.w + static_cast<int64_t>(d.channel + i) * g.k;
    }
    return d;
}

constexpr int kDotAhead = 4;                   // pieces of each weight row under way at once

// Requests the first pieces of a wave's weight rows; they may be asked for before the input rows are known.
__device__ __forceinline__ void dot_request(const DotRows& d, int k, int k0, uint4 (&piece)[kDotAhead][kDotRows]) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int u = 0; u < kDotAhead; ++u) {
        const int at = k0 + u * 512 + lane * 8;
#pragma unroll
        for (int i = 0; i < kDotRows; ++i)
            piece[u][i] = at < k ? *reinterpret_cast<const uint4*>(d.row[i] + at) : make_uint4(0, 0, 0, 0);
    }
}

// One tile: xs holds R input rows [R][k] in LDS; `piece` the pieces requested for k0 = 0.
template <class T, int R>
__device__ __forceinline__ void dot_finish(const DecLinearGroup& g, const DotRows& d, uint4 (&piece)[kDotAhead][kDotRows], const T* xs, int row0,
                                           int rows) {
    const int lane = threadIdx.x & 63;
    const int k = g.k;
    float acc[kDotRows][R];
#pragma unroll
    for (int i = 0; i < kDotRows; ++i)
#pragma unroll
        for (int r = 0; r < R; ++r) acc[i][r] = 0.0f;
    for (int k0 = 0;;) {
#pragma unroll
        for (int u = 0; u < kDotAhead; ++u) {
            const int at = k0 + u * 512 + lane * 8;
            if (at < k) {
#pragma unroll
                for (int r = 0; r < R; ++r)
#pragma unroll
                    for (int i = 0; i < kDotRows; ++i) acc[i][r] = dot8(piece[u][i], xs + r * k + at, acc[i][r]);
            }
        }
        k0 += kDotAhead * 512;
        if (k0 >= k) break;
        dot_request(d, k, k0, piece);
    }
#pragma unroll
    for (int i = 0; i < kDotRows; ++i)
#pragma unroll
        for (int r = 0; r < R; ++r) acc[i][r] = wave_sum(acc[i][r]);
    if (lane != 0) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        if (r >= rows) break;
        const int64_t base = (row0 + r) * g.ldo + d.channel;
        if (g.w_up) {
#pragma unroll
            for (int i = 0; i < kDotRows / 2; ++i)
                static_cast<T*>(g.out)[base + i] = from_f32<T>(silu_f32(acc[2 * i][r]) * acc[2 * i + 1][r]);
        } else {
#pragma unroll
            for (int i = 0; i < kDotRows; ++i) g.out32[base + i] = acc[i][r];
        }
    }
}

template <class T, int R>
__device__ __forceinline__ void dot_tile(const DecLinearGroup& g, const T* xs, int tile, int row0, int rows) {
    const DotRows d = dot_rows(g, tile);
    uint4 piece[kDotAhead][kDotRows];
    dot_request(d, g.k, 0, piece);
    dot_finish<T, R>(g, d, piece, xs, row0, rows);
}

}  // namespace qm
