// qm_decoder_device.h — device helpers shared by the decoder language models' kernels (gfx950, wave64).
//
// Activations that a matrix product reads are bf16 (T = uint16_t) when the model is served and fp32 (T = float) in the
// 32-bit mode; weights are bf16 in both (the checkpoint's own format, so nothing is lost).  Everything else — the residual
// stream, projections on their way into a mixer, norms, scores, recurrent state — is fp32 throughout.
#pragma once

#include "../qm_device.h"
#include "qm_decoder_ops.h"

namespace qm {

constexpr int kDecThreads = 256;

__device__ __forceinline__ float to_f32(uint16_t v) { return bf2f(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
template <class T> __device__ __forceinline__ T from_f32(float v);
template <> __device__ __forceinline__ uint16_t from_f32<uint16_t>(float v) { return f2bf(v); }
template <> __device__ __forceinline__ float from_f32<float>(float v) { return v; }

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }

// Sum / maximum over the 64 lanes of a wave, in every lane.
__device__ __forceinline__ float wave_sum(float v) {
    v = row16_allreduce_sum(v);
    v += __shfl_xor(v, 16, 64);
    v += __shfl_xor(v, 32, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int m = 1; m < 64; m *= 2) v = fmaxf(v, __shfl_xor(v, m, 64));
    return v;
}

// N sums over the 256 threads of a block at once, in every thread.  sh: 4 * N floats of LDS, free again for the next call
// after the caller's next barrier (two calls in a row take two areas).
template <int N>
__device__ __forceinline__ void block_sums(float (&v)[N], float* sh) {
    const int wave = threadIdx.x >> 6;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        v[i] = wave_sum(v[i]);
        if ((threadIdx.x & 63) == 0) sh[i * 4 + wave] = v[i];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = (sh[i * 4] + sh[i * 4 + 1]) + (sh[i * 4 + 2] + sh[i * 4 + 3]);
}

// A position is known to the host, or lives in device memory where a captured graph finds it.
__device__ __forceinline__ int position_of(const int32_t* device, int host) { return device ? *device : host; }

// One row by a block of 256 threads.  sh_x: width floats, sh_red: 16 floats, both LDS; h may be LDS or global memory.
// The caller puts a barrier between this and any use of sh_x, sh_red or h by other threads.
template <class T>
__device__ __forceinline__ void residual_norm_row(const ResidualParams& prm, int row, float* sh_x, float* sh_red, T* h, bool write_x) {
    const int tid = threadIdx.x;
    const int width = prm.width;
    const int64_t src = prm.row_map ? prm.row_map[row] : row;
    const float* y0 = prm.terms > 0 ? prm.term[0].y + src * prm.term[0].ld : nullptr;
    const float* y1 = prm.terms > 1 ? prm.term[1].y + src * prm.term[1].ld : nullptr;
    const float* y2 = prm.terms > 2 ? prm.term[2].y + src * prm.term[2].ld : nullptr;
    float sq[3] = {0.0f, 0.0f, 0.0f};
    const bool n0 = y0 && prm.term[0].norm_w, n1 = y1 && prm.term[1].norm_w, n2 = y2 && prm.term[2].norm_w;
    if (n0 || n1 || n2) {
        for (int c = tid; c < width; c += kDecThreads) {
            if (n0) sq[0] = fmaf(y0[c], y0[c], sq[0]);
            if (n1) sq[1] = fmaf(y1[c], y1[c], sq[1]);
            if (n2) sq[2] = fmaf(y2[c], y2[c], sq[2]);
        }
        block_sums<3>(sq, sh_red);
    }
    const float inv_width = 1.0f / static_cast<float>(width);
    const float f0 = y0 ? prm.term[0].scale * (n0 ? 1.0f / sqrtf(sq[0] * inv_width + prm.eps) : 1.0f) : 0.0f;
    const float f1 = y1 ? prm.term[1].scale * (n1 ? 1.0f / sqrtf(sq[1] * inv_width + prm.eps) : 1.0f) : 0.0f;
    const float f2 = y2 ? prm.term[2].scale * (n2 ? 1.0f / sqrtf(sq[2] * inv_width + prm.eps) : 1.0f) : 0.0f;
    const uint16_t* embedding = nullptr;
    if (!prm.x_in) {
        const int token = min(max(prm.tokens[src], 0), prm.vocab - 1);
        embedding = prm.embed + static_cast<int64_t>(token) * width;
    }
    float total[1] = {0.0f};
    for (int c = tid; c < width; c += kDecThreads) {
        float x = embedding ? bf2f(embedding[c]) : prm.x_in[src * width + c];
        float add = 0.0f;
        if (y0) add = fmaf(f0 * y0[c], n0 ? prm.term[0].norm_w[c] : 1.0f, add);
        if (y1) add = fmaf(f1 * y1[c], n1 ? prm.term[1].norm_w[c] : 1.0f, add);
        if (y2) add = fmaf(f2 * y2[c], n2 ? prm.term[2].norm_w[c] : 1.0f, add);
        x += add;
        if (prm.step_vec) x += prm.step_vec[c];
        sh_x[c] = x;
        if (write_x && prm.x_out) prm.x_out[static_cast<int64_t>(row) * width + c] = x;
        total[0] = fmaf(x, x, total[0]);
    }
    block_sums<1>(total, sh_red + 12);
    const float inverse = 1.0f / sqrtf(total[0] * inv_width + prm.eps);
    for (int c = tid; c < prm.ld_h; c += kDecThreads)
        h[c] = c < width ? from_f32<T>(sh_x[c] * inverse * prm.norm_w[c]) : from_f32<T>(0.0f);
}

// One row of the gated norm by a block of 256 threads; sh_red: 4 floats of LDS.
template <class T>
__device__ __forceinline__ void gated_norm_row(const GatedNormParams& prm, int64_t row, float* sh_red, T* out) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const float* o = prm.o + row * prm.ld_o;
    const float* gate = prm.gate + row * prm.ld_gate;
    const int total = prm.groups * prm.size;
    const float inv_size = 1.0f / static_cast<float>(prm.size);
    if (prm.groups == 1) {
        float sq[1] = {0.0f};
        for (int c = tid; c < total; c += kDecThreads) sq[0] = fmaf(o[c], o[c], sq[0]);
        block_sums<1>(sq, sh_red);
        const float inverse = 1.0f / sqrtf(sq[0] * inv_size + prm.eps);
        for (int c = tid; c < total; c += kDecThreads)
            out[c] = from_f32<T>(o[c] * inverse * prm.weight[c] * sigmoid_f32(gate[c]));
    } else {
        for (int g = wave; g < prm.groups; g += kDecThreads / 64) {
            float sq = 0.0f;
            for (int c = lane; c < prm.size; c += 64) {
                const float v = o[g * prm.size + c];
                sq = fmaf(v, v, sq);
            }
            const float inverse = 1.0f / sqrtf(wave_sum(sq) * inv_size + prm.eps);
            for (int c = lane; c < prm.size; c += 64) {
                const int at = g * prm.size + c;
                out[at] = from_f32<T>(o[at] * inverse * prm.weight[at] * sigmoid_f32(gate[at]));
            }
        }
    }
    for (int c = total + tid; c < prm.ld_out; c += kDecThreads) out[c] = from_f32<T>(0.0f);
}

// One row's heads, combined, by a block of 256 threads; `active` splits hold keys.
template <class T>
__device__ __forceinline__ void merge_attention_row(const AttentionPartials& p, int64_t row, int active, T* out, int64_t ld_out) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int h = wave; h < p.heads; h += kDecThreads / 64) {
        const int64_t base = (row * p.heads + h) * p.splits;
        const float m = lane < active ? p.ml[(base + lane) * 2] : -INFINITY;
        const float l = lane < active ? p.ml[(base + lane) * 2 + 1] : 0.0f;
        const float largest = wave_max(m);
        float w = lane < active ? expf(m - largest) : 0.0f;
        w = w / wave_sum(w * l);
        for (int e0 = 0; e0 < p.vdim; e0 += 64) {
            const int e = e0 + lane;
            float sum = 0.0f;
            for (int s = 0; s < active; ++s) {
                const float ws = __shfl(w, s, 64);
                if (e < p.vdim) sum = fmaf(ws, p.acc[(base + s) * p.vdim + e], sum);
            }
            if (e < p.vdim) out[h * p.vdim + e] = from_f32<T>(sum);
        }
    }
    for (int c = p.heads * p.vdim + threadIdx.x; c < ld_out; c += kDecThreads) out[c] = from_f32<T>(0.0f);
}

// Rotary factors of pair i at a position: the angle in double (position * frequency, reduced to one turn), its sine and
// cosine in fp32.
__device__ __forceinline__ void rotary(int position, double frequency, float& cosine, float& sine) {
    const double angle = static_cast<double>(position) * frequency;
    const double turns = rint(angle * 0.15915494309189535);
    const float reduced = static_cast<float>(fma(-turns, 6.283185307179586, angle));
    sincosf(reduced, &sine, &cosine);
}

}  // namespace qm
