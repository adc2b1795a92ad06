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

// (v_exp_f32 and v_rcp_f32 are good to one unit in the last place)
__device__ __forceinline__ float reciprocal(float x) { return __builtin_amdgcn_rcpf(x); }
__device__ __forceinline__ float sigmoid_f32(float z) { return reciprocal(1.0f + fast_exp2(-z * kLog2e)); }
__device__ __forceinline__ float silu_f32(float z) { return z * sigmoid_f32(z); }

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

// The residual sum and its norm for one row by a block of 256 threads.  Rows are padded with zeros to ld_h columns, and a
// thread owns the float4s tid, tid + 256, ... of a row (NV of them): everything the row needs is requested before the first
// sum waits.  sh_red: 16 floats of LDS; h may be LDS or global memory.  The caller puts a barrier between this and any use
// of sh_red or h by other threads.
__device__ __forceinline__ float4 load4(const float* p, int v) { return reinterpret_cast<const float4*>(p)[v]; }
__device__ __forceinline__ float4 load4(const uint16_t* p, int v) {
    const uint2 w = reinterpret_cast<const uint2*>(p)[v];
    return make_float4(lo_bf16(w.x), hi_bf16(w.x), lo_bf16(w.y), hi_bf16(w.y));
}
__device__ __forceinline__ void store4(float* p, int v, float a, float b, float c, float d) { reinterpret_cast<float4*>(p)[v] = make_float4(a, b, c, d); }
__device__ __forceinline__ void store4(uint16_t* p, int v, float a, float b, float c, float d) {
    reinterpret_cast<uint2*>(p)[v] = make_uint2(pack_bf16_pair(a, b), pack_bf16_pair(c, d));
}
__device__ __forceinline__ float square_sum(float4 v, float sum) { return fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sum)))); }
// Element v, or zeros where it is not wanted: the load is made either way (from the first element), because a load under a
// condition would wait its turn behind a branch.
template <class P>
__device__ __forceinline__ float4 load4_if(bool wanted, const P* p, int v) {
    const float4 x = load4(p, wanted ? v : 0);
    return make_float4(wanted ? x.x : 0.0f, wanted ? x.y : 0.0f, wanted ? x.z : 0.0f, wanted ? x.w : 0.0f);
}
// acc + f * y * w
__device__ __forceinline__ float4 weighted(float4 acc, float f, float4 y, float4 w) {
    return make_float4(fmaf(f * y.x, w.x, acc.x), fmaf(f * y.y, w.y, acc.y), fmaf(f * y.z, w.z, acc.z), fmaf(f * y.w, w.w, acc.w));
}

template <class T, int NV>
__device__ __forceinline__ void residual_norm_row(const ResidualParams& prm, int row, float* sh_red, T* h, bool write_x) {
    const int tid = threadIdx.x;
    const int64_t src = prm.row_map ? prm.row_map[row] : row;
    const int vectors = static_cast<int>(prm.ld_h >> 2);
    const float* y_row[3];
    bool normed[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        y_row[i] = i < prm.terms ? prm.term[i].y + src * prm.term[i].ld : nullptr;
        normed[i] = i < prm.terms && prm.term[i].norm_w;
    }
    const uint16_t *embedding = nullptr, *bigram = nullptr;
    if (!prm.x_in) {
        const int64_t token = min(max(prm.tokens[src], 0), prm.vocab - 1);
        embedding = prm.embed + token * prm.ld_h;
        if (prm.buckets > 0) {
            const int64_t before = prm.tokens[src - 1];
            bigram = prm.bigram + (before < 0 ? prm.buckets : (before * prm.mul_prev + token * prm.mul_cur) % prm.buckets) * prm.ld_h;
        }
    }
    const float4 zero = make_float4(0.0f, 0.0f, 0.0f, 0.0f), one = make_float4(1.0f, 1.0f, 1.0f, 1.0f);
    float4 x[NV], y[3][NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int v = tid + i * kDecThreads;
        const bool in = v < vectors;
        x[i] = embedding ? load4_if(in, embedding, v) : load4_if(in, prm.x_in + src * prm.ld_h, v);
        if (bigram) x[i] = weighted(x[i], 1.0f, load4_if(in, bigram, v), one);
#pragma unroll
        for (int t = 0; t < 3; ++t) y[t][i] = y_row[t] ? load4_if(in, y_row[t], v) : zero;
    }
    const float inv_width = 1.0f / static_cast<float>(prm.width);
    float factor[3] = {0.0f, 0.0f, 0.0f};
    if (normed[0] || normed[1] || normed[2]) {
#pragma unroll
        for (int t = 0; t < 3; ++t)
#pragma unroll
            for (int i = 0; i < NV; ++i) factor[t] = square_sum(y[t][i], factor[t]);
        block_sums<3>(factor, sh_red);
    }
#pragma unroll
    for (int t = 0; t < 3; ++t) {
        const float inverse = normed[t] ? 1.0f / sqrtf(factor[t] * inv_width + prm.eps) : 1.0f;
        factor[t] = t < prm.terms ? prm.term[t].scale * inverse : 0.0f;
    }
    float total[1] = {0.0f};
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int v = tid + i * kDecThreads;
        if (v >= vectors) continue;
        float4 add = zero;
#pragma unroll
        for (int t = 0; t < 3; ++t)
            if (y_row[t]) add = weighted(add, factor[t], y[t][i], normed[t] ? load4(prm.term[t].norm_w, v) : one);
        x[i] = weighted(x[i], 1.0f, add, one);
        if (prm.step_vec) x[i] = weighted(x[i], 1.0f, load4(prm.step_vec, v), one);
        if (write_x && prm.x_out) reinterpret_cast<float4*>(prm.x_out + static_cast<int64_t>(row) * prm.ld_h)[v] = x[i];
        total[0] = square_sum(x[i], total[0]);
    }
    block_sums<1>(total, sh_red + 12);
    const float inverse = 1.0f / sqrtf(total[0] * inv_width + prm.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int v = tid + i * kDecThreads;
        if (v >= vectors) continue;
        const float4 w = load4(prm.norm_w, v);
        store4(h, v, x[i].x * inverse * w.x, x[i].y * inverse * w.y, x[i].z * inverse * w.z, x[i].w * inverse * w.w);
    }
}

// The factor that a gate's projection g becomes.
__device__ __forceinline__ float gate_f32(float g, bool silu) { return silu ? silu_f32(g) : sigmoid_f32(g); }

// One row of the gated norm by a block of 256 threads; sh_red: 4 floats of LDS.
template <class T>
__device__ __forceinline__ void gated_norm_row(const GatedNormParams& prm, int64_t row, float* sh_red, T* out) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const float* o = prm.o + row * prm.ld_o;
    const float* gate = prm.gate + row * prm.ld_gate;
    const bool silu = prm.silu != 0;
    const int total = prm.groups * prm.size;
    const float inv_size = 1.0f / static_cast<float>(prm.size);
    auto weight_at = [&](int at) { return prm.weight ? prm.weight[at] : 1.0f; };
    constexpr int kHeld = 4;                   // float4s a thread holds between its two uses of a value
    if (prm.groups == 1 && total % 4 == 0 && prm.ld_o % 4 == 0 && total <= kHeld * 4 * kDecThreads) {
        const int vectors = total >> 2;
        float4 held[kHeld], g[kHeld];
        float sq[1] = {0.0f};
#pragma unroll
        for (int i = 0; i < kHeld; ++i) {
            const int v = tid + i * kDecThreads;
            held[i] = load4_if(v < vectors, o, v);
            g[i] = load4_if(v < vectors, gate, v);
            sq[0] = square_sum(held[i], sq[0]);
        }
        block_sums<1>(sq, sh_red);
        const float inverse = 1.0f / sqrtf(sq[0] * inv_size + prm.eps);
#pragma unroll
        for (int i = 0; i < kHeld; ++i) {
            const int v = tid + i * kDecThreads;
            if (v >= vectors) continue;
            const float4 w = prm.weight ? load4(prm.weight, v) : make_float4(1.0f, 1.0f, 1.0f, 1.0f);
            store4(out, v, held[i].x * inverse * w.x * gate_f32(g[i].x, silu), held[i].y * inverse * w.y * gate_f32(g[i].y, silu),
                   held[i].z * inverse * w.z * gate_f32(g[i].z, silu), held[i].w * inverse * w.w * gate_f32(g[i].w, silu));
        }
    } else if (prm.groups == 1) {
        float sq[1] = {0.0f};
        for (int c = tid; c < total; c += kDecThreads) sq[0] = fmaf(o[c], o[c], sq[0]);
        block_sums<1>(sq, sh_red);
        const float inverse = 1.0f / sqrtf(sq[0] * inv_size + prm.eps);
        for (int c = tid; c < total; c += kDecThreads)
            out[c] = from_f32<T>(o[c] * inverse * weight_at(c) * gate_f32(gate[c], silu));
    } else {
        // a wave per slice, a slice of up to 256 values held by its lanes
        for (int g = wave; g < prm.groups; g += kDecThreads / 64) {
            float held[4], gates[4], sq = 0.0f;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int c = lane + 64 * i;
                const bool in = c < prm.size;
                const int at = g * prm.size + (in ? c : 0);
                const float value = o[at];
                gates[i] = gate[at];
                held[i] = in ? value : 0.0f;
                sq = fmaf(held[i], held[i], sq);
            }
            for (int c = lane + 256; c < prm.size; c += 64) sq = fmaf(o[g * prm.size + c], o[g * prm.size + c], sq);
            const float inverse = 1.0f / sqrtf(wave_sum(sq) * inv_size + prm.eps);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int c = lane + 64 * i, at = g * prm.size + c;
                if (c < prm.size) out[at] = from_f32<T>(held[i] * inverse * weight_at(at) * gate_f32(gates[i], silu));
            }
            for (int c = lane + 256; c < prm.size; c += 64) {
                const int at = g * prm.size + c;
                out[at] = from_f32<T>(o[at] * inverse * weight_at(at) * gate_f32(gate[at], silu));
            }
        }
    }
    for (int c = total + tid; c < prm.ld_out; c += kDecThreads) out[c] = from_f32<T>(0.0f);
}

// One row's heads, combined, by a block of 256 threads; `active` splits hold keys.  sh_w: heads * active floats of LDS.
template <class T>
__device__ __forceinline__ void merge_attention_row(const AttentionPartials& p, int64_t row, int active, float* sh_w, T* out, int64_t ld_out) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int h = wave; h < p.heads; h += kDecThreads / 64) {      // each split's factor: a wave per head, a lane per split
        const int64_t at = ((row * p.heads + h) * p.splits + min(lane, active - 1)) * 2;
        const float m_read = p.ml[at], l_read = p.ml[at + 1];
        const float m = lane < active ? m_read : -INFINITY, l = lane < active ? l_read : 0.0f;
        const float w = fast_exp2((m - wave_max(m)) * kLog2e);
        const float total = wave_sum(w * l);
        if (lane < active) sh_w[h * active + lane] = w / total;
    }
    __syncthreads();
    const int n = p.heads * p.vdim;
    const float* acc = p.acc + row * p.heads * p.splits * p.vdim;
    if (p.vdim % 4 == 0) {
        const int per_head = p.vdim >> 2;
        for (int i = threadIdx.x; i < n >> 2; i += kDecThreads) {
            const int h = i / per_head, e = i - h * per_head;
            const float4* from = reinterpret_cast<const float4*>(acc + static_cast<int64_t>(h) * p.splits * p.vdim) + e;
            float4 sum = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
            for (int s0 = 0; s0 < active; s0 += 8) {               // (splits past the last: the last one, with factor zero)
                float4 v[8];
#pragma unroll
                for (int s = 0; s < 8; ++s) v[s] = from[min(s0 + s, active - 1) * per_head];
#pragma unroll
                for (int s = 0; s < 8; ++s) {
                    const float w = s0 + s < active ? sh_w[h * active + min(s0 + s, active - 1)] : 0.0f;
                    sum.x = fmaf(w, v[s].x, sum.x); sum.y = fmaf(w, v[s].y, sum.y);
                    sum.z = fmaf(w, v[s].z, sum.z); sum.w = fmaf(w, v[s].w, sum.w);
                }
            }
            store4(out, i, sum.x, sum.y, sum.z, sum.w);
        }
    } else {
        for (int i = threadIdx.x; i < n; i += kDecThreads) {
            const int h = i / p.vdim, e = i - h * p.vdim;
            float sum = 0.0f;
            for (int s = 0; s < active; ++s) sum = fmaf(sh_w[h * active + s], acc[(static_cast<int64_t>(h) * p.splits + s) * p.vdim + e], sum);
            out[i] = from_f32<T>(sum);
        }
    }
    for (int c = n + threadIdx.x; c < ld_out; c += kDecThreads) out[c] = from_f32<T>(0.0f);
}

// Rotary factors of pair i at a position: the angle in double (position * frequency, reduced to one turn), its sine and
// cosine in fp32.
__device__ __forceinline__ void rotary(int position, double frequency, float& cosine, float& sine) {
    const double angle = static_cast<double>(position) * frequency;
    const double turns = rint(angle * 0.15915494309189535);
    const float reduced = static_cast<float>(fma(-turns, 6.283185307179586, angle));
    sincosf(reduced, &sine, &cosine);
}

// n values divided by their root mean square and weighted, by a block of 256 threads, zeros behind them up to `padded`;
// sh_red: 4 floats of LDS.
template <class T>
__device__ __forceinline__ void slice_norm_row(const float* x, const float* weight, int n, int64_t padded, float eps, float* sh_red, T* out) {
    const int tid = threadIdx.x;
    constexpr int kHeld = 4;
    float held[kHeld], sq[1] = {0.0f};
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
        const int c = tid + i * kDecThreads;
        const float value = x[min(c, n - 1)];
        held[i] = c < n ? value : 0.0f;
        sq[0] = fmaf(held[i], held[i], sq[0]);
    }
    for (int c = tid + kHeld * kDecThreads; c < n; c += kDecThreads) sq[0] = fmaf(x[c], x[c], sq[0]);
    block_sums<1>(sq, sh_red);
    const float inverse = 1.0f / sqrtf(sq[0] / static_cast<float>(n) + eps);
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
        const int c = tid + i * kDecThreads;
        if (c < n) out[c] = from_f32<T>(held[i] * inverse * weight[c]);
    }
    for (int c = tid + kHeld * kDecThreads; c < n; c += kDecThreads) out[c] = from_f32<T>(x[c] * inverse * weight[c]);
    for (int64_t c = n + tid; c < padded; c += kDecThreads) out[c] = from_f32<T>(0.0f);
}

}  // namespace qm
