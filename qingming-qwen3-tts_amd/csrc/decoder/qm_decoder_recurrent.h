// qm_decoder_recurrent.h — the two recurrences, token by token: a head's state [dim][columns] is cut along its columns
// (value channels), which never interact.  A wave owns 16 columns; its four lane groups of 16 hold a quarter of the
// state's rows each, in registers, so a sum over the rows is RD fmafs and two exchanges between lanes.  The vectors that
// all columns share are put into LDS a few tokens at a time.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

constexpr int kRecTokens = 8;                  // tokens whose vectors are in LDS at once
constexpr int kRecColumns = 64;                // state columns of a block
// a lane group's quarter of a vector starts 4 floats further on than the last one ended: the four quarters of one read lie
// in different banks
__host__ __device__ inline int rec_stride(int rd) { return 4 * (rd + 4); }
template <int RD>
__device__ __forceinline__ int rec_at(int channel) { return (channel / RD) * (RD + 4) + channel % RD; }

// (Rows and columns past the state repeat its last ones: no branch around a load.  Their vectors are zeros, and they are
// not stored.)
template <int RD>
__device__ __forceinline__ void load_state(float (&s)[RD], const float* state, int dim, int columns, int sub, int column) {
    column = min(column, columns - 1);
#pragma unroll
    for (int i = 0; i < RD; ++i) s[i] = state[min(sub * RD + i, dim - 1) * columns + column];
}
template <int RD>
__device__ __forceinline__ void store_state(const float (&s)[RD], float* state, int dim, int columns, int sub, int column) {
#pragma unroll
    for (int i = 0; i < RD; ++i) {
        const int d = sub * RD + i;
        if (d < dim && column < columns) state[static_cast<int64_t>(d) * columns + column] = s[i];
    }
}
__device__ __forceinline__ float quarter_sum(float v) {
    v += __shfl_xor(v, 16, 64);
    v += __shfl_xor(v, 32, 64);
    return v;
}

__host__ __device__ inline int decay_lds_floats(int rd) { return kRecTokens * 2 * rec_stride(rd); }

// Channel c of a head's q and k as they enter the recurrence: silu of the projections, or rotated (channels i and
// i + rot_dims / 2 together) and k scaled.
__device__ __forceinline__ void decay_channel(const DecayAttentionParams& prm, const float* q_head, const float* k_head, int c, int position, float& q,
                                              float& k) {
    q = q_head[c];
    k = k_head[c];
    if (!(prm.options & QM_DECAY_ROTARY)) {
        q = silu_f32(q);
        k = silu_f32(k);
        return;
    }
    if (c < prm.rot_dims) {
        const int half = prm.rot_dims >> 1, pair = c < half ? c : c - half, other = c < half ? c + half : pair;
        float cosine, sine;
        rotary(position, prm.frequency[pair], cosine, sine);
        if (c < half) sine = -sine;
        q = q * cosine + q_head[other] * sine;
        k = k * cosine + k_head[other] * sine;
    }
    k *= prm.k_scale;
}
__device__ __forceinline__ float decay_value(const DecayAttentionParams& prm, float v) { return prm.options & QM_DECAY_ROTARY ? v : silu_f32(v); }

// Linear attention with decay: head `head`, state columns [64 slice, 64 slice + 64).
template <int RD>
__device__ __forceinline__ void decay_attention_block(const DecayAttentionParams& prm, int head, int slice, float* lds) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane >> 4;
    const int column = slice * kRecColumns + wave * 16 + (lane & 15);
    constexpr int kStride = 4 * (RD + 4);
    float* state = prm.state + static_cast<int64_t>(head) * prm.dim * prm.vdim;
    const float decay = prm.powers[head * kDecayPowers + 1];
    const int position = position_of(prm.position_dev, prm.position);
    float s[RD];
    load_state<RD>(s, state, prm.dim, prm.vdim, sub, column);
    for (int t0 = 0; t0 < prm.rows; t0 += kRecTokens) {
        const int tokens = min(kRecTokens, prm.rows - t0);
        __syncthreads();
        for (int i = tid; i < tokens * 4 * RD; i += kDecThreads) {
            const int t = i / (4 * RD), c = i % (4 * RD);
            const float* p = prm.proj + (t0 + t) * prm.ld_proj + head * prm.dim;
            float* to = lds + t * 2 * kStride + rec_at<RD>(c);
            float q = 0.0f, k = 0.0f;
            if (c < prm.dim) decay_channel(prm, p + prm.q_column, p + prm.k_column, c, position + t0 + t, q, k);
            to[0] = q;
            to[kStride] = k;
        }
        float v[kRecTokens];
#pragma unroll
        for (int t = 0; t < kRecTokens; ++t)
            v[t] = t < tokens && column < prm.vdim ? decay_value(prm, prm.proj[(t0 + t) * prm.ld_proj + prm.v_column + head * prm.vdim + column]) : 0.0f;
        __syncthreads();
#pragma unroll
        for (int t = 0; t < kRecTokens; ++t) {
            if (t >= tokens) break;
            const float* q = lds + t * 2 * kStride + sub * (RD + 4);
            const float* k = q + kStride;
            float o = 0.0f;
#pragma unroll
            for (int i = 0; i < RD; i += 4) {
                const float4 kk = *reinterpret_cast<const float4*>(k + i), qq = *reinterpret_cast<const float4*>(q + i);
                s[i] = fmaf(kk.x, v[t], decay * s[i]); o = fmaf(qq.x, s[i], o);
                s[i + 1] = fmaf(kk.y, v[t], decay * s[i + 1]); o = fmaf(qq.y, s[i + 1], o);
                s[i + 2] = fmaf(kk.z, v[t], decay * s[i + 2]); o = fmaf(qq.z, s[i + 2], o);
                s[i + 3] = fmaf(kk.w, v[t], decay * s[i + 3]); o = fmaf(qq.w, s[i + 3], o);
            }
            o = quarter_sum(o);
            if (sub == 0 && column < prm.vdim) prm.out[static_cast<int64_t>(t0 + t) * prm.heads * prm.vdim + head * prm.vdim + column] = o;
        }
    }
    store_state<RD>(s, state, prm.dim, prm.vdim, sub, column);
}

__host__ __device__ inline int delta_lds_floats(int rd, int rank) { return kRecTokens * (5 * rec_stride(rd) + 1 + rank); }

// exp(-exp(-1/2) sigmoid(z))
__device__ __forceinline__ float delta_decay_of(float z) { return expf(-0.60653065971263342f * sigmoid_f32(z)); }

// The decay of channel `at` (of all heads') at one token, given tanh of the token's rank-sized projection in LDS.
__device__ __forceinline__ float delta_channel_decay(const DeltaParams& prm, const float* tanh_z, int at) {
    float z = prm.w0[at];
    const int all = prm.heads * prm.dim;
#pragma unroll 16
    for (int r = 0; r < prm.rank; ++r) z = fmaf(prm.w2[static_cast<int64_t>(r) * all + at], tanh_z[r], z);
    return delta_decay_of(z);
}

// Generalized delta rule: head `head`, state columns [64 slice, 64 slice + 64).
template <int RD>
__device__ __forceinline__ void general_delta_block(const DeltaParams& prm, int head, int slice, float* lds) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane >> 4;
    const int column = slice * kRecColumns + wave * 16 + (lane & 15);
    constexpr int kStride = 4 * (RD + 4);
    float* state = prm.state + static_cast<int64_t>(head) * prm.dim * prm.dim;
    float* inverse = lds + kRecTokens * 5 * kStride;              // [kRecTokens]
    float* tanh_z = inverse + kRecTokens;                          // [kRecTokens][rank]
    float s[RD];
    load_state<RD>(s, state, prm.dim, prm.dim, sub, column);
    for (int t0 = 0; t0 < prm.rows; t0 += kRecTokens) {
        const int tokens = min(kRecTokens, prm.rows - t0);
        __syncthreads();
        for (int i = tid; i < tokens * prm.rank; i += kDecThreads) {
            const int t = i / prm.rank, r = i - t * prm.rank;
            tanh_z[i] = tanhf(prm.proj[(t0 + t) * prm.ld_proj + prm.z_column + r]);
        }
        __syncthreads();
        for (int t = wave; t < tokens; t += 4) {                   // a wave per token: the unit key's factor
            const float* p = prm.proj + (t0 + t) * prm.ld_proj + head * prm.dim + prm.k_column;
            float sq = 0.0f;
            for (int c = lane; c < prm.dim; c += 64) sq = fmaf(p[c], p[c], sq);
            sq = wave_sum(sq);
            if (lane == 0) inverse[t] = 1.0f / sqrtf(sq + prm.unit_eps);
        }
        __syncthreads();
        for (int i = tid; i < tokens * 4 * RD; i += kDecThreads) { // w, a u, u, k, r of every token and channel of the head
            const int t = i / (4 * RD), c = i % (4 * RD);
            const float* p = prm.proj + (t0 + t) * prm.ld_proj + head * prm.dim + c;
            float w = 0.0f, au = 0.0f, u = 0.0f, k = 0.0f, r = 0.0f;
            if (c < prm.dim) {
                const int at = head * prm.dim + c;
                k = p[prm.k_column];
                r = p[prm.r_column];
                u = k * inverse[t];
                au = sigmoid_f32(p[prm.a_column] + prm.a_bias[at]) * u;
                w = delta_channel_decay(prm, tanh_z + t * prm.rank, at);
            }
            float* put = lds + t * 5 * kStride + rec_at<RD>(c);
            put[0] = w; put[kStride] = au; put[2 * kStride] = u; put[3 * kStride] = k; put[4 * kStride] = r;
        }
        float v[kRecTokens];
#pragma unroll
        for (int t = 0; t < kRecTokens; ++t)
            v[t] = t < tokens && column < prm.dim ? prm.proj[(t0 + t) * prm.ld_proj + prm.v_column + head * prm.dim + column] : 0.0f;
        __syncthreads();
#pragma unroll
        for (int t = 0; t < kRecTokens; ++t) {
            if (t >= tokens) break;
            const float* w = lds + t * 5 * kStride + sub * (RD + 4);
            float seen = 0.0f;
#pragma unroll
            for (int i = 0; i < RD; i += 4) {
                const float4 u = *reinterpret_cast<const float4*>(w + 2 * kStride + i);
                seen = fmaf(u.x, s[i], seen); seen = fmaf(u.y, s[i + 1], seen);
                seen = fmaf(u.z, s[i + 2], seen); seen = fmaf(u.w, s[i + 3], seen);
            }
            seen = quarter_sum(seen);
            float o = 0.0f;
#pragma unroll
            for (int i = 0; i < RD; i += 4) {
                const float4 ww = *reinterpret_cast<const float4*>(w + i), au = *reinterpret_cast<const float4*>(w + kStride + i);
                const float4 k = *reinterpret_cast<const float4*>(w + 3 * kStride + i), r = *reinterpret_cast<const float4*>(w + 4 * kStride + i);
                s[i] = fmaf(k.x, v[t], fmaf(-au.x, seen, ww.x * s[i])); o = fmaf(r.x, s[i], o);
                s[i + 1] = fmaf(k.y, v[t], fmaf(-au.y, seen, ww.y * s[i + 1])); o = fmaf(r.y, s[i + 1], o);
                s[i + 2] = fmaf(k.z, v[t], fmaf(-au.z, seen, ww.z * s[i + 2])); o = fmaf(r.z, s[i + 2], o);
                s[i + 3] = fmaf(k.w, v[t], fmaf(-au.w, seen, ww.w * s[i + 3])); o = fmaf(r.w, s[i + 3], o);
            }
            o = quarter_sum(o);
            if (sub == 0 && column < prm.dim) prm.out[static_cast<int64_t>(t0 + t) * prm.heads * prm.dim + head * prm.dim + column] = o;
        }
    }
    store_state<RD>(s, state, prm.dim, prm.dim, sub, column);
}

// One token of the delta rule: everything from memory is requested before anything waits, a channel's decay is summed by
// 256 / (4 RD) threads.
__host__ __device__ inline int delta_step_lds_floats(int rd, int rank) { return 5 * rec_stride(rd) + rank + 256 + 8; }
template <int RD>
__device__ __forceinline__ void general_delta_step(const DeltaParams& prm, int head, int slice, float* lds) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane >> 4;
    const int column = slice * kRecColumns + wave * 16 + (lane & 15);
    constexpr int kStride = 4 * (RD + 4), kChannels = 4 * RD, kParts = kDecThreads / kChannels, kAhead = 16;
    const int c = tid % kChannels, part = tid / kChannels;
    float* sh_z = lds + 5 * kStride;                               // [rank]
    float* sh_sum = sh_z + prm.rank;                               // [parts][channels]
    float* sh_sq = sh_sum + kDecThreads;                           // [4]
    const bool in = c < prm.dim;
    const int at = head * prm.dim + (in ? c : 0), all = prm.heads * prm.dim;
    const float* p = prm.proj + at;
    const float k_read = p[prm.k_column], r = p[prm.r_column], a = p[prm.a_column];
    const float k = in ? k_read : 0.0f;
    const float bias = prm.a_bias[at], w0 = prm.w0[at];
    const float v = prm.proj[prm.v_column + head * prm.dim + min(column, prm.dim - 1)];
    const int ranks = (prm.rank + kParts - 1) / kParts, first = part * ranks, last = min(prm.rank, first + ranks);
    const float* w2 = prm.w2 + at;
    float piece[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead; ++i) piece[i] = w2[static_cast<int64_t>(min(first + i, prm.rank - 1)) * all];
    const float z0 = tid < prm.rank ? prm.proj[prm.z_column + tid] : 0.0f;
    float* state = prm.state + static_cast<int64_t>(head) * prm.dim * prm.dim;
    float s[RD];
    load_state<RD>(s, state, prm.dim, prm.dim, sub, column);
    if (tid < prm.rank) sh_z[tid] = tanhf(z0);
    for (int i = tid + kDecThreads; i < prm.rank; i += kDecThreads) sh_z[i] = tanhf(prm.proj[prm.z_column + i]);
    const float sq = wave_sum(part == 0 ? k * k : 0.0f);
    if (lane == 0) sh_sq[wave] = sq;
    __syncthreads();
    float z = 0.0f;
    for (int i0 = first; i0 < last; i0 += kAhead) {
        float now[kAhead];
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            now[i] = piece[i];
            piece[i] = w2[static_cast<int64_t>(min(i0 + kAhead + i, prm.rank - 1)) * all];
        }
#pragma unroll
        for (int i = 0; i < kAhead; ++i)
            if (i0 + i < last) z = fmaf(now[i], sh_z[i0 + i], z);
    }
    sh_sum[tid] = z;
    __syncthreads();
    if (part == 0) {
        float sum = w0;
#pragma unroll
        for (int i = 0; i < kParts; ++i) sum += sh_sum[i * kChannels + c];
        const float u = k * (1.0f / sqrtf((sh_sq[0] + sh_sq[1]) + (sh_sq[2] + sh_sq[3]) + prm.unit_eps));
        float* put = lds + rec_at<RD>(c);
        put[0] = in ? delta_decay_of(sum) : 0.0f;
        put[kStride] = in ? sigmoid_f32(a + bias) * u : 0.0f;
        put[2 * kStride] = u;
        put[3 * kStride] = k;
        put[4 * kStride] = in ? r : 0.0f;
    }
    __syncthreads();
    const float* w = lds + sub * (RD + 4);
    float seen = 0.0f, o = 0.0f;
#pragma unroll
    for (int i = 0; i < RD; ++i) seen = fmaf(w[2 * kStride + i], s[i], seen);
    seen = quarter_sum(seen);
#pragma unroll
    for (int i = 0; i < RD; ++i) {
        s[i] = fmaf(w[3 * kStride + i], v, fmaf(-w[kStride + i], seen, w[i] * s[i]));
        o = fmaf(w[4 * kStride + i], s[i], o);
    }
    o = quarter_sum(o);
    if (sub == 0 && column < prm.dim) prm.out[head * prm.dim + column] = o;
    store_state<RD>(s, state, prm.dim, prm.dim, sub, column);
}

}  // namespace qm
