// qm_decoder_decay_chunks.hip — linear attention with a per-head decay over a prompt's rows, in chunks of 64 tokens (gfx950).
//
// With S the state before a chunk and d the head's decay, token i of the chunk gives
//   o_i = d^(i+1) S^T q_i + sum_{j <= i} d^(i-j) (q_i . k_j) v_j,      S' = d^n S + sum_j d^(n-1-j) k_j v_j^T.
// Three launches: every chunk's own contribution to the state, all at once; a walk over the chunks that turns the
// contributions into the state before each chunk (element by element, so the whole state is walked in parallel); every
// chunk's outputs, all at once.  All products are fp32 on the matrix cores, powers of d have non-negative exponents only.
// Bound: the bytes of the states between the launches and the fp32 matrix cores, whichever is longer.
#include "../qm_host.h"
#include "qm_decoder_mfma32.h"

namespace qm {

constexpr int kDecaySlice = 64;                // value channels staged at once
constexpr int kDecayVStride = kDecaySlice + 4;

// Rotation of every row's q and k in place, k scaled: a block per row, a pair's angle once for all heads.
__global__ __launch_bounds__(kDecThreads) void decay_rotate_kernel(DecayAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int row = static_cast<int>(blockIdx.x), half = prm.rot_dims >> 1;
    const int position = position_of(prm.position_dev, prm.position) + row;
    float* sh_cos = lds;
    float* sh_sin = lds + half;
    for (int i = threadIdx.x; i < half; i += kDecThreads) rotary(position, prm.frequency[i], sh_cos[i], sh_sin[i]);
    __syncthreads();
    float* q = prm.proj + row * prm.ld_proj + prm.q_column;
    float* k = prm.proj + row * prm.ld_proj + prm.k_column;
#pragma unroll 2
    for (int i = threadIdx.x; i < prm.heads * prm.dim; i += kDecThreads) {
        const int c = i % prm.dim;
        if (c < half) {
            const float cosine = sh_cos[c], sine = sh_sin[c];
            const float qu = q[i], qv = q[i + half], ku = k[i] * prm.k_scale, kv = k[i + half] * prm.k_scale;
            q[i] = qu * cosine - qv * sine;
            q[i + half] = qv * cosine + qu * sine;
            k[i] = ku * cosine - kv * sine;
            k[i + half] = kv * cosine + ku * sine;
        } else if (c >= prm.rot_dims) {
            k[i] *= prm.k_scale;
        }
    }
}

// Rows [t0, t0 + 64) of a head's q, k or v columns into LDS, through silu unless they were rotated (zeros past the rows or
// the head), times factor(j): sixteen threads take 64 columns of a row, four each.  request_rows asks for columns c4 .. c4 + 3
// of the thread's four rows, put_rows stores them.
__device__ __forceinline__ void request_rows(const DecayAttentionParams& prm, int t0, int column, int columns, int c, float4 (&x)[4]) {
    const int row = threadIdx.x >> 4;
    const bool vectors = ((column | columns | prm.ld_proj) & 3) == 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {              // (rows past the last repeat it, with factor zero: no branch around a load)
        const float* p = prm.proj + min(t0 + row + 16 * i, prm.rows - 1) * prm.ld_proj + column;
        if (vectors) {
            x[i] = load4_if(c < columns, p, c >> 2);
        } else {
            float e[4];
#pragma unroll
            for (int n = 0; n < 4; ++n) {
                const float v = p[min(c + n, columns - 1)];
                e[n] = c + n < columns ? v : 0.0f;
            }
            x[i] = make_float4(e[0], e[1], e[2], e[3]);
        }
    }
}
template <class F>
__device__ __forceinline__ void put_rows(const DecayAttentionParams& prm, float* to, int stride, int t0, int c, float4 (&x)[4], F factor) {
    const int row = threadIdx.x >> 4;
    const bool silu = !(prm.options & QM_DECAY_ROTARY);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = row + 16 * i;
        const float f = t0 + j < prm.rows ? factor(j) : 0.0f;
        if (silu) x[i] = make_float4(silu_f32(x[i].x), silu_f32(x[i].y), silu_f32(x[i].z), silu_f32(x[i].w));
        *reinterpret_cast<float4*>(to + j * stride + c) = make_float4(x[i].x * f, x[i].y * f, x[i].z * f, x[i].w * f);
    }
}
// `padded`: a multiple of 16
template <class F>
__device__ __forceinline__ void stage_rows(const DecayAttentionParams& prm, float* to, int stride, int t0, int column, int columns, int padded, F factor) {
#pragma unroll 2
    for (int c = (threadIdx.x & 15) * 4; c < padded; c += 64) {
        float4 x[4];
        request_rows(prm, t0, column, columns, c, x);
        put_rows(prm, to, stride, t0, c, x, factor);
    }
}

__global__ __launch_bounds__(kDecThreads) void decay_chunk_state_kernel(DecayAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, l16 = lane & 15;
    const int head = static_cast<int>(blockIdx.x), chunk = static_cast<int>(blockIdx.y), e0 = static_cast<int>(blockIdx.z) * kDecaySlice;
    const int t0 = chunk * kDecayChunk, tokens = min(kDecayChunk, prm.rows - t0);
    const int dp = mfma32_pad(prm.dim), stride = mfma32_stride(prm.dim);
    const float* powers = prm.powers + head * kDecayPowers;
    float* ks = lds;                           // [64][stride]
    float* vs = ks + kDecayChunk * stride;     // [64][kDecayVStride]
    stage_rows(prm, ks, stride, t0, prm.k_column + head * prm.dim, prm.dim, dp, [&](int j) { return powers[tokens - 1 - j]; });
    stage_rows(prm, vs, kDecayVStride, t0, prm.v_column + head * prm.vdim + e0, prm.vdim - e0, kDecaySlice, [](int) { return 1.0f; });
    __syncthreads();
    float* out = prm.scratch + (static_cast<int64_t>(chunk) * prm.heads + head) * prm.dim * prm.vdim;
    for (int d0 = 16 * wave; d0 < dp; d0 += 64) {
        f32x4_t acc[4] = {};
        for (int j0 = 0; j0 < kDecayChunk; j0 += 4) {
            const float a = ks[(j0 + g) * stride + d0 + l16];
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[e] = mfma32(a, vs[(j0 + g) * kDecayVStride + 16 * e + l16], acc[e]);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int column = e0 + 16 * e + l16;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = d0 + 4 * g + r;
                if (d < prm.dim && column < prm.vdim) out[static_cast<int64_t>(d) * prm.vdim + column] = acc[e][r];
            }
        }
    }
}

// scratch[chunk] := the state before the chunk; state := the state behind the last one.
__global__ __launch_bounds__(kDecThreads) void decay_chunk_walk_kernel(DecayAttentionParams prm, int chunks) {
    const int per_head = prm.dim * prm.vdim;
    const int64_t plane = static_cast<int64_t>(prm.heads) * per_head;
    const int64_t at = static_cast<int64_t>(blockIdx.x) * kDecThreads + threadIdx.x;
    if (at >= plane) return;
    const float* powers = prm.powers + at / per_head * kDecayPowers;
    const float whole = powers[kDecayChunk], rest = powers[prm.rows - (chunks - 1) * kDecayChunk];
    float s = prm.state[at];
    constexpr int kAhead = 8;
    for (int c0 = 0; c0 < chunks; c0 += kAhead) {
        float own[kAhead];
#pragma unroll
        for (int c = 0; c < kAhead; ++c) own[c] = c0 + c < chunks ? prm.scratch[(c0 + c) * plane + at] : 0.0f;
#pragma unroll
        for (int c = 0; c < kAhead; ++c) {
            if (c0 + c >= chunks) break;
            prm.scratch[(c0 + c) * plane + at] = s;
            s = fmaf(c0 + c == chunks - 1 ? rest : whole, s, own[c]);
        }
    }
    prm.state[at] = s;
}

__global__ __launch_bounds__(kDecThreads) void decay_chunk_output_kernel(DecayAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, l16 = lane & 15;
    const int head = static_cast<int>(blockIdx.x), chunk = static_cast<int>(blockIdx.y);
    const int t0 = chunk * kDecayChunk, e0 = static_cast<int>(blockIdx.z) * kDecaySlice;
    const int dp = mfma32_pad(prm.dim), stride = mfma32_stride(prm.dim);
    const float* powers = prm.powers + head * kDecayPowers;
    float* qs = lds;                           // [64][stride]
    float* ks = qs + kDecayChunk * stride;     // [64][stride], then the weights and the values, [64][kDecayVStride] each
    float* ps = ks;
    float* vs = ks + kDecayChunk * kDecayVStride;
    auto one = [](int) { return 1.0f; };
    const int c4 = (threadIdx.x & 15) * 4;
    float4 value[4];
    request_rows(prm, t0, prm.v_column + head * prm.vdim + e0, prm.vdim - e0, c4, value);
    const float* before = prm.scratch + (static_cast<int64_t>(chunk) * prm.heads + head) * prm.dim * prm.vdim;
    const int column = e0 + 16 * wave + l16;
    auto request_state = [&](int d0, float (&s)[4]) __attribute__((always_inline)) {          // (q is zero past the head)
#pragma unroll
        for (int t = 0; t < 4; ++t) s[t] = before[min(d0 + 4 * g + t, prm.dim - 1) * prm.vdim + min(column, prm.vdim - 1)];
    };
    constexpr int kAhead = 4;                  // blocks of 16 state rows under way
    float state[kAhead][4];
#pragma unroll
    for (int u = 0; u < kAhead; ++u) request_state(16 * u, state[u]);
    stage_rows(prm, qs, stride, t0, prm.q_column + head * prm.dim, prm.dim, dp, one);
    stage_rows(prm, ks, stride, t0, prm.k_column + head * prm.dim, prm.dim, dp, one);
    __syncthreads();
    f32x4_t score[4] = {};                     // rows of tile `wave`, column tiles 0 .. wave
    for (int d0 = 0; d0 < dp; d0 += 16) {
        const float4 a = *reinterpret_cast<const float4*>(qs + (16 * wave + l16) * stride + d0 + 4 * g);
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j <= wave) score[j] = mfma32_block(a, *reinterpret_cast<const float4*>(ks + (16 * j + l16) * stride + d0 + 4 * g), score[j]);
    }
    __syncthreads();
    put_rows(prm, vs, kDecayVStride, t0, c4, value, one);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j > wave) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * wave + 4 * g + r, column = 16 * j + l16;
            ps[row * kDecayVStride + column] = column <= row ? score[j][r] * powers[row - column] : 0.0f;
        }
    }
    float decayed[4];                          // d^(i+1) of the lane's row of each tile
#pragma unroll
    for (int i = 0; i < 4; ++i) decayed[i] = powers[16 * i + l16 + 1];
    __syncthreads();
    f32x4_t acc[4] = {};
    for (int base = 0; base < dp; base += 16 * kAhead) {
#pragma unroll
        for (int u = 0; u < kAhead; ++u) {
            const int d0 = base + 16 * u;
            if (d0 >= dp) break;
            const float4 b = make_float4(state[u][0], state[u][1], state[u][2], state[u][3]);
            if (base + 16 * kAhead < dp) request_state(d0 + 16 * kAhead, state[u]);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                float4 a = *reinterpret_cast<const float4*>(qs + (16 * i + l16) * stride + d0 + 4 * g);
                a.x *= decayed[i]; a.y *= decayed[i]; a.z *= decayed[i]; a.w *= decayed[i];
                acc[i] = mfma32_block(a, b, acc[i]);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const float* v = vs + (16 * j + 4 * g) * kDecayVStride + 16 * wave + l16;
        const float4 b = make_float4(v[0], v[kDecayVStride], v[2 * kDecayVStride], v[3 * kDecayVStride]);
#pragma unroll
        for (int i = j; i < 4; ++i)
            acc[i] = mfma32_block(*reinterpret_cast<const float4*>(ps + (16 * i + l16) * kDecayVStride + 16 * j + 4 * g), b, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = t0 + 16 * i + 4 * g + r;
            if (t < prm.rows && column < prm.vdim) prm.out[static_cast<int64_t>(t) * prm.heads * prm.vdim + head * prm.vdim + column] = acc[i][r];
        }
}

int64_t decay_scratch_floats(int rows, int heads, int dim, int vdim) {
    if (rows < kChunkedRows || heads <= 0 || dim <= 0 || vdim <= 0) return 0;
    return static_cast<int64_t>((rows + kDecayChunk - 1) / kDecayChunk) * heads * dim * vdim;
}

int32_t launch_decay_chunks(const DecayAttentionParams& prm, hipStream_t stream) {
    const int chunks = (prm.rows + kDecayChunk - 1) / kDecayChunk;
    const int stride = mfma32_stride(prm.dim), slices = (prm.vdim + kDecaySlice - 1) / kDecaySlice;
    const int state_lds = static_cast<int>(sizeof(float)) * kDecayChunk * (stride + kDecayVStride);
    const int output_lds = static_cast<int>(sizeof(float)) * kDecayChunk * (stride + (stride > 2 * kDecayVStride ? stride : 2 * kDecayVStride));
    static std::atomic<bool> raised[2][kMaxDevices];
    int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(decay_chunk_state_kernel), kDotLdsMost, raised[0]);
    if (rc == QM_OK) rc = ensure_dynamic_lds(reinterpret_cast<const void*>(decay_chunk_output_kernel), kDotLdsMost, raised[1]);
    if (rc != QM_OK) return rc;
    if (output_lds > kDotLdsMost || chunks > 65535 || prm.scratch_floats < decay_scratch_floats(prm.rows, prm.heads, prm.dim, prm.vdim)) return QM_ERR_WORKSPACE;
    if (prm.options & QM_DECAY_ROTARY)
        hipLaunchKernelGGL(decay_rotate_kernel, dim3(prm.rows), dim3(kDecThreads), sizeof(float) * (prm.rot_dims + 1), stream, prm);
    hipLaunchKernelGGL(decay_chunk_state_kernel, dim3(prm.heads, chunks, slices), dim3(kDecThreads), state_lds, stream, prm);
    const int64_t plane = static_cast<int64_t>(prm.heads) * prm.dim * prm.vdim;
    hipLaunchKernelGGL(decay_chunk_walk_kernel, dim3(static_cast<unsigned>((plane + kDecThreads - 1) / kDecThreads)), dim3(kDecThreads), 0, stream, prm,
                       chunks);
    hipLaunchKernelGGL(decay_chunk_output_kernel, dim3(prm.heads, chunks, slices), dim3(kDecThreads), output_lds, stream, prm);
    return launch_status();
}

}  // namespace qm
