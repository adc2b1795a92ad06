// qm_decoder_delta_chunks.hip — the generalized delta rule over a prompt's rows, in chunks of 32 tokens (gfx950).
//
// S_t = diag(w_t) S_{t-1} - (a_t u_t)(u_t^T S_{t-1}) + k_t v_t^T,  o_t = S_t^T r_t.  Let W_t be the product of the decays of
// the chunk's tokens up to t (per channel, W before the first token 1), S the state before the chunk, and
//   U_t = u_t W_{t-1},  A_t = a_t u_t / W_t,  K_t = k_t / W_t,  R_t = r_t W_t   (rows of [32][dim] matrices).
// What the removal terms read, p_t = u_t^T S_{t-1}, solves a triangular system:  (I + L_A) P = U S + L_K V  with
// L_A[t][s] = U_t . A_s and L_K[t][s] = U_t . K_s for s < t.  So P = M S + N V with M = (I + L_A)^-1 U, N = (I + L_A)^-1 L_K,
// and with the lower triangles (diagonal included) D_A[t][s] = R_t . A_s, D_K[t][s] = R_t . K_s:
//   O = (R - D_A M) S + (D_K - D_A N) V,      S' = diag(W) (S - A^T P + K^T V),  W the whole chunk's product.
// M, N, R - D_A M, D_K - D_A N do not depend on S: one launch computes them for every chunk and head at once.  A second one
// walks the chunks; columns of S never interact, so its blocks take 16 columns each, four waves sharing the rows.  A decay is
// never below exp(-e^(-1/2)) = 0.545, so 1 / W stays under 3e8 and everything fits fp32; A and K enter the state already
// multiplied by W.  All products are fp32 on the matrix cores.
// Bound: the walk, a chain of rows / 32 dependent steps.
#include "../qm_host.h"
#include "qm_decoder_mfma32.h"
#include "qm_decoder_recurrent.h"

namespace qm {

constexpr int kDeltaChunk = 32;
constexpr int kDeltaMat = kDeltaChunk + 4;     // row stride of a [32][32] matrix in LDS

// Channels of a head as the prepared matrices have them: what lies behind the head's own is zero (decays: one).
__host__ __device__ inline int delta_pad(int dim) { return (dim + 63) / 64 * 64; }

// Scratch of a (chunk, head), floats: M, X (32 x dp), -A^T W, K^T W (dp x 32), N, Y [32][32], W [dp].  The first four are kept
// as the walk's left operands: 16 x 16 blocks of 64 float4s, lane l's being row l % 16, columns 4 (l / 16) .. + 3 of the block.
struct DeltaScratch {
    int m, x, at, kt, n, y, w, floats;
};
__host__ __device__ inline DeltaScratch delta_scratch(int dim) {
    const int dp = delta_pad(dim), rows = kDeltaChunk * dp, square = kDeltaChunk * kDeltaChunk;
    DeltaScratch s;
    s.m = 0; s.x = rows; s.at = 2 * rows; s.kt = 3 * rows; s.n = 4 * rows; s.y = s.n + square; s.w = s.y + square;
    s.floats = s.w + dp;
    return s;
}
__host__ __device__ inline int delta_z_stride(int rank) { return (rank + 3) / 4 * 4; }
// the float4 of row r, columns c .. c + 3 of block `block` (16 x 16)
__device__ __forceinline__ int operand_at(int block, int r, int c) { return (block * 64 + (c >> 2 & 3) * 16 + (r & 15)) * 4; }
inline int delta_prepare_lds(int dim) {
    const int half = 2 * kDeltaChunk * mfma32_stride(dim), squares = 5 * kDeltaChunk * kDeltaMat;
    return kDeltaChunk + half + (half > squares ? half : squares);
}

__global__ __launch_bounds__(kDecThreads) void delta_chunk_prepare_kernel(DeltaParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, l16 = lane & 15;
    const int chunk = static_cast<int>(blockIdx.x), head = static_cast<int>(blockIdx.y);
    const int t0 = chunk * kDeltaChunk, tokens = min(kDeltaChunk, prm.rows - t0);
    const int dim = prm.dim, dp = delta_pad(dim), stride = mfma32_stride(dim);
    const DeltaScratch at = delta_scratch(dim);
    float* scratch = prm.scratch + (static_cast<int64_t>(chunk) * prm.heads + head) * at.floats;
    float* inverse = lds;                      // [32]
    float* us = inverse + kDeltaChunk;         // [32][stride] each; us holds the decays first
    float* rs = us + kDeltaChunk * stride;
    float* as = rs + kDeltaChunk * stride;
    float* ks = as + kDeltaChunk * stride;
    float* mats = as;                          // once A and K are used up: L_A, L_K, D_A, D_K, each [32][kDeltaMat]
    float* inverted = mats + 4 * kDeltaChunk * kDeltaMat;          // and (I + L_A)^-1
    float* zs = rs;                            // tanh of the rank-sized projection, [32][z_stride], until the decays are there
    const int z_stride = delta_z_stride(prm.rank);

    for (int i = tid; i < kDeltaChunk * z_stride; i += kDecThreads) {
        const int t = i / z_stride, r = i - t * z_stride;
        zs[i] = t < tokens && r < prm.rank ? tanhf(prm.proj[(t0 + t) * prm.ld_proj + prm.z_column + r]) : 0.0f;
    }
    for (int t = wave; t < tokens; t += 4) {
        const float* k = prm.proj + (t0 + t) * prm.ld_proj + prm.k_column + head * dim;
        float sq = 0.0f;
        for (int c = lane; c < dim; c += 64) sq = fmaf(k[c], k[c], sq);
        sq = wave_sum(sq);
        if (lane == 0) inverse[t] = 1.0f / sqrtf(sq + prm.unit_eps);
    }
    __syncthreads();
    const int all = prm.heads * dim;
    for (int i = tid; i < 2 * dp; i += kDecThreads) {              // decays: a thread takes a channel of sixteen tokens
        const int c = i % dp, first = i / dp * 16;
        float z[16];
        const float bias = c < dim ? prm.w0[head * dim + c] : 0.0f;
#pragma unroll
        for (int t = 0; t < 16; ++t) z[t] = bias;
        if (c < dim) {
            const float* w2 = prm.w2 + head * dim + c;
#pragma unroll 4
            for (int r = 0; r < prm.rank; r += 4) {
                float w[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) w[e] = w2[static_cast<int64_t>(min(r + e, prm.rank - 1)) * all];      // (zs is zero past the rank)
#pragma unroll
                for (int t = 0; t < 16; ++t) {
                    const float4 x = *reinterpret_cast<const float4*>(zs + (first + t) * z_stride + r);
                    z[t] = fmaf(w[0], x.x, z[t]); z[t] = fmaf(w[1], x.y, z[t]);
                    z[t] = fmaf(w[2], x.z, z[t]); z[t] = fmaf(w[3], x.w, z[t]);
                }
            }
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) us[(first + t) * stride + c] = first + t < tokens && c < dim ? delta_decay_of(z[t]) : 1.0f;
    }
    __syncthreads();
    if (tid < dp) {                                                // products of decays, into rs
        float product = 1.0f;
#pragma unroll 8
        for (int t = 0; t < kDeltaChunk; ++t) {
            product *= us[t * stride + tid];
            rs[t * stride + tid] = product;
        }
        scratch[at.w + tid] = product;
    }
    __syncthreads();
    // a thread takes a channel of sixteen tokens, last token first: a token needs the products up to it and up to the one
    // before, and leaves its row of R in the product's place
    float edge[2], whole[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
        const int i = tid + n * kDecThreads, c = i % dp, first = i / dp * 16;
        const bool in = i < 2 * dp;
        edge[n] = in && first > 0 ? rs[(first - 1) * stride + c] : 1.0f;
        whole[n] = in ? rs[(kDeltaChunk - 1) * stride + c] : 1.0f;
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < 2; ++n) {
        const int i = tid + n * kDecThreads, c = i % dp, first = i / dp * 16;
        if (i >= 2 * dp) break;
        const float bias = c < dim ? prm.a_bias[head * dim + c] : 0.0f;
        for (int t1 = first + 12; t1 >= first; t1 -= 4) {
            float k[4], r[4], a[4], at_[4], kt_[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const bool in = t1 + e < tokens && c < dim;
                const float* p = prm.proj + min(t0 + t1 + e, prm.rows - 1) * prm.ld_proj + head * dim + min(c, dim - 1);
                const float k_read = p[prm.k_column], r_read = p[prm.r_column];
                a[e] = p[prm.a_column];
                k[e] = in ? k_read : 0.0f;
                r[e] = in ? r_read : 0.0f;
            }
#pragma unroll
            for (int e = 3; e >= 0; --e) {
                const int t = t1 + e;
                const float after = rs[t * stride + c], before = t > first ? rs[(t - 1) * stride + c] : edge[n];
                const float u = k[e] * inverse[min(t, tokens - 1)];
                const float removal = sigmoid_f32(a[e] + bias) * u, over = reciprocal(after);
                us[t * stride + c] = u * before;
                as[t * stride + c] = removal * over;
                ks[t * stride + c] = k[e] * over;
                rs[t * stride + c] = r[e] * after;
                at_[e] = -whole[n] * removal * over;
                kt_[e] = whole[n] * k[e] * over;
            }
            const int to = operand_at(c / 16 * 2 + t1 / 16, c, t1);
            *reinterpret_cast<float4*>(scratch + at.at + to) = make_float4(at_[0], at_[1], at_[2], at_[3]);
            *reinterpret_cast<float4*>(scratch + at.kt + to) = make_float4(kt_[0], kt_[1], kt_[2], kt_[3]);
        }
    }
    __syncthreads();
    {                                                              // wave 0: L_A, 1: L_K, 2: D_A, 3: D_K
        const float* left = wave < 2 ? us : rs;
        const float* right = wave & 1 ? ks : as;
        f32x4_t acc[2][2] = {};
        for (int d0 = 0; d0 < dp; d0 += 16) {
            float4 a[2], b[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                a[i] = *reinterpret_cast<const float4*>(left + (16 * i + l16) * stride + d0 + 4 * g);
                b[i] = *reinterpret_cast<const float4*>(right + (16 * i + l16) * stride + d0 + 4 * g);
            }
            acc[0][0] = mfma32_block(a[0], b[0], acc[0][0]);
            acc[1][0] = mfma32_block(a[1], b[0], acc[1][0]);
            acc[1][1] = mfma32_block(a[1], b[1], acc[1][1]);
        }
        __syncthreads();
        float* mat = mats + wave * kDeltaChunk * kDeltaMat;
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int j = 0; j < 2; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = 16 * i + 4 * g + r, s = 16 * j + l16;
                    mat[t * kDeltaMat + s] = s < t || (s == t && wave >= 2) ? acc[i][j][r] : 0.0f;
                }
    }
    __syncthreads();
    // (I + L_A)^-1 = [[T1, 0], [-T2 L21 T1, T2]]: the two 16 x 16 inverses by a column per thread, the third block by products
    const float* l_a = mats;
    const float* l_k = mats + kDeltaChunk * kDeltaMat;
    const float* d_a = mats + 2 * kDeltaChunk * kDeltaMat;
    const float* d_k = mats + 3 * kDeltaChunk * kDeltaMat;
    if (tid < kDeltaChunk) {
        const int b = tid & 16, c = tid & 15;
        float solved[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float v = t == c ? 1.0f : 0.0f;
#pragma unroll
            for (int s = 0; s < t; s += 4) {
                const float4 m = *reinterpret_cast<const float4*>(l_a + (b + t) * kDeltaMat + b + s);
                v = fmaf(-m.x, solved[s], v);
                if (s + 1 < t) v = fmaf(-m.y, solved[s + 1], v);
                if (s + 2 < t) v = fmaf(-m.z, solved[s + 2], v);
                if (s + 3 < t) v = fmaf(-m.w, solved[s + 3], v);
            }
            solved[t] = v;
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) inverted[(b + t) * kDeltaMat + b + c] = solved[t];
    }
    __syncthreads();
    auto left_operand = [&](const float* m, int rows, int terms) { return *reinterpret_cast<const float4*>(m + (rows + l16) * kDeltaMat + terms + 4 * g); };
    auto right_operand = [&](const float* m, int step, int terms, int columns) {
        const float* p = m + (terms + 4 * g) * step + columns + l16;
        return make_float4(p[0], p[step], p[2 * step], p[3 * step]);
    };
    auto as_operand = [](f32x4_t v) { return make_float4(v[0], v[1], v[2], v[3]); };
    if (wave == 0) {
        const f32x4_t none = {};
        const f32x4_t lower = mfma32_block(left_operand(l_a, 16, 0), right_operand(inverted, kDeltaMat, 0, 0), none);      // L21 T1
        const f32x4_t third = mfma32_block(left_operand(inverted, 16, 16), as_operand(lower), none);
#pragma unroll
        for (int r = 0; r < 4; ++r) inverted[(16 + 4 * g + r) * kDeltaMat + l16] = -third[r];
    }
    __syncthreads();
    // sixteen columns at a time of (U, L_K): times the inverse, and of (R, D_K) less D_A times that
    for (int n = wave; n < dp / 16 + 2; n += 4) {
        const bool wide = n < dp / 16;
        const int c = wide ? 16 * n : 16 * (n - dp / 16), step = wide ? stride : kDeltaMat;
        const float* y = wide ? us : l_k;
        const float* z = wide ? rs : d_k;
        float* solved_out = scratch + (wide ? at.m : at.n);
        float* rest_out = scratch + (wide ? at.x : at.y);
        const float4 y0 = right_operand(y, step, 0, c), y1 = right_operand(y, step, 16, c);
        f32x4_t m[2] = {}, x[2];
        m[0] = mfma32_block(left_operand(inverted, 0, 0), y0, m[0]);
        m[1] = mfma32_block(left_operand(inverted, 16, 0), y0, m[1]);
        m[1] = mfma32_block(left_operand(inverted, 16, 16), y1, m[1]);
#pragma unroll
        for (int b = 0; b < 2; ++b) {
#pragma unroll
            for (int r = 0; r < 4; ++r) x[b][r] = -z[(16 * b + 4 * g + r) * step + c + l16];
            x[b] = mfma32_block(left_operand(d_a, 16 * b, 0), as_operand(m[0]), x[b]);
        }
        x[1] = mfma32_block(left_operand(d_a, 16, 16), as_operand(m[1]), x[1]);
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * b + 4 * g + r;
                const int to = wide ? operand_at(2 * n + b, t, l16) + (l16 & 3) : t * kDeltaChunk + c + l16;
                solved_out[to] = m[b][r];
                rest_out[to] = -x[b][r];
            }
    }
}

// What a wave needs of a chunk besides the state: its shares of the prepared matrices, and the values of the block's columns.
template <int TW>
struct DeltaStep {
    float4 m[2][TW], x[2][TW], at[TW][2], kt[TW][2], w[TW];
    float2 n[2], y[2];
    float v[2][4], own[2];
};

// A barrier for what went into LDS: unlike __syncthreads it leaves the loads under way (the next chunk's) in flight.
__device__ __forceinline__ void block_exchange() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// TW: 16-row tiles of the state per wave (tile = wave + 4 i)
template <int TW>
__global__ __launch_bounds__(kDecThreads) void delta_chunk_walk_kernel(DeltaParams prm, int chunks) {
    constexpr int kStride = 20;                                    // the four row groups of a store lie in different banks
    __shared__ float sh[2][4][2][kDeltaChunk * kStride];           // by turns: each wave's share of P and of O
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, l16 = lane & 15;
    // (block numbers go round the dies: the blocks of a head, which read the same matrices, share one's L2)
    const int head = static_cast<int>(blockIdx.x), column = static_cast<int>(blockIdx.y) * 16 + l16;
    const int dim = prm.dim;
    const DeltaScratch at = delta_scratch(dim);
    float* state = prm.state + static_cast<int64_t>(head) * dim * dim;
    const int part = wave >> 1, pair = 2 * (wave & 1);             // the wave's terms of N V and Y V: tokens 16 part + 4 g + pair, + 1
    f32x4_t s[TW];
#pragma unroll
    for (int i = 0; i < TW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (wave + 4 * i) + 4 * g + r;
            const float value = state[min(d, dim - 1) * dim + min(column, dim - 1)];
            s[i][r] = d < dim ? value : 0.0f;
        }
    // (a token past the last meets zeros, a column past the head is not stored: both repeat the last, no branch around a load)
    const float* values = prm.proj + prm.v_column + head * dim + min(column, dim - 1);
    auto value_at = [&](int token) { return values[min(token, prm.rows - 1) * prm.ld_proj]; };
    auto request = [&](int chunk, DeltaStep<TW>& f) __attribute__((always_inline)) {
        const float* from = prm.scratch + (static_cast<int64_t>(chunk) * prm.heads + head) * at.floats;
#pragma unroll
        for (int i = 0; i < TW; ++i) {
            const int tile = wave + 4 * i;
#pragma unroll
            for (int b = 0; b < 2; ++b) {
                const int operand = ((2 * tile + b) * 64 + lane) * 4;
                f.m[b][i] = *reinterpret_cast<const float4*>(from + at.m + operand);
                f.x[b][i] = *reinterpret_cast<const float4*>(from + at.x + operand);
                f.at[i][b] = *reinterpret_cast<const float4*>(from + at.at + operand);
                f.kt[i][b] = *reinterpret_cast<const float4*>(from + at.kt + operand);
            }
            f.w[i] = *reinterpret_cast<const float4*>(from + at.w + 16 * tile + 4 * g);
        }
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const int row = (16 * b + l16) * kDeltaChunk + 16 * part + 4 * g + pair;
            f.n[b] = *reinterpret_cast<const float2*>(from + at.n + row);
            f.y[b] = *reinterpret_cast<const float2*>(from + at.y + row);
#pragma unroll
            for (int t = 0; t < 4; ++t) f.v[b][t] = value_at(chunk * kDeltaChunk + 16 * b + 4 * g + t);
            f.own[b] = value_at(chunk * kDeltaChunk + 16 * part + 4 * g + pair + b);
        }
    };
    auto walk = [&](int chunk, DeltaStep<TW>& f, DeltaStep<TW>& next) __attribute__((always_inline)) {
        // this chunk's loads, a whole step under way, have to be there; then the next one's go out
        __builtin_amdgcn_s_waitcnt((7 << 4) | (15 << 8));          // vmcnt(0), nothing else
        __builtin_amdgcn_sched_barrier(0);
        request(min(chunk + 1, chunks - 1), next);
        __builtin_amdgcn_sched_barrier(0);
        f32x4_t p[2] = {}, o[2] = {};
#pragma unroll
        for (int i = 0; i < TW; ++i) {
            const float4 b = make_float4(s[i][0], s[i][1], s[i][2], s[i][3]);
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                p[half] = mfma32_block(f.m[half][i], b, p[half]);
                o[half] = mfma32_block(f.x[half][i], b, o[half]);
            }
        }
        float (*mine)[kDeltaChunk * kStride] = sh[chunk & 1][wave];
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            p[half] = mfma32(f.n[half].y, f.own[1], mfma32(f.n[half].x, f.own[0], p[half]));
            o[half] = mfma32(f.y[half].y, f.own[1], mfma32(f.y[half].x, f.own[0], o[half]));
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                mine[0][(16 * half + 4 * g + r) * kStride + l16] = p[half][r];
                mine[1][(16 * half + 4 * g + r) * kStride + l16] = o[half][r];
            }
        }
        // (what does not need P, while the others arrive)
#pragma unroll
        for (int i = 0; i < TW; ++i) {
            s[i][0] *= f.w[i].x; s[i][1] *= f.w[i].y; s[i][2] *= f.w[i].z; s[i][3] *= f.w[i].w;
#pragma unroll
            for (int b = 0; b < 2; ++b) s[i] = mfma32_block(f.kt[i][b], make_float4(f.v[b][0], f.v[b][1], f.v[b][2], f.v[b][3]), s[i]);
        }
        block_exchange();
        float share[4][2][4], read[2][4];
#pragma unroll
        for (int w = 0; w < 4; ++w)
#pragma unroll
            for (int b = 0; b < 2; ++b)
#pragma unroll
                for (int t = 0; t < 4; ++t) share[w][b][t] = sh[chunk & 1][w][0][(16 * b + 4 * g + t) * kStride + l16];
        __builtin_amdgcn_sched_barrier(0);                         // (all of them requested before the first is waited for)
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int t = 0; t < 4; ++t) read[b][t] = (share[0][b][t] + share[1][b][t]) + (share[2][b][t] + share[3][b][t]);
#pragma unroll
        for (int i = 0; i < TW; ++i)
#pragma unroll
            for (int b = 0; b < 2; ++b) s[i] = mfma32_block(f.at[i][b], make_float4(read[b][0], read[b][1], read[b][2], read[b][3]), s[i]);
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int t = 8 * wave + 4 * j + g, from = t * kStride + l16, token = chunk * kDeltaChunk + t;
            const float out = (sh[chunk & 1][0][1][from] + sh[chunk & 1][1][1][from]) + (sh[chunk & 1][2][1][from] + sh[chunk & 1][3][1][from]);
            if (token < prm.rows && column < dim) prm.out[static_cast<int64_t>(token) * prm.heads * dim + head * dim + column] = out;
        }
    };
    DeltaStep<TW> even, odd;
    request(0, even);
    for (int chunk = 0; chunk < chunks; chunk += 2) {
        walk(chunk, even, odd);
        if (chunk + 1 < chunks) walk(chunk + 1, odd, even);
    }
#pragma unroll
    for (int i = 0; i < TW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (wave + 4 * i) + 4 * g + r;
            if (d < dim && column < dim) state[static_cast<int64_t>(d) * dim + column] = s[i][r];
        }
}

int64_t delta_scratch_floats(int rows, int heads, int dim) {
    if (rows < kChunkedRows || heads <= 0 || dim <= 0) return 0;
    return static_cast<int64_t>((rows + kDeltaChunk - 1) / kDeltaChunk) * heads * delta_scratch(dim).floats;
}

// (the rank-sized projection's tanh shares the LDS of three matrices)
bool delta_chunks_fit(const DeltaParams& prm) { return delta_z_stride(prm.rank) <= 3 * mfma32_stride(prm.dim); }

int32_t launch_delta_chunks(const DeltaParams& prm, hipStream_t stream) {
    const int chunks = (prm.rows + kDeltaChunk - 1) / kDeltaChunk;
    const int lds = static_cast<int>(sizeof(float)) * delta_prepare_lds(prm.dim);
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(delta_chunk_prepare_kernel), kDotLdsMost, raised);
    if (rc != QM_OK) return rc;
    if (lds > kDotLdsMost || prm.scratch_floats < delta_scratch_floats(prm.rows, prm.heads, prm.dim)) return QM_ERR_WORKSPACE;
    hipLaunchKernelGGL(delta_chunk_prepare_kernel, dim3(chunks, prm.heads), dim3(kDecThreads), lds, stream, prm);
    const dim3 grid(prm.heads, (prm.dim + 15) / 16);
    if (prm.dim <= 64) hipLaunchKernelGGL(delta_chunk_walk_kernel<1>, grid, dim3(kDecThreads), 0, stream, prm, chunks);
    else if (prm.dim <= 128) hipLaunchKernelGGL(delta_chunk_walk_kernel<2>, grid, dim3(kDecThreads), 0, stream, prm, chunks);
    else if (prm.dim <= 192) hipLaunchKernelGGL(delta_chunk_walk_kernel<3>, grid, dim3(kDecThreads), 0, stream, prm, chunks);
    else hipLaunchKernelGGL(delta_chunk_walk_kernel<4>, grid, dim3(kDecThreads), 0, stream, prm, chunks);
    return launch_status();
}

}  // namespace qm
