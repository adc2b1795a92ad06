// qm_decoder_latent_mfma.hip — few rows' attention over latents on the bf16 matrix cores (gfx950).
//
// All heads share keys and values, so sixteen queries (rows x heads) meet every cached latent that a block fetches.  A block of
// four waves takes sixteen queries and one key split, in passes of 64 keys: a latent goes from memory into registers once and
// from there into LDS twice, as it is (the score's operand) and transposed (the second product's).  Scores are
// S^T = K Q^T (v_mfma_f32_16x16x32_bf16): a lane then holds eight keys of one query in two tiles, the softmax is in the lane but
// for two exchanges, and the weights stand where O^T = L^T P^T wants its operand if it takes the 32 keys in the order the scores
// left them.  A weight enters as the sum of two bf16 numbers.  Two waves share the 64 keys, two halves of the latent's channels
// share the second product.  Bound by HBM: a cached latent and key part are read once per sixteen queries.
#include "../qm_host.h"
#include "qm_decoder_latent.h"

namespace qm {

typedef uint32_t lat_u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t lat_u32x2 __attribute__((ext_vector_type(2)));

constexpr int kLatQueries = 16;                // queries of a block
constexpr int kLatRotary = 64;                 // channels of the key part, padded

// C: channels of a latent, padded to 64, 128, 256 or 512
template <int C>
struct LatentShape {
    static constexpr int kKStride = C + kLatRotary + 8;            // bf16 per key in LDS
    static constexpr int kVStride = kLatentKeys + 4;               // bf16 per channel in LDS
    static constexpr int kKBytes = kLatentKeys * kKStride * 2;
    static constexpr int kLds = kKBytes + C * kVStride * 2;
    static constexpr int kTiles = C / 2 / 16;                      // of a wave's half of the channels
    static_assert(2 * (kTiles * 4 * 64 + 128) * 4 <= kLds, "the parts' sums fit where the keys were");
};

template <int C>
__global__ __launch_bounds__(kDecThreads) void latent_partials_mfma_kernel(LatentAttentionParams prm) {
    using Shape = LatentShape<C>;
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    uint16_t* ks = reinterpret_cast<uint16_t*>(smem);                          // [keys][kKStride]: latent, key part
    uint16_t* vt = reinterpret_cast<uint16_t*>(smem + Shape::kKBytes);         // [C][kVStride]
    constexpr int kKb = (C + kLatRotary) / 32, kTiles = Shape::kTiles;
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l16 = lane & 15;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int part = wave & 1, half = wave >> 1;
    const int split = static_cast<int>(blockIdx.x), total = prm.rows * prm.heads;
    const int query = static_cast<int>(blockIdx.y) * kLatQueries + l16;
    const int asked = min(query, total - 1);
    const int start = position_of(prm.position_dev, prm.position);
    const int all = start + prm.rows, each = latent_keys_per_split(all, prm.splits);
    const int begin = split * each;
    lat_u32x4 q[kKb];
    const uint16_t* q_row = static_cast<const uint16_t*>(prm.q_scratch) + static_cast<int64_t>(asked) * (C + kLatRotary) + 8 * g;
#pragma unroll
    for (int kb = 0; kb < kKb; ++kb) q[kb] = *reinterpret_cast<const lat_u32x4*>(q_row + kb * 32);
    if (begin >= all) return;
    const int block_last = min(static_cast<int>(blockIdx.y) * kLatQueries + kLatQueries - 1, total - 1);
    const int end = min(begin + each, start + block_last / prm.heads + 1);     // what any of the block's queries sees
    const int position = start + asked / prm.heads;

    f32x4_t o[kTiles];
#pragma unroll
    for (int t = 0; t < kTiles; ++t) o[t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    float m = -INFINITY, l = 0.0f;
    const float to_log2 = prm.scale * kLog2e;

    const uint16_t* latent = static_cast<const uint16_t*>(prm.latent_cache);
    const uint16_t* key_part = static_cast<const uint16_t*>(prm.key_cache);
    const int ld = static_cast<int>(prm.ld_latent), key_stride = prm.key_stride;
    // blocks of four keys x eight channels, dealt to the threads: sixteen lanes take the same channels of all keys, so that both
    // ways of storing them spread over the LDS banks; and pieces of the key part
    constexpr int kGroups = kLatentKeys / 4, kUnits = kGroups * (C / 8), kBlocks = (kUnits + kDecThreads - 1) / kDecThreads;
    constexpr int kRotaryPieces = kLatentKeys * (kLatRotary / 8) / kDecThreads;
    lat_u32x4 piece[kBlocks][4], rotary_piece[kRotaryPieces];
    // (keys past the last repeat it and are masked; channels past the latent's meet zeros of the query or are not stored)
    auto request = [&](int tile) __attribute__((always_inline)) {
        const int last = end - 1;
#pragma unroll
        for (int i = 0; i < kBlocks; ++i) {
            const int at = min(tid + i * kDecThreads, kUnits - 1), key = at % kGroups * 4, c = at / kGroups * 8;
#pragma unroll
            for (int j = 0; j < 4; ++j)
                piece[i][j] = *reinterpret_cast<const lat_u32x4*>(latent + static_cast<int64_t>(min(tile + key + j, last)) * ld + min(c, ld - 8));
        }
#pragma unroll
        for (int i = 0; i < kRotaryPieces; ++i) {
            const int at = tid + i * kDecThreads, key = at / (kLatRotary / 8), c = at % (kLatRotary / 8) * 8;
            rotary_piece[i] = *reinterpret_cast<const lat_u32x4*>(key_part + static_cast<int64_t>(min(tile + key, last)) * key_stride + min(c, key_stride - 8));
        }
    };
    auto deposit = [&]() __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kBlocks; ++i) {
            const int at = tid + i * kDecThreads, key = at % kGroups * 4, c = at / kGroups * 8;
            if (at >= kUnits) break;
#pragma unroll
            for (int j = 0; j < 4; ++j) *reinterpret_cast<lat_u32x4*>(ks + (key + j) * Shape::kKStride + c) = piece[i][j];
            auto low = [](uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x05040100U); };
            auto high = [](uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x07060302U); };
#pragma unroll
            for (int w = 0; w < 4; ++w) {
                const uint32_t p0 = piece[i][0][w], p1 = piece[i][1][w], p2 = piece[i][2][w], p3 = piece[i][3][w];
                uint16_t* to = vt + (c + 2 * w) * Shape::kVStride + key;
                *reinterpret_cast<lat_u32x2*>(to) = lat_u32x2{low(p0, p1), low(p2, p3)};
                *reinterpret_cast<lat_u32x2*>(to + Shape::kVStride) = lat_u32x2{high(p0, p1), high(p2, p3)};
            }
        }
#pragma unroll
        for (int i = 0; i < kRotaryPieces; ++i) {
            const int at = tid + i * kDecThreads, key = at / (kLatRotary / 8), c = at % (kLatRotary / 8) * 8;
            *reinterpret_cast<lat_u32x4*>(ks + key * Shape::kKStride + C + c) = rotary_piece[i];
        }
    };

    if (begin < end) request(begin);
    for (int tile = begin; tile < end; tile += kLatentKeys) {
        __syncthreads();                                           // the pass before has been read
        deposit();
        __syncthreads();
        if (tile + kLatentKeys < end) request(tile + kLatentKeys);
        const int k0 = tile + 32 * part;
        if (k0 >= end) continue;
        f32x4_t s[2] = {f32x4_t{0.0f, 0.0f, 0.0f, 0.0f}, f32x4_t{0.0f, 0.0f, 0.0f, 0.0f}};
        const uint16_t* k_row = ks + (32 * part + l16) * Shape::kKStride + 8 * g;
#pragma unroll
        for (int kb = 0; kb < kKb; ++kb) {
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const lat_u32x4 a = *reinterpret_cast<const lat_u32x4*>(k_row + 16 * j * Shape::kKStride + kb * 32);
                s[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, q[kb]), s[j], 0, 0, 0);
            }
        }
        // s[j][r] is key k0 + 16 j + 4 g + r of query l16
        const int last = min(position, end - 1) - k0 - 4 * g;
        float p[8], largest = -INFINITY;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            p[i] = 16 * (i >> 2) + (i & 3) <= last ? s[i >> 2][i & 3] * to_log2 : -INFINITY;
            largest = fmaxf(largest, p[i]);
        }
        largest = fmaxf(largest, __shfl_xor(largest, 16, 64));
        largest = fmaxf(largest, __shfl_xor(largest, 32, 64));
        const float before = m;
        m = fmaxf(m, largest);
        const float reference = m == -INFINITY ? 0.0f : m;         // (a query that has seen no key yet: all its weights are zero)
        const float alpha = fast_exp2(before - reference);
        float sum = 0.0f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            p[i] = fast_exp2(p[i] - reference);
            sum += p[i];
        }
        l = l * alpha + sum;
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int t = 0; t < kTiles; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[t][r] *= alpha;
        }
        lat_u32x4 upper, lower;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float x = p[2 * e], y = p[2 * e + 1];
            const uint32_t pair_of = pack_bf16_pair(x, y);
            upper[e] = pair_of;
            lower[e] = pack_bf16_pair(x - lo_bf16(pair_of), y - hi_bf16(pair_of));
        }
#pragma unroll
        for (int t = 0; t < kTiles; ++t) {
            const uint16_t* v_row = vt + (half * (C / 2) + 16 * t + l16) * Shape::kVStride + 32 * part + 4 * g;
            const lat_u32x2 first = *reinterpret_cast<const lat_u32x2*>(v_row), second = *reinterpret_cast<const lat_u32x2*>(v_row + 16);
            const lat_u32x4 a = {first[0], first[1], second[0], second[1]};
            o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, upper), o[t], 0, 0, 0);
            o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, lower), o[t], 0, 0, 0);
        }
    }
    // the two parts of the keys, combined by the first
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    float* shared = reinterpret_cast<float*>(smem) + half * (kTiles * 4 * 64 + 128);
    __syncthreads();
    if (part == 1) {
#pragma unroll
        for (int t = 0; t < kTiles; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) shared[(t * 4 + r) * 64 + lane] = o[t][r];
        shared[kTiles * 4 * 64 + lane] = m;
        shared[kTiles * 4 * 64 + 64 + lane] = l;
    }
    __syncthreads();
    if (part == 1 || query >= total) return;
    const float m_other = shared[kTiles * 4 * 64 + lane], l_other = shared[kTiles * 4 * 64 + 64 + lane];
    const float most = fmaxf(m, m_other), reference = most == -INFINITY ? 0.0f : most;
    const float own = fast_exp2(m - reference), other = fast_exp2(m_other - reference);
    const int64_t at = static_cast<int64_t>(query) * prm.splits + split;
    if (half == 0 && g == 0) {
        prm.ml[at * 2] = most;
        prm.ml[at * 2 + 1] = l * own + l_other * other;
    }
    float* out = prm.acc + at * prm.kv_rank;
#pragma unroll
    for (int t = 0; t < kTiles; ++t) {
        const int c = half * (C / 2) + 16 * t + 4 * g;             // o[t][r] is channel c + r
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = o[t][r] * own + shared[(t * 4 + r) * 64 + lane] * other;
        if (prm.kv_rank % 4 == 0) {
            if (c < prm.kv_rank) *reinterpret_cast<float4*>(out + c) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (c + r < prm.kv_rank) out[c + r] = v[r];
        }
    }
}

template <int C>
static int32_t partials_as(const LatentAttentionParams& prm, hipStream_t stream) {
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(latent_partials_mfma_kernel<C>), LatentShape<C>::kLds, raised);
    if (rc != QM_OK) return rc;
    const int tiles = (prm.rows * prm.heads + kLatQueries - 1) / kLatQueries;
    hipLaunchKernelGGL(latent_partials_mfma_kernel<C>, dim3(prm.splits, tiles), dim3(kDecThreads), LatentShape<C>::kLds, stream, prm);
    return launch_status();
}

bool latent_partials_fit_mfma(const LatentAttentionParams& prm) {
    return prm.kv_rank <= 512 && prm.rot_dim <= kLatRotary && prm.key_stride >= 8 && static_cast<int64_t>(prm.rows) * prm.heads <= 16 * 65535;
}

int32_t launch_latent_partials_mfma(const LatentAttentionParams& prm, hipStream_t stream) {
    switch (latent_pad(prm.kv_rank)) {
        case 64: return partials_as<64>(prm, stream);
        case 128: return partials_as<128>(prm, stream);
        case 256: return partials_as<256>(prm, stream);
        default: return partials_as<512>(prm, stream);
    }
}

}  // namespace qm
