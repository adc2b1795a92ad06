// qm_decoder_attention_mfma.hip — the chunked attention of a prompt's rows on the bf16 matrix cores (gfx950).
//
// A block of eight waves takes 64 query rows of one key/value head (a query row is a position and one of the head's query
// heads: they share keys and values) and walks the keys that any of them sees in tiles of 128.  Four waves work on the same
// 32 rows, each on a quarter of every tile, and combine at the end: a prompt of a thousand tokens gives a grid that fills the
// chip, its longest block walks eight tiles, and a wave needs nothing from another while it walks.  Blocks of one key/value
// head share a die's L2 (block numbers go round the dies).
//
// Scores are S^T = K Q^T (v_mfma_f32_32x32x16_bf16): a lane then holds sixteen keys of one query, the softmax is in the lane
// but for one exchange with the other half of the wave, and the weights stand where the second product O^T = V^T P^T wants
// its operand, if it takes the keys of a block in the order the scores left them.  Scores and weights are fp32; the second
// product takes a weight as the sum of two bf16 numbers (its rounding and the rounding of what is left: 16 bits).  Values
// are transposed on their way into LDS.  Bound: bf16 MFMA and the vector work per score; flops 2 (dim + vdim) per visible
// key and query (the second product's doubled weights not counted).
#include "../qm_host.h"
#include "qm_decoder_device.h"

namespace qm {

typedef float dec_f32x16 __attribute__((ext_vector_type(16)));
typedef uint32_t dec_u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t dec_u32x2 __attribute__((ext_vector_type(2)));

constexpr int kFlashKeys = 128;                // keys per tile
constexpr int kFlashParts = kFlashKeys / 32;   // waves that share 32 query rows
constexpr int kFlashThreads = 2 * kFlashParts * 64;
constexpr int kFlashRows = 64;                 // query rows per block
constexpr int kFlashVStride = kFlashKeys + 4;  // bf16 per value channel in LDS: the 32 rows of a fragment lie in different banks

// CK, CV: channels of a key and of a value, rounded up to multiples of 32
template <int CK, int CV>
struct FlashShape {
    static constexpr int kKStride = CK + 8;
    static constexpr int kKBytes = kFlashKeys * kKStride * 2;
    static constexpr int kVBytes = CV * kFlashVStride * 2;
    // (the other parts' sums arrive two channel tiles at a time)
    static constexpr int kCombineTiles = CV / 32 < 2 ? 1 : 2;
    static constexpr int kCombineBytes = 2 * (kFlashParts - 1) * (kCombineTiles * 16 * 64 + 2 * 32) * 4;
    static constexpr int kLds = kKBytes + kVBytes > kCombineBytes ? kKBytes + kVBytes : kCombineBytes;
};

template <int CK, int CV>
__global__ __launch_bounds__(kFlashThreads) void chunk_attention_mfma_kernel(ChunkAttentionParams prm) {
    using Shape = FlashShape<CK, CV>;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    uint16_t* ks = reinterpret_cast<uint16_t*>(smem);                          // [keys][kKStride]
    uint16_t* vt = reinterpret_cast<uint16_t*>(smem + Shape::kKBytes);         // [CV][kFlashVStride]
    constexpr int kKb = CK / 16, kVt = CV / 32;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pair = wave / kFlashParts, part = wave % kFlashParts, half = lane >> 5;
    const int kv_head = static_cast<int>(blockIdx.x);
    const int group = prm.heads / prm.kv_heads;
    const int total = prm.rows * group;
    const int row0 = static_cast<int>(gridDim.y - 1 - blockIdx.y) * kFlashRows;      // (late rows, which may see more keys, first)
    auto position_at = [&](int query_row) { return prm.position + min(query_row, total - 1) / group; };
    auto chunk_start = [&](int position) { return position - position % prm.chunk; };
    // what the block, this wave and this lane see: keys [.., ..]
    const int block_lo = chunk_start(position_at(row0)), block_hi = position_at(row0 + kFlashRows - 1);
    const int wave_first = position_at(row0 + 32 * pair), wave_last = position_at(row0 + 32 * pair + 31);
    const int wave_lo = chunk_start(wave_first), wave_lo_most = chunk_start(wave_last);
    const int query_row = row0 + 32 * pair + (lane & 31);
    const int local = min(query_row, total - 1) / group;
    const int head = kv_head * group + min(query_row, total - 1) % group;
    const int position = prm.position + local;
    const int lo = chunk_start(position);

    dec_u32x4 q[kKb];
    const uint16_t* q_row = static_cast<const uint16_t*>(prm.q_rot) + (static_cast<int64_t>(local) * prm.heads + head) * prm.k_stride;
#pragma unroll
    for (int kb = 0; kb < kKb; ++kb) {
        const int c = kb * 16 + 8 * half;
        const dec_u32x4 read = *reinterpret_cast<const dec_u32x4*>(q_row + min(c, prm.k_stride - 8));
        q[kb] = c < prm.k_stride ? read : dec_u32x4{0, 0, 0, 0};
    }
    dec_f32x16 o[kVt];
#pragma unroll
    for (int t = 0; t < kVt; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[t][r] = 0.0f;
    float m = -INFINITY, l = 0.0f;
    const float to_log2 = prm.scale * kLog2e;

    const uint16_t* k_head = static_cast<const uint16_t*>(prm.k_cache) + static_cast<int64_t>(kv_head) * prm.ring * prm.k_stride;
    const uint16_t* v_head = static_cast<const uint16_t*>(prm.v_cache) + static_cast<int64_t>(kv_head) * prm.ring * prm.v_stride;
    constexpr int kKPieces = kFlashKeys * (CK / 8) / kFlashThreads;                // 16-byte pieces of keys per thread
    constexpr int kVBlocks = (kFlashKeys / 4 * (CV / 4) + kFlashThreads - 1) / kFlashThreads;    // blocks of 4 keys x 4 channels per thread
    dec_u32x4 k_piece[kKPieces];
    dec_u32x2 v_piece[kVBlocks][4];
    // (keys past the last one that the block sees repeat it, channels past the head's repeat others: the first are masked,
    // the second meet zeros of the query or are not stored; no branch around a load)
    auto request = [&](int tile) __attribute__((always_inline)) {
        const int base = tile % prm.ring, last = block_hi - tile;
        auto slot_of = [&](int key) {
            const int s = base + min(key, last);
            return s >= prm.ring ? s - prm.ring : s;
        };
#pragma unroll
        for (int i = 0; i < kKPieces; ++i) {
            const int at = tid + i * kFlashThreads, key = at / (CK / 8), c = at % (CK / 8) * 8;
            k_piece[i] = *reinterpret_cast<const dec_u32x4*>(k_head + slot_of(key) * prm.k_stride + min(c, prm.k_stride - 8));
        }
#pragma unroll
        for (int i = 0; i < kVBlocks; ++i) {
            const int at = tid + i * kFlashThreads, key = at / (CV / 4) * 4, c = at % (CV / 4) * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j)
                v_piece[i][j] = *reinterpret_cast<const dec_u32x2*>(v_head + slot_of(key + j) * prm.v_stride + min(c, prm.v_stride - 4));
        }
    };
    auto deposit = [&]() __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kKPieces; ++i) {
            const int at = tid + i * kFlashThreads, key = at / (CK / 8), c = at % (CK / 8) * 8;
            *reinterpret_cast<dec_u32x4*>(ks + key * Shape::kKStride + c) = k_piece[i];
        }
#pragma unroll
        for (int i = 0; i < kVBlocks; ++i) {
            const int at = tid + i * kFlashThreads, key = at / (CV / 4) * 4, c = at % (CV / 4) * 4;
            if (at >= kFlashKeys / 4 * (CV / 4)) break;
            const dec_u32x2 p0 = v_piece[i][0], p1 = v_piece[i][1], p2 = v_piece[i][2], p3 = v_piece[i][3];
            uint16_t* to = vt + c * kFlashVStride + key;
            auto pair_low = [](uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x05040100U); };
            auto pair_high = [](uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x07060302U); };
            *reinterpret_cast<dec_u32x2*>(to) = dec_u32x2{pair_low(p0[0], p1[0]), pair_low(p2[0], p3[0])};
            *reinterpret_cast<dec_u32x2*>(to + kFlashVStride) = dec_u32x2{pair_high(p0[0], p1[0]), pair_high(p2[0], p3[0])};
            *reinterpret_cast<dec_u32x2*>(to + 2 * kFlashVStride) = dec_u32x2{pair_low(p0[1], p1[1]), pair_low(p2[1], p3[1])};
            *reinterpret_cast<dec_u32x2*>(to + 3 * kFlashVStride) = dec_u32x2{pair_high(p0[1], p1[1]), pair_high(p2[1], p3[1])};
        }
    };

    request(block_lo);
    for (int tile = block_lo; tile <= block_hi; tile += kFlashKeys) {
        __syncthreads();                                           // the tile before has been read
        deposit();
        __syncthreads();
        if (tile + kFlashKeys <= block_hi) request(tile + kFlashKeys);
        const int k0 = tile + 32 * part;
        if (k0 > wave_last || k0 + 31 < wave_lo) continue;         // nothing here for this wave's rows
        dec_f32x16 s;
#pragma unroll
        for (int r = 0; r < 16; ++r) s[r] = 0.0f;
        const uint16_t* k_row = ks + (32 * part + (lane & 31)) * Shape::kKStride + 8 * half;
#pragma unroll
        for (int kb = 0; kb < kKb; ++kb) {
            const dec_u32x4 a = *reinterpret_cast<const dec_u32x4*>(k_row + kb * 16);
            s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, q[kb]), s, 0, 0, 0);
        }
        // register r is key k0 + 8 (r / 4) + 4 half + r % 4
        float p[16];
        const bool whole = k0 >= wave_lo_most && k0 + 31 <= wave_first;
#pragma unroll
        for (int r = 0; r < 16; ++r) p[r] = s[r] * to_log2;
        if (!whole) {
            const int first = lo - k0 - 4 * half, last = position - k0 - 4 * half;
#pragma unroll
            for (int r = 0; r < 16; ++r) p[r] = 8 * (r / 4) + r % 4 >= first && 8 * (r / 4) + r % 4 <= last ? p[r] : -INFINITY;
        }
        float largest = p[0];
#pragma unroll
        for (int r = 1; r < 16; ++r) largest = fmaxf(largest, p[r]);
        largest = fmaxf(largest, __shfl_xor(largest, 32, 64));
        const float before = m;
        m = fmaxf(m, largest);
        const float reference = m == -INFINITY ? 0.0f : m;         // (a row that has seen no key yet: all its weights are zero)
        const float alpha = fast_exp2(before - reference);
        float sum = 0.0f;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            p[r] = fast_exp2(p[r] - reference);
            sum += p[r];
        }
        l = l * alpha + sum;
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int t = 0; t < kVt; ++t)
#pragma unroll
                for (int r = 0; r < 16; ++r) o[t][r] *= alpha;
        }
        dec_u32x4 high[2], low[2];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float x = p[8 * b + 2 * e], y = p[8 * b + 2 * e + 1];
                const uint32_t pair_of = pack_bf16_pair(x, y);
                high[b][e] = pair_of;
                low[b][e] = pack_bf16_pair(x - lo_bf16(pair_of), y - hi_bf16(pair_of));
            }
        }
#pragma unroll
        for (int t = 0; t < kVt; ++t) {
            const uint16_t* v_row = vt + (32 * t + (lane & 31)) * kFlashVStride + 32 * part + 4 * half;
#pragma unroll
            for (int b = 0; b < 2; ++b) {
                const dec_u32x2 first = *reinterpret_cast<const dec_u32x2*>(v_row + 16 * b), second = *reinterpret_cast<const dec_u32x2*>(v_row + 16 * b + 8);
                const dec_u32x4 a = {first[0], first[1], second[0], second[1]};
                o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, high[b]), o[t], 0, 0, 0);
                o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, low[b]), o[t], 0, 0, 0);
            }
        }
    }

    // the four parts of the keys, combined by the first
    l += __shfl_xor(l, 32, 64);
    constexpr int kAtOnce = Shape::kCombineTiles;
    float* shared = reinterpret_cast<float*>(smem);
    float* sh_ml = shared + 2 * (kFlashParts - 1) * kAtOnce * 16 * 64;         // [2 pairs][parts - 1][2][32]
    auto sums_of = [&](int p) { return shared + (pair * (kFlashParts - 1) + p - 1) * kAtOnce * 16 * 64; };
    auto ml_of = [&](int p) { return sh_ml + (pair * (kFlashParts - 1) + p - 1) * 64; };
    float factor[kFlashParts], scale = 0.0f;
#pragma unroll
    for (int t0 = 0; t0 < kVt; t0 += kAtOnce) {
        __syncthreads();
        if (part > 0) {
#pragma unroll
            for (int t = 0; t < kAtOnce; ++t)
#pragma unroll
                for (int r = 0; r < 16; ++r) sums_of(part)[(t * 16 + r) * 64 + lane] = o[t0 + t][r];
            if (t0 == 0 && lane < 32) {
                ml_of(part)[lane] = m;
                ml_of(part)[32 + lane] = l;
            }
        }
        __syncthreads();
        if (part > 0) continue;
        if (t0 == 0) {
            float most = m;
#pragma unroll
            for (int p = 1; p < kFlashParts; ++p) most = fmaxf(most, ml_of(p)[lane & 31]);
            factor[0] = fast_exp2(m - most);
            float total_l = l * factor[0];
#pragma unroll
            for (int p = 1; p < kFlashParts; ++p) {
                factor[p] = fast_exp2(ml_of(p)[lane & 31] - most);
                total_l = fmaf(ml_of(p)[32 + (lane & 31)], factor[p], total_l);
            }
            scale = 1.0f / total_l;
        }
        if (query_row >= total) continue;
        uint16_t* out = static_cast<uint16_t*>(prm.out) + local * prm.ld_out + head * prm.vdim;
#pragma unroll
        for (int t = 0; t < kAtOnce; ++t) {
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int c = 32 * (t0 + t) + 8 * g + 4 * half;
                float v[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    v[e] = o[t0 + t][4 * g + e] * factor[0];
#pragma unroll
                    for (int p = 1; p < kFlashParts; ++p) v[e] = fmaf(sums_of(p)[(t * 16 + 4 * g + e) * 64 + lane], factor[p], v[e]);
                    v[e] *= scale;
                }
                if (prm.vdim % 4 == 0) {
                    if (c < prm.vdim) *reinterpret_cast<uint2*>(out + c) = make_uint2(pack_bf16_pair(v[0], v[1]), pack_bf16_pair(v[2], v[3]));
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (c + e < prm.vdim) out[c + e] = f2bf(v[e]);
                }
            }
        }
    }
    // zeros behind the heads' columns, by the last head's blocks
    if (kv_head == prm.kv_heads - 1) {
        const int first = row0 / group, last = min(row0 + kFlashRows - 1, total - 1) / group;
        const int from = prm.heads * prm.vdim, behind = static_cast<int>(prm.ld_out) - from;
        for (int i = tid; i < (last - first + 1) * behind; i += kFlashThreads)
            static_cast<uint16_t*>(prm.out)[(first + i / behind) * prm.ld_out + from + i % behind] = 0;
    }
}

template <int CK, int CV>
static int32_t flash_as(const ChunkAttentionParams& prm, hipStream_t stream) {
    constexpr int kLds = FlashShape<CK, CV>::kLds;
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(chunk_attention_mfma_kernel<CK, CV>), kLds, raised);
    if (rc != QM_OK) return rc;
    const int64_t total = static_cast<int64_t>(prm.rows) * (prm.heads / prm.kv_heads);
    if ((total + kFlashRows - 1) / kFlashRows > 65535) return QM_ERR_GEOMETRY;
    hipLaunchKernelGGL((chunk_attention_mfma_kernel<CK, CV>), dim3(prm.kv_heads, static_cast<unsigned>((total + kFlashRows - 1) / kFlashRows)),
                       dim3(kFlashThreads), kLds, stream, prm);
    return launch_status();
}

int32_t launch_chunk_attention_mfma(const ChunkAttentionParams& prm, hipStream_t stream) {
    if (prm.ld_out % 4 || (reinterpret_cast<uintptr_t>(prm.out) & 7)) return QM_ERR_GEOMETRY;
    const int c = prm.dim > prm.vdim ? prm.dim : prm.vdim;
    if (c <= 32) return flash_as<32, 32>(prm, stream);
    if (c <= 64) return flash_as<64, 64>(prm, stream);
    if (c <= 128) return flash_as<128, 128>(prm, stream);
    if (prm.dim <= 192 && prm.vdim <= 128) return flash_as<192, 128>(prm, stream);
    return flash_as<256, 256>(prm, stream);
}

}  // namespace qm
