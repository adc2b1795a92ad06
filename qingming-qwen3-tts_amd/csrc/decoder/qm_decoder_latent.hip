// qm_decoder_latent.hip — softmax attention whose keys and values are made from one latent per token, for gfx950.
//
// Cached per token: the latent (kv_rank channels) and one rotated key part that all heads share.  Two ways to the same scores:
//   few rows (decode), and fp32   the query goes through the head's up_k once, then latents are the keys and the values of all
//                                 heads; the weighted latent goes through the head's up_v.  A step reads each cached latent once.
//   many bf16 rows                keys and values of every position are made by the matrix-core linear and the heads attend as in
//                                 any other model: dim + rot_dim and vdim channels per score instead of kv_rank + rot_dim and kv_rank.
#include "../qm_host.h"
#include "qm_decoder_attention.h"
#include "qm_decoder_dot.h"
#include "qm_decoder_latent.h"

namespace qm {

constexpr int kLatentSlice = 64;               // columns of up_k per block
constexpr int kLatentOutputs = 32;             // rows of up_v per block
constexpr int kExpandRows = 2048;              // positions expanded by one linear

template <class T>
__global__ __launch_bounds__(kDecThreads) void latent_rows_kernel(LatentRowsParams prm) {
    __shared__ float sh_red[8];
    const int row = static_cast<int>(blockIdx.x);
    if (prm.q_latent)
        slice_norm_row<T>(prm.proj + row * prm.ld_proj + prm.q_column, prm.q_norm, prm.q_rank, prm.ld_q, prm.eps, sh_red,
                          static_cast<T*>(prm.q_latent) + row * prm.ld_q);
    if (prm.latent_cache) latent_keep_row<T>(prm, row, sh_red + 4);
}

// Queries through up_k: a block takes 64 columns of one head's up_k and R rows; eight threads cover the columns of a matrix row,
// 32 matrix rows are under way at once.  The blocks of head number `heads` write what the step's token leaves in the cache.
template <class T, int R>
__global__ __launch_bounds__(kDecThreads) void latent_query_kernel(LatentAttentionParams prm, LatentRowsParams keep) {
    request_arguments(prm, keep);
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float sh_red[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int head = static_cast<int>(blockIdx.y), column0 = static_cast<int>(blockIdx.x) * kLatentSlice, row0 = static_cast<int>(blockIdx.z) * R;
    if (head == prm.heads) {
        if (column0 == 0 && row0 == 0) latent_keep_row<T>(keep, 0, sh_red);
        return;
    }
    const int per_head = prm.dim + prm.rot_dim;
    float* sh_q = lds;                         // [R][dim]
    float* sh_sum = lds + R * prm.dim;         // [4 waves][R][64]
    const int column = column0 + (tid & 7) * 8;
    const uint16_t* w = prm.up_k + static_cast<int64_t>(head) * prm.dim * prm.ld_latent + min(column, static_cast<int>(prm.ld_latent) - 8);
    constexpr int kAhead = 4;
    uint4 piece[kAhead];
    const int first = tid >> 3;
#pragma unroll
    for (int u = 0; u < kAhead; ++u) piece[u] = *reinterpret_cast<const uint4*>(w + min(first + 32 * u, prm.dim - 1) * prm.ld_latent);
    for (int i = tid; i < R * prm.dim; i += kDecThreads) {
        const int r = i / prm.dim, d = i - r * prm.dim;
        sh_q[i] = prm.q[min(row0 + r, prm.rows - 1) * prm.ld_query + head * per_head + d];
    }
    __syncthreads();
    float acc[R][8];
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[r][e] = 0.0f;
    for (int d0 = first; d0 < prm.dim; d0 += 32 * kAhead) {
#pragma unroll
        for (int u = 0; u < kAhead; ++u) {
            const int d = d0 + 32 * u;
            Raw8<uint16_t> raw;
            raw.w = piece[u];
            float v[8];
            raw.widen(v);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const float q = d < prm.dim ? sh_q[r * prm.dim + d] : 0.0f;
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[r][e] = fmaf(q, v[e], acc[r][e]);
            }
            piece[u] = *reinterpret_cast<const uint4*>(w + min(d + 32 * kAhead, prm.dim - 1) * prm.ld_latent);
        }
    }
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float v = acc[r][e];
            v += __shfl_xor(v, 8, 64);
            v += __shfl_xor(v, 16, 64);
            v += __shfl_xor(v, 32, 64);
            if (lane < 8) sh_sum[(wave * R + r) * 64 + lane * 8 + e] = v;
        }
    __syncthreads();
    const int stride = latent_pad(prm.kv_rank) + latent_rotary_pad(prm.rot_dim);
    T* q_scratch = static_cast<T*>(prm.q_scratch);
    for (int i = tid; i < R * 64; i += kDecThreads) {
        const int r = i >> 6, c = i & 63;
        if (row0 + r >= prm.rows) break;
        const float v = (sh_sum[r * 64 + c] + sh_sum[(R + r) * 64 + c]) + (sh_sum[(2 * R + r) * 64 + c] + sh_sum[(3 * R + r) * 64 + c]);
        q_scratch[(static_cast<int64_t>(row0 + r) * prm.heads + head) * stride + column0 + c] = from_f32<T>(column0 + c < prm.kv_rank ? v : 0.0f);
    }
    if (column0 != 0) return;
    const int position = position_of(prm.position_dev, prm.position);
    const int rotary_pad = latent_rotary_pad(prm.rot_dim);
    for (int i = tid; i < R * rotary_pad; i += kDecThreads) {
        const int r = i / rotary_pad, c = i - r * rotary_pad, row = row0 + r;
        if (row >= prm.rows) break;
        float v = 0.0f;
        if (c < prm.rot_dim)
            v = turned_neighbour(prm.q + row * prm.ld_query + head * per_head + prm.dim, c, prm.frequency, position + row, prm.magnitude);
        q_scratch[(static_cast<int64_t>(row) * prm.heads + head) * stride + latent_pad(prm.kv_rank) + c] = from_f32<T>(v);
    }
}

// One (row, head, key split): scores against latents and key parts, the softmax's partial sums, the weighted latents.  Sixteen
// lanes hold a key; a thread owns up to four channels of the result.
template <class T>
__global__ __launch_bounds__(kDecThreads) void latent_partials_kernel(LatentAttentionParams prm) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float sc[kLatentKeys], sh_f[1];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane >> 4, l16 = lane & 15;
    const int split = static_cast<int>(blockIdx.x), head = static_cast<int>(blockIdx.y), row = static_cast<int>(blockIdx.z);
    const int start = position_of(prm.position_dev, prm.position);
    const int all = start + prm.rows, each = latent_keys_per_split(all, prm.splits);
    const int begin = split * each, end = min(start + row + 1, begin + each);
    if (begin >= all) return;
    const int pad = latent_pad(prm.kv_rank), stride = pad + latent_rotary_pad(prm.rot_dim);
    const T* q = static_cast<const T*>(prm.q_scratch) + (static_cast<int64_t>(row) * prm.heads + head) * stride;
    for (int c = tid; c < stride; c += kDecThreads) lds[c] = to_f32(q[c]);
    __syncthreads();
    const T* latent = static_cast<const T*>(prm.latent_cache);
    const T* key_part = static_cast<const T*>(prm.key_cache);
    constexpr int kOwn = kLatentMaxRank / kDecThreads;
    float acc[kOwn] = {}, m = -INFINITY, l = 0.0f;
    for (int tile = begin; tile < end; tile += kLatentKeys) {
        const int keys = min(kLatentKeys, end - tile);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int j = wave * 16 + i * 4 + sub;
            const int64_t key = tile + min(j, keys - 1);
            float s = 0.0f;
            for (int c = l16 * 8; c < prm.kv_rank; c += 128) {     // (zeros behind the latent)
                Raw8<T> raw;
                raw.load(latent + key * prm.ld_latent + c);
                float v[8];
                raw.widen(v);
#pragma unroll
                for (int e = 0; e < 8; ++e) s = fmaf(v[e], lds[c + e], s);
            }
            for (int c = l16 * 8; c < prm.key_stride; c += 128) {
                Raw8<T> raw;
                raw.load(key_part + key * prm.key_stride + c);
                float v[8];
                raw.widen(v);
#pragma unroll
                for (int e = 0; e < 8; ++e) s = fmaf(v[e], lds[pad + c + e], s);
            }
            s = row16_allreduce_sum(s);
            if (l16 == 0) sc[j] = s * (prm.scale * kLog2e);
        }
        __syncthreads();
        if (wave == 0) {
            const float s = lane < keys ? sc[lane] : -INFINITY;
            const float largest = fmaxf(m, wave_max(s));
            const float p = lane < keys ? exp2f(s - largest) : 0.0f, factor = exp2f(m - largest);
            l = l * factor + wave_sum(p);
            m = largest;
            sc[lane] = p;
            if (lane == 0) sh_f[0] = factor;
        }
        __syncthreads();
        const float factor = sh_f[0];
#pragma unroll
        for (int x = 0; x < kOwn; ++x) {
            const int c = tid + x * kDecThreads;
            if (c >= prm.kv_rank) break;
            float sum = acc[x] * factor;
            const T* from = latent + static_cast<int64_t>(tile) * prm.ld_latent + c;
#pragma unroll 8
            for (int j = 0; j < keys; ++j) sum = fmaf(sc[j], to_f32(from[j * prm.ld_latent]), sum);
            acc[x] = sum;
        }
        __syncthreads();
    }
    const int64_t at = (static_cast<int64_t>(row) * prm.heads + head) * prm.splits + split;
    if (tid == 0) {
        prm.ml[at * 2] = m;
        prm.ml[at * 2 + 1] = l;
    }
#pragma unroll
    for (int x = 0; x < kOwn; ++x)
        if (tid + x * kDecThreads < prm.kv_rank) prm.acc[at * prm.kv_rank + tid + x * kDecThreads] = acc[x];
}

// The splits of a (row, head) combined and sent through 32 rows of the head's up_v.
template <class T>
__global__ __launch_bounds__(kDecThreads) void latent_output_kernel(LatentAttentionParams prm) {
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) float sh_o[];               // [kv_rank, padded to 512s]
    __shared__ float sh_w[kDecMaxSplits];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int e0 = static_cast<int>(blockIdx.x) * kLatentOutputs + wave * (kLatentOutputs / 4), head = static_cast<int>(blockIdx.y);
    const int64_t row = blockIdx.z;
    constexpr int kEach = kLatentOutputs / 4;
    const uint16_t* w = prm.up_v + static_cast<int64_t>(head) * prm.vdim * prm.ld_latent;
    const uint16_t* w_row[kEach];
    uint4 piece[kEach];
    const int ld = static_cast<int>(prm.ld_latent);
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
        w_row[i] = w + static_cast<int64_t>(min(e0 + i, prm.vdim - 1)) * ld;
        piece[i] = *reinterpret_cast<const uint4*>(w_row[i] + min(lane * 8, ld - 8));
    }
    const int all = position_of(prm.position_dev, prm.position) + prm.rows;
    const int each = latent_keys_per_split(all, prm.splits), active = (all + each - 1) / each;
    const int64_t at = (row * prm.heads + head) * prm.splits;
    const float* acc = prm.acc + at * prm.kv_rank;
    constexpr int kFirst = 16, kOwn = 2;       // splits and channels of the thread that are asked for before the factors are known
    float held[kOwn][kFirst];
#pragma unroll
    for (int x = 0; x < kOwn; ++x)
#pragma unroll
        for (int s = 0; s < kFirst; ++s)
            held[x][s] = acc[static_cast<int64_t>(min(s, active - 1)) * prm.kv_rank + min(tid + x * kDecThreads, prm.kv_rank - 1)];
    if (wave == 0) {
        const float m_read = prm.ml[(at + min(lane, active - 1)) * 2], l_read = prm.ml[(at + min(lane, active - 1)) * 2 + 1];
        const float m = lane < active ? m_read : -INFINITY, l = lane < active ? l_read : 0.0f;
        const float factor = fast_exp2(m - wave_max(m));
        const float total = wave_sum(factor * l);
        if (lane < active) sh_w[lane] = factor / total;
    }
    __syncthreads();
    const int padded = (prm.kv_rank + 511) / 512 * 512;
#pragma unroll
    for (int x = 0; x < kOwn; ++x) {
        float sum = 0.0f;
#pragma unroll
        for (int s = 0; s < kFirst; ++s) sum = fmaf(s < active ? sh_w[min(s, active - 1)] : 0.0f, held[x][s], sum);
        held[x][0] = sum;
    }
    for (int c = tid; c < padded; c += kDecThreads) {
        const int own = (c - tid) / kDecThreads;
        float sum = own == 0 ? held[0][0] : own == 1 ? held[1][0] : 0.0f;
        const int from = min(c, prm.kv_rank - 1);
        for (int s0 = own < kOwn ? kFirst : 0; s0 < active; s0 += 8) {
            float v[8];
#pragma unroll
            for (int s = 0; s < 8; ++s) v[s] = acc[static_cast<int64_t>(min(s0 + s, active - 1)) * prm.kv_rank + from];
#pragma unroll
            for (int s = 0; s < 8; ++s) sum = fmaf(s0 + s < active ? sh_w[s0 + s] : 0.0f, v[s], sum);
        }
        sh_o[c] = c < prm.kv_rank ? sum : 0.0f;
    }
    __syncthreads();
    float out[kEach];
#pragma unroll
    for (int i = 0; i < kEach; ++i) out[i] = 0.0f;
    for (int c0 = 0; c0 < padded; c0 += 512) {
#pragma unroll
        for (int i = 0; i < kEach; ++i) {
            out[i] = dot8(piece[i], sh_o + c0 + lane * 8, out[i]);             // (zeros behind the latent)
            piece[i] = *reinterpret_cast<const uint4*>(w_row[i] + min(c0 + 512 + lane * 8, ld - 8));
        }
    }
    T* to = static_cast<T*>(prm.out) + row * prm.ld_out;
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
        const float v = wave_sum(out[i]);
        if (lane == 0 && e0 + i < prm.vdim) to[head * prm.vdim + e0 + i] = from_f32<T>(v);
    }
    if (head == prm.heads - 1 && blockIdx.x == 0)
        for (int c = prm.heads * prm.vdim + tid; c < prm.ld_out; c += kDecThreads) to[c] = from_f32<T>(0.0f);
}

// ---- many rows: keys and values of every position ------------------------------------------------------------------------
struct ExpandParams {
    const float* up;               // [positions][ld]: keys of every head, values of every head at v_column
    const uint16_t* key_cache;
    uint16_t* k;                   // [heads][ring][k_stride]
    uint16_t* v;                   // [heads][ring][v_stride]
    int64_t ld;
    int first, ring, heads, dim, rot_dim, vdim, k_stride, v_stride, key_stride, v_column;
};
__device__ __forceinline__ void put8(uint16_t* to, const float (&v)[8]) {
    *reinterpret_cast<uint4*>(to) = make_uint4(pack_bf16_pair(v[0], v[1]), pack_bf16_pair(v[2], v[3]), pack_bf16_pair(v[4], v[5]), pack_bf16_pair(v[6], v[7]));
}
// The linear's rows dealt to the heads, the shared key part behind each head's keys: a block per position.
__global__ __launch_bounds__(kDecThreads) void latent_expand_kernel(ExpandParams prm) {
    const int at = static_cast<int>(blockIdx.x), position = prm.first + at;
    const float* up = prm.up + at * prm.ld;
    const uint16_t* shared = prm.key_cache + static_cast<int64_t>(position) * prm.key_stride;
    const int k_pieces = prm.k_stride >> 3, v_pieces = prm.v_stride >> 3, vector_k = !(prm.dim & 7), vector_v = !(prm.vdim & 7) && !(prm.v_column & 3);
    for (int i = threadIdx.x; i < prm.heads * k_pieces; i += kDecThreads) {
        const int h = i / k_pieces, c = (i - h * k_pieces) * 8;
        const float* head = up + h * prm.dim;
        uint16_t* to = prm.k + (static_cast<int64_t>(h) * prm.ring + position) * prm.k_stride + c;
        float v[8];
        if (vector_k && c + 8 <= prm.dim) {
            const float4 a = load4(head, c >> 2), b = load4(head, (c >> 2) + 1);
            v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int channel = c + e;
                v[e] = channel < prm.dim ? head[channel] : channel < prm.dim + prm.rot_dim ? bf2f(shared[channel - prm.dim]) : 0.0f;
            }
        }
        put8(to, v);
    }
    for (int i = threadIdx.x; i < prm.heads * v_pieces; i += kDecThreads) {
        const int h = i / v_pieces, c = (i - h * v_pieces) * 8;
        const float* head = up + prm.v_column + h * prm.vdim;
        float v[8];
        if (vector_v) {
            const float4 a = load4(head, c >> 2), b = load4(head, (c >> 2) + 1);
            v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = c + e < prm.vdim ? head[c + e] : 0.0f;
        }
        put8(prm.v + (static_cast<int64_t>(h) * prm.ring + position) * prm.v_stride + c, v);
    }
}
// The rows' queries, their part behind `dim` turned: a block per row.
__global__ __launch_bounds__(kDecThreads) void latent_rotate_query_kernel(LatentAttentionParams prm, uint16_t* to, int k_stride) {
    __shared__ float sh_cos[kLatentMaxRotary / 2], sh_sin[kLatentMaxRotary / 2];
    const int64_t row = blockIdx.x;
    const int position = prm.position + static_cast<int>(row);
    for (int i = threadIdx.x; i < prm.rot_dim / 2; i += kDecThreads) {
        rotary(position, prm.frequency[i], sh_cos[i], sh_sin[i]);
        sh_cos[i] *= prm.magnitude;
        sh_sin[i] *= prm.magnitude;
    }
    __syncthreads();
    const int pieces = k_stride >> 3, per_head = prm.dim + prm.rot_dim;
    const bool vectors = ((prm.dim | per_head) & 7) == 0;
    const float* q = prm.q + row * prm.ld_query;
    for (int i = threadIdx.x; i < prm.heads * pieces; i += kDecThreads) {
        const int h = i / pieces, c0 = (i - h * pieces) * 8;
        const float* head = q + h * per_head;
        float v[8];
        if (vectors && c0 + 8 <= prm.dim) {
            const float4 a = load4(head, c0 >> 2), b = load4(head, (c0 >> 2) + 1);
            v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
            put8(to + (row * prm.heads + h) * k_stride + c0, v);
            continue;
        }
        if (vectors && c0 >= prm.dim && c0 + 8 <= per_head) {
            const float4 a = load4(head, c0 >> 2), b = load4(head, (c0 >> 2) + 1);
            const float x[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
            for (int e = 0; e < 8; e += 2) {
                const float cosine = sh_cos[(c0 - prm.dim + e) >> 1], sine = sh_sin[(c0 - prm.dim + e) >> 1];
                v[e] = x[e] * cosine - x[e + 1] * sine;
                v[e + 1] = x[e + 1] * cosine + x[e] * sine;
            }
            put8(to + (row * prm.heads + h) * k_stride + c0, v);
            continue;
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int c = c0 + e, r = c - prm.dim;
            const float own = c < per_head ? head[min(c, per_head - 1)] : 0.0f;
            const bool turns = r >= 0 && r < prm.rot_dim;
            const float other = turns ? head[prm.dim + (r ^ 1)] : 0.0f;
            v[e] = turns ? own * sh_cos[r >> 1] + (r & 1 ? other : -other) * sh_sin[r >> 1] : own;
        }
        put8(to + (row * prm.heads + h) * k_stride + c0, v);
    }
}

int latent_q_stride(int kv_rank, int rot_dim) { return latent_pad(kv_rank) + latent_rotary_pad(rot_dim); }

static int expand_rows(int positions) { return positions < kExpandRows ? positions : kExpandRows; }
static int64_t aligned(int64_t bytes) { return (bytes + 255) / 256 * 256; }
static int pad8(int n) { return (n + 7) / 8 * 8; }

static int64_t expanded_bytes(int positions, int heads, int dim, int rot_dim, int vdim, int up_rows) {
    const int64_t each = static_cast<int64_t>(positions) * heads * 2;
    return aligned(static_cast<int64_t>(expand_rows(positions)) * up_rows * 4) + 2 * aligned(each * pad8(dim + rot_dim)) + aligned(each * pad8(vdim));
}

static int32_t attend_expanded(const LatentAttentionParams& prm, hipStream_t stream) {
    const int positions = prm.position + prm.rows, k_stride = pad8(prm.dim + prm.rot_dim), v_stride = pad8(prm.vdim);
    char* at = reinterpret_cast<char*>(prm.expanded);
    float* up = prm.expanded;
    at += aligned(static_cast<int64_t>(expand_rows(positions)) * prm.up_rows * 4);
    const int64_t each = static_cast<int64_t>(positions) * prm.heads * 2;
    uint16_t* q = reinterpret_cast<uint16_t*>(at);
    at += aligned(each * k_stride);
    uint16_t* k = reinterpret_cast<uint16_t*>(at);
    at += aligned(each * k_stride);
    uint16_t* v = reinterpret_cast<uint16_t*>(at);
    for (int first = 0; first < positions; first += kExpandRows) {
        DecLinearParams linear = {};
        linear.groups = 1;
        linear.rows = positions - first < kExpandRows ? positions - first : kExpandRows;
        DecLinearGroup& g = linear.group[0];
        g.x = static_cast<const uint16_t*>(prm.latent_cache) + first * prm.ld_latent;
        g.w = prm.up_k;
        g.out32 = up;
        g.ldx = prm.ld_latent;
        g.ldo = g.n = prm.up_rows;
        g.k = static_cast<int32_t>(prm.ld_latent);
        const int32_t rc = launch_decoder_linears(linear, 0, stream);
        if (rc != QM_OK) return rc;
        const ExpandParams e = {up, static_cast<const uint16_t*>(prm.key_cache), k, v, prm.up_rows, first, positions, prm.heads, prm.dim, prm.rot_dim, prm.vdim,
                                k_stride, v_stride, prm.key_stride, prm.up_v_row};
        hipLaunchKernelGGL(latent_expand_kernel, dim3(linear.rows), dim3(kDecThreads), 0, stream, e);
    }
    hipLaunchKernelGGL(latent_rotate_query_kernel, dim3(prm.rows), dim3(kDecThreads), 0, stream, prm, q, k_stride);
    const int32_t rc = launch_status();
    if (rc != QM_OK) return rc;
    ChunkAttentionParams a = {};
    a.q_rot = q; a.k_cache = k; a.v_cache = v; a.out = prm.out;
    a.ld_out = prm.ld_out;
    a.position = prm.position; a.rows = prm.rows;
    a.heads = a.kv_heads = prm.heads;
    a.dim = prm.dim + prm.rot_dim; a.vdim = prm.vdim;
    a.k_stride = k_stride; a.v_stride = v_stride;
    a.ring = a.chunk = positions;              // (one chunk: every key up to the row's own)
    a.scale = prm.scale;
    return launch_chunk_attention_mfma(a, stream);
}

static int32_t check_rows(const LatentRowsParams& p) {
    if (p.rows < 0 || p.position < 0) return QM_ERR_ARGUMENT;
    if (!p.proj || (p.q_latent && !p.q_norm) || (p.latent_cache && (!p.kv_norm || !p.key_cache || !p.frequency))) return QM_ERR_NULL;
    if (p.q_latent && (p.q_rank <= 0 || p.ld_q < p.q_rank)) return QM_ERR_GEOMETRY;
    if (p.latent_cache && (p.kv_rank <= 0 || p.kv_rank > kLatentMaxRank || p.ld_latent < p.kv_rank || p.ld_latent % 8 || p.rot_dim < 0 || p.rot_dim % 2 ||
                           p.rot_dim > kLatentMaxRotary || p.key_stride < p.rot_dim || p.key_stride % 8))
        return QM_ERR_GEOMETRY;
    return QM_OK;
}

int32_t launch_latent_rows(const LatentRowsParams& prm, int f32, hipStream_t stream) {
    const int32_t rc = check_rows(prm);
    if (rc != QM_OK || prm.rows == 0) return rc;
    if (f32) hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(prm.rows), dim3(kDecThreads), 0, stream, prm);
    else hipLaunchKernelGGL(latent_rows_kernel<uint16_t>, dim3(prm.rows), dim3(kDecThreads), 0, stream, prm);
    return launch_status();
}

template <class T, int R>
static int32_t query_as(const LatentAttentionParams& prm, const LatentRowsParams* keep, hipStream_t stream) {
    const dim3 grid(latent_pad(prm.kv_rank) / kLatentSlice, prm.heads + (keep ? 1 : 0), (prm.rows + R - 1) / R);
    const size_t lds = sizeof(float) * (R * prm.dim + 4 * R * 64);
    hipLaunchKernelGGL((latent_query_kernel<T, R>), grid, dim3(kDecThreads), lds, stream, prm, keep ? *keep : LatentRowsParams{});
    return launch_status();
}

template <class T>
static int32_t attend_latents(const LatentAttentionParams& prm, const LatentRowsParams* keep, bool matrix, hipStream_t stream) {
    int32_t rc = prm.rows > 2 ? query_as<T, 4>(prm, keep, stream) : query_as<T, 1>(prm, keep, stream);
    if (rc != QM_OK) return rc;
    if (matrix) {
        rc = launch_latent_partials_mfma(prm, stream);
    } else {
        hipLaunchKernelGGL(latent_partials_kernel<T>, dim3(prm.splits, prm.heads, prm.rows), dim3(kDecThreads),
                           sizeof(float) * latent_q_stride(prm.kv_rank, prm.rot_dim), stream, prm);
        rc = launch_status();
    }
    if (rc != QM_OK) return rc;
    hipLaunchKernelGGL(latent_output_kernel<T>, dim3((prm.vdim + kLatentOutputs - 1) / kLatentOutputs, prm.heads, prm.rows), dim3(kDecThreads),
                       sizeof(float) * ((prm.kv_rank + 511) / 512 * 512), stream, prm);
    return launch_status();
}

int32_t launch_latent_attention(const LatentAttentionParams& prm, const LatentRowsParams* keep, int f32, hipStream_t stream) {
    if (prm.rows < 0 || prm.position < 0) return QM_ERR_ARGUMENT;
    if (!prm.q || !prm.up_k || !prm.up_v || !prm.latent_cache || !prm.key_cache || !prm.out || !prm.q_scratch || !prm.ml || !prm.acc ||
        (prm.rot_dim > 0 && !prm.frequency))
        return QM_ERR_NULL;
    if (prm.heads <= 0 || prm.heads > 65534 || prm.dim <= 0 || prm.dim > 1024 || prm.rot_dim < 0 || prm.rot_dim % 2 || prm.rot_dim > kLatentMaxRotary ||
        prm.vdim <= 0 || prm.kv_rank <= 0 || prm.kv_rank > kLatentMaxRank)
        return QM_ERR_GEOMETRY;
    if (prm.ld_latent < prm.kv_rank || prm.ld_latent % 8 || prm.key_stride < prm.rot_dim || prm.key_stride % 8 || prm.splits < 1 ||
        prm.splits > kDecMaxSplits || prm.rows > 65535 || prm.ld_out % 4 || prm.ld_out < static_cast<int64_t>(prm.heads) * prm.vdim ||
        prm.ld_query < static_cast<int64_t>(prm.heads) * (prm.dim + prm.rot_dim))
        return QM_ERR_GEOMETRY;
    if (keep) {
        const int32_t rc = check_rows(*keep);
        if (rc != QM_OK) return rc;
        if (prm.rows != 1 || !keep->latent_cache) return QM_ERR_ARGUMENT;
    }
    if (prm.rows == 0) return QM_OK;
    const bool rows_only = (prm.options & QM_ATTENTION_ROWS) != 0;
    if (!f32 && !rows_only && !keep && prm.expanded && prm.rows >= kAttentionMatrixRows && !prm.position_dev && prm.dim + prm.rot_dim <= kDecMaxHead &&
        prm.vdim <= kDecMaxHead && prm.ld_latent % 128 == 0) {
        if (prm.up_rows <= 0 || prm.up_rows % 128 || prm.up_v_row < prm.heads * prm.dim || prm.up_v_row + prm.heads * prm.vdim > prm.up_rows ||
            prm.up_v != prm.up_k + static_cast<int64_t>(prm.up_v_row) * prm.ld_latent)
            return QM_ERR_GEOMETRY;
        if (prm.expanded_bytes < expanded_bytes(prm.position + prm.rows, prm.heads, prm.dim, prm.rot_dim, prm.vdim, prm.up_rows)) return QM_ERR_WORKSPACE;
        return attend_expanded(prm, stream);
    }
    if (f32) return attend_latents<float>(prm, keep, false, stream);
    return attend_latents<uint16_t>(prm, keep, !rows_only && latent_partials_fit_mfma(prm), stream);
}

}  // namespace qm

extern "C" int32_t qm_latent_rows_norm(const qm_latent_rows* op, int32_t f32, void* hip_stream) {
    return op ? qm::launch_latent_rows(*op, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
extern "C" int32_t qm_latent_query_stride(int32_t kv_rank, int32_t rot_dim) { return qm::latent_q_stride(kv_rank, rot_dim); }
extern "C" int64_t qm_latent_expanded_bytes(int32_t positions, int32_t heads, int32_t dim, int32_t rot_dim, int32_t vdim, int32_t up_rows) {
    return qm::expanded_bytes(positions, heads, dim, rot_dim, vdim, up_rows);
}
extern "C" int32_t qm_latent_attention_rows(const qm_latent_attention* op, int32_t f32, void* hip_stream) {
    return op ? qm::launch_latent_attention(*op, nullptr, f32, static_cast<hipStream_t>(hip_stream)) : QM_ERR_NULL;
}
