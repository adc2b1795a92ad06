// qm_decoder_step.hip — one token through a layer run in three launches, for gfx950: everything that reads the layer's
// norm, the mixer, everything that leaves the layer.  The small vector work between two linears (residual sum, norms, the
// attention's merge, gates) is repeated by every block that needs its result rather than handed over through a launch of
// its own, while the block's first weights are already on their way.
//
// Bound by HBM (each weight is read once) and, for narrow models, by the latency of the launches.
#include "../qm_host.h"
#include "qm_decoder_attention.h"
#include "qm_decoder_dot.h"
#include "qm_decoder_recurrent.h"

namespace qm {

constexpr int kInRows = 4;                     // weight rows per wave: input linears
constexpr int kOutRows = 2;                    // output linears (few, long rows)
constexpr int kInBlocks = 1024;                // most blocks of the input launch: each repeats the norm

template <class T, int NV>
__global__ __launch_bounds__(kDecThreads) void layer_in_kernel(LayerInParams prm, int tiles) {
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    __shared__ float sh_red[16];
    T* hs = reinterpret_cast<T*>(smem);                                        // [ld_h]
    int tile = static_cast<int>(blockIdx.x);
    int g = dot_group<kInRows>(prm.linears, tile);
    DotRows<kInRows> d = dot_rows<kInRows>(prm.linears.group[g], tile);
    uint4 piece[kDotAhead][kInRows];
    dot_request<kInRows>(d, prm.linears.group[g].k, piece);
    residual_norm_row<T, NV>(prm.residual, 0, sh_red, hs, blockIdx.x == 0);
    __syncthreads();
    if (prm.residual.h && blockIdx.x == 0) {
        T* out = static_cast<T*>(prm.residual.h);
        for (int c = threadIdx.x; c < prm.residual.ld_h; c += kDecThreads) out[c] = hs[c];
    }
    for (int next = static_cast<int>(blockIdx.x) + static_cast<int>(gridDim.x);; next += static_cast<int>(gridDim.x)) {
        dot_finish<T, 1, kInRows>(prm.linears.group[g], d, piece, hs, 0, 1);
        if (next >= tiles) break;
        tile = next;
        g = dot_group<kInRows>(prm.linears, tile);
        d = dot_rows<kInRows>(prm.linears.group[g], tile);
        dot_request<kInRows>(d, prm.linears.group[g].k, piece);
    }
}

template <class T>
__global__ __launch_bounds__(kDecThreads) void layer_out_kernel(LayerOutParams prm, int most_k) {
    request_arguments(prm);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    __shared__ float sh_red[4];
    T* xs = reinterpret_cast<T*>(smem);
    int tile = static_cast<int>(blockIdx.x);
    const int g = dot_group<kOutRows>(prm.linears, tile);
    const DecLinearGroup& group = prm.linears.group[g];
    const DotRows<kOutRows> d = dot_rows<kOutRows>(group, tile);
    uint4 piece[kDotAhead][kOutRows];
    dot_request<kOutRows>(d, group.k, piece);
    if (prm.input[g] == 1) {
        merge_attention_row<T>(prm.part, 0, attention_active_splits(*prm.position_dev, prm.chunk, prm.part.keys_per_split),
                               reinterpret_cast<float*>(xs + most_k), xs, group.k);
    } else if (prm.input[g] == 2) {
        gated_norm_row<T>(prm.gated, 0, sh_red, xs);
    } else if (prm.input[g] == 3) {
        slice_norm_row<T>(prm.slice.x, prm.slice.weight, prm.slice.n, group.k, prm.slice.eps, sh_red, xs);
    } else {
        constexpr int kVec = 16 / sizeof(T);
        const T* x = static_cast<const T*>(group.x);
        for (int c = threadIdx.x * kVec; c < group.k; c += kDecThreads * kVec)
            *reinterpret_cast<uint4*>(xs + c) = *reinterpret_cast<const uint4*>(x + c);
    }
    __syncthreads();
    dot_finish<T, 1, kOutRows>(group, d, piece, xs, 0, 1);
}

template <class T, int GQ, int VC>
__global__ __launch_bounds__(kDecThreads) void mixer_step_kernel(ChunkAttentionParams attention, DecayAttentionParams decay) {
    request_arguments(attention, decay);
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int attention_blocks = attention.part.splits * attention.kv_heads;
    int block = static_cast<int>(blockIdx.x);
    if (block < attention_blocks) {
        chunk_attention_block<T, GQ, VC, true>(attention, block % attention.part.splits, block / attention.part.splits, 0, lds);
        return;
    }
    block -= attention_blocks;
    const int slices = (decay.vdim + kRecColumns - 1) / kRecColumns;
    const int head = block / slices, slice = block % slices;
    if (decay.dim <= 32) decay_attention_block<8>(decay, head, slice, lds);
    else if (decay.dim <= 64) decay_attention_block<16>(decay, head, slice, lds);
    else if (decay.dim <= 128) decay_attention_block<32>(decay, head, slice, lds);
    else decay_attention_block<64>(decay, head, slice, lds);
}

constexpr int kArgmaxThreads = 1024;
__global__ __launch_bounds__(kArgmaxThreads) void argmax_kernel(const float* scores, int vocab, int32_t* token) {
    __shared__ float sh_best[kArgmaxThreads / 64];
    __shared__ int sh_id[kArgmaxThreads / 64];
    float best = -INFINITY;
    int id = 0x7fffffff;
    for (int i = threadIdx.x; i < vocab; i += kArgmaxThreads) {
        const float v = scores[i];
        if (v > best || id == 0x7fffffff) {
            best = v;
            id = i;
        }
    }
    auto take = [&](float v, int i) {
        if (v > best || (v == best && i < id)) {
            best = v;
            id = i;
        }
    };
#pragma unroll
    for (int m = 1; m < 64; m *= 2) {
        const float v = __shfl_xor(best, m, 64);
        const int i = __shfl_xor(id, m, 64);
        take(v, i);
    }
    if ((threadIdx.x & 63) == 0) {
        sh_best[threadIdx.x >> 6] = best;
        sh_id[threadIdx.x >> 6] = id;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < kArgmaxThreads / 64; ++w) take(sh_best[w], sh_id[w]);
        *token = id < vocab ? id : 0;
    }
}

__global__ void emit_kernel(int32_t* step, int32_t* out, int advance) {
    out[step[kStepEmitted]++] = step[kStepChosen];
    step[kStepBefore] = step[kStepToken];
    step[kStepToken] = step[kStepChosen];
    step[kStepPosition] += advance;
}

static int most_k(const DecLinearParams& prm) {
    int k = 0;
    for (int g = 0; g < prm.groups; ++g) k = prm.group[g].k > k ? prm.group[g].k : k;
    return k;
}

template <class T, int NV>
static int32_t layer_in_as(const LayerInParams& prm, hipStream_t stream) {
    const int tiles = dot_tiles_of<kInRows>(prm.linears);
    const size_t lds = static_cast<size_t>(prm.residual.ld_h) * sizeof(T);
    hipLaunchKernelGGL((layer_in_kernel<T, NV>), dim3(tiles < kInBlocks ? tiles : kInBlocks), dim3(kDecThreads), lds, stream, prm, tiles);
    return launch_status();
}
template <class T>
static int32_t layer_in(const LayerInParams& prm, hipStream_t stream) {
    switch (row_vectors(prm.residual.ld_h)) {
        case 1: return layer_in_as<T, 1>(prm, stream);
        case 2: return layer_in_as<T, 2>(prm, stream);
        case 4: return layer_in_as<T, 4>(prm, stream);
        default: return layer_in_as<T, 12>(prm, stream);
    }
}

int32_t launch_layer_in(const LayerInParams& prm, int f32, hipStream_t stream) {
    if (prm.linears.groups < 1 || prm.linears.groups > kDecGroups || prm.linears.rows != 1) return QM_ERR_ARGUMENT;
    for (int g = 0; g < prm.linears.groups; ++g) {
        const DecLinearGroup& d = prm.linears.group[g];
        if (!d.w || (d.w_up ? !d.out : !d.out32)) return QM_ERR_NULL;
        if (d.n <= 0 || d.n % (d.w_up ? 128 : 16) || d.k % 128 || d.k != prm.residual.ld_h) return QM_ERR_GEOMETRY;
    }
    const int32_t rc = check_residual(prm.residual);
    if (rc != QM_OK) return rc;
    return f32 ? layer_in<float>(prm, stream) : layer_in<uint16_t>(prm, stream);
}

template <class T>
static int32_t layer_out_as(const LayerOutParams& prm, hipStream_t stream) {
    const size_t merge = prm.part.ml ? static_cast<size_t>(prm.part.heads) * prm.part.splits * sizeof(float) : 0;
    const int k = most_k(prm.linears);
    const size_t lds = static_cast<size_t>(k) * sizeof(T) + merge;
    static std::atomic<bool> raised[kMaxDevices];
    const int32_t rc = ensure_dynamic_lds(reinterpret_cast<const void*>(layer_out_kernel<T>), kDotLdsMost, raised);
    if (rc != QM_OK) return rc;
    if (lds > static_cast<size_t>(kDotLdsMost)) return QM_ERR_GEOMETRY;
    hipLaunchKernelGGL(layer_out_kernel<T>, dim3(dot_tiles_of<kOutRows>(prm.linears)), dim3(kDecThreads), lds, stream, prm, k);
    return launch_status();
}

int32_t launch_layer_out(const LayerOutParams& prm, int f32, hipStream_t stream) {
    if (prm.linears.groups < 1 || prm.linears.groups > kDecGroups || prm.linears.rows != 1) return QM_ERR_ARGUMENT;
    for (int g = 0; g < prm.linears.groups; ++g) {
        const DecLinearGroup& d = prm.linears.group[g];
        if (!d.w || !d.out32 || (prm.input[g] == 0 && !d.x) || (prm.input[g] == 1 && (!prm.part.ml || !prm.part.acc || !prm.position_dev))) return QM_ERR_NULL;
        if (d.n <= 0 || d.n % 128 || d.k % 128) return QM_ERR_GEOMETRY;
        if (prm.input[g] == 1 && d.k < prm.part.heads * prm.part.vdim) return QM_ERR_GEOMETRY;
        if (prm.input[g] == 2 && (d.k < prm.gated.groups * prm.gated.size || prm.gated.ld_out != d.k)) return QM_ERR_GEOMETRY;
        if (prm.input[g] == 3 && (!prm.slice.x || !prm.slice.weight || prm.slice.n <= 0 || prm.slice.n > d.k)) return QM_ERR_GEOMETRY;
    }
    return f32 ? layer_out_as<float>(prm, stream) : layer_out_as<uint16_t>(prm, stream);
}

template <class T, int GQ, int VC>
static int32_t mixer_step_as(const ChunkAttentionParams& a, const DecayAttentionParams& d, hipStream_t stream) {
    const int rd = d.dim <= 32 ? 8 : d.dim <= 64 ? 16 : d.dim <= 128 ? 32 : 64;
    const int attention = attention_lds_floats(GQ, a.k_stride, a.v_stride), decay = decay_lds_floats(rd);
    const int blocks = a.part.splits * a.kv_heads + d.heads * ((d.vdim + kRecColumns - 1) / kRecColumns);
    hipLaunchKernelGGL((mixer_step_kernel<T, GQ, VC>), dim3(blocks), dim3(kDecThreads), sizeof(float) * (attention > decay ? attention : decay), stream,
                       a, d);
    return launch_status();
}
template <class T, int GQ>
static int32_t mixer_step_group(const ChunkAttentionParams& a, const DecayAttentionParams& d, hipStream_t stream) {
    return a.v_stride <= 128 && a.k_stride <= 128 ? mixer_step_as<T, GQ, 1>(a, d, stream) : mixer_step_as<T, GQ, 2>(a, d, stream);
}
template <class T>
static int32_t mixer_step(const ChunkAttentionParams& a, const DecayAttentionParams& d, hipStream_t stream) {
    const int group = a.heads / a.kv_heads;
    return group == 1 ? mixer_step_group<T, 1>(a, d, stream) : group == 2 ? mixer_step_group<T, 2>(a, d, stream) : mixer_step_group<T, 4>(a, d, stream);
}

int32_t launch_mixer_step(const ChunkAttentionParams& attention, const DecayAttentionParams& decay, int f32, hipStream_t stream) {
    int32_t rc = check_attention(attention);
    if (rc == QM_OK) rc = check_decay_attention(decay);
    if (rc != QM_OK) return rc;
    if (attention.rows != 1 || decay.rows != 1) return QM_ERR_ARGUMENT;
    return f32 ? mixer_step<float>(attention, decay, stream) : mixer_step<uint16_t>(attention, decay, stream);
}

int32_t launch_argmax(const float* scores, int vocab, int32_t* token, hipStream_t stream) {
    if (!scores || !token) return QM_ERR_NULL;
    if (vocab <= 0) return QM_ERR_ARGUMENT;
    hipLaunchKernelGGL(argmax_kernel, dim3(1), dim3(kArgmaxThreads), 0, stream, scores, vocab, token);
    return launch_status();
}

int32_t launch_emit(int32_t* step, int32_t* out, int advance, hipStream_t stream) {
    if (!step || !out) return QM_ERR_NULL;
    hipLaunchKernelGGL(emit_kernel, dim3(1), dim3(1), 0, stream, step, out, advance);
    return launch_status();
}

}  // namespace qm
