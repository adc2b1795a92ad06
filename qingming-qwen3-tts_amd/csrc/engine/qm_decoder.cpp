// qm_decoder.cpp — the engine of the decoder language models: weights from safetensors, the caches and states of every
// live sequence, the step over a sequence's next tokens, and generation.
//
// A model is a list of layer runs (a repeated layer runs several times, each pass with caches and states of its own).  One
// sequence's memory is one allocation: per run the ring caches of its attention, the fp32 states of its recurrences.  A
// step takes what earlier steps left there, so a prompt may be cut anywhere.
//
// A pass of many rows, per layer run:
//   qm_residual_norm_rows   the last layer's sublayers onto the stream, the vector of a loop's pass, norm1
//   linears                 every projection of the mixer as one matrix (fp32 out), gate/up with SwiGLU
//   mixer                   rotation + cache write + attention and decayed linear attention, or the delta rule, or retention,
//                           or attention over latents; gated norm
//   linears                 the output projections and the feed-forward's down projection in one launch
// Where a layer's feed-forward has norms of its own it follows in the same way: residual + norm, gate/up, down, or the experts.
// One token: the same in few fused launches per layer run, replayed from a graph that reads tokens and position from device
// memory.
#include "../../../include/qm_decoder.h"

#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>
#include <cstring>
#include <memory>
#include <string>
#include <vector>

#include "../decoder/qm_decoder_ops.h"
#include "qm_decoder_config.hpp"
#include "qm_engine_common.hpp"

namespace qm_engine {

std::string& last_error() {
    thread_local std::string text;
    return text;
}

namespace {

constexpr float kUnitEps = 1.0e-6f;       // inside the root of the delta rule's unit key
constexpr int kLogitRows = 256;           // rows of the head at once
using qm::kStepWords;                      // device words of a one-token step

int padded(int n, int to) { return (n + to - 1) / to * to; }

// a named section of a fused projection: `columns` outputs from column `at` on
struct Section {
    int at = 0, columns = 0;
};

struct Matrix {
    DeviceBuffer data;                    // [n][k] bf16, zero rows and columns behind
    int n = 0, k = 0;
    const uint16_t* u16() const { return data.u16(); }
};

float widen(uint16_t v) {
    const uint32_t bits = static_cast<uint32_t>(v) << 16;
    float f;
    std::memcpy(&f, &bits, sizeof f);
    return f;
}

struct DecoderLayer {
    DecoderLayerConfig config;
    DeviceBuffer norm1;
    Matrix in, gate, up, down, o_left, o_right;     // delta rule: its output projection is o_right
    Section q, k, v;                                // attention's
    Section dq, dk, dv, dg;                         // decayed attention's q, k, v, gate
    Section r, kk, vv, a, g, z;                     // delta rule's
    DeviceBuffer out_left, out_right, mix_norm, powers, frequency, w2, w0, a_bias;
    int rank = 0;
    DeviceBuffer norm2, after_mixer, after_ff;      // a sandwich layer's other norms
    Section q_latent, kv_latent, up_v;              // latent attention's: in `in`, and the values in `up_latent` (keys at 0)
    Matrix q_up, up_latent, router;
    DeviceBuffer q_norm, kv_norm;
    double magnitude = 1.0;
};

struct RunState {                                   // byte offsets inside a sequence's memory
    size_t k = 0, v = 0, decay = 0, delta = 0, latent = 0, key = 0;
};

}  // namespace
}  // namespace qm_engine

struct qm_decoder {
    qm_engine::DecoderConfig config;
    std::vector<qm_engine::DecoderLayer> layers;
    std::vector<qm_engine::LayerRun> runs;
    std::vector<qm_engine::RunState> states;
    std::vector<qm_engine::DeviceBuffer> memory;    // one per sequence
    std::vector<int> length;                        // tokens of each live sequence, -1: free
    std::vector<int32_t> before;                    // its last token, -1: none
    size_t sequence_bytes = 0;
    qm_engine::DeviceBuffer final_norm, loop_step;
    qm_engine::Matrix embed, bigram, head;
    int capacity = 0, max_rows = 0, f32 = 0, path = 0;
    bool warm = false;
    int width_p = 0, vocab_p = 0;
    hipStream_t stream = nullptr;
    bool own_stream = false;
    qm_engine::DeviceBuffer x[2], h, proj, mlp, attended, gated, y[3], q_rot, raw, ml, acc, scratch, tokens, wanted, head_h, logits, tap, tap_h,
        step_words, q_latent, queries, q_scratch, expanded, expert_logits, expert_scratch;
    std::vector<hipGraphExec_t> graphs;             // one-token step of each sequence

    ~qm_decoder() {
        for (hipGraphExec_t g : graphs)
            if (g) (void)hipGraphExecDestroy(g);
        if (own_stream && stream) (void)hipStreamDestroy(stream);
    }
};

namespace qm_engine {
namespace {

// ---- weights -------------------------------------------------------------------------------------------------------

class Loader {
public:
    explicit Loader(const std::string& dir) : files_(dir) {}
    const TensorView& get(const std::string& name, const std::vector<int64_t>& shape) const {
        const TensorView* t = files_.find(name);
        if (!t) throw TensorError("tensor missing: " + name);
        if (t->dtype != "BF16") throw TensorError("expected BF16 tensor: " + name);
        if (t->shape != shape) throw TensorError("unexpected shape of " + name);
        return *t;
    }
    int64_t extent(const std::string& name, size_t axis) const {
        const TensorView* t = files_.find(name);
        if (!t) throw TensorError("tensor missing: " + name);
        if (axis >= t->shape.size() || t->shape[axis] <= 0) throw TensorError("unexpected shape of " + name);
        return t->shape[axis];
    }
    // a vector, or a small matrix, as fp32
    DeviceBuffer floats(const std::string& name, const std::vector<int64_t>& shape) const {
        return padded_floats(name, shape, static_cast<int>(shape.back()));
    }
    // the same with zeros behind each row, up to `columns`
    DeviceBuffer padded_floats(const std::string& name, const std::vector<int64_t>& shape, int columns) const {
        const TensorView& t = get(name, shape);
        const size_t from = static_cast<size_t>(shape.back()), rows = t.elements() / from;
        std::vector<float> host(rows * columns, 0.0f);
        for (size_t r = 0; r < rows; ++r)
            for (size_t c = 0; c < from; ++c) host[r * columns + c] = element(t, r * from + c);
        return upload(host.data(), host.size() * sizeof(float));
    }
    // a norm's weight, stored less one or as it is, times `scale`
    DeviceBuffer norm(const std::string& name, int width, bool around_zero, double scale = 1.0) const {
        const TensorView& t = get(name, {width});
        std::vector<float> host(static_cast<size_t>(padded(width, 128)), 0.0f);
        for (int c = 0; c < width; ++c)
            host[static_cast<size_t>(c)] = static_cast<float>(((around_zero ? 1.0 : 0.0) + element(t, static_cast<size_t>(c))) * scale);
        return upload(host.data(), host.size() * sizeof(float));
    }
    DeviceBuffer transposed_floats(const std::string& name, int64_t rows, int64_t columns) const {
        const TensorView& t = get(name, {rows, columns});
        std::vector<float> host(t.elements());
        for (int64_t r = 0; r < rows; ++r)
            for (int64_t c = 0; c < columns; ++c) host[c * rows + r] = element(t, r * columns + c);
        return upload(host.data(), host.size() * sizeof(float));
    }
    static float element(const TensorView& t, size_t i) {
        uint16_t bits;
        std::memcpy(&bits, t.data + 2 * i, 2);
        return widen(bits);
    }
    static DeviceBuffer upload(const void* data, size_t bytes) {
        DeviceBuffer b(bytes);
        hip_check(hipMemcpy(b.raw(), data, bytes, hipMemcpyHostToDevice), "weight upload");
        return b;
    }
    // linears of one input stacked into one matrix, each from a multiple of 8 rows on
    struct Part {
        std::string name;
        int columns;
        Section* section;
    };
    Matrix stacked(const std::vector<Part>& parts, int k, int rows_to = 128) const {
        Matrix m;
        int n = 0;
        for (const Part& p : parts) {
            if (p.section) *p.section = {n, p.columns};
            n += padded(p.columns, 8);
        }
        m.n = padded(n, rows_to);
        m.k = padded(k, 128);
        std::vector<uint16_t> host(static_cast<size_t>(m.n) * m.k, 0);
        int at = 0;
        for (const Part& p : parts) {
            const TensorView& t = get(p.name, {p.columns, k});
            for (int r = 0; r < p.columns; ++r)
                std::memcpy(host.data() + static_cast<size_t>(at + r) * m.k, t.data + static_cast<size_t>(r) * k * 2, static_cast<size_t>(k) * 2);
            at += padded(p.columns, 8);
        }
        m.data = upload(host.data(), host.size() * 2);
        return m;
    }
    Matrix matrix(const std::string& name, int n, int k) const { return stacked({{name, n, nullptr}}, k); }
    // `count` matrices of one shape one behind the other, each padded for itself (n: rows of one)
    template <class Name>
    Matrix each(int count, Name name, int n, int k) const {
        Matrix m;
        m.n = padded(n, 128);
        m.k = padded(k, 128);
        m.data = DeviceBuffer(static_cast<size_t>(count) * m.n * m.k * 2);
        std::vector<uint16_t> host(static_cast<size_t>(m.n) * m.k, 0);
        for (int i = 0; i < count; ++i) {
            const TensorView& t = get(name(i), {n, k});
            for (int r = 0; r < n; ++r)
                std::memcpy(host.data() + static_cast<size_t>(r) * m.k, t.data + static_cast<size_t>(r) * k * 2, static_cast<size_t>(k) * 2);
            hip_check(hipMemcpy(m.data.u16() + static_cast<size_t>(i) * m.n * m.k, host.data(), host.size() * 2, hipMemcpyHostToDevice), "weight upload");
        }
        return m;
    }

private:
    ModelDirectory files_;
};

DeviceBuffer upload_doubles(std::vector<double> values) {
    if (values.empty()) values.push_back(0.0);
    return Loader::upload(values.data(), values.size() * sizeof(double));
}
DeviceBuffer decay_powers(const std::vector<double>& decays) {
    std::vector<float> powers;
    for (double decay : decays)
        for (int i = 0; i < QM_DECAY_POWERS; ++i) powers.push_back(static_cast<float>(i == 0 ? 1.0 : std::pow(decay, i)));
    return Loader::upload(powers.data(), powers.size() * sizeof(float));
}

DecoderLayer load_layer(const Loader& from, const DecoderConfig& model, int index) {
    DecoderLayer w;
    const DecoderLayerConfig& config = w.config = model.layers[static_cast<size_t>(index)];
    const int width = model.width;
    const std::string base = "l" + std::to_string(index) + ".", mix = base + "mix.";
    w.norm1 = from.norm(base + "norm1", width, model.norms_around_zero);
    if (config.form == LayerForm::Sandwich) {
        w.after_mixer = from.norm(base + "norm1b", width, model.norms_around_zero);
        if (config.ff) {
            w.norm2 = from.norm(base + "norm2", width, model.norms_around_zero);
            w.after_ff = from.norm(base + "norm2b", width, model.norms_around_zero);
        }
    }
    if (config.mixer == MixerKind::AttentionBesideDecay) {
        const ChunkAttentionConfig& a = config.attention;
        const DecayAttentionConfig& d = config.decay;
        w.in = from.stacked({{mix + "left.q", a.heads * a.dim, &w.q}, {mix + "left.k", a.kv_heads * a.dim, &w.k},
                             {mix + "left.v", a.kv_heads * a.vdim, &w.v}, {mix + "right.q", d.heads * d.dim, &w.dq},
                             {mix + "right.k", d.heads * d.dim, &w.dk}, {mix + "right.v", d.heads * d.vdim, &w.dv},
                             {mix + "right.g", d.heads * d.vdim, &w.dg}}, width);
        w.o_left = from.matrix(mix + "left.o", width, a.heads * a.vdim);
        w.o_right = from.matrix(mix + "right.o", width, d.heads * d.vdim);
        w.mix_norm = from.floats(mix + "right.norm", {d.heads * d.vdim});
        w.out_left = from.padded_floats(mix + "left.out", {width}, padded(width, 128));
        w.out_right = from.padded_floats(mix + "right.out", {width}, padded(width, 128));
        w.frequency = upload_doubles(rotary_frequencies(a.rot_dims, a.rot_base, {}, nullptr));
        w.powers = decay_powers(d.decay);
    } else if (config.mixer == MixerKind::Retention) {
        const RetentionConfig& c = config.retention;
        w.in = from.stacked({{mix + "q", c.heads * c.dim, &w.dq}, {mix + "k", c.heads * c.dim, &w.dk}, {mix + "v", c.heads * c.vdim, &w.dv},
                             {mix + "g", c.heads * c.vdim, &w.dg}}, width);
        w.o_right = from.matrix(mix + "o", width, c.heads * c.vdim);
        w.frequency = upload_doubles(rotary_frequencies(c.rot_dims, c.rot_base, {}, nullptr));
        w.powers = decay_powers(c.decay);
    } else if (config.mixer == MixerKind::LatentAttention) {
        const LatentAttentionConfig& c = config.latent;
        std::vector<Loader::Part> in = {{mix + "dq", c.q_rank, &w.q_latent}};
        if (c.kv_from < 0) {
            in.push_back({mix + "dkv", c.kv_rank + c.rot_dim, &w.kv_latent});
            w.kv_norm = from.floats(mix + "dkv.norm", {c.kv_rank});
        }
        w.in = from.stacked(in, width);
        w.q_norm = from.floats(mix + "dq.norm", {c.q_rank});
        w.q_up = from.matrix(mix + "uq", c.heads * (c.dim + c.rot_dim), c.q_rank);
        w.up_latent = from.stacked({{mix + "uk", c.heads * c.dim, nullptr}, {mix + "uv", c.heads * c.vdim, &w.up_v}}, c.kv_rank);
        w.o_left = from.matrix(mix + "o", width, c.heads * c.vdim);
        w.frequency = upload_doubles(rotary_frequencies(c.rot_dim, c.rot_base, c.scaling, &w.magnitude));
    } else {
        const int all = config.delta.heads * config.delta.dim;
        w.rank = static_cast<int>(from.extent(mix + "w1", 0));
        w.in = from.stacked({{mix + "r", all, &w.r}, {mix + "k", all, &w.kk}, {mix + "v", all, &w.vv}, {mix + "a", all, &w.a},
                             {mix + "g", all, &w.g}, {mix + "w1", w.rank, &w.z}}, width);
        w.w2 = from.transposed_floats(mix + "w2", all, w.rank);
        w.w0 = from.floats(mix + "w0", {all});
        w.a_bias = from.floats(mix + "a.b", {all});
        w.mix_norm = from.floats(mix + "norm", {all});
        w.o_right = from.matrix(mix + "o", width, all);
    }
    if (config.experts) {
        auto named = [&](const char* which) { return [&base, which](int e) { return base + "mlp.e" + std::to_string(e) + "." + which; }; };
        w.gate = from.each(config.experts, named("gate"), config.ff, width);
        w.up = from.each(config.experts, named("up"), config.ff, width);
        w.down = from.each(config.experts, named("down"), width, config.ff);
        w.router = from.stacked({{base + "mlp.router", config.experts, nullptr}}, width, config.experts <= 64 ? 16 : 128);
    } else if (config.ff) {
        w.gate = from.matrix(base + "mlp.gate", config.ff, width);
        w.up = from.matrix(base + "mlp.up", config.ff, width);
        w.down = from.matrix(base + "mlp.down", width, config.ff);
    }
    return w;
}

int ring_of(const qm_decoder& d, const ChunkAttentionConfig& a) { return std::min<int64_t>(d.capacity, static_cast<int64_t>(a.chunk) + d.max_rows); }
int chunk_of(const qm_decoder& d, const ChunkAttentionConfig& a) { return std::min(a.chunk, d.capacity); }

// Key splits of one token's attention over latents: passes of 64 keys, as many splits as there may be.
int latent_splits(int capacity) { return std::clamp((capacity + qm::kLatentKeys - 1) / qm::kLatentKeys, 1, qm::kDecMaxSplits); }

// A chunk's keys in at most 16 splits of whole passes of 128 keys.
int keys_per_split(int chunk) { return padded(std::max(128, (chunk + 15) / 16), 128); }
int key_splits(int chunk) { return (chunk + keys_per_split(chunk) - 1) / keys_per_split(chunk); }

std::unique_ptr<qm_decoder> create_decoder(const std::string& dir, int f32, int capacity, int sequences, int max_rows, hipStream_t stream) {
    if (capacity <= 0 || sequences <= 0 || max_rows < 0 || (f32 != 0 && f32 != 1))
        throw ApiError(QM_ERR_ARGUMENT, "capacity and sequences must be positive");
    auto d = std::make_unique<qm_decoder>();
    d->config = read_decoder_config(dir + "/config.json");
    d->runs = layer_runs(d->config);
    d->capacity = capacity;
    d->max_rows = std::min(capacity, max_rows ? max_rows : 2048);
    d->f32 = f32;
    const int width = d->config.width;
    if (padded(width, 128) > qm::kDecMaxWidth) throw ApiError(QM_ERR_GEOMETRY, "model width beyond the kernels' limit");
    d->stream = stream;
    if (!stream) {
        hip_check(hipStreamCreateWithFlags(&d->stream, hipStreamNonBlocking), "decoder stream");
        d->own_stream = true;
    }
    const Loader from(dir);
    d->width_p = padded(width, 128);
    d->vocab_p = padded(d->config.vocab, 128);
    d->embed = from.matrix("embed", d->config.vocab, width);
    if (d->config.bigram_buckets) d->bigram = from.matrix("bigram", d->config.bigram_buckets + 1, width);
    d->final_norm = from.norm("final.norm", width, d->config.norms_around_zero, d->config.logit_scale);    // (the scores' scale is linear in it)
    d->head = from.matrix("head", d->config.vocab, width);
    if (d->config.loop_times) d->loop_step = from.padded_floats("loop.step", {d->config.loop_times, width}, d->width_p);
    for (size_t i = 0; i < d->config.layers.size(); ++i)
        d->layers.push_back(load_layer(from, d->config, static_cast<int>(i)));

    // one sequence's memory
    const size_t item = f32 ? 4 : 2;
    size_t at = 0;
    auto take = [&](size_t bytes) {
        const size_t here = at;
        at += (bytes + 255) / 256 * 256;
        return here;
    };
    for (const LayerRun& run : d->runs) {
        const DecoderLayerConfig& c = d->config.layers[static_cast<size_t>(run.layer)];
        RunState s;
        if (c.mixer == MixerKind::AttentionBesideDecay) {
            const size_t ring = static_cast<size_t>(ring_of(*d, c.attention)) * c.attention.kv_heads * item;
            s.k = take(ring * padded(c.attention.dim, 8));
            s.v = take(ring * padded(c.attention.vdim, 8));
            s.decay = take(static_cast<size_t>(c.decay.heads) * c.decay.dim * c.decay.vdim * 4);
        } else if (c.mixer == MixerKind::Retention) {
            s.decay = take(static_cast<size_t>(c.retention.heads) * c.retention.dim * c.retention.vdim * 4);
        } else if (c.mixer == MixerKind::LatentAttention) {
            if (c.latent.kv_from >= 0) {
                s = d->states[static_cast<size_t>(c.latent.kv_from)];          // (such models have no loop: run i is layer i)
            } else {
                s.latent = take(static_cast<size_t>(capacity) * padded(c.latent.kv_rank, 128) * item);
                s.key = take(static_cast<size_t>(capacity) * padded(c.latent.rot_dim, 8) * item);
            }
        } else {
            s.delta = take(static_cast<size_t>(c.delta.heads) * c.delta.dim * c.delta.dim * 4);
        }
        d->states.push_back(s);
    }
    d->sequence_bytes = at;
    for (int i = 0; i < sequences; ++i) {
        d->memory.emplace_back(at);
        d->length.push_back(-1);
        d->before.push_back(-1);
    }
    d->graphs.assign(static_cast<size_t>(sequences), nullptr);

    // activations of a pass
    const size_t rows = static_cast<size_t>(d->max_rows);
    size_t proj = 0, mlp = 0, attended = 0, gated = 0, q_rot = 0, raw = 0, ml = 0, acc = 0, scratch = 0;
    size_t q_latent = 0, queries = 0, q_scratch = 0, expanded = 0, expert_logits = 0, expert_scratch = 0;
    for (const DecoderLayer& w : d->layers) {
        const DecoderLayerConfig& c = w.config;
        proj = std::max(proj, static_cast<size_t>(w.in.n));
        if (!c.experts) mlp = std::max(mlp, static_cast<size_t>(w.down.k));
        if (c.experts) {
            expert_logits = std::max(expert_logits, static_cast<size_t>(w.router.n));
            expert_scratch = std::max(expert_scratch, static_cast<size_t>(qm::expert_scratch_bytes(d->max_rows, c.experts, c.top, d->width_p, w.gate.n, f32)));
        }
        gated = std::max(gated, static_cast<size_t>(w.o_right.k));
        if (c.mixer == MixerKind::AttentionBesideDecay) {
            const int splits = key_splits(chunk_of(*d, c.attention));
            attended = std::max(attended, static_cast<size_t>(w.o_left.k));
            q_rot = std::max(q_rot, static_cast<size_t>(c.attention.heads) * padded(c.attention.dim, 8));
            // (many rows are not split: one record per row and head)
            const size_t records = std::max(rows, static_cast<size_t>(16) * splits) * c.attention.heads;
            ml = std::max(ml, records * 2);
            acc = std::max(acc, records * c.attention.vdim);
            raw = std::max(raw, static_cast<size_t>(c.decay.heads) * c.decay.vdim);
            scratch = std::max(scratch, static_cast<size_t>(qm::decay_scratch_floats(d->max_rows, c.decay.heads, c.decay.dim, c.decay.vdim)));
        } else if (c.mixer == MixerKind::Retention) {
            const RetentionConfig& r = c.retention;
            raw = std::max(raw, static_cast<size_t>(r.heads) * r.vdim);
            scratch = std::max(scratch, static_cast<size_t>(qm::decay_scratch_floats(d->max_rows, r.heads, r.dim, r.vdim)));
        } else if (c.mixer == MixerKind::LatentAttention) {
            const LatentAttentionConfig& l = c.latent;
            attended = std::max(attended, static_cast<size_t>(w.o_left.k));
            q_latent = std::max(q_latent, static_cast<size_t>(w.q_up.k));
            queries = std::max(queries, static_cast<size_t>(w.q_up.n));
            q_scratch = std::max(q_scratch, rows * l.heads * qm::latent_q_stride(l.kv_rank, l.rot_dim));
            const size_t records = std::max(rows, static_cast<size_t>(qm::kAttentionMatrixRows) * latent_splits(capacity)) * l.heads;
            ml = std::max(ml, records * 2);
            acc = std::max(acc, records * l.kv_rank);
            if (!f32)
                expanded = std::max(expanded, static_cast<size_t>(qm_latent_expanded_bytes(capacity, l.heads, l.dim, l.rot_dim, l.vdim, w.up_latent.n)));
        } else {
            raw = std::max(raw, static_cast<size_t>(c.delta.heads) * c.delta.dim);
            scratch = std::max(scratch, static_cast<size_t>(qm::delta_scratch_floats(d->max_rows, c.delta.heads, c.delta.dim)));
        }
    }
    // (buffers a matrix product reads begin as zeros: what lies behind a narrower layer's columns is then always finite)
    auto zeros = [&](size_t bytes) {
        DeviceBuffer b(std::max<size_t>(bytes, 256));
        hip_check(hipMemset(b.raw(), 0, b.bytes()), "activation reset");
        return b;
    };
    const size_t stream_floats = rows * static_cast<size_t>(d->width_p);
    d->x[0] = zeros(stream_floats * 4);
    d->x[1] = zeros(stream_floats * 4);
    d->h = zeros(rows * d->width_p * item);
    d->proj = zeros(rows * proj * 4);
    d->mlp = zeros(rows * mlp * item);
    d->attended = zeros(rows * attended * item);
    d->gated = zeros(rows * gated * item);
    for (DeviceBuffer& y : d->y) y = zeros(rows * d->width_p * 4);
    d->q_rot = zeros(rows * q_rot * item);
    d->raw = zeros(rows * raw * 4);
    d->ml = zeros(ml * 4);
    d->acc = zeros(acc * 4);
    d->scratch = zeros(scratch * 4);
    d->tokens = zeros((rows + 1) * 4);                                         // the token before, then the pass's
    d->q_latent = zeros(rows * q_latent * item);
    d->queries = zeros(rows * queries * 4);
    d->q_scratch = zeros(q_scratch * item);
    d->expanded = zeros(expanded);
    d->expert_logits = zeros(rows * expert_logits * 4);
    d->expert_scratch = zeros(expert_scratch);
    d->wanted = zeros(kLogitRows * 4);
    d->head_h = zeros(static_cast<size_t>(kLogitRows) * d->width_p * item);
    d->logits = zeros(static_cast<size_t>(kLogitRows) * d->vocab_p * 4);
    d->step_words = zeros(kStepWords * 4);
    hip_check(hipDeviceSynchronize(), "decoder setup");
    return d;
}

// ---- a pass over the rows of one sequence ------------------------------------------------------------------------------

// What the layers so far have left to add to the stream.
struct Pending {
    qm_residual_term term[3] = {};
    int count = 0;
};

qm_residual_norm residual_of(const qm_decoder& d, const Pending& pending, const float* x_in, float* x_out, const float* step_vec, const float* norm,
                             void* h) {
    qm_residual_norm p = {};
    p.x_in = x_in;
    p.embed = d.embed.u16();
    p.tokens = static_cast<const int32_t*>(d.tokens.raw()) + 1;
    p.bigram = d.bigram.u16();
    p.buckets = d.config.bigram_buckets; p.mul_prev = d.config.bigram_mul_prev; p.mul_cur = d.config.bigram_mul_cur;
    p.step_vec = step_vec;
    p.norm_w = norm;
    p.x_out = x_out;
    p.h = h;
    p.ld_h = d.width_p;
    p.width = d.config.width;
    p.vocab = d.config.vocab;
    p.eps = static_cast<float>(d.config.eps);
    p.terms = pending.count;
    for (int i = 0; i < pending.count; ++i) p.term[i] = pending.term[i];
    return p;
}

float* f32_of(const DeviceBuffer& b) { return static_cast<float*>(b.raw()); }
char* at_of(const DeviceBuffer& b, size_t offset) { return static_cast<char*>(b.raw()) + offset; }

const float* step_vec_of(const qm_decoder& d, const LayerRun& run) {
    return run.opens_pass < 0 ? nullptr : f32_of(d.loop_step) + static_cast<size_t>(run.opens_pass) * d.width_p;
}

qm_chunk_attention attention_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows, int position) {
    const ChunkAttentionConfig& a = w.config.attention;
    const DeviceBuffer& memory = d.memory[static_cast<size_t>(sequence)];
    qm_chunk_attention p = {};
    p.proj = f32_of(d.proj);
    p.frequency = static_cast<const double*>(w.frequency.raw());
    p.q_rot = d.q_rot.raw();
    p.k_cache = at_of(memory, s.k);
    p.v_cache = at_of(memory, s.v);
    p.out = d.attended.raw();
    p.ld_proj = w.in.n;
    p.ld_out = w.o_left.k;
    p.position = position;
    p.rows = rows;
    p.heads = a.heads; p.kv_heads = a.kv_heads; p.dim = a.dim; p.vdim = a.vdim;
    p.k_stride = padded(a.dim, 8); p.v_stride = padded(a.vdim, 8);
    p.ring = ring_of(d, a);
    p.chunk = chunk_of(d, a);
    p.rot_dims = a.rot_dims;
    p.k_column = w.k.at; p.v_column = w.v.at;
    p.scale = static_cast<float>(a.scale);
    p.options = d.path & 4 ? QM_ATTENTION_ROWS : 0;
    p.part.ml = f32_of(d.ml);
    p.part.acc = f32_of(d.acc);
    p.part.heads = a.heads; p.part.vdim = a.vdim;
    // (many rows fill the chip by themselves: their keys stay whole)
    p.part.keys_per_split = rows < 16 ? keys_per_split(p.chunk) : p.chunk;
    p.part.splits = rows < 16 ? key_splits(p.chunk) : 1;
    return p;
}

qm_decay_attention decay_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows, int position) {
    const DecayAttentionConfig& c = w.config.decay;
    const RetentionConfig& retention = w.config.retention;
    const bool rotary = w.config.mixer == MixerKind::Retention;
    qm_decay_attention p = {};
    p.proj = f32_of(d.proj);
    p.powers = f32_of(w.powers);
    p.state = reinterpret_cast<float*>(at_of(d.memory[static_cast<size_t>(sequence)], s.decay));
    p.out = f32_of(d.raw);
    p.ld_proj = w.in.n;
    if (!(d.path & 4)) {
        p.scratch = f32_of(d.scratch);
        p.scratch_floats = static_cast<int64_t>(d.scratch.bytes() / 4);
    }
    p.rows = rows;
    p.heads = rotary ? retention.heads : c.heads;
    p.dim = rotary ? retention.dim : c.dim;
    p.vdim = rotary ? retention.vdim : c.vdim;
    p.q_column = w.dq.at; p.k_column = w.dk.at; p.v_column = w.dv.at;
    if (rotary) {
        p.options = QM_DECAY_ROTARY;
        p.frequency = static_cast<const double*>(w.frequency.raw());
        p.rot_dims = retention.rot_dims;
        p.position = position;
        p.k_scale = static_cast<float>(1.0 / std::sqrt(static_cast<double>(retention.dim)));
    }
    return p;
}

qm_latent_rows latent_rows_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows, int position) {
    const LatentAttentionConfig& c = w.config.latent;
    const DeviceBuffer& memory = d.memory[static_cast<size_t>(sequence)];
    qm_latent_rows p = {};
    p.proj = f32_of(d.proj);
    p.q_norm = f32_of(w.q_norm); p.kv_norm = f32_of(w.kv_norm);
    p.frequency = static_cast<const double*>(w.frequency.raw());
    p.q_latent = d.q_latent.raw();
    if (c.kv_from < 0) {
        p.latent_cache = at_of(memory, s.latent);
        p.key_cache = at_of(memory, s.key);
    }
    p.ld_proj = w.in.n; p.ld_q = w.q_up.k; p.ld_latent = w.up_latent.k;
    p.position = position; p.rows = rows;
    p.q_rank = c.q_rank; p.kv_rank = c.kv_rank; p.rot_dim = c.rot_dim;
    p.key_stride = padded(c.rot_dim, 8);
    p.q_column = w.q_latent.at; p.kv_column = w.kv_latent.at;
    p.eps = static_cast<float>(d.config.eps);
    p.magnitude = static_cast<float>(w.magnitude);
    return p;
}

qm_latent_attention latent_attention_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows, int position) {
    const LatentAttentionConfig& c = w.config.latent;
    const DeviceBuffer& memory = d.memory[static_cast<size_t>(sequence)];
    qm_latent_attention p = {};
    p.q = f32_of(d.queries);
    p.frequency = static_cast<const double*>(w.frequency.raw());
    p.up_k = w.up_latent.u16();
    p.up_v = w.up_latent.u16() + static_cast<size_t>(w.up_v.at) * w.up_latent.k;
    p.latent_cache = at_of(memory, s.latent);
    p.key_cache = at_of(memory, s.key);
    p.out = d.attended.raw();
    p.q_scratch = d.q_scratch.raw();
    p.ml = f32_of(d.ml); p.acc = f32_of(d.acc);
    if (!d.f32) {
        p.expanded = f32_of(d.expanded);
        p.expanded_bytes = static_cast<int64_t>(d.expanded.bytes());
    }
    p.ld_query = w.q_up.n; p.ld_latent = w.up_latent.k; p.ld_out = w.o_left.k;
    p.position = position; p.rows = rows;
    p.heads = c.heads; p.dim = c.dim; p.rot_dim = c.rot_dim; p.vdim = c.vdim; p.kv_rank = c.kv_rank;
    p.key_stride = padded(c.rot_dim, 8);
    p.splits = rows < qm::kAttentionMatrixRows ? latent_splits(d.capacity) : 1;
    p.up_rows = w.up_latent.n; p.up_v_row = w.up_v.at;
    p.options = d.path & 4 ? QM_ATTENTION_ROWS : 0;
    p.scale = static_cast<float>(c.scale);
    p.magnitude = static_cast<float>(w.magnitude);
    return p;
}

qm_experts experts_of(const qm_decoder& d, const DecoderLayer& w, int rows, float* y) {
    qm_experts p = {};
    p.x = d.h.raw();
    p.logits = f32_of(d.expert_logits);
    p.gate = w.gate.u16(); p.up = w.up.u16(); p.down = w.down.u16();
    p.out32 = y;
    p.scratch = d.expert_scratch.raw();
    p.ld_logits = w.router.n;
    p.scratch_bytes = static_cast<int64_t>(d.expert_scratch.bytes());
    p.rows = rows; p.experts = w.config.experts; p.top = w.config.top; p.width_p = w.gate.k; p.ff_p = w.gate.n;
    p.options = d.path & 4 ? QM_EXPERTS_ROWS : 0;
    return p;
}

qm_general_delta delta_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows) {
    const GeneralDeltaConfig& c = w.config.delta;
    qm_general_delta p = {};
    p.proj = f32_of(d.proj);
    p.w2 = f32_of(w.w2); p.w0 = f32_of(w.w0); p.a_bias = f32_of(w.a_bias);
    p.state = reinterpret_cast<float*>(at_of(d.memory[static_cast<size_t>(sequence)], s.delta));
    p.out = f32_of(d.raw);
    p.ld_proj = w.in.n;
    if (!(d.path & 4)) {
        p.scratch = f32_of(d.scratch);
        p.scratch_floats = static_cast<int64_t>(d.scratch.bytes() / 4);
    }
    p.rows = rows; p.heads = c.heads; p.dim = c.dim; p.rank = w.rank;
    p.r_column = w.r.at; p.k_column = w.kk.at; p.v_column = w.vv.at; p.a_column = w.a.at; p.z_column = w.z.at;
    p.unit_eps = kUnitEps;
    return p;
}

qm_gated_norm gated_of(const qm_decoder& d, const DecoderLayer& w) {
    qm_gated_norm p = {};
    p.o = f32_of(d.raw);
    p.weight = f32_of(w.mix_norm);
    p.out = d.gated.raw();
    int gate = w.dg.at;
    switch (w.config.mixer) {
        case MixerKind::GeneralDelta:                 // a norm per head
            gate = w.g.at;
            p.groups = w.config.delta.heads;
            p.size = w.config.delta.dim;
            break;
        case MixerKind::Retention:                    // the same, without a weight
            p.groups = w.config.retention.heads;
            p.size = w.config.retention.vdim;
            p.silu = 1;
            break;
        default:                                      // one over all heads
            p.groups = 1;
            p.size = w.config.decay.heads * w.config.decay.vdim;
    }
    p.gate = f32_of(d.proj) + gate;
    p.ld_o = static_cast<int64_t>(p.groups) * p.size;
    p.ld_gate = w.in.n;
    p.ld_out = w.o_right.k;
    p.eps = static_cast<float>(d.config.eps);
    return p;
}

qm_decoder_linear linear_of(const Matrix& m, const void* x, float* out) {
    qm_decoder_linear l = {};
    l.x = x; l.w = m.u16(); l.out32 = out;
    l.ldx = m.k; l.ldo = m.n; l.n = m.n; l.k = m.k;
    return l;
}
qm_decoder_linear gate_up_of(const DecoderLayer& w, const void* x, void* out) {
    qm_decoder_linear l = {};
    l.x = x; l.w = w.gate.u16(); l.w_up = w.up.u16(); l.out = out;
    l.ldx = w.gate.k; l.ldo = w.gate.n; l.n = w.gate.n; l.k = w.gate.k;
    return l;
}

bool sandwich(const DecoderLayer& w) { return w.config.form == LayerForm::Sandwich; }

// The linears that read a layer's norm, and those that leave its sublayers' outputs in y[0 ..]; the terms they become.
qm::DecLinearParams linears_in(const qm_decoder& d, const DecoderLayer& w, int rows) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    p.group[p.groups++] = linear_of(w.in, d.h.raw(), f32_of(d.proj));
    if (w.config.ff && !sandwich(w)) p.group[p.groups++] = gate_up_of(w, d.h.raw(), d.mlp.raw());
    return p;
}
void add_term(const qm_decoder& d, Pending& pending, const float* y, const float* norm, float scale) {
    qm_residual_term& t = pending.term[pending.count++];
    t.y = y; t.norm_w = norm; t.ld = d.width_p; t.scale = scale;
}
qm::DecLinearParams linears_out(const qm_decoder& d, const DecoderLayer& w, int rows, Pending& pending) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    pending = Pending();
    auto add = [&](const Matrix& m, const void* x, const float* norm, float scale) {
        float* y = f32_of(d.y[p.groups]);
        p.group[p.groups++] = linear_of(m, x, y);
        add_term(d, pending, y, norm, scale);
    };
    const float mult = static_cast<float>(d.config.residual_mult);
    switch (w.config.mixer) {
        case MixerKind::AttentionBesideDecay:
            add(w.o_left, d.attended.raw(), f32_of(w.out_left), 0.5f);
            add(w.o_right, d.gated.raw(), f32_of(w.out_right), 0.5f);
            break;
        case MixerKind::GeneralDelta: add(w.o_right, d.gated.raw(), nullptr, 1.0f); break;
        case MixerKind::Retention: add(w.o_right, d.gated.raw(), f32_of(w.after_mixer), mult); break;
        case MixerKind::LatentAttention: add(w.o_left, d.attended.raw(), f32_of(w.after_mixer), mult); break;
    }
    if (w.config.ff && !sandwich(w)) add(w.down, d.mlp.raw(), nullptr, 1.0f);
    return p;
}

// A sandwich layer's feed-forward: what reads norm2, and (dense) the linear behind it.
qm::DecLinearParams feed_in(const qm_decoder& d, const DecoderLayer& w, int rows) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    p.group[p.groups++] = w.config.experts ? linear_of(w.router, d.h.raw(), f32_of(d.expert_logits)) : gate_up_of(w, d.h.raw(), d.mlp.raw());
    return p;
}
qm::DecLinearParams feed_out(const qm_decoder& d, const DecoderLayer& w, int rows) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    p.group[p.groups++] = linear_of(w.down, d.mlp.raw(), f32_of(d.y[0]));
    return p;
}
Pending feed_term(const qm_decoder& d, const DecoderLayer& w) {
    Pending pending;
    add_term(d, pending, f32_of(d.y[0]), f32_of(w.after_ff), static_cast<float>(d.config.residual_mult));
    return pending;
}

// Every layer run over `rows` tokens of d.tokens at `position`; leaves the stream and what is pending for the head.
void run_layers(qm_decoder& d, int sequence, int rows, int position, const float** stream_out, Pending& pending, float* taps) {
    hipStream_t s = d.stream;
    const float* x = nullptr;
    int next = 0;
    pending = Pending();
    for (size_t i = 0; i < d.runs.size(); ++i) {
        const LayerRun& run = d.runs[i];
        const DecoderLayer& w = d.layers[static_cast<size_t>(run.layer)];
        float* x_new = f32_of(d.x[next]);
        op_check(qm::launch_residual_norm(residual_of(d, pending, x, x_new, step_vec_of(d, run), f32_of(w.norm1), d.h.raw()), rows, d.f32, s),
                 "residual + norm");
        x = x_new;
        next ^= 1;
        op_check(qm::launch_decoder_linears(linears_in(d, w, rows), d.f32, s), "input projections");
        if (w.config.mixer == MixerKind::AttentionBesideDecay) {
            op_check(qm::launch_chunk_attention(attention_of(d, w, d.states[i], sequence, rows, position), d.f32, s), "chunked attention");
            op_check(qm::launch_decay_attention(decay_of(d, w, d.states[i], sequence, rows, position), s), "decayed linear attention");
        } else if (w.config.mixer == MixerKind::Retention) {
            op_check(qm::launch_decay_attention(decay_of(d, w, d.states[i], sequence, rows, position), s), "retention");
        } else if (w.config.mixer == MixerKind::LatentAttention) {
            op_check(qm::launch_latent_rows(latent_rows_of(d, w, d.states[i], sequence, rows, position), d.f32, s), "latents");
            qm::DecLinearParams up = {};
            up.rows = rows;
            up.group[up.groups++] = linear_of(w.q_up, d.q_latent.raw(), f32_of(d.queries));
            op_check(qm::launch_decoder_linears(up, d.f32, s), "queries");
            op_check(qm::launch_latent_attention(latent_attention_of(d, w, d.states[i], sequence, rows, position), nullptr, d.f32, s),
                     "attention over latents");
        } else {
            op_check(qm::launch_general_delta(delta_of(d, w, d.states[i], sequence, rows), s), "generalized delta rule");
        }
        if (w.config.mixer != MixerKind::LatentAttention) op_check(qm::launch_gated_norm(gated_of(d, w), rows, d.f32, s), "gated norm");
        op_check(qm::launch_decoder_linears(linears_out(d, w, rows, pending), d.f32, s), "output projections");
        if (sandwich(w) && w.config.ff) {
            x_new = f32_of(d.x[next]);
            op_check(qm::launch_residual_norm(residual_of(d, pending, x, x_new, nullptr, f32_of(w.norm2), d.h.raw()), rows, d.f32, s), "residual + norm");
            x = x_new;
            next ^= 1;
            op_check(qm::launch_decoder_linears(feed_in(d, w, rows), d.f32, s), "feed-forward");
            if (w.config.experts) op_check(qm::launch_experts(experts_of(d, w, rows, f32_of(d.y[0])), d.f32, s), "experts");
            else op_check(qm::launch_decoder_linears(feed_out(d, w, rows), d.f32, s), "feed-forward");
            pending = feed_term(d, w);
        }
        if (taps) {
            // the stream behind this run, before anything is added ahead of the next one
            op_check(qm::launch_residual_norm(residual_of(d, pending, x, f32_of(d.tap), nullptr, f32_of(d.final_norm), d.tap_h.raw()), rows, d.f32, s),
                     "stream");
            const size_t row_bytes = static_cast<size_t>(d.config.width) * 4;
            hip_check(hipMemcpy2DAsync(taps + i * rows * d.config.width, row_bytes, d.tap.raw(), static_cast<size_t>(d.width_p) * 4, row_bytes,
                                       static_cast<size_t>(rows), hipMemcpyDeviceToHost, s), "stream read");
            hip_check(hipStreamSynchronize(s), "stream read");
        }
    }
    *stream_out = x;
}

// Logits of the rows that `places` (host) names, as rows of `out` (host).
void run_head(qm_decoder& d, const float* x, const Pending& pending, const int32_t* places, int count, float* out) {
    hipStream_t s = d.stream;
    for (int first = 0; first < count; first += kLogitRows) {
        const int rows = std::min(kLogitRows, count - first);
        hip_check(hipMemcpyAsync(d.wanted.raw(), places + first, static_cast<size_t>(rows) * 4, hipMemcpyHostToDevice, s), "wanted rows");
        qm_residual_norm p = residual_of(d, pending, x, nullptr, nullptr, f32_of(d.final_norm), d.head_h.raw());
        p.row_map = static_cast<const int32_t*>(d.wanted.raw());
        op_check(qm::launch_residual_norm(p, rows, d.f32, s), "final norm");
        qm::DecLinearParams l = {};
        l.rows = rows;
        l.group[l.groups++] = linear_of(d.head, d.head_h.raw(), f32_of(d.logits));
        op_check(qm::launch_decoder_linears(l, d.f32, s), "head");
        const size_t vocab_bytes = static_cast<size_t>(d.config.vocab) * 4;
        if (out)
            hip_check(hipMemcpy2DAsync(out + static_cast<size_t>(first) * d.config.vocab, vocab_bytes, d.logits.raw(),
                                       static_cast<size_t>(d.vocab_p) * 4, vocab_bytes, static_cast<size_t>(rows), hipMemcpyDeviceToHost, s),
                      "logits read");
        hip_check(hipStreamSynchronize(s), "logits read");
    }
}

// ---- one token -----------------------------------------------------------------------------------------------------------

int32_t* step_words(const qm_decoder& d) { return static_cast<int32_t*>(d.step_words.raw()); }

// The token and position that the step words name, through every layer run and the head: logits in row 0 of d.logits.
void enqueue_one(qm_decoder& d, int sequence) {
    hipStream_t s = d.stream;
    const float* x = nullptr;
    int next = 0;
    Pending pending;
    auto residual = [&](float* x_new, const float* step_vec, const float* norm) {
        qm_residual_norm p = residual_of(d, pending, x, x_new, step_vec, norm, nullptr);
        p.tokens = step_words(d) + qm::kStepToken;
        return p;
    };
    for (size_t i = 0; i < d.runs.size(); ++i) {
        const LayerRun& run = d.runs[i];
        const DecoderLayer& w = d.layers[static_cast<size_t>(run.layer)];
        float* x_new = f32_of(d.x[next]);
        qm::LayerInParams in = {};
        in.residual = residual(x_new, step_vec_of(d, run), f32_of(w.norm1));
        in.linears = linears_in(d, w, 1);
        op_check(qm::launch_layer_in(in, d.f32, s), "residual + norm + input projections");
        x = x_new;
        next ^= 1;
        qm::LayerOutParams out = {};
        out.position_dev = step_words(d);
        switch (w.config.mixer) {
            case MixerKind::AttentionBesideDecay: {
                qm_chunk_attention a = attention_of(d, w, d.states[i], sequence, 1, 0);
                a.position_dev = step_words(d);
                op_check(qm::launch_mixer_step(a, decay_of(d, w, d.states[i], sequence, 1, 0), d.f32, s), "attention beside decayed attention");
                out.part = a.part;
                out.chunk = a.chunk;
                out.input[0] = 1;
                out.input[1] = 2;
                break;
            }
            case MixerKind::GeneralDelta:
                op_check(qm::launch_general_delta(delta_of(d, w, d.states[i], sequence, 1), s), "generalized delta rule");
                out.input[0] = 2;
                break;
            case MixerKind::Retention: {
                qm_decay_attention r = decay_of(d, w, d.states[i], sequence, 1, 0);
                r.position_dev = step_words(d);
                op_check(qm::launch_decay_attention(r, s), "retention");
                out.input[0] = 2;
                break;
            }
            case MixerKind::LatentAttention: {
                qm_latent_rows rows = latent_rows_of(d, w, d.states[i], sequence, 1, 0);
                qm_latent_attention a = latent_attention_of(d, w, d.states[i], sequence, 1, 0);
                rows.position_dev = a.position_dev = step_words(d);
                qm::LayerOutParams up = {};
                up.linears.rows = 1;
                up.linears.group[up.linears.groups++] = linear_of(w.q_up, nullptr, f32_of(d.queries));
                up.input[0] = 3;
                up.slice = {rows.proj + rows.q_column, rows.q_norm, rows.q_rank, rows.eps};
                op_check(qm::launch_layer_out(up, d.f32, s), "queries");
                rows.q_latent = nullptr;
                op_check(qm::launch_latent_attention(a, rows.latent_cache ? &rows : nullptr, d.f32, s), "attention over latents");
                break;
            }
        }
        out.linears = linears_out(d, w, 1, pending);
        if (w.config.mixer != MixerKind::LatentAttention) out.gated = gated_of(d, w);
        op_check(qm::launch_layer_out(out, d.f32, s), "output projections");
        if (sandwich(w) && w.config.ff) {
            x_new = f32_of(d.x[next]);
            qm::LayerInParams feed = {};
            feed.residual = residual(x_new, nullptr, f32_of(w.norm2));
            if (w.config.experts) feed.residual.h = d.h.raw();
            feed.linears = feed_in(d, w, 1);
            op_check(qm::launch_layer_in(feed, d.f32, s), "residual + norm + feed-forward");
            x = x_new;
            next ^= 1;
            if (w.config.experts) {
                op_check(qm::launch_experts(experts_of(d, w, 1, f32_of(d.y[0])), d.f32, s), "experts");
            } else {
                qm::LayerOutParams down = {};
                down.linears = feed_out(d, w, 1);
                op_check(qm::launch_layer_out(down, d.f32, s), "feed-forward");
            }
            pending = feed_term(d, w);
        }
    }
    qm::LayerInParams head = {};
    head.residual = residual(nullptr, nullptr, f32_of(d.final_norm));
    head.linears.rows = 1;
    head.linears.group[head.linears.groups++] = linear_of(d.head, nullptr, f32_of(d.logits));
    op_check(qm::launch_layer_in(head, d.f32, s), "final norm + head");
}

// The same by the operators of the prompt pass.
void enqueue_one_by_operators(qm_decoder& d, int sequence, int position) {
    hip_check(hipMemcpyAsync(d.tokens.raw(), step_words(d) + qm::kStepBefore, 8, hipMemcpyDeviceToDevice, d.stream), "token");
    const float* x = nullptr;
    Pending pending;
    run_layers(d, sequence, 1, position, &x, pending, nullptr);
    op_check(qm::launch_residual_norm(residual_of(d, pending, x, nullptr, nullptr, f32_of(d.final_norm), d.head_h.raw()), 1, d.f32, d.stream), "final norm");
    qm::DecLinearParams l = {};
    l.rows = 1;
    l.group[l.groups++] = linear_of(d.head, d.head_h.raw(), f32_of(d.logits));
    op_check(qm::launch_decoder_linears(l, d.f32, d.stream), "head");
}

// One token of the sequence, whose words are in place; logits in row 0 of d.logits.
void run_one(qm_decoder& d, int sequence) {
    int& length = d.length[static_cast<size_t>(sequence)];
    if (length >= d.capacity) throw ApiError(QM_ERR_SLOT_RANGE, "the sequence exceeds its capacity");
    hipGraphExec_t& graph = d.graphs[static_cast<size_t>(sequence)];
    if ((d.path & 3) == 2) {
        enqueue_one_by_operators(d, sequence, length);
    } else if ((d.path & 3) == 1 || !d.warm) {
        enqueue_one(d, sequence);          // (the first of all sets the kernels' attributes, outside of any capture)
        d.warm = true;
    } else {
        if (!graph) {
            hipGraph_t captured = nullptr;
            hip_check(hipStreamBeginCapture(d.stream, hipStreamCaptureModeThreadLocal), "step capture");
            try {
                enqueue_one(d, sequence);
            } catch (...) {
                (void)hipStreamEndCapture(d.stream, &captured);
                if (captured) (void)hipGraphDestroy(captured);
                throw;
            }
            hip_check(hipStreamEndCapture(d.stream, &captured), "step capture");
            const hipError_t e = hipGraphInstantiate(&graph, captured, nullptr, nullptr, 0);
            (void)hipGraphDestroy(captured);
            hip_check(e, "step graph");
        }
        hip_check(hipGraphLaunch(graph, d.stream), "step graph launch");
    }
    ++length;
}

void put_step_words(qm_decoder& d, int position, int before, int token) {
    const int32_t words[kStepWords] = {position, before, token, 0, 0};
    hip_check(hipMemcpyAsync(d.step_words.raw(), words, sizeof words, hipMemcpyHostToDevice, d.stream), "step words");
}

void check_tokens(const qm_decoder& d, const int32_t* tokens, int count) {
    if (!tokens) throw ApiError(QM_ERR_NULL, "no tokens");
    for (int i = 0; i < count; ++i)
        if (tokens[i] < 0 || tokens[i] >= d.config.vocab) throw ApiError(QM_ERR_ARGUMENT, "a token is outside the vocabulary");
}

int& length_of(qm_decoder& d, int sequence) {
    if (sequence < 0 || sequence >= static_cast<int>(d.length.size()) || d.length[static_cast<size_t>(sequence)] < 0)
        throw ApiError(QM_ERR_ARGUMENT, "not a live sequence");
    return d.length[static_cast<size_t>(sequence)];
}

void step(qm_decoder& d, int sequence, const int32_t* tokens, int count, const int32_t* want, int wanted, float* logits, float* streams,
          bool read_back = true) {
    int& length = length_of(d, sequence);
    int32_t& before = d.before[static_cast<size_t>(sequence)];
    if (count <= 0) throw ApiError(QM_ERR_ARGUMENT, "a step has at least one token");
    check_tokens(d, tokens, count);
    if (count > d.capacity - length) throw ApiError(QM_ERR_SLOT_RANGE, "the sequence exceeds its capacity");
    if (wanted < 0 || (wanted > 0 && (!want || !logits))) throw ApiError(QM_ERR_NULL, "no room for the logits");
    for (int i = 0; i < wanted; ++i)
        if (want[i] < 0 || want[i] >= count) throw ApiError(QM_ERR_ARGUMENT, "a wanted place is outside the step");
    if (streams && count > d.max_rows) throw ApiError(QM_ERR_ARGUMENT, "streams of one pass only");
    if (streams && !d.tap.raw()) {
        d.tap = DeviceBuffer(static_cast<size_t>(d.max_rows) * d.width_p * 4);
        d.tap_h = DeviceBuffer(static_cast<size_t>(d.max_rows) * d.width_p * 4);
    }
    if (count == 1 && !streams) {
        put_step_words(d, length, before, tokens[0]);
        run_one(d, sequence);
        before = tokens[0];
        for (int i = 0; i < wanted; ++i)
            hip_check(hipMemcpyAsync(logits + static_cast<size_t>(i) * d.config.vocab, d.logits.raw(), static_cast<size_t>(d.config.vocab) * 4,
                                     hipMemcpyDeviceToHost, d.stream), "logits read");
        if (read_back) hip_check(hipStreamSynchronize(d.stream), "step");
        return;
    }
    for (int first = 0; first < count; first += d.max_rows) {
        const int rows = std::min(d.max_rows, count - first);
        std::vector<int32_t> places;
        std::vector<int> order;
        for (int i = 0; i < wanted; ++i)
            if (want[i] >= first && want[i] < first + rows) {
                places.push_back(want[i] - first);
                order.push_back(i);
            }
        std::vector<int32_t> fed(static_cast<size_t>(rows) + 1, before);
        std::copy(tokens + first, tokens + first + rows, fed.begin() + 1);
        hip_check(hipMemcpyAsync(d.tokens.raw(), fed.data(), fed.size() * 4, hipMemcpyHostToDevice, d.stream), "token upload");
        const float* x = nullptr;
        Pending pending;
        run_layers(d, sequence, rows, length, &x, pending, streams);
        length += rows;
        before = tokens[first + rows - 1];
        if (!places.empty()) {
            std::vector<float> some(places.size() * static_cast<size_t>(d.config.vocab));
            run_head(d, x, pending, places.data(), static_cast<int>(places.size()), some.data());
            for (size_t i = 0; i < order.size(); ++i)
                std::memcpy(logits + static_cast<size_t>(order[i]) * d.config.vocab, some.data() + i * d.config.vocab,
                            static_cast<size_t>(d.config.vocab) * 4);
        }
    }
    if (read_back) hip_check(hipStreamSynchronize(d.stream), "step");
}

// The prompt, then token by token: the head's scores, the token they give into the step words, the step that reads it.
int generate(qm_decoder& d, int sequence, const int32_t* prompt, int count, int maximum, int stop_token, int top_k, float temperature, uint64_t seed,
             int32_t* out) {
    int& length = length_of(d, sequence);
    if (maximum <= 0 || !out) throw ApiError(QM_ERR_ARGUMENT, "no room for the tokens");
    if (count <= 0) throw ApiError(QM_ERR_ARGUMENT, "a prompt has at least one token");
    if (top_k > 0 && (d.config.vocab > 4096 || top_k > 256 || !(temperature > 0.0f)))
        throw ApiError(QM_ERR_GEOMETRY, "the sampler takes a vocabulary of at most 4096, top_k <= 256 and a positive temperature");
    // (the last token emitted is not fed back)
    if (static_cast<int64_t>(length) + count + maximum - 1 > d.capacity) throw ApiError(QM_ERR_SLOT_RANGE, "prompt and tokens exceed the capacity");
    std::vector<float> last(static_cast<size_t>(d.config.vocab));
    const int32_t want = count - 1;
    step(d, sequence, prompt, count, &want, 1, last.data(), nullptr);    // leaves the scores in row 0 of d.logits
    DeviceBuffer emitted(static_cast<size_t>(maximum) * 4), generator(8);
    hip_check(hipMemcpyAsync(generator.raw(), &seed, 8, hipMemcpyHostToDevice, d.stream), "generator state");
    int32_t& before = d.before[static_cast<size_t>(sequence)];
    put_step_words(d, length, 0, before);
    StreamDrain drain(d.stream);          // (the two buffers outlive what reads them, also on an error)
    int produced = 0;
    for (;;) {
        if (top_k > 0)
            op_check(qm_sample_topk(d.logits.raw(), 0, 0, d.config.vocab, top_k, temperature, static_cast<uint64_t*>(generator.raw()),
                                    step_words(d) + qm::kStepChosen, d.stream), "sampler");
        else
            op_check(qm::launch_argmax(f32_of(d.logits), d.config.vocab, step_words(d) + qm::kStepChosen, d.stream), "arg-max");
        op_check(qm::launch_emit(step_words(d), static_cast<int32_t*>(emitted.raw()), produced > 0, d.stream), "emit");
        ++produced;
        if (stop_token >= 0) {
            int32_t token = 0;
            hip_check(hipMemcpyAsync(&token, step_words(d) + qm::kStepToken, 4, hipMemcpyDeviceToHost, d.stream), "token read");
            hip_check(hipStreamSynchronize(d.stream), "token read");
            if (token == stop_token) break;
        }
        if (produced == maximum) break;
        run_one(d, sequence);
    }
    hip_check(hipMemcpyAsync(out, emitted.raw(), static_cast<size_t>(produced) * 4, hipMemcpyDeviceToHost, d.stream), "tokens read");
    hip_check(hipStreamSynchronize(d.stream), "tokens read");
    if (produced > 1) before = out[produced - 2];             // (the last token emitted was not fed)
    return produced;
}

}  // namespace
}  // namespace qm_engine

using namespace qm_engine;

extern "C" const char* qm_decoder_last_error(void) { return last_error().c_str(); }

extern "C" const char* qm_decoder_architecture(int32_t index) {
    const auto& names = decoder_architectures();
    return index >= 0 && index < static_cast<int32_t>(names.size()) ? names[static_cast<size_t>(index)].c_str() : nullptr;
}

extern "C" int32_t qm_decoder_check_config(const char* path) {
    if (!path) return QM_ERR_NULL;
    return guarded([&] { read_decoder_config(path); });
}

extern "C" int32_t qm_decoder_create(const char* model_dir, int32_t f32, int32_t capacity, int32_t sequences, int32_t max_rows, void* hip_stream,
                                     qm_decoder** out) {
    if (!model_dir || !out) return QM_ERR_NULL;
    *out = nullptr;
    return guarded([&] { *out = create_decoder(model_dir, f32, capacity, sequences, max_rows, static_cast<hipStream_t>(hip_stream)).release(); });
}

extern "C" void qm_decoder_destroy(qm_decoder* decoder) {
    if (decoder) (void)hipStreamSynchronize(decoder->stream);
    delete decoder;
}

extern "C" int32_t qm_decoder_info(const qm_decoder* d, int64_t info[8]) {
    if (!d || !info) return QM_ERR_NULL;
    const int64_t values[8] = {d->config.vocab, d->config.width, static_cast<int64_t>(d->layers.size()), static_cast<int64_t>(d->runs.size()),
                               d->capacity, static_cast<int64_t>(d->memory.size()), d->max_rows, static_cast<int64_t>(d->sequence_bytes)};
    std::copy(values, values + 8, info);
    return QM_OK;
}

extern "C" int32_t qm_decoder_open(qm_decoder* d, int32_t* sequence) {
    if (!d || !sequence) return QM_ERR_NULL;
    return guarded([&] {
        const auto free = std::find(d->length.begin(), d->length.end(), -1);
        if (free == d->length.end()) throw ApiError(QM_ERR_SLOT_RANGE, "every sequence is in use");
        const size_t at = static_cast<size_t>(free - d->length.begin());
        hip_check(hipMemsetAsync(d->memory[at].raw(), 0, d->memory[at].bytes(), d->stream), "sequence reset");
        *free = 0;
        d->before[at] = -1;
        *sequence = static_cast<int32_t>(at);
    });
}

extern "C" int32_t qm_decoder_close(qm_decoder* d, int32_t sequence) {
    if (!d) return QM_ERR_NULL;
    return guarded([&] { length_of(*d, sequence) = -1; });
}

extern "C" int32_t qm_decoder_step(qm_decoder* d, int32_t sequence, const int32_t* tokens, int32_t count, const int32_t* want, int32_t wanted,
                                   float* logits, float* streams) {
    if (!d) return QM_ERR_NULL;
    return guarded([&] { step(*d, sequence, tokens, count, want, wanted, logits, streams); });
}

extern "C" int32_t qm_decoder_synchronize(qm_decoder* d) {
    if (!d) return QM_ERR_NULL;
    return guarded([&] { hip_check(hipStreamSynchronize(d->stream), "decoder synchronize"); });
}

extern "C" int32_t qm_decoder_set_path(qm_decoder* d, int32_t path) {
    if (!d) return QM_ERR_NULL;
    if (path < 0 || (path & 3) == 3 || path > 7) return QM_ERR_ARGUMENT;
    d->path = path;
    return QM_OK;
}

extern "C" int32_t qm_decoder_enqueue(qm_decoder* d, int32_t sequence, const int32_t* tokens, int32_t count) {
    if (!d) return QM_ERR_NULL;
    return guarded([&] { step(*d, sequence, tokens, count, nullptr, 0, nullptr, nullptr, false); });
}

extern "C" int32_t qm_decoder_generate(qm_decoder* d, int32_t sequence, const int32_t* prompt, int32_t count, int32_t maximum, int32_t stop_token,
                                       int32_t top_k, float temperature, uint64_t seed, int32_t* tokens_out, int32_t* produced) {
    if (!d || !produced) return QM_ERR_NULL;
    *produced = 0;
    return guarded([&] { *produced = generate(*d, sequence, prompt, count, maximum, stop_token, top_k, temperature, seed, tokens_out); });
}
