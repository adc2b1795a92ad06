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
//   mixer                   rotation + cache write + attention and decayed linear attention, or the delta rule; gated norm
//   linears                 the output projections and the feed-forward's down projection in one launch
// One token: three fused launches per layer run (qm_decoder_step_ops.h), replayed from a graph that reads token and
// position from device memory.
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
constexpr int kStepWords = 4;             // device words of a one-token step: position, token, tokens emitted

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
};

struct RunState {                                   // byte offsets inside a sequence's memory
    size_t k = 0, v = 0, decay = 0, delta = 0;
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
    size_t sequence_bytes = 0;
    qm_engine::DeviceBuffer final_norm, loop_step;
    qm_engine::Matrix embed, head;
    int capacity = 0, max_rows = 0, f32 = 0, path = 0;
    bool warm = false;
    int width_p = 0, vocab_p = 0;
    hipStream_t stream = nullptr;
    bool own_stream = false;
    qm_engine::DeviceBuffer x[2], h, proj, mlp, attended, gated, y[3], q_rot, raw, ml, acc, scratch, tokens, wanted, head_h, logits, tap, tap_h,
        step_words;
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
    Matrix stacked(const std::vector<Part>& parts, int k) const {
        Matrix m;
        int n = 0;
        for (const Part& p : parts) {
            if (p.section) *p.section = {n, p.columns};
            n += padded(p.columns, 8);
        }
        m.n = padded(n, 128);
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

private:
    ModelDirectory files_;
};

DecoderLayer load_layer(const Loader& from, const DecoderLayerConfig& config, int index, int width) {
    DecoderLayer w;
    w.config = config;
    const std::string base = "l" + std::to_string(index) + ".", mix = base + "mix.";
    w.norm1 = from.padded_floats(base + "norm1", {width}, padded(width, 128));
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
        std::vector<double> frequency(static_cast<size_t>(std::max(1, a.rot_dims / 2)), 0.0);
        for (int i = 0; i < a.rot_dims / 2; ++i) frequency[static_cast<size_t>(i)] = std::pow(a.rot_base, -2.0 * i / a.rot_dims);
        w.frequency = Loader::upload(frequency.data(), frequency.size() * sizeof(double));
        std::vector<float> powers;
        for (double decay : d.decay)
            for (int i = 0; i < QM_DECAY_POWERS; ++i) powers.push_back(static_cast<float>(i == 0 ? 1.0 : std::pow(decay, i)));
        w.powers = Loader::upload(powers.data(), powers.size() * sizeof(float));
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
    if (config.ff) {
        w.gate = from.matrix(base + "mlp.gate", config.ff, width);
        w.up = from.matrix(base + "mlp.up", config.ff, width);
        w.down = from.matrix(base + "mlp.down", width, config.ff);
    }
    return w;
}

int ring_of(const qm_decoder& d, const ChunkAttentionConfig& a) { return std::min<int64_t>(d.capacity, static_cast<int64_t>(a.chunk) + d.max_rows); }
int chunk_of(const qm_decoder& d, const ChunkAttentionConfig& a) { return std::min(a.chunk, d.capacity); }

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
    d->final_norm = from.padded_floats("final.norm", {width}, d->width_p);
    d->head = from.matrix("head", d->config.vocab, width);
    if (d->config.loop_times) d->loop_step = from.padded_floats("loop.step", {d->config.loop_times, width}, d->width_p);
    for (size_t i = 0; i < d->config.layers.size(); ++i)
        d->layers.push_back(load_layer(from, d->config.layers[i], static_cast<int>(i), width));

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
        } else {
            s.delta = take(static_cast<size_t>(c.delta.heads) * c.delta.dim * c.delta.dim * 4);
        }
        d->states.push_back(s);
    }
    d->sequence_bytes = at;
    for (int i = 0; i < sequences; ++i) {
        d->memory.emplace_back(at);
        d->length.push_back(-1);
    }
    d->graphs.assign(static_cast<size_t>(sequences), nullptr);

    // activations of a pass
    const size_t rows = static_cast<size_t>(d->max_rows);
    size_t proj = 0, mlp = 0, attended = 0, gated = 0, q_rot = 0, raw = 0, ml = 0, acc = 0, scratch = 0;
    for (const DecoderLayer& w : d->layers) {
        const DecoderLayerConfig& c = w.config;
        proj = std::max(proj, static_cast<size_t>(w.in.n));
        mlp = std::max(mlp, static_cast<size_t>(w.down.k));
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
    d->tokens = zeros(rows * 4);
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
    p.tokens = static_cast<const int32_t*>(d.tokens.raw());
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

qm_decay_attention decay_of(const qm_decoder& d, const DecoderLayer& w, const RunState& s, int sequence, int rows) {
    const DecayAttentionConfig& c = w.config.decay;
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
    p.rows = rows; p.heads = c.heads; p.dim = c.dim; p.vdim = c.vdim;
    p.q_column = w.dq.at; p.k_column = w.dk.at; p.v_column = w.dv.at;
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
    const bool delta = w.config.mixer == MixerKind::GeneralDelta;
    qm_gated_norm p = {};
    p.o = f32_of(d.raw);
    p.weight = f32_of(w.mix_norm);
    p.gate = f32_of(d.proj) + (delta ? w.g.at : w.dg.at);
    p.out = d.gated.raw();
    p.groups = delta ? w.config.delta.heads : 1;      // a norm per head, or one over all of them
    p.size = delta ? w.config.delta.dim : w.config.decay.heads * w.config.decay.vdim;
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

// The linears that read a layer's norm, and those that leave its sublayers' outputs in y[0 ..]; the terms they become.
qm::DecLinearParams linears_in(const qm_decoder& d, const DecoderLayer& w, int rows) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    p.group[p.groups++] = linear_of(w.in, d.h.raw(), f32_of(d.proj));
    if (w.config.ff) p.group[p.groups++] = gate_up_of(w, d.h.raw(), d.mlp.raw());
    return p;
}
qm::DecLinearParams linears_out(const qm_decoder& d, const DecoderLayer& w, int rows, Pending& pending) {
    qm::DecLinearParams p = {};
    p.rows = rows;
    pending = Pending();
    auto add = [&](const Matrix& m, const void* x, const float* norm, float scale) {
        float* y = f32_of(d.y[p.groups]);
        p.group[p.groups++] = linear_of(m, x, y);
        qm_residual_term& t = pending.term[pending.count++];
        t.y = y; t.norm_w = norm; t.ld = d.width_p; t.scale = scale;
    };
    if (w.config.mixer == MixerKind::AttentionBesideDecay) {
        add(w.o_left, d.attended.raw(), f32_of(w.out_left), 0.5f);
        add(w.o_right, d.gated.raw(), f32_of(w.out_right), 0.5f);
    } else {
        add(w.o_right, d.gated.raw(), nullptr, 1.0f);
    }
    if (w.config.ff) add(w.down, d.mlp.raw(), nullptr, 1.0f);
    return p;
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
            op_check(qm::launch_decay_attention(decay_of(d, w, d.states[i], sequence, rows), s), "decayed linear attention");
        } else {
            op_check(qm::launch_general_delta(delta_of(d, w, d.states[i], sequence, rows), s), "generalized delta rule");
        }
        op_check(qm::launch_gated_norm(gated_of(d, w), rows, d.f32, s), "gated norm");
        op_check(qm::launch_decoder_linears(linears_out(d, w, rows, pending), d.f32, s), "output projections");
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
        p.tokens = step_words(d) + 1;
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
        out.linears = linears_out(d, w, 1, pending);
        out.gated = gated_of(d, w);
        out.position_dev = step_words(d);
        if (w.config.mixer == MixerKind::AttentionBesideDecay) {
            qm_chunk_attention a = attention_of(d, w, d.states[i], sequence, 1, 0);
            a.position_dev = step_words(d);
            op_check(qm::launch_mixer_step(a, decay_of(d, w, d.states[i], sequence, 1), d.f32, s), "attention beside decayed attention");
            out.part = a.part;
            out.chunk = a.chunk;
            out.input[0] = 1;
            out.input[1] = 2;
        } else {
            op_check(qm::launch_general_delta(delta_of(d, w, d.states[i], sequence, 1), s), "generalized delta rule");
            out.input[0] = 2;
        }
        op_check(qm::launch_layer_out(out, d.f32, s), "output projections");
    }
    qm::LayerInParams head = {};
    head.residual = residual(nullptr, nullptr, f32_of(d.final_norm));
    head.linears.rows = 1;
    head.linears.group[head.linears.groups++] = linear_of(d.head, nullptr, f32_of(d.logits));
    op_check(qm::launch_layer_in(head, d.f32, s), "final norm + head");
}

// The same by the operators of the prompt pass.
void enqueue_one_by_operators(qm_decoder& d, int sequence, int position) {
    hip_check(hipMemcpyAsync(d.tokens.raw(), step_words(d) + 1, 4, hipMemcpyDeviceToDevice, d.stream), "token");
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

void put_step_words(qm_decoder& d, int position, int token) {
    const int32_t words[3] = {position, token, 0};
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
        put_step_words(d, length, tokens[0]);
        run_one(d, sequence);
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
        hip_check(hipMemcpyAsync(d.tokens.raw(), tokens + first, static_cast<size_t>(rows) * 4, hipMemcpyHostToDevice, d.stream), "token upload");
        const float* x = nullptr;
        Pending pending;
        run_layers(d, sequence, rows, length, &x, pending, streams);
        length += rows;
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
    put_step_words(d, length, 0);
    StreamDrain drain(d.stream);          // (the two buffers outlive what reads them, also on an error)
    int produced = 0;
    for (;;) {
        if (top_k > 0)
            op_check(qm_sample_topk(d.logits.raw(), 0, 0, d.config.vocab, top_k, temperature, static_cast<uint64_t*>(generator.raw()),
                                    step_words(d) + 1, d.stream), "sampler");
        else
            op_check(qm::launch_argmax(f32_of(d.logits), d.config.vocab, step_words(d), d.stream), "arg-max");
        op_check(qm::launch_emit(step_words(d), static_cast<int32_t*>(emitted.raw()), produced > 0, d.stream), "emit");
        ++produced;
        if (stop_token >= 0) {
            int32_t token = 0;
            hip_check(hipMemcpyAsync(&token, step_words(d) + 1, 4, hipMemcpyDeviceToHost, d.stream), "token read");
            hip_check(hipStreamSynchronize(d.stream), "token read");
            if (token == stop_token) break;
        }
        if (produced == maximum) break;
        run_one(d, sequence);
    }
    hip_check(hipMemcpyAsync(out, emitted.raw(), static_cast<size_t>(produced) * 4, hipMemcpyDeviceToHost, d.stream), "tokens read");
    hip_check(hipStreamSynchronize(d.stream), "tokens read");
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
