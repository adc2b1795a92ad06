// qm_decoder_config.cpp — see qm_decoder_config.hpp.
#include "qm_decoder_config.hpp"

#include <algorithm>
#include <cmath>
#include <cstdint>
#include <fstream>
#include <iterator>

#include "qm_json.hpp"

namespace qm_engine {

namespace {

[[noreturn]] void fail(const std::string& what) { throw IoError("config.json: " + what); }

const Json& member(const Json& object, const char* key) {
    const Json* v = object.kind == Json::Object ? object.member(key) : nullptr;
    if (!v) fail(std::string("missing key '") + key + "'");
    return *v;
}
double number(const Json& object, const char* key) {
    const Json& v = member(object, key);
    if (v.kind != Json::Number || !std::isfinite(v.number)) fail(std::string("'") + key + "' is not a number");
    return v.number;
}
int count(const Json& object, const char* key, int least = 1) {
    const double v = number(object, key);
    if (v < least || v > 1.0e9 || v != std::floor(v)) fail(std::string("'") + key + "' is not a count");
    return static_cast<int>(v);
}
// a whole factor of which only the remainder matters
int factor(const Json& object, const char* key, int modulus) {
    const double v = number(object, key);
    if (v < 0.0 || v > 9007199254740992.0 || v != std::floor(v)) fail(std::string("'") + key + "' is not a whole number");
    return static_cast<int>(static_cast<int64_t>(v) % modulus);
}
std::string text(const Json& object, const char* key) {
    const Json& v = member(object, key);
    if (v.kind != Json::String) fail(std::string("'") + key + "' is not a string");
    return v.text;
}
bool absent(const Json& object, const char* key) {
    const Json* v = object.member(key);
    return !v || v->kind == Json::Null;
}

double rotary_base(const Json& rot) {
    const double base = number(rot, "base");
    if (!(base > 0.0)) fail("'rot.base' is not positive");
    return base;
}

ChunkAttentionConfig chunk_attention(const Json& j) {
    ChunkAttentionConfig c;
    c.heads = count(j, "heads");
    c.kv_heads = count(j, "kv_heads");
    c.dim = count(j, "dim");
    c.vdim = count(j, "vdim");
    c.scale = number(j, "scale");
    c.chunk = count(member(j, "mask"), "size");
    if (!absent(j, "rot")) {
        const Json& rot = member(j, "rot");
        c.rot_dims = count(rot, "dims", 0);
        c.rot_base = rotary_base(rot);
    }
    if (c.heads % c.kv_heads) fail("'heads' is not a multiple of 'kv_heads'");
    if (c.rot_dims % 2 || c.rot_dims > c.dim) fail("'rot.dims' does not fit the head");
    return c;
}

std::vector<double> decays(const Json& j, int heads) {
    const Json& decay = member(j, "decay");
    if (decay.kind != Json::Array || static_cast<int>(decay.items.size()) != heads) fail("'decay' does not name one value per head");
    std::vector<double> values;
    for (const Json& v : decay.items) {
        if (v.kind != Json::Number || !std::isfinite(v.number)) fail("a decay is not a number");
        values.push_back(v.number);
    }
    return values;
}

DecayAttentionConfig decay_attention(const Json& j) {
    DecayAttentionConfig c;
    c.heads = count(j, "heads");
    c.dim = count(j, "dim");
    c.vdim = count(j, "vdim");
    c.decay = decays(j, c.heads);
    return c;
}

RetentionConfig retention(const Json& j) {
    RetentionConfig c;
    c.heads = count(j, "heads");
    c.dim = count(j, "dim");
    c.vdim = count(j, "vdim");
    c.decay = decays(j, c.heads);
    if (!absent(j, "rot")) {
        const Json& rot = member(j, "rot");
        c.rot_dims = count(rot, "dims", 0);
        c.rot_base = rotary_base(rot);
    }
    if (c.rot_dims % 2 || c.rot_dims > c.dim) fail("'rot.dims' does not fit the head");
    return c;
}

LatentAttentionConfig latent_attention(const Json& j) {
    LatentAttentionConfig c;
    c.heads = count(j, "heads");
    c.dim = count(j, "dim");
    c.rot_dim = count(j, "rot_dim");
    c.vdim = count(j, "vdim");
    c.q_rank = count(j, "q_rank");
    c.kv_rank = count(j, "kv_rank");
    c.scale = number(j, "scale");
    if (!absent(j, "kv_from")) c.kv_from = count(j, "kv_from", 0);
    const Json& rot = member(j, "rot");
    c.rot_base = rotary_base(rot);
    if (c.rot_dim % 2 || count(rot, "dims") != c.rot_dim) fail("'rot.dims' is not the rotated key part's size");
    if (!absent(rot, "scaling")) {
        const Json& scaling = member(rot, "scaling");
        c.scaling = {number(scaling, "factor"), number(scaling, "original"), number(scaling, "fast"), number(scaling, "slow")};
        if (!(c.scaling.factor > 0.0 && c.scaling.original > 0.0 && c.scaling.fast > 0.0 && c.scaling.slow > 0.0) || c.rot_base == 1.0)
            fail("'rot.scaling' is not a stretching of frequencies");
    }
    return c;
}

bool same_scaling(const RotaryScaling& a, const RotaryScaling& b) {
    return a.factor == b.factor && a.original == b.original && a.fast == b.fast && a.slow == b.slow;
}

// Vabevik: parallel layers (one norm, mixer and feed-forward side by side), each mixer either chunked attention beside
// decayed linear attention or the generalized delta rule, with a run of layers that is repeated.
DecoderConfig read_vabevik(const Json& j) {
    DecoderConfig c;
    c.vocab = count(j, "vocab");
    c.width = count(j, "width");
    c.eps = number(member(j, "norm"), "eps");
    const Json& layers = member(j, "layers");
    if (layers.kind != Json::Array || layers.items.empty()) fail("'layers' is not a list of layers");
    for (const Json& entry : layers.items) {
        DecoderLayerConfig layer;
        const std::string type = text(entry, "type");
        const Json& mixer = member(entry, "mixer");
        if (type == "parallel") {
            layer.mixer = MixerKind::AttentionBesideDecay;
            layer.attention = chunk_attention(member(mixer, "left"));
            layer.decay = decay_attention(member(mixer, "right"));
        } else if (type == "general_delta") {
            layer.mixer = MixerKind::GeneralDelta;
            layer.delta.heads = count(mixer, "heads");
            layer.delta.dim = count(mixer, "dim");
        } else {
            fail("unknown mixer '" + type + "'");
        }
        if (!absent(entry, "mlp")) {
            const Json& mlp = member(entry, "mlp");
            if (text(mlp, "kind") != "dense") fail("unknown feed-forward '" + text(mlp, "kind") + "'");
            layer.ff = count(mlp, "ff");
        }
        c.layers.push_back(std::move(layer));
    }
    if (!absent(j, "loop")) {
        const Json& loop = member(j, "loop");
        c.loop_start = count(loop, "start", 0);
        c.loop_stop = count(loop, "stop", 0);
        c.loop_times = count(loop, "times", 0);
        if (c.loop_start >= c.loop_stop || c.loop_stop > static_cast<int>(c.layers.size()) || c.loop_times < 1) fail("'loop' does not name a run of layers");
    }
    return c;
}

// Tuzavik: mixer and feed-forward each between two norms; retention or latent attention (whose latent another layer may
// share), dense feed-forwards or mixtures of experts, a bigram embedding.
DecoderConfig read_tuzavik(const Json& j) {
    DecoderConfig c;
    c.vocab = count(j, "vocab");
    c.width = count(j, "width");
    c.eps = number(member(j, "norm"), "eps");
    c.norms_around_zero = true;
    c.residual_mult = number(j, "residual_mult");
    c.logit_scale = number(j, "logit_scale");
    const Json& bigram = member(member(j, "embedding"), "bigram");
    c.bigram_buckets = count(bigram, "buckets");
    c.bigram_mul_prev = factor(bigram, "mul_prev", c.bigram_buckets);
    c.bigram_mul_cur = factor(bigram, "mul_cur", c.bigram_buckets);
    const Json& layers = member(j, "layers");
    if (layers.kind != Json::Array || layers.items.empty()) fail("'layers' is not a list of layers");
    for (const Json& entry : layers.items) {
        DecoderLayerConfig layer;
        layer.form = LayerForm::Sandwich;
        const std::string type = text(entry, "type");
        const Json& mixer = member(entry, "mixer");
        if (type == "retention") {
            layer.mixer = MixerKind::Retention;
            layer.retention = retention(mixer);
        } else if (type == "latent_attention") {
            layer.mixer = MixerKind::LatentAttention;
            layer.latent = latent_attention(mixer);
            const LatentAttentionConfig& l = layer.latent;
            if (l.kv_from >= 0) {
                if (l.kv_from >= static_cast<int>(c.layers.size()) || c.layers[static_cast<size_t>(l.kv_from)].mixer != MixerKind::LatentAttention)
                    fail("'kv_from' does not name an earlier latent layer");
                const LatentAttentionConfig& from = c.layers[static_cast<size_t>(l.kv_from)].latent;
                if (from.kv_from >= 0 || from.kv_rank != l.kv_rank || from.rot_dim != l.rot_dim || from.rot_base != l.rot_base ||
                    !same_scaling(from.scaling, l.scaling))
                    fail("'kv_from' names a layer whose latent does not fit");
            }
        } else {
            fail("unknown mixer '" + type + "'");
        }
        if (!absent(entry, "mlp")) {
            const Json& mlp = member(entry, "mlp");
            const std::string kind = text(mlp, "kind");
            if (kind == "dense") {
                layer.ff = count(mlp, "ff");
            } else if (kind == "moe") {
                layer.ff = count(member(mlp, "expert"), "ff");
                layer.experts = count(member(mlp, "router"), "experts");
                layer.top = count(member(mlp, "router"), "top");
                if (layer.top > layer.experts) fail("'router.top' is more than there are experts");
            } else {
                fail("unknown feed-forward '" + kind + "'");
            }
        }
        c.layers.push_back(std::move(layer));
    }
    return c;
}

struct Architecture {
    const char* name;
    DecoderConfig (*read)(const Json&);
};
constexpr Architecture kArchitectures[] = {
    {"Vabevik", read_vabevik},
    {"Tuzavik", read_tuzavik},
};

}  // namespace

const std::vector<std::string>& decoder_architectures() {
    static const std::vector<std::string> names = [] {
        std::vector<std::string> n;
        for (const Architecture& a : kArchitectures) n.push_back(a.name);
        return n;
    }();
    return names;
}

DecoderConfig read_decoder_config(const std::string& path) {
    std::ifstream in(path, std::ios::binary);
    if (!in) throw IoError("open failed: " + path);
    const std::string bytes((std::istreambuf_iterator<char>(in)), std::istreambuf_iterator<char>());
    const Json root = JsonReader(bytes.data(), bytes.size(), "config.json").document();
    const std::string name = text(root, "architecture");
    for (const Architecture& a : kArchitectures) {
        if (name != a.name) continue;
        DecoderConfig c = a.read(root);
        c.architecture = name;
        return c;
    }
    fail("no model of the registry has the architecture '" + name + "'");
}

std::vector<double> rotary_frequencies(int dims, double base, const RotaryScaling& scaling, double* magnitude) {
    std::vector<double> f(static_cast<size_t>(dims / 2));
    for (int i = 0; i < dims / 2; ++i) f[static_cast<size_t>(i)] = std::pow(base, -2.0 * i / dims);
    if (magnitude) *magnitude = 1.0;
    if (scaling.factor == 0.0) return f;
    // the pair that turns t times over the original context; pairs up to `fast` turns stay, from `slow` turns on stretched
    auto pair_of = [&](double turns) { return dims * std::log(scaling.original / (2.0 * M_PI * turns)) / (2.0 * std::log(base)); };
    const double lo = std::max(std::floor(pair_of(scaling.fast)), 0.0), hi = std::min(std::ceil(pair_of(scaling.slow)), dims - 1.0);
    for (int i = 0; i < dims / 2; ++i) {
        const double ramp = std::clamp((i - lo) / std::max(hi - lo, 0.001), 0.0, 1.0);
        double& value = f[static_cast<size_t>(i)];
        value = value / scaling.factor * ramp + value * (1.0 - ramp);
    }
    if (magnitude) *magnitude = 0.1 * std::log(scaling.factor) + 1.0;
    return f;
}

std::vector<LayerRun> layer_runs(const DecoderConfig& c) {
    const int layers = static_cast<int>(c.layers.size());
    std::vector<LayerRun> runs;
    const int start = c.loop_times ? c.loop_start : layers;
    for (int i = 0; i < start; ++i) runs.push_back({i, -1});
    for (int t = 0; t < c.loop_times; ++t)
        for (int i = c.loop_start; i < c.loop_stop; ++i) runs.push_back({i, i == c.loop_start ? t : -1});
    for (int i = c.loop_times ? c.loop_stop : layers; i < layers; ++i) runs.push_back({i, -1});
    return runs;
}

}  // namespace qm_engine
