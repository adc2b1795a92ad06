// qm_decoder_config.cpp — see qm_decoder_config.hpp.
#include "qm_decoder_config.hpp"

#include <cmath>
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
std::string text(const Json& object, const char* key) {
    const Json& v = member(object, key);
    if (v.kind != Json::String) fail(std::string("'") + key + "' is not a string");
    return v.text;
}
bool absent(const Json& object, const char* key) {
    const Json* v = object.member(key);
    return !v || v->kind == Json::Null;
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
        c.rot_base = number(rot, "base");
        if (!(c.rot_base > 0.0)) fail("'rot.base' is not positive");
    }
    if (c.heads % c.kv_heads) fail("'heads' is not a multiple of 'kv_heads'");
    if (c.rot_dims % 2 || c.rot_dims > c.dim) fail("'rot.dims' does not fit the head");
    return c;
}

DecayAttentionConfig decay_attention(const Json& j) {
    DecayAttentionConfig c;
    c.heads = count(j, "heads");
    c.dim = count(j, "dim");
    c.vdim = count(j, "vdim");
    const Json& decay = member(j, "decay");
    if (decay.kind != Json::Array || static_cast<int>(decay.items.size()) != c.heads) fail("'decay' does not name one value per head");
    for (const Json& v : decay.items) {
        if (v.kind != Json::Number || !std::isfinite(v.number)) fail("a decay is not a number");
        c.decay.push_back(v.number);
    }
    return c;
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

struct Architecture {
    const char* name;
    DecoderConfig (*read)(const Json&);
};
constexpr Architecture kArchitectures[] = {
    {"Vabevik", read_vabevik},
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
