// qm_decoder_config.hpp — what a decoder language model consists of, read from its config.json, and the registry of
// architectures.  A configuration is a list of layers made of mechanisms with their sizes and constants; an architecture's
// reader fills it, the engine knows only the mechanisms.
#pragma once

#include <string>
#include <vector>

namespace qm_engine {

// softmax attention inside chunks of positions, grouped query heads, rotary positions on the first rot_dims channels
struct ChunkAttentionConfig {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, chunk = 0, rot_dims = 0;
    double rot_base = 0.0, scale = 0.0;
};
// linear attention with a per-head decay, a norm over all heads and an output gate
struct DecayAttentionConfig {
    int heads = 0, dim = 0, vdim = 0;
    std::vector<double> decay;
};
// generalized delta rule with data-dependent decays and removal rates, per-head norms and an output gate
struct GeneralDeltaConfig {
    int heads = 0, dim = 0;
};
enum class MixerKind { AttentionBesideDecay, GeneralDelta };

// One norm; the mixer and the feed-forward (ff = 0: none) both read its output and are added to the stream together.
struct DecoderLayerConfig {
    MixerKind mixer = MixerKind::GeneralDelta;
    ChunkAttentionConfig attention;
    DecayAttentionConfig decay;
    GeneralDeltaConfig delta;
    int ff = 0;
};

struct DecoderConfig {
    std::string architecture;
    int vocab = 0, width = 0;
    double eps = 0.0;
    std::vector<DecoderLayerConfig> layers;
    // layers loop_start .. loop_stop - 1 run loop_times times in a row, a vector added before each pass (0 times: no loop)
    int loop_start = 0, loop_stop = 0, loop_times = 0;
};

// One pass through a layer: which layer, and the pass of the loop it opens (-1: none).
struct LayerRun {
    int layer = 0, opens_pass = -1;
};
std::vector<LayerRun> layer_runs(const DecoderConfig& config);

// The names the registry knows, in order.
const std::vector<std::string>& decoder_architectures();
// Reads and checks a config.json; throws IoError with the reason.
DecoderConfig read_decoder_config(const std::string& path);

}  // namespace qm_engine
