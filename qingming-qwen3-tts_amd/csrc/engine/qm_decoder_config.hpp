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
// rotary frequencies stretched for longer contexts (YaRN); factor 0: not stretched
struct RotaryScaling {
    double factor = 0.0, original = 0.0, fast = 0.0, slow = 0.0;
};
// linear attention with a per-head decay, q and k rotated, k scaled, a norm per head and an output gate
struct RetentionConfig {
    int heads = 0, dim = 0, vdim = 0, rot_dims = 0;
    double rot_base = 0.0;
    std::vector<double> decay;
};
// softmax attention over a latent per token that every head makes its key and value from, beside one rotated key part that
// all heads share; kv_from >= 0: latent and key part are those of that layer
struct LatentAttentionConfig {
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0, kv_from = -1;
    double rot_base = 0.0, scale = 0.0;
    RotaryScaling scaling;
};
enum class MixerKind { AttentionBesideDecay, GeneralDelta, Retention, LatentAttention };

// How a layer's norms, mixer and feed-forward are arranged.
//   Parallel  one norm; mixer and feed-forward both read its output and are added to the stream together
//   Sandwich  mixer, then feed-forward, each between two norms of its own, added to the stream times residual_mult
enum class LayerForm { Parallel, Sandwich };

struct DecoderLayerConfig {
    LayerForm form = LayerForm::Parallel;
    MixerKind mixer = MixerKind::GeneralDelta;
    ChunkAttentionConfig attention;
    DecayAttentionConfig decay;
    GeneralDeltaConfig delta;
    RetentionConfig retention;
    LatentAttentionConfig latent;
    int ff = 0;                      // of the feed-forward, or of each expert (0: no feed-forward)
    int experts = 0, top = 0;        // mixture of experts, weights sigmoid(router) of the chosen ones (0: one dense feed-forward)
};

struct DecoderConfig {
    std::string architecture;
    int vocab = 0, width = 0;
    double eps = 0.0;
    std::vector<DecoderLayerConfig> layers;
    bool norms_around_zero = false;  // norm weights are stored less one
    double residual_mult = 1.0, logit_scale = 1.0;
    // a second embedding, of the token and the one before it: row (before * mul_prev + token * mul_cur) mod buckets, row
    // `buckets` for a sequence's first token (0: none)
    int bigram_buckets = 0, bigram_mul_prev = 0, bigram_mul_cur = 0;
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
// The frequencies of rotary pairs 0 .. dims / 2 - 1, and what both cosine and sine are multiplied by.
std::vector<double> rotary_frequencies(int dims, double base, const RotaryScaling& scaling, double* magnitude);
// Reads and checks a config.json; throws IoError with the reason.
DecoderConfig read_decoder_config(const std::string& path);

}  // namespace qm_engine
