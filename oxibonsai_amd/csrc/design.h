// design.h — model designs described by a config.json: what a layer program consists of, and the registry that turns an
// "architecture" name into one (host only).
//
// A design is a list of layers (a mixer and an optional feed-forward each, with sizes of their own), an optional range of
// layers that runs several times, and a head.  Another design is one more entry in the registry that fills the same
// structures; another mixer, feed-forward or norm is one more kind in them.
#pragma once
#include <stdint.h>

#include <string>
#include <vector>

#include "json.h"

namespace oxb {

enum class MixerKind { LatentAttention, GroupedAttention, StateSpace, GatedDelta, Parallel };
enum class MlpKind { Dense, Gated };                // W_down gelu_tanh(W_up h); W_down (gelu_tanh(W_gate h) * (W_up h))
enum class NormKind { DynamicTanh, RmsAroundOne };  // tanh(alpha x) w + b; x / rms(x) (1 + w)
// Sequential: x += mixer(norm1 x), x += mlp(norm2 x).  Parallel: x += m (mixer(h) + mlp(h)), h = norm1 x.
enum class BlockKind { Sequential, Parallel };

// Rotation: pair i of dims / 2 turns by base^(-2 i / dims) per position.  factor != 0: turns longer than original / low
// positions are slowed by it, those shorter than original / high stay, the ones between are blended.
struct RopeConfig {
    double base = 10000.0;
    uint32_t dims = 0;
    double factor = 0, low = 0, high = 0, original = 0;
    bool operator==(const RopeConfig& o) const {
        return base == o.base && dims == o.dims && factor == o.factor && low == o.low && high == o.high && original == o.original;
    }
};
double rope_frequency(const RopeConfig& r, uint32_t i);

struct MixerConfig {
    MixerKind kind = MixerKind::LatentAttention;
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    RopeConfig rope;
    float scale = 1.0f;                                    // of attention scores
    uint32_t rot_dim = 0, kv_rank = 0;                     // latent attention
    uint32_t conv = 0;                                     // taps of the recurrent mixers' convolutions
    uint32_t state = 0, groups = 0, norm_groups = 0;       // state space
    std::vector<MixerConfig> parts;                        // Parallel: mixers that read the same input ..
    std::vector<float> part_scales;                        // .. and what their results are multiplied by
    std::vector<std::string> part_names;                   // .. and their tensors' prefixes
};
struct MlpConfig {
    MlpKind kind = MlpKind::Dense;
    uint32_t ff = 0;
};
struct LayerConfig {
    MixerConfig mixer;
    bool has_mlp = false;
    MlpConfig mlp;
};
struct LoopConfig {   // layers start .. stop - 1 run `times` times; 0: no loop
    uint32_t start = 0, stop = 0, times = 0;
};
struct DesignConfig {
    std::string architecture;
    NormKind norm = NormKind::DynamicTanh;
    BlockKind block = BlockKind::Sequential;
    float eps = 1e-6f, logit_scale = 1.0f, embed_scale = 1.0f, residual_mult = 1.0f;
    uint32_t vocab = 0, width = 0;
    std::vector<LayerConfig> layers;
    LoopConfig loop;
};

struct LayerRun {   // one entry per run of a layer, in order
    uint32_t layer;
    int pass;       // number of the pass through the loop, -1 outside
    bool first;     // first layer of a pass
};
std::vector<LayerRun> layer_runs(const DesignConfig& c);

struct Design {
    const char* architecture;
    bool (*read)(const Json& j, DesignConfig* c, std::string* err);
};
const std::vector<Design>& designs();

// config.json text -> configuration, through the registry entry its "architecture" names.
bool read_design(const std::string& text, DesignConfig* c, std::string* err);

}  // namespace oxb
