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

enum class MixerKind { LatentAttention };
enum class MlpKind { Dense };              // W_down gelu_tanh(W_up h)
enum class NormKind { DynamicTanh };       // tanh(alpha x) w + b

struct MixerConfig {
    MixerKind kind = MixerKind::LatentAttention;
    uint32_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0;
    double rot_base = 10000.0;
    uint32_t rot_dims = 0;
    float scale = 1.0f;
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
    float eps = 1e-6f, logit_scale = 1.0f;
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
