/*
 * tk_layer_spec.h — decoders described layer by layer (config.json): what a layer's mixer and feed-forward are, with every size and constant.
 * The registry maps config.json's "architecture" to the function that reads that design's keys into this description; the model and session
 * (tk_layered.h) know only the description.  Host only.
 */
#ifndef TK_LAYER_SPEC_H
#define TK_LAYER_SPEC_H

#include <stdint.h>

#include <string>
#include <vector>

/* softmax attention over a paged cache */
struct TkAttnSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    int rot_dims = 0;        /* leading dimensions of a head that rotate, "rotate half" pairs (i, i + rot_dims / 2) */
    double rot_base = 10000.0;
    float scale = 1.0f;
    int window = 0;          /* position i reads j with i - j < window (0: no window) ... */
    int keep_first = 0;      /* ... or j < keep_first */
    int chunk = 0;           /* positions [n chunk, (n + 1) chunk) of a sequence read one another only (0: no chunks) */
    float softcap = 0.0f;    /* scores become softcap * tanh(score / softcap) (0: left as they are) */
    int taps = 0;            /* short causal convolution on the channels of q, k and v, before the rotation (0: none) */
    bool bias = false;       /* q, k, v and o have biases */
    bool qk_norm = false;    /* per-head RMS norm of q and k before the rotation, weights shared by the heads */
};

/* gated delta rule: short causal convolutions, unit q and k, one decay per head and key channel, low-rank decay and output gates */
struct TkDeltaSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0;
    float unit_eps = 1e-6f;
};

/* retention: linear attention with one constant decay per head, rotated q and k, a per-head RMS norm and a SiLU gate on the output */
struct TkRetentionSpec {
    int heads = 0, dim = 0, vdim = 0;
    int rot_dims = 0;
    double rot_base = 10000.0;
    std::vector<double> decay; /* [heads], 0 .. 1 */
};

/* one token mixer of a layer; a layer's branches read the same input and their scaled results are added */
struct TkBranchSpec {
    enum Kind { ATTENTION, DELTA, RETENTION } kind = ATTENTION;
    float scale = 1.0f;
    std::string prefix; /* tensors are <prefix>q, <prefix>k, ... */
    TkAttnSpec attn;
    TkDeltaSpec delta;
    TkRetentionSpec retention;
};

struct TkMlpSpec {
    enum Kind { NONE, DENSE, MOE } kind = NONE;
    int ff = 0;                                    /* of the layer or of one expert */
    /* gate activation: silu(g) * u; CLAMPED: g = min(g, limit), u = clamp(u, -limit, limit), then g * sigmoid(slope * g) * (u + shift) */
    enum Act { SWIGLU, CLAMPED } act = SWIGLU;
    float limit = 0.0f, slope = 1.0f, shift = 0.0f;
    int experts = 0, top = 0, groups = 1, keep = 1; /* sigmoid router: the top experts of the best `keep` of `groups` groups, scores not renormalised */
    std::string prefix;
};

struct TkLayerSpec {
    std::vector<TkBranchSpec> branches;
    TkMlpSpec mlp;
    std::string norm1, norm2; /* tensors of the norms on the mixer's and the feed-forward's output */
    std::string pre1, pre2;   /* of the norms on their input ("": they read the stream itself) */
    int weights_of = -1;      /* the layer whose tensors this one uses, itself one with tensors of its own (-1: its own); cache and state are its own always */
};

struct TkLayeredConfig {
    std::string architecture;
    int width = 0, vocab = 0;
    float eps = 1e-5f;
    float embed_scale = 1.0f;
    enum Norm { RMS, LAYER } norm = RMS; /* LAYER: mean taken off, weight and bias (tensor <name>.b) */
    std::vector<TkLayerSpec> layers;
};

/* false with *err: not JSON, an unknown architecture, a missing key or a size this build has no kernel for */
bool tk_layered_parse(const std::string& config_json, TkLayeredConfig* out, std::string* err);
/* names of the registered architectures */
std::vector<std::string> tk_layered_architectures();

/* limits of the kernels (csrc/llm/tk_mixer_kernels.hip) */
#define TK_MAX_HEAD_DIM 256
#define TK_MAX_DELTA_DIM 256
#define TK_MAX_DELTA_VDIM 256
#define TK_MAX_RETENTION_DIM 256
#define TK_MAX_RETENTION_VDIM 256
#define TK_MAX_CONV_TAPS 16
#define TK_MAX_EXPERTS 256
#define TK_MAX_TOP 64

#endif
