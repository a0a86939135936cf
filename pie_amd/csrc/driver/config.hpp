// Driver configuration: the per-launch TOML the Pie server writes for a driver
// (`[model] [batching] [runtime]`, driver/portable/src/config.hpp:52-116,
// server/src/embedded_driver.rs:319-358), parsed by a small TOML subset reader
// (sections, `key = value` with string / integer / float / boolean values, comments).
// Unknown `[batching]` keys are rejected like the reference does.
#pragma once

#include <cstdint>
#include <cstdlib>
#include <fstream>
#include <map>
#include <sstream>
#include <stdexcept>
#include <cctype>
#include <string>
#include <vector>

namespace pie_hip_driver {

// ---- layer stacks: models whose layers differ from one another ----------------------------------
// Each layer names a mixer (what exchanges information between tokens) with its own sizes, and an
// optional feed-forward.  Mixers are listed here once, with every constant a parameter.

// Rotary embedding of the first `dims` entries of a vector (which entries pair up is the mixer's: neighbours,
// or entry i with entry i + dims / 2).
struct RotarySpec {
    int dims = 0;
    double base = 10000.0;
    bool yarn = false;   // frequencies ramped between f and f / factor, cos / sin scaled
    double factor = 1.0, original = 0.0, fast = 32.0, slow = 1.0;
    bool operator==(const RotarySpec& o) const {
        return dims == o.dims && base == o.base && yarn == o.yarn && factor == o.factor && original == o.original &&
               fast == o.fast && slow == o.slow;
    }
};

// Attention over a cached low-rank latent per token and one rotated key part shared by the heads (or none);
// optionally on another layer's cached latents, with a learned sink per head (exp(sink) joins the sum of
// exponentials), and with logistic gates on the heads' outputs: one per value or one per head.
enum class OutputGate { None, PerValue, PerHead };
struct LatentAttentionSpec {
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    double scale = 0.0;
    RotarySpec rot;
    bool half_split = false;   // rotated pairs (i, i + dims / 2) instead of neighbours
    bool sinks = false;
    OutputGate gate = OutputGate::None;
    int kv_from = -1;          // the layer whose cache rows this one reads (-1: its own)
};

// Gated delta rule with one decay per head and key channel; a short causal convolution before it.
struct ChannelDeltaSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1;
    int decay_rank = 0, gate_rank = 0;   // low-rank decay and output gate (a checkpoint's tensors fix them)
};

// Grouped-query attention: optional sliding window (0: none), optional sink (added to the sum of
// exponentials), query and key projections with or without biases, normed per head, over the whole projection
// or not at all before the rotation, values of their own or the keys as projected, an optional logistic gate on
// the concatenated heads.
enum class QueryKeyNorm { None, PerHead, WholeProjection };
struct GroupAttentionSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, window = 0;
    double scale = 0.0;
    float sink = 0.f;
    RotarySpec rot;
    bool half_split = true, biases = true, own_values = false, gate = false;
    QueryKeyNorm norm = QueryKeyNorm::PerHead;
    int widest() const { return dim > vdim ? dim : vdim; }
};

// A memory S [dim, vdim] with one decay per head and token.  Retention: constant decays; MatrixLstm:
// exponential gates with a running maximum and a normaliser; StateSpace (Mamba-2): step sizes, query and
// key heads shared by groups, a short convolution with biases, a skip per head.
enum class DecayKind { Retention, MatrixLstm, StateSpace };
struct DecayMemorySpec {
    DecayKind kind = DecayKind::Retention;
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1;
    int norm_parts = 1;            // StateSpace: equal parts of the gated output that are normed on their own
    double gate_cap = 0.0;         // MatrixLstm
    std::vector<double> decay;     // Retention, one per head
};

// Parallel: attention and a memory side by side on the same input, attention_scale * a + memory_scale * m.
enum class MixerKind { LatentAttention, ChannelDelta, DecayMemory, Parallel, Attention };

// A mixture of feed-forwards: a router over `experts`, of which a token uses `top`.
// GroupSoftmax: chosen from the best `keep` of `groups` equal groups of neighbours; the chosen probabilities are
// divided by their sum and multiplied by `scale`.  CorrectedScores: logistic scores, the largest after a learned
// correction are chosen, the scores themselves are the weights.
// Expert, ClampedPair: g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(alpha g) (u + shift);
// SquaredRelu: max(up, 0)^2.  `shared_ff`: width of one more expert that every token uses, behind a logistic gate
// (0: none); it is cut into parts as wide as the (padded) experts, which then run and join like chosen ones.
enum class RouterKind { GroupSoftmax, CorrectedScores };
enum class ExpertKind { ClampedPair, SquaredRelu };
struct MixtureSpec {
    RouterKind router = RouterKind::GroupSoftmax;
    ExpertKind expert = ExpertKind::ClampedPair;
    int experts = 0, top = 0, ff = 0, groups = 1, keep = 1, shared_ff = 0;
    float scale = 1.f, limit = 0.f, alpha = 1.f, shift = 0.f;
    int padded_ff() const { return (ff + 127) / 128 * 128; }
    int shared_parts() const { return shared_ff > 0 ? (shared_ff + padded_ff() - 1) / padded_ff() : 0; }
    int all_experts() const { return experts + shared_parts(); }   // shared parts first
    int routes() const { return top + shared_parts(); }            // of a token
    int router_columns() const { return experts + (shared_ff > 0 ? 1 : 0); }   // the last: the shared expert's gate
};

struct LayerSpec {
    MixerKind mixer = MixerKind::LatentAttention;
    LatentAttentionSpec latent;
    ChannelDeltaSpec delta;
    GroupAttentionSpec attn;       // Parallel, Attention
    DecayMemorySpec memory;        // DecayMemory, Parallel
    float attention_scale = 1.f, memory_scale = 1.f;
    int ff = 0;   // width of the dense feed-forward (ModelConfig::ff_act); 0: the layer has none
    MixtureSpec moe;   // experts 0: the layer has none
    bool has_attn() const { return mixer == MixerKind::Parallel || mixer == MixerKind::Attention; }
    bool has_memory() const { return mixer == MixerKind::Parallel || mixer == MixerKind::DecayMemory; }
};

// Layers start .. stop - 1 run `times` times in a row with the same weights; every pass keeps its own
// cache and state.
struct LayerLoop {
    int start = 0, stop = 0, times = 1;
};
struct LayerRun {
    int layer, pass;
    bool begins_pass;   // first layer of a pass of the loop
};

// (GatedSilu: silu(gate) * up between three matrices, with biases or without)
enum class FeedForwardAct { SquaredRelu, Gelu, GatedSilu };

// A second embedding row per token, by a hash of the previous token and its own: row (previous * mul_prev + token *
// mul_cur) mod buckets, row `buckets` for a sequence's first token (buckets 0: none).
struct BigramSpec {
    std::uint64_t buckets = 0, mul_prev = 0, mul_cur = 0;
};

struct ModelConfig {
    // architecture: "llama3" (dense, adjacent-pair RoPE) | "qwen3" (dense, qk-norm, half-split
    // RoPE) | "qwen3_moe" | "varasun", "lofudra", "fobanex", "minodra" (layer stacks)
    std::string arch = "llama3";
    int hidden = 0, layers = 0, q_heads = 0, kv_heads = 0, head_dim = 0, intermediate = 0;
    int vocab = 0;
    float rope_theta = 500000.f, rms_eps = 1e-5f;
    // llama3 wavelength-band RoPE scaling; factor <= 0 disables it
    float rope_factor = 0.f, rope_low_freq_factor = 1.f, rope_high_freq_factor = 4.f;
    int rope_original_max_pos = 8192;
    // rope_scaling = "llama3" (wavelength bands, the default when rope_factor > 0) or "yarn"
    // (ramp over the rotation dims between beta_fast and beta_slow, cos / sin times the
    // attention factor; 0 = 0.1 ln(factor) + 1)
    std::string rope_scaling;
    float rope_beta_fast = 32.f, rope_beta_slow = 1.f, rope_attention_factor = 0.f;
    int rope_interleaved = -1;  // -1: half split, the pairing of Llama / Mistral / Qwen checkpoints
    bool tie_embeddings = false;
    // storage format of the decoder linears: "int4b8" | "int8" | "fp8" | "bf16"
    std::string quant = "int4b8";
    int group_size = 128;
    std::string scale_dtype = "bf16";  // row scales of int8/fp8: "bf16" | "f32"
    // MoE (qwen3_moe)
    int num_experts = 0, top_k = 0, expert_intermediate = 0;
    bool norm_topk = true;
    int sliding_window = 0;   // > 0: a query at position p sees keys p - W + 1 .. p only
    // synthetic random-init weights: N(0, init_std) in bf16, then quantised
    std::uint64_t seed = 0x9E3779B97F4A7C15ull;
    float init_std = 0.02f;
    float router_std = 0.f;  // MoE router rows; 0 = init_std
    float embed_std = 0.f;   // embedding rows; 0 = init_std (a large value lets a token's own embedding
                             // dominate the residual stream, so distinct tokens take distinct MoE routes)
    // `[model] hf_path` (portable driver's key) or `snapshot_dir` (CUDA driver's key): a Hugging
    // Face snapshot directory; its config.json then fixes the shape fields above and the weights
    // come from its safetensors files instead of the synthetic initialiser
    std::string checkpoint_dir;
    // with checkpoint_dir: take only config.json from it and fill the weights synthetically
    bool random_weights = false;
    // layer stacks: the layers, and what follows the last one (logits = cap * tanh(scale * y / cap);
    // cap 0: no cap).  Empty for the uniform architectures above.
    std::vector<LayerSpec> stack;
    LayerLoop loop;                // stop 0: none
    bool sandwich_norms = false;   // a norm ahead of every sublayer besides the one on its output
    bool shared_norm = false;      // one norm per layer: mixer and feed-forward read it and join the stream together
    // sublayers read a normed row plus a convolution over it and its last canon_taps - 1 predecessors; their outputs
    // pass a logistic gate of the normed row; norms have one weight for all columns; the embedding is normed
    bool gated_sublayers = false;
    int canon_taps = 0;
    BigramSpec bigram;
    float embed_scale = 1.f;       // (with shared_norm or gated_sublayers)
    FeedForwardAct ff_act = FeedForwardAct::SquaredRelu;
    bool ff_biases = false;        // GatedSilu
    std::vector<LayerRun> layer_runs() const {
        std::vector<LayerRun> runs;
        const int n = static_cast<int>(stack.size());
        for (int l = 0; l < n; ++l) {
            if (loop.stop > loop.start && l == loop.start) {
                for (int t = 0; t < loop.times; ++t)
                    for (int k = loop.start; k < loop.stop; ++k) runs.push_back({k, t, k == loop.start});
                l = loop.stop - 1;
            } else {
                runs.push_back({l, 0, false});
            }
        }
        return runs;
    }
    float logit_scale = 1.f, logit_softcap = 0.f;
    bool is_stack() const { return !stack.empty(); }
    // activations and products: "bfloat16" | "float32" (layer stacks only: true 32-bit throughout)
    std::string compute_dtype = "bfloat16";
    bool f32() const { return compute_dtype == "float32"; }
};

struct BatchingConfig {
    int kv_page_size = 32;       // driver/portable/src/config.hpp:30
    int total_pages = 1024;      // server/src/config.rs:727-743
    int max_forward_tokens = 10240;
    int max_forward_requests = 512;
    int cpu_pages = 0;
    // recurrent state of layer stacks: sequences that can hold state at a time (0: one per request
    // of a batch), and host slots they can be swapped to
    int rs_cache_slots = 0, cpu_rs_slots = 0;
    // KV-cache storage (driver/cuda/src/config.hpp:66, kv_cache_format.cpp:46-110): auto | bf16 |
    // bfloat16 | fp8_e4m3 | int8_per_token_head | fp8_per_token_head
    std::string kv_cache_dtype = "auto";
};

struct RuntimeConfig {
    bool verbose = false;
    bool use_graphs = true;
    // a second copy of every decoder linear in the skinny GEMM's tile-major layout (doubles the
    // weight memory, ~25 % off the 5-32-row and MoE grouped GEMMs)
    bool tiled_weights = true;
    // one synthetic full-size prefill chunk and a decode step at start-up, so that the first
    // request does not pay one-time costs (measured: 58 ms cold against 47 ms for a 2048-token
    // prefill of an 8B model); writes only KV pages nobody owns yet
    bool warmup = true;
    // time the candidate kernels of every decoder linear at start-up (2-4 and 17-128 rows, a few
    // tens of milliseconds) and dispatch on the measurements instead of the fitted cost model
    bool tune_linears = true;
    // one or two decode rows: the attention output projection merges the attention's splits in
    // its prologue where that is measured to pay (no separate merge launch; the attention output
    // rows are then never stored)
    bool attn_merge_proj = true;
    std::string snapshot_dir;
};

struct DriverConfig {
    ModelConfig model;
    BatchingConfig batching;
    RuntimeConfig runtime;
};

namespace detail {
inline std::string trim(const std::string& s) {
    const auto b = s.find_first_not_of(" \t\r\n");
    if (b == std::string::npos) return "";
    const auto e = s.find_last_not_of(" \t\r\n");
    return s.substr(b, e - b + 1);
}
inline std::string unquote(const std::string& v) {
    if (v.size() >= 2 && (v.front() == '"' || v.front() == '\'') && v.back() == v.front())
        return v.substr(1, v.size() - 2);
    return v;
}
inline bool to_bool(const std::string& v, const std::string& key) {
    if (v == "true") return true;
    if (v == "false") return false;
    throw std::runtime_error("config: " + key + " must be true or false");
}
inline long long to_int(const std::string& v, const std::string& key) {
    std::string t;
    for (char c : v)
        if (c != '_') t.push_back(c);
    char* end = nullptr;
    const long long r = std::strtoll(t.c_str(), &end, 0);
    if (end == t.c_str() || *end != '\0') throw std::runtime_error("config: " + key + " must be an integer");
    return r;
}
inline double to_float(const std::string& v, const std::string& key) {
    char* end = nullptr;
    const double r = std::strtod(v.c_str(), &end);
    if (end == v.c_str() || *end != '\0') throw std::runtime_error("config: " + key + " must be a number");
    return r;
}
}  // namespace detail

// Parses TOML text into section -> key -> raw value.
inline std::map<std::string, std::map<std::string, std::string>> parse_toml_lite(
    const std::string& text) {
    std::map<std::string, std::map<std::string, std::string>> out;
    std::istringstream in(text);
    std::string line, section;
    int lineno = 0;
    while (std::getline(in, line)) {
        ++lineno;
        // strip comments outside quotes
        bool inq = false;
        char qc = 0;
        for (size_t i = 0; i < line.size(); ++i) {
            const char c = line[i];
            if (inq) {
                if (c == qc) inq = false;
            } else if (c == '"' || c == '\'') {
                inq = true;
                qc = c;
            } else if (c == '#') {
                line.erase(i);
                break;
            }
        }
        line = detail::trim(line);
        if (line.empty()) continue;
        if (line.front() == '[') {
            if (line.back() != ']') throw std::runtime_error("config: bad section at line " + std::to_string(lineno));
            section = detail::trim(line.substr(1, line.size() - 2));
            out[section];
            continue;
        }
        const auto eq = line.find('=');
        if (eq == std::string::npos) throw std::runtime_error("config: expected key = value at line " + std::to_string(lineno));
        out[section][detail::trim(line.substr(0, eq))] = detail::trim(line.substr(eq + 1));
    }
    return out;
}

// The kernel library's PIE_HIP_KV_* code of a kv_cache_dtype value; the reference's other values
// (fp8_e5m2, fp4_e2m1, nvfp4) are recognised and refused, anything else is invalid
// (driver/cuda/src/kv_cache_format.cpp:105-108).
inline int kv_format_code(const std::string& value) {
    std::string v;
    for (char ch : value) v.push_back(static_cast<char>(std::tolower(static_cast<unsigned char>(ch))));
    if (v.empty() || v == "auto" || v == "bf16" || v == "bfloat16") return 0;
    if (v == "fp8_e4m3") return 1;
    if (v == "int8_per_token_head") return 2;
    if (v == "fp8_per_token_head") return 3;
    if (v == "fp8_e5m2") return 4;
    if (v == "fp4_e2m1" || v == "nvfp4") return 5;   // one scheme under two names (kv_cache_format.cpp:99-107)
    throw std::runtime_error("invalid kv_cache_dtype '" + value +
                             "'; expected one of: auto, bf16, bfloat16, fp8_e4m3, fp8_e5m2, "
                             "int8_per_token_head, fp8_per_token_head, fp4_e2m1, nvfp4");
}

// Shape and range checks, defaults that depend on other fields.
inline void finalize_batching(const BatchingConfig& b) {
    if (b.kv_page_size <= 0 || b.kv_page_size % 16 != 0)
        throw std::runtime_error("config: kv_page_size must be a positive multiple of 16");
    if (b.total_pages <= 0 || b.max_forward_tokens <= 0 || b.max_forward_requests <= 0)
        throw std::runtime_error("config: [batching] sizes must be positive");
    if (b.rs_cache_slots < 0 || b.cpu_rs_slots < 0)
        throw std::runtime_error("config: rs_cache_slots and cpu_rs_slots must not be negative");
    (void)kv_format_code(b.kv_cache_dtype);
}

// Layer stacks: every layer's sizes, and the storage choices the stack executor has.
inline void finalize_stack(DriverConfig& c) {
    auto& m = c.model;
    if (m.hidden <= 0 || m.vocab <= 0) throw std::runtime_error("config: a layer stack needs a width and a vocabulary");
    for (size_t i = 0; i < m.stack.size(); ++i) {
        const LayerSpec& l = m.stack[i];
        const std::string at = "config: layer " + std::to_string(i) + ": ";
        if (l.ff < 0) throw std::runtime_error(at + "negative feed-forward width");
        if (l.mixer == MixerKind::LatentAttention) {
            const auto& a = l.latent;
            if (a.heads <= 0 || a.dim <= 0 || a.rot_dim < 0 || a.vdim <= 0 || a.q_rank <= 0 || a.kv_rank <= 0)
                throw std::runtime_error(at + "latent_attention needs heads, dim, vdim, q_rank, kv_rank");
            if (a.rot.dims < 0 || a.rot.dims % 2 != 0 || a.rot.dims > a.rot_dim)
                throw std::runtime_error(at + "rot.dims must be even and at most rot_dim");
            if (a.rot.dims > 0 && !(a.rot.base > 0.0)) throw std::runtime_error(at + "rot.base must be positive");
            if (a.kv_from >= 0) {
                const LayerSpec* from = a.kv_from < static_cast<int>(i) ? &m.stack[static_cast<size_t>(a.kv_from)] : nullptr;
                if (!from || from->mixer != MixerKind::LatentAttention || from->latent.kv_from >= 0)
                    throw std::runtime_error(at + "kv_from must name an earlier latent_attention layer with latents of its own");
                const auto& b = from->latent;
                if (b.kv_rank != a.kv_rank || b.rot_dim != a.rot_dim || !(b.rot == a.rot) || b.half_split != a.half_split)
                    throw std::runtime_error(at + "kv_from: kv_rank, rot_dim and the rotation must be equal");
                if (m.loop.stop != 0) throw std::runtime_error(at + "kv_from cannot be combined with a loop");
            }
        } else if (l.mixer == MixerKind::ChannelDelta) {
            const auto& d = l.delta;
            if (d.heads <= 0 || d.kv_heads <= 0 || d.dim <= 0 || d.vdim <= 0 || d.taps <= 0)
                throw std::runtime_error(at + "channel_delta needs heads, kv_heads, dim, vdim, conv");
            if (d.heads % d.kv_heads != 0) throw std::runtime_error(at + "heads must be a multiple of kv_heads");
        }
        if (l.has_attn()) {
            const auto& a = l.attn;
            if (a.heads <= 0 || a.kv_heads <= 0 || a.dim <= 0 || a.window < 0)
                throw std::runtime_error(at + "attention needs heads, kv_heads, dim and a window that is not negative");
            if (a.heads % a.kv_heads != 0) throw std::runtime_error(at + "heads must be a multiple of kv_heads");
            if (a.vdim <= 0) throw std::runtime_error(at + "attention needs a positive vdim");
            if (!a.own_values && a.vdim != a.dim) throw std::runtime_error(at + "values that are the keys have the keys' size");
            if (a.widest() > 1024) throw std::runtime_error(at + "attention heads are limited to 1024 values");
            if (a.rot.dims < 0 || a.rot.dims % 2 != 0 || a.rot.dims > a.dim)
                throw std::runtime_error(at + "rot.dims must be even and at most dim");
            if (a.rot.dims > 0 && !(a.rot.base > 0.0)) throw std::runtime_error(at + "rot.base must be positive");
        }
        if (l.moe.experts != 0) {
            const auto& e = l.moe;
            if (!m.shared_norm && !m.gated_sublayers)
                throw std::runtime_error(at + "this architecture has no mixtures");
            if (e.experts <= 0 || e.ff <= 0 || e.top <= 0 || e.groups <= 0 || e.keep <= 0 || e.keep > e.groups || e.experts % e.groups != 0)
                throw std::runtime_error(at + "a mixture needs experts in equal groups, a positive width, top and kept groups");
            if (e.top > e.keep * (e.experts / e.groups)) throw std::runtime_error(at + "fewer experts in the kept groups than a token uses");
            if (e.shared_ff < 0) throw std::runtime_error(at + "shared.ff must not be negative");
            if (e.all_experts() > 512 || e.routes() > 64)
                throw std::runtime_error(at + "mixtures are limited to 512 experts, 64 per token (a shared expert counts by its parts)");
            if (!(e.limit >= 0.f)) throw std::runtime_error(at + "expert.limit must not be negative");
        }
        if (l.has_memory()) {
            const auto& d = l.memory;
            if (d.heads <= 0 || d.kv_heads <= 0 || d.dim <= 0 || d.vdim <= 0 || d.taps <= 0)
                throw std::runtime_error(at + "a memory needs heads, key heads, dim, vdim (and conv)");
            if (d.heads % d.kv_heads != 0) throw std::runtime_error(at + "heads must be a multiple of the groups");
            if (d.dim > 512) throw std::runtime_error(at + "memories are limited to 512 key channels");
            if (d.kind == DecayKind::Retention && d.decay.size() != static_cast<size_t>(d.heads))
                throw std::runtime_error(at + "retention needs one decay per head");
            for (double v : d.decay)
                if (!(v >= 0.0 && v <= 1.0)) throw std::runtime_error(at + "decays must be between 0 and 1");
            if (d.kind == DecayKind::MatrixLstm && !(d.gate_cap > 0.0)) throw std::runtime_error(at + "gate_cap must be positive");
            if (d.norm_parts <= 0 || (d.heads * d.vdim) % d.norm_parts != 0)
                throw std::runtime_error(at + "norm_groups must divide heads * vdim");
        }
    }
    if (m.loop.stop != 0 || m.loop.start != 0) {
        if (m.loop.start < 0 || m.loop.stop <= m.loop.start || m.loop.stop > static_cast<int>(m.stack.size()) || m.loop.times <= 0)
            throw std::runtime_error("config: loop needs 0 <= start < stop <= layers and times > 0");
    }
    if (m.gated_sublayers && m.canon_taps <= 0) throw std::runtime_error("config: canon.taps must be positive");
    if (m.compute_dtype != "bfloat16" && m.compute_dtype != "float32")
        throw std::runtime_error("config: compute_dtype must be bfloat16 or float32");
    m.quant = "bf16";   // the linears of layer stacks are kept as stored
    m.layers = static_cast<int>(m.stack.size());
    if (kv_format_code(c.batching.kv_cache_dtype) != 0)
        throw std::runtime_error("config: layer stacks keep their cache in the compute type (kv_cache_dtype = auto)");
    if (c.batching.rs_cache_slots == 0) c.batching.rs_cache_slots = c.batching.max_forward_requests;
    finalize_batching(c.batching);
}

inline void finalize_config(DriverConfig& c) {
    auto& m = c.model;
    if (m.is_stack()) return finalize_stack(c);
    if (m.f32()) throw std::runtime_error("config: compute_dtype float32 is available for layer stacks only");
    if (m.hidden <= 0 || m.layers <= 0 || m.q_heads <= 0 || m.kv_heads <= 0 || m.vocab <= 0)
        throw std::runtime_error("config: [model] needs hidden, layers, q_heads, kv_heads, vocab");
    if (m.head_dim <= 0) m.head_dim = m.hidden / m.q_heads;
    if (m.q_heads % m.kv_heads != 0) throw std::runtime_error("config: q_heads must be a multiple of kv_heads");
    const bool moe = m.arch == "qwen3_moe";
    if (m.arch != "llama3" && m.arch != "qwen3" && !moe)
        throw std::runtime_error("config: unsupported arch '" + m.arch + "'");
    if (moe) {
        if (m.num_experts <= 0 || m.top_k <= 0 || m.expert_intermediate <= 0 || m.top_k > m.num_experts)
            throw std::runtime_error("config: qwen3_moe needs num_experts, top_k, expert_intermediate");
    } else if (m.intermediate <= 0) {
        throw std::runtime_error("config: [model] needs intermediate");
    }
    if (m.quant != "int4b8" && m.quant != "int8" && m.quant != "fp8" && m.quant != "bf16")
        throw std::runtime_error("config: unsupported quant '" + m.quant + "'");
    if (m.scale_dtype != "bf16" && m.scale_dtype != "f32")
        throw std::runtime_error("config: scale_dtype must be bf16 or f32");
    // (i, i + d/2) pairs for every architecture here, as the reference rotates them
    // (driver/cuda/src/kernels/rope.cu:10-21 keeps adjacent pairs for GLM only)
    if (m.rope_interleaved < 0) m.rope_interleaved = 0;
    if (m.rope_scaling.empty()) m.rope_scaling = "llama3";
    if (m.rope_scaling != "llama3" && m.rope_scaling != "yarn")
        throw std::runtime_error("config: rope_scaling must be llama3 or yarn");
    finalize_batching(c.batching);
}

inline DriverConfig parse_config_text(const std::string& text) {
    using namespace detail;
    DriverConfig c;
    const auto t = parse_toml_lite(text);
    for (const auto& [sec, kv] : t) {
        for (const auto& [k, raw] : kv) {
            const std::string v = unquote(raw);
            const std::string key = sec + "." + k;
            if (sec == "model") {
                auto& m = c.model;
                if (k == "arch") m.arch = v;
                else if (k == "hidden" || k == "hidden_size") m.hidden = (int)to_int(v, key);
                else if (k == "layers" || k == "num_hidden_layers") m.layers = (int)to_int(v, key);
                else if (k == "q_heads" || k == "num_attention_heads") m.q_heads = (int)to_int(v, key);
                else if (k == "kv_heads" || k == "num_key_value_heads") m.kv_heads = (int)to_int(v, key);
                else if (k == "head_dim") m.head_dim = (int)to_int(v, key);
                else if (k == "intermediate" || k == "intermediate_size") m.intermediate = (int)to_int(v, key);
                else if (k == "vocab" || k == "vocab_size") m.vocab = (int)to_int(v, key);
                else if (k == "rope_theta") m.rope_theta = (float)to_float(v, key);
                else if (k == "rms_eps" || k == "rms_norm_eps") m.rms_eps = (float)to_float(v, key);
                else if (k == "rope_factor") m.rope_factor = (float)to_float(v, key);
                else if (k == "rope_low_freq_factor") m.rope_low_freq_factor = (float)to_float(v, key);
                else if (k == "rope_high_freq_factor") m.rope_high_freq_factor = (float)to_float(v, key);
                else if (k == "rope_original_max_pos") m.rope_original_max_pos = (int)to_int(v, key);
                else if (k == "rope_scaling") m.rope_scaling = v;
                else if (k == "rope_beta_fast") m.rope_beta_fast = (float)to_float(v, key);
                else if (k == "rope_beta_slow") m.rope_beta_slow = (float)to_float(v, key);
                else if (k == "rope_attention_factor") m.rope_attention_factor = (float)to_float(v, key);
                else if (k == "rope_interleaved") m.rope_interleaved = to_bool(v, key) ? 1 : 0;
                else if (k == "tie_embeddings") m.tie_embeddings = to_bool(v, key);
                else if (k == "quant") m.quant = v;
                else if (k == "group_size") m.group_size = (int)to_int(v, key);
                else if (k == "scale_dtype") m.scale_dtype = v;
                else if (k == "num_experts") m.num_experts = (int)to_int(v, key);
                else if (k == "top_k") m.top_k = (int)to_int(v, key);
                else if (k == "expert_intermediate") m.expert_intermediate = (int)to_int(v, key);
                else if (k == "norm_topk") m.norm_topk = to_bool(v, key);
                else if (k == "sliding_window") m.sliding_window = (int)to_int(v, key);
                else if (k == "seed") m.seed = (std::uint64_t)to_int(v, key);
                else if (k == "init_std") m.init_std = (float)to_float(v, key);
                else if (k == "router_std") m.router_std = (float)to_float(v, key);
                else if (k == "embed_std") m.embed_std = (float)to_float(v, key);
                else if (k == "random_weights") m.random_weights = to_bool(v, key);
                else if (k == "compute_dtype") m.compute_dtype = v;
                else if (k == "hf_path" || k == "snapshot_dir") m.checkpoint_dir = v;
                // other [model] keys (paths, dtype hints) belong to loaders this driver lacks
            } else if (sec == "batching") {
                auto& b = c.batching;
                if (k == "kv_page_size") b.kv_page_size = (int)to_int(v, key);
                else if (k == "total_pages") b.total_pages = (int)to_int(v, key);
                else if (k == "max_forward_tokens") b.max_forward_tokens = (int)to_int(v, key);
                else if (k == "max_forward_requests") b.max_forward_requests = (int)to_int(v, key);
                else if (k == "cpu_pages") b.cpu_pages = (int)to_int(v, key);
                else if (k == "rs_cache_slots") b.rs_cache_slots = (int)to_int(v, key);
                else if (k == "cpu_rs_slots") b.cpu_rs_slots = (int)to_int(v, key);
                else if (k == "kv_cache_dtype") b.kv_cache_dtype = v;
                else throw std::runtime_error("config: unknown [batching] key '" + k + "'");
            } else if (sec == "runtime") {
                auto& r = c.runtime;
                if (k == "verbose") r.verbose = to_bool(v, key);
                else if (k == "use_graphs") r.use_graphs = to_bool(v, key);
                else if (k == "tiled_weights") r.tiled_weights = to_bool(v, key);
                else if (k == "warmup") r.warmup = to_bool(v, key);
                else if (k == "tune_linears") r.tune_linears = to_bool(v, key);
                else if (k == "attn_merge_proj") r.attn_merge_proj = to_bool(v, key);
                else if (k == "snapshot_dir") r.snapshot_dir = v;
            }
        }
    }
    if (c.model.checkpoint_dir.empty()) finalize_config(c);   // else after config.json is applied
    return c;
}

// `src` is a file path, or inline TOML when it contains a newline.
inline DriverConfig load_config(const std::string& src) {
    if (src.find('\n') != std::string::npos) return parse_config_text(src);
    std::ifstream f(src);
    if (!f) throw std::runtime_error("config: cannot open '" + src + "'");
    std::stringstream ss;
    ss << f.rdbuf();
    return parse_config_text(ss.str());
}

}  // namespace pie_hip_driver
