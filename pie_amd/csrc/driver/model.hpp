// Model weights resident in HBM, in the storage formats the kernels stream.
//
// Layout per decoder layer (llama-like; op sequence of
// driver/portable/src/graph_qwen3.cpp:225-829 and driver/cuda/src/model/llama_like.cpp:364-762):
//   attn_norm [H] bf16, wqkv [(hq+2hk)d, H] (q rows, then k rows, then v rows — per-row /
//   per-group scales make the fusion exact), optional q_norm/k_norm [d], wo [H, hq*d],
//   ffn_norm [H], then either wgu [2I, H] (rows interleaved gate_0, up_0, gate_1, ... for the
//   fused SwiGLU epilogue) + wdown [H, I], or the
//   MoE block: router [E, H] bf16, experts stacked along the rows — wgu [E * 2Ie, H] (gate/up
//   interleaved inside each expert) and wdown [E * H, Ie].
// embed [V, H] bf16, final_norm [H], lm_head [V, H] bf16 (aliases embed when tied); those
// three stay unquantised like the reference (driver/cuda/src/config.hpp:20-30).
#pragma once

#include <array>
#include <hip/hip_runtime.h>

#include <cstdint>
#include <map>
#include <string>
#include <vector>

#include "config.hpp"

namespace pie_hip_driver {

enum class Quant { Int4b8, Int8, Fp8, Bf16 };

struct Linear {
    Quant kind = Quant::Bf16;
    void* data = nullptr;   // packed weights, [N, K] in the format's element size
    void* scale = nullptr;  // int4: bf16 [N, K/G]; int8/fp8: f32 or bf16 [N]; bf16: null
    bool scale_bf16 = true;
    int N = 0, K = 0, group = 0;
    // optional copies in the skinny GEMM's tile-major layout (pie_hip_repack_mfma_tiles)
    void* data_tiled = nullptr;
    void* scale_tiled = nullptr;   // int4 group scales; other formats keep `scale`
    // kernel that measured fastest for M activation rows at start-up (index M, 0..128):
    // 0 GEMV, 1 skinny GEMM, 2 tiled GEMM, 3 tiled GEMM in K shares; -1: not measured, the cost
    // model decides
    std::array<int8_t, 129> tuned = [] { std::array<int8_t, 129> t{}; t.fill(-1); return t; }();
    size_t data_bytes() const {
        const size_t nk = static_cast<size_t>(N) * K;
        switch (kind) {
            case Quant::Int4b8: return nk / 2;
            case Quant::Bf16: return nk * 2;
            default: return nk;
        }
    }
    size_t scale_bytes() const {
        switch (kind) {
            case Quant::Int4b8: return static_cast<size_t>(N) * (K / group) * 2;
            case Quant::Bf16: return 0;
            default: return static_cast<size_t>(N) * (scale_bf16 ? 2 : 4);
        }
    }
};

struct LayerWeights {
    uint16_t* attn_norm = nullptr;
    uint16_t* ffn_norm = nullptr;
    uint16_t* q_norm = nullptr;
    uint16_t* k_norm = nullptr;
    Linear wqkv, wo, wgu, wdown;  // MoE: wgu / wdown hold the experts stacked along the rows
    Linear router;                // MoE: [E, H] bf16
};

// Where everything sits in a layer-stack layer's padded matrices and rows.  Sizes that are the K of
// a product are rounded up so that every product takes the matrix-core kernels (zero columns in
// the weights, zero or ignored entries in the rows).
constexpr int pad_to(int v, int a) { return (v + a - 1) / a * a; }
// (the latent ranks the matrix-core attention is built for; wider ones take the plain kernel)
constexpr int pad_latent(int v) {
    return v <= 256 ? pad_to(v, 64) : v <= 512 ? pad_to(v, 128) : pad_to(v, 64);
}
struct LatentShape {
    int heads, dimp, rotp, vdp, kvp;   // per-head sizes and the latent, rounded up
    int kv_off, gate_off, gate_cols, ld_in;   // fused projection: query latent | latent, rotated key part | gates (heads of
                                              // gate_cols: vdp, 1 or 0)
    int ld_cq, hd, ld_q;               // query latent rows; q rows: heads of [dimp | rotp]
    int ld_row;                        // cache row: [kvp | rotp] (rotp 0: no rotated part)
    int ld_o;                          // attention output rows: heads of vdp
    explicit LatentShape(const LatentAttentionSpec& a)
        : heads(a.heads), dimp(pad_to(a.dim, 32)), rotp(pad_to(a.rot_dim, 32)), vdp(pad_to(a.vdim, 32)),
          kvp(pad_latent(a.kv_rank)), kv_off(pad_to(a.q_rank, 16)),
          gate_off(pad_to(kv_off + (a.kv_from < 0 ? a.kv_rank + a.rot_dim : 0), 8)),
          gate_cols(a.gate == OutputGate::PerValue ? vdp : a.gate == OutputGate::PerHead ? 1 : 0), ld_in(pad_to(gate_off + heads * gate_cols, 16)),
          ld_cq(pad_to(a.q_rank, 128)), hd(dimp + rotp), ld_q(heads * hd), ld_row(kvp + rotp),
          ld_o(pad_to(heads * vdp, 128)) {}
};
struct DeltaShape {
    int kd, vd, channels;                       // q (= k) channels, v channels, all three
    int decay_off, gate_off, ld_in;             // fused projection: q | k | v | step sizes | decay | gate inputs
    int ld_a1, ld_g1, ld_gate, ld_o;            // columns of the low-rank second factors, gate rows, output rows
    explicit DeltaShape(const ChannelDeltaSpec& d)
        : kd(d.kv_heads * d.dim), vd(d.heads * d.vdim), channels(2 * kd + vd), decay_off(pad_to(channels + d.heads, 8)),
          gate_off(pad_to(decay_off + d.decay_rank, 8)), ld_in(pad_to(gate_off + d.gate_rank, 16)),
          ld_a1(pad_to(d.decay_rank, 32)), ld_g1(pad_to(d.gate_rank, 32)),
          ld_gate(pad_to(vd, 16)), ld_o(pad_to(vd, 128)) {}
};

// (the head sizes the matrix-core attention is built for; wider ones take the plain kernel)
constexpr int pad_head(int v) { return v <= 128 ? pad_to(v, 32) : v <= 256 ? pad_to(v, 64) : pad_to(v, 32); }
// Grouped attention beside or without a memory, and a memory alone, behind one fused projection.
struct MixShape {
    int q_off = 0, k_off = 0, dimp = 0, ld_attn = 0;   // attention: query and key columns; output heads of dimp
    int v_off = -1, attn_gate_off = -1;                // its own values, its gates (heads of dimp)
    int mq_off = 0, mk_off = 0, mv_off = 0, gate_off = 0;   // memory: columns of the fused projection
    int channels = 0, ld_conv = 0;                     // StateSpace: convolved columns [values | keys | queries]
    int gates = 0;                                     // fp32 gate columns, a product of their own
    int out_off = 0, ld_in = 0, ld_o = 0;              // where the memory's output starts in the rows of W_o's input
    explicit MixShape(const LayerSpec& l) {
        int at = 0, out = 0;
        auto place = [&](int n) {
            const int here = at;
            at = pad_to(at + n, 8);
            return here;
        };
        const auto& d = l.memory;
        const int kd = d.kv_heads * d.dim, vd = d.heads * d.vdim;
        if (l.has_attn()) {
            dimp = pad_head(l.attn.widest());
            q_off = place(l.attn.heads * l.attn.dim);
            k_off = place(l.attn.kv_heads * l.attn.dim);
            if (l.attn.own_values) v_off = place(l.attn.kv_heads * l.attn.vdim);
            if (l.attn.gate) attn_gate_off = place(l.attn.heads * dimp);
            out = ld_attn = pad_to(l.attn.heads * dimp, 16);
        }
        if (l.has_memory()) {
            if (d.kind == DecayKind::StateSpace) {   // contiguous, so that one convolution covers them
                mv_off = at;
                mk_off = mv_off + vd;
                mq_off = mk_off + kd;
                channels = vd + 2 * kd;
                ld_conv = pad_to(channels, 8);
                at = pad_to(at + channels, 8);
                gates = pad_to(d.heads, 16);
            } else {
                mq_off = place(kd);
                mk_off = place(kd);
                mv_off = place(vd);
                if (d.kind == DecayKind::MatrixLstm) gates = pad_to(2 * d.heads, 16);
            }
            gate_off = place(vd);
            out_off = out;
            out += vd;
        }
        ld_in = pad_to(at, 16);
        ld_o = pad_to(out, 128);
    }
};

struct StackLayer {
    LayerSpec spec;
    float *norm1 = nullptr, *norm2 = nullptr;   // on the sublayers' outputs
    float *pre1 = nullptr, *pre2 = nullptr;     // ahead of the sublayers (null: none)
    Linear w_in;            // everything the mixer projects its input to, fused
    Linear wo;
    Linear w_up, w_down;    // feed-forward (none: data null).  Gated: w_up's rows are (gate_i, up_i) pairs; a mixture's
                            // experts are stacked along the rows
    float *up_bias = nullptr, *down_bias = nullptr;   // gated: in the order of the rows
    uint16_t* w_router = nullptr;                     // mixture: [router columns rounded up to 16, width]
    float* correction = nullptr;                      // mixture: added to the scores for the choice (CorrectedScores)
    // gated sublayers: gate product and bias, convolution [taps, width] ahead of mixer and feed-forward
    Linear w_gate1, w_gate2;
    float *gate1_bias = nullptr, *gate2_bias = nullptr;
    uint16_t *canon1 = nullptr, *canon2 = nullptr;
    // latent attention
    Linear w_uq;
    Linear w_ukv;                                // [heads * (dimp + vdp), kvp]: keys and values out of the latent
    uint16_t *w_uk_t = nullptr, *w_uv = nullptr; // per head [kvp, dimp] (transposed keys) and [vdp, kvp]
    float *q_norm = nullptr, *kv_norm = nullptr, *sinks = nullptr;
    int rotary = -1;                             // index into Model::rotary
    // channel delta
    uint16_t *w_decay = nullptr, *w_gate = nullptr;   // second factors of the low-rank decay and output gate
    // grouped attention, decay memories (conv_w, dt_bias and out_norm as below)
    float *q_bias = nullptr, *k_bias = nullptr, *k_norm = nullptr;
    uint16_t* w_gates = nullptr;                     // [MixShape::gates, width]: the products that drive the recurrence
    float *conv_b = nullptr, *skip = nullptr, *gate_bias = nullptr, *decay_log2 = nullptr;
    float *conv_w = nullptr, *decay_rate = nullptr /* -exp(A_log) log2(e) */, *dt_bias = nullptr, *out_norm = nullptr;
};

struct RotaryTable {
    RotarySpec spec;
    double* freq = nullptr;   // [dims / 2] device
    float mscale = 1.f;
};

struct TensorRef {
    void* ptr;
    size_t bytes;
};

class Model {
  public:
    Model() = default;
    ~Model();
    Model(const Model&) = delete;
    Model& operator=(const Model&) = delete;

    // Allocates every tensor and fills it with seeded synthetic weights on the device:
    // N(0, init_std) rounded to bf16, then quantised by the library's quantiser kernels.
    void init_synthetic(const ModelConfig& cfg, hipStream_t stream);

    // The same layout filled from a Hugging Face snapshot (cfg.checkpoint_dir): bf16 / f16 / f32
    // `*.weight` tensors are fused (q|k|v rows, gate/up interleaved, experts stacked) and
    // quantised on the device to cfg.quant; compressed-tensors int4 checkpoints
    // (`weight_packed` int32 [N, K/8] + `weight_scale` [N, K/group]) are taken as stored.
    void load_snapshot(const ModelConfig& cfg, hipStream_t stream);

    // Builds the tile-major copies of every decoder linear whose shape the skinny GEMM takes.
    void build_tiled_copies(hipStream_t stream);

    // Layer stacks (cfg.stack): weights from the snapshot, or synthetic with cfg.random_weights.
    void load_stack(const ModelConfig& cfg, hipStream_t stream);

    const ModelConfig& cfg() const { return cfg_; }
    bool is_moe() const { return cfg_.arch == "qwen3_moe"; }
    bool has_qk_norm() const { return cfg_.arch != "llama3"; }
    // True when the q and k rows of every layer's wqkv were re-ordered at load so that rows
    // (2i, 2i+1) of a head hold the half-split RoPE pair (i, i + d/2): the fused projection
    // epilogues then rotate neighbouring outputs and store them at i and i + d/2.
    bool qk_rows_paired() const { return qk_rows_paired_; }
    Quant quant() const { return quant_; }

    uint16_t* embed = nullptr;
    uint16_t* lm_head = nullptr;
    uint16_t* final_norm = nullptr;
    float* inv_freq = nullptr;  // [d/2] device
    std::vector<LayerWeights> layers;
    // layer stacks
    std::vector<StackLayer> stack;
    std::vector<RotaryTable> rotary;   // the stack's distinct rotations
    Linear head;                       // lm_head, padded
    float* stack_norm = nullptr;       // norm ahead of it
    uint16_t* bigram = nullptr;        // [buckets + 1, hidden]
    float* embed_norm = nullptr;       // norm of the embedding (gated sublayers)
    float* loop_step = nullptr;        // [times, hidden]: added ahead of every pass of the loop
    std::vector<LayerRun> runs;        // the layers in the order they are run
    int ld_x() const { return pad_to(cfg_.hidden, 128); }

    // bytes streamed from HBM by one decode step at batch 1 (every weight once)
    size_t decode_weight_bytes() const { return decode_bytes_; }
    const std::map<std::string, TensorRef>& tensors() const { return names_; }

  private:
    void* alloc(size_t bytes, const std::string& name);
    void make_linear(Linear& lin, int N, int K, const std::string& name, std::uint64_t seed,
                     hipStream_t stream);
    void prepare_linear(Linear& lin, int N, int K, const std::string& name);
    void quantise_scratch(Linear& lin, const std::string& name, hipStream_t stream);
    void interleave_gate_up(Linear& lin, int blocks, hipStream_t stream);
    void interleave_row_blocks(Linear& lin, size_t half, size_t rows, hipStream_t stream);
    void pair_qk_rows(hipStream_t stream);
    bool qk_rows_paired_ = false;
    ModelConfig cfg_;
    Quant quant_ = Quant::Bf16;
    std::vector<void*> allocs_;
    std::map<std::string, TensorRef> names_;
    uint16_t* tmp_bf16_ = nullptr;  // scratch for the largest bf16 tensor being quantised
    size_t tmp_elems_ = 0;
    size_t decode_bytes_ = 0;
};

// Host-side inv_freq table (theta^(-2i/d) with optional llama3 band scaling,
// driver/portable/src/model.cpp:1414-1448: the stored factor divides the base frequency).
std::vector<float> rope_inv_freq(const ModelConfig& cfg);
// Frequencies of a rotation spec, and what its cos and sin are multiplied by.
std::vector<double> rotary_frequencies(const RotarySpec& r);
float rotary_mscale(const RotarySpec& r);
// bf16 N(mean, std) on the device, a pure function of (seed, index)
void fill_normal(uint16_t* dst, size_t n, uint64_t seed, float mean, float std, hipStream_t stream);
// What cos and sin are multiplied by: YaRN's attention factor (0.1 ln(factor) + 1 unless the
// config states one), 1 for every other scheme.
float rope_mscale(const ModelConfig& cfg);

}  // namespace pie_hip_driver
