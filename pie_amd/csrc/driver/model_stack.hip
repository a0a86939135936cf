// Weights of layer-stack models: checkpoint tensors ("embed", "l<i>.norm1", "l<i>.mix.*",
// "l<i>.mlp.*", "final.norm", "head") into the padded, fused matrices the kernels read.
#include <cmath>
#include <cstring>
#include <memory>
#include <stdexcept>

#include "model.hpp"
#include "pie_hip_kernels.h"
#include "snapshot.hpp"

namespace pie_hip_driver {

#define PIE_HIP_CHECK(expr)                                                              \
    do {                                                                                 \
        hipError_t e_ = (expr);                                                          \
        if (e_ != hipSuccess)                                                            \
            throw std::runtime_error(std::string(#expr) + ": " + hipGetErrorString(e_)); \
    } while (0)

// f_i = base^(-2i/dims); with YaRN scaling f_i / factor above the pair that turns `slow` times
// over the original context, f_i below the one that turns `fast` times, a linear ramp between.
std::vector<double> rotary_frequencies(const RotarySpec& r) {
    std::vector<double> out(static_cast<size_t>(r.dims / 2));
    double lo = 0.0, hi = 0.0;
    if (r.yarn) {
        auto pair_with_turns = [&](double turns) {
            return r.dims * std::log(r.original / (2.0 * 3.14159265358979323846 * turns)) / (2.0 * std::log(r.base));
        };
        lo = std::max(std::floor(pair_with_turns(r.fast)), 0.0);
        hi = std::min(std::ceil(pair_with_turns(r.slow)), static_cast<double>(r.dims) - 1.0);
    }
    for (size_t i = 0; i < out.size(); ++i) {
        const double f = std::pow(r.base, -2.0 * static_cast<double>(i) / r.dims);
        out[i] = f;
        if (r.yarn) {
            const double ramp = std::min(1.0, std::max(0.0, (static_cast<double>(i) - lo) / std::max(hi - lo, 0.001)));
            out[i] = f / r.factor * ramp + f * (1.0 - ramp);
        }
    }
    return out;
}

float rotary_mscale(const RotarySpec& r) {
    return r.yarn ? static_cast<float>(0.1 * std::log(r.factor) + 1.0) : 1.f;
}

namespace {

// A checkpoint matrix on the host: bf16 bits [rows, cols].
struct HostMatrix {
    std::vector<uint16_t> v;
    int rows = 0, cols = 0;
    const uint16_t* row(int r) const { return v.data() + static_cast<size_t>(r) * cols; }
};

float bf16_value(uint16_t b) {
    const uint32_t u = static_cast<uint32_t>(b) << 16;
    float f;
    std::memcpy(&f, &u, 4);
    return f;
}

}  // namespace

void Model::load_stack(const ModelConfig& cfg, hipStream_t stream) {
    cfg_ = cfg;
    quant_ = Quant::Bf16;
    const bool random = cfg.random_weights;
    std::unique_ptr<Snapshot> snap;
    if (!random) snap = std::make_unique<Snapshot>(cfg.checkpoint_dir);
    std::uint64_t seed = cfg.seed;
    auto next_seed = [&]() { return seed += 0xA0761D6478BD642Full; };
    const int H = cfg.hidden, Hp = ld_x(), V = cfg.vocab;

    auto matrix = [&](const std::string& name, int rows, int cols) {
        const StTensor& t = snap->at(name);
        expect_shape(t, name, rows, cols);
        HostMatrix m;
        std::vector<uint16_t> staging;
        const uint16_t* p = as_bf16(t, staging);
        m.v.assign(p, p + t.elems());
        m.rows = rows;
        m.cols = cols;
        return m;
    };
    // fp32 vector parameter; `dflt` fills it for random weights, `map` changes its values
    auto identity = [](float v) { return v; };
    auto vec_mapped = [&](const std::string& name, size_t n, auto dflt, auto map) {
        std::vector<float> v(n);
        if (random) {
            for (size_t i = 0; i < n; ++i) v[i] = dflt(i);
        } else {
            const StTensor& t = snap->at(name);
            if (t.elems() != static_cast<int64_t>(n)) throw std::runtime_error("snapshot: tensor '" + name + "' has an unexpected shape");
            if (t.dtype == "F32") {   // kept to the last bit
                std::memcpy(v.data(), t.data, 4 * n);
            } else {
                std::vector<uint16_t> staging;
                const uint16_t* p = as_bf16(t, staging);
                for (size_t i = 0; i < n; ++i) v[i] = bf16_value(p[i]);
            }
        }
        for (float& x : v) x = map(x);
        float* d = static_cast<float*>(alloc(4 * n, name));
        PIE_HIP_CHECK(hipMemcpyAsync(d, v.data(), 4 * n, hipMemcpyHostToDevice, stream));
        PIE_HIP_CHECK(hipStreamSynchronize(stream));
        return d;
    };
    auto vec = [&](const std::string& name, size_t n, auto dflt) { return vec_mapped(name, n, dflt, identity); };
    auto ones = [](size_t) { return 1.f; };
    auto upload = [&](uint16_t* dst, const std::vector<uint16_t>& host) {
        PIE_HIP_CHECK(hipMemcpyAsync(dst, host.data(), host.size() * 2, hipMemcpyHostToDevice, stream));
        PIE_HIP_CHECK(hipStreamSynchronize(stream));
    };
    auto device_matrix = [&](const std::string& name, size_t elems, int fan_in, auto fill) {
        auto* d = static_cast<uint16_t*>(alloc(elems * 2, name));
        if (random) {
            fill_normal(d, elems, next_seed(), 0.f, 0.7f / std::sqrt(static_cast<float>(fan_in)), stream);
        } else {
            std::vector<uint16_t> host(elems, 0);
            fill(host);
            upload(d, host);
        }
        return d;
    };
    // [N, K] zero-padded linear; fill(put) places checkpoint rows: put(row, first column, values, n)
    auto linear = [&](Linear& lin, const std::string& name, int N, int K, int fan_in, auto fill) {
        lin.kind = Quant::Bf16;
        lin.N = N;
        lin.K = K;
        lin.data = device_matrix(name, static_cast<size_t>(N) * K, fan_in, [&](std::vector<uint16_t>& host) {
            fill([&](int row, int col, const uint16_t* src, int n) {
                std::memcpy(host.data() + static_cast<size_t>(row) * K + col, src, static_cast<size_t>(n) * 2);
            });
        });
        decode_bytes_ += lin.data_bytes();
    };
    // rows [row0, row0 + rows) = the tensor's rows as they are
    auto plain_rows = [&](const auto& put, const std::string& name, int row0, int rows, int cols) {
        const HostMatrix m = matrix(name, rows, cols);
        for (int r = 0; r < rows; ++r) put(row0 + r, 0, m.row(r), cols);
    };
    auto rotary_of = [&](const RotarySpec& spec) {
        if (spec.dims == 0) return -1;
        for (size_t i = 0; i < rotary.size(); ++i)
            if (rotary[i].spec == spec) return static_cast<int>(i);
        RotaryTable t;
        t.spec = spec;
        t.mscale = rotary_mscale(spec);
        const std::vector<double> f = rotary_frequencies(spec);
        t.freq = static_cast<double*>(alloc(f.size() * 8, "rotary." + std::to_string(rotary.size())));
        PIE_HIP_CHECK(hipMemcpyAsync(t.freq, f.data(), f.size() * 8, hipMemcpyHostToDevice, stream));
        PIE_HIP_CHECK(hipStreamSynchronize(stream));
        rotary.push_back(t);
        return static_cast<int>(rotary.size()) - 1;
    };

    embed = device_matrix("embed", static_cast<size_t>(V) * H, 1,
                          [&](std::vector<uint16_t>& host) { host = matrix("embed", V, H).v; });
    linear(head, "head", pad_to(V, 16), Hp, H, [&](auto put) { plain_rows(put, "head", 0, V, H); });
    // a norm with one weight for all columns, spread over them
    auto scalar_norm = [&](const std::string& name) {
        float g = 1.f;
        if (!random) {
            const StTensor& t = snap->at(name);
            if (t.elems() != 1) throw std::runtime_error("snapshot: tensor '" + name + "' has an unexpected shape");
            std::vector<uint16_t> staging;
            if (t.dtype == "F32") std::memcpy(&g, t.data, 4);
            else g = bf16_value(as_bf16(t, staging)[0]);
        }
        const std::vector<float> v(static_cast<size_t>(H), g);
        float* d = static_cast<float*>(alloc(4 * v.size(), name));
        PIE_HIP_CHECK(hipMemcpyAsync(d, v.data(), 4 * v.size(), hipMemcpyHostToDevice, stream));
        PIE_HIP_CHECK(hipStreamSynchronize(stream));
        return d;
    };
    // a convolution's taps, one after the other: [width, taps] -> [taps, width]
    auto tap_major = [&](const std::string& name, int taps) {
        return device_matrix(name, static_cast<size_t>(taps) * H, taps, [&](std::vector<uint16_t>& host) {
            const HostMatrix m = matrix(name, H, taps);
            for (int c = 0; c < H; ++c)
                for (int j = 0; j < taps; ++j) host[static_cast<size_t>(j) * H + c] = m.row(c)[j];
        });
    };
    stack_norm = cfg.gated_sublayers ? scalar_norm("final.norm") : vec("final.norm", H, ones);
    if (cfg.gated_sublayers) embed_norm = scalar_norm("embed.norm");
    if (cfg.bigram.buckets > 0) {
        if (cfg.bigram.buckets >= (1ull << 31) - 1) throw std::runtime_error("model: too many bigram buckets");
        const int rows = static_cast<int>(cfg.bigram.buckets) + 1;
        bigram = device_matrix("bigram", static_cast<size_t>(rows) * H, 1, [&](std::vector<uint16_t>& host) { host = matrix("bigram", rows, H).v; });
    }

    runs = cfg.layer_runs();
    if (cfg.loop.stop > cfg.loop.start)
        loop_step = vec("loop.step", static_cast<size_t>(cfg.loop.times) * H, [](size_t) { return 0.f; });
    stack.resize(cfg.stack.size());
    for (size_t l = 0; l < stack.size(); ++l) {
        StackLayer& w = stack[l];
        w.spec = cfg.stack[l];
        // a gated pair of matrices as rows (gate_0, up_0, gate_1, ..)
        auto paired_rows = [&](const auto& put, const std::string& at, int row0, int ff) {
            int half = 0;
            for (const char* name : {"gate", "up"}) {
                const HostMatrix mat = matrix(at + name, ff, H);
                for (int r = 0; r < ff; ++r) put(row0 + 2 * r + half, 0, mat.row(r), H);
                ++half;
            }
        };
        const char *post1 = cfg.sandwich_norms ? "norm1b" : "norm1", *post2 = cfg.sandwich_norms ? "norm2b" : "norm2";
        const std::string p = "l" + std::to_string(l) + ".", mix = p + "mix.";
        // what surrounds sublayer n of a gated pair
        auto gated_sublayer = [&](const std::string& n, float*& norm, uint16_t*& canon, Linear& gate, float*& bias) {
            norm = scalar_norm(p + "norm" + n);
            canon = tap_major(p + "canon" + n, cfg.canon_taps);
            linear(gate, p + "rg" + n, Hp, Hp, H, [&](auto put) { plain_rows(put, p + "rg" + n, 0, H, H); });
            bias = vec(p + "rg" + n + ".b", H, [](size_t) { return 0.f; });
        };
        if (cfg.gated_sublayers) {
            gated_sublayer("1", w.pre1, w.canon1, w.w_gate1, w.gate1_bias);
            if (w.spec.ff > 0 || w.spec.moe.experts > 0) gated_sublayer("2", w.pre2, w.canon2, w.w_gate2, w.gate2_bias);
        } else if (!cfg.shared_norm) w.norm1 = vec(p + post1, H, ones);
        if (cfg.sandwich_norms || cfg.shared_norm) w.pre1 = vec(p + "norm1", H, ones);
        if (w.spec.mixer == MixerKind::LatentAttention) {
            const LatentAttentionSpec& a = w.spec.latent;
            const LatentShape s(a);
            w.rotary = rotary_of(a.rot);
            w.q_norm = vec(mix + "dq.norm", a.q_rank, ones);
            if (a.kv_from < 0) w.kv_norm = vec(mix + "dkv.norm", a.kv_rank, ones);
            // The kernels rotate neighbours: of half-split vectors entry i goes to place 2 i and entry i + dims / 2 to
            // 2 i + 1, in queries and keys alike (scores do not change).
            auto rotated_place = [&](int i) {
                const int half = a.rot.dims / 2;
                return !a.half_split || i >= a.rot.dims ? i : i < half ? 2 * i : 2 * (i - half) + 1;
            };
            linear(w.w_in, mix + "in", s.ld_in, Hp, H, [&](auto put) {
                plain_rows(put, mix + "dq", 0, a.q_rank, H);
                if (a.kv_from < 0) {
                    const HostMatrix m = matrix(mix + "dkv", a.kv_rank + a.rot_dim, H);
                    for (int r = 0; r < a.kv_rank + a.rot_dim; ++r)
                        put(s.kv_off + (r < a.kv_rank ? r : a.kv_rank + rotated_place(r - a.kv_rank)), 0, m.row(r), H);
                }
                if (a.gate == OutputGate::PerHead) plain_rows(put, mix + "g", s.gate_off, a.heads, H);
                if (a.gate == OutputGate::PerValue) {
                    const HostMatrix m = matrix(mix + "g", a.heads * a.vdim, H);
                    for (int r = 0; r < a.heads * a.vdim; ++r) put(s.gate_off + r / a.vdim * s.vdp + r % a.vdim, 0, m.row(r), H);
                }
            });
            linear(w.w_uq, mix + "uq", s.ld_q, s.ld_cq, a.q_rank, [&](auto put) {
                const HostMatrix m = matrix(mix + "uq", a.heads * (a.dim + a.rot_dim), a.q_rank);
                for (int h = 0; h < a.heads; ++h)
                    for (int i = 0; i < a.dim + a.rot_dim; ++i)
                        put(h * s.hd + (i < a.dim ? i : s.dimp + rotated_place(i - a.dim)), 0, m.row(h * (a.dim + a.rot_dim) + i), a.q_rank);
            });
            if (a.sinks) w.sinks = vec(mix + "sink", a.heads, [](size_t) { return 0.f; });
            HostMatrix uk, uv;
            if (!random) {
                uk = matrix(mix + "uk", a.heads * a.dim, a.kv_rank);
                uv = matrix(mix + "uv", a.heads * a.vdim, a.kv_rank);
            }
            w.w_uk_t = device_matrix(mix + "uk_t", static_cast<size_t>(a.heads) * s.kvp * s.dimp, a.dim,
                                     [&](std::vector<uint16_t>& host) {
                                         for (int h = 0; h < a.heads; ++h)
                                             for (int d = 0; d < a.dim; ++d)
                                                 for (int r = 0; r < a.kv_rank; ++r)
                                                     host[(static_cast<size_t>(h) * s.kvp + r) * s.dimp + d] = uk.row(h * a.dim + d)[r];
                                     });
            w.w_uv = device_matrix(mix + "uv", static_cast<size_t>(a.heads) * s.vdp * s.kvp, a.kv_rank,
                                   [&](std::vector<uint16_t>& host) {
                                       for (int h = 0; h < a.heads; ++h)
                                           for (int c = 0; c < a.vdim; ++c)
                                               std::memcpy(&host[(static_cast<size_t>(h) * s.vdp + c) * s.kvp],
                                                           uv.row(h * a.vdim + c), static_cast<size_t>(a.kv_rank) * 2);
                                   });
            const size_t before = decode_bytes_;
            linear(w.w_ukv, mix + "ukv", a.heads * (s.dimp + s.vdp), s.kvp, a.kv_rank, [&](auto put) {
                for (int h = 0; h < a.heads; ++h) {
                    for (int d = 0; d < a.dim; ++d) put(h * (s.dimp + s.vdp) + d, 0, uk.row(h * a.dim + d), a.kv_rank);
                    for (int c = 0; c < a.vdim; ++c)
                        put(h * (s.dimp + s.vdp) + s.dimp + c, 0, uv.row(h * a.vdim + c), a.kv_rank);
                }
            });
            decode_bytes_ = before + static_cast<size_t>(a.heads) * s.kvp * (s.dimp + s.vdp) * 2;   // (decode reads uk_t and uv instead)
            linear(w.wo, mix + "o", Hp, s.ld_o, a.heads * a.vdim, [&](auto put) {
                const HostMatrix m = matrix(mix + "o", H, a.heads * a.vdim);
                for (int r = 0; r < H; ++r)
                    for (int h = 0; h < a.heads; ++h) put(r, h * s.vdp, m.row(r) + h * a.vdim, a.vdim);
            });
        } else if (w.spec.mixer == MixerKind::ChannelDelta) {
            ChannelDeltaSpec& d = w.spec.delta;
            // the ranks of the decay and the output gate are the shapes of their first factors
            auto rank_of = [&](const std::string& name, int dflt) {
                if (random) return dflt;
                const StTensor& t = snap->at(name);
                if (t.shape.size() != 2 || t.shape[0] <= 0 || t.shape[0] > (1 << 20))
                    throw std::runtime_error("snapshot: tensor '" + name + "' has an unexpected shape");
                return static_cast<int>(t.shape[0]);
            };
            d.decay_rank = rank_of(mix + "a1", d.decay_rank > 0 ? d.decay_rank : d.dim);
            d.gate_rank = rank_of(mix + "g1", d.gate_rank > 0 ? d.gate_rank : d.vdim);
            const DeltaShape s(d);
            linear(w.w_in, mix + "in", s.ld_in, Hp, H, [&](auto put) {
                plain_rows(put, mix + "q", 0, s.kd, H);
                plain_rows(put, mix + "k", s.kd, s.kd, H);
                plain_rows(put, mix + "v", 2 * s.kd, s.vd, H);
                plain_rows(put, mix + "b", s.channels, d.heads, H);
                plain_rows(put, mix + "a1", s.decay_off, d.decay_rank, H);
                plain_rows(put, mix + "g1", s.gate_off, d.gate_rank, H);
            });
            auto low_rank = [&](const std::string& name, int rows, int rank, int ld) {
                decode_bytes_ += static_cast<size_t>(rows) * ld * 2;
                return device_matrix(name, static_cast<size_t>(rows) * ld, rank, [&](std::vector<uint16_t>& host) {
                    const HostMatrix m = matrix(name, rows, rank);
                    for (int r = 0; r < rows; ++r) std::memcpy(&host[static_cast<size_t>(r) * ld], m.row(r), static_cast<size_t>(rank) * 2);
                });
            };
            w.w_decay = low_rank(mix + "a2", d.heads * d.dim, d.decay_rank, s.ld_a1);
            w.w_gate = low_rank(mix + "g2", s.vd, d.gate_rank, s.ld_g1);
            linear(w.wo, mix + "o", Hp, s.ld_o, s.vd, [&](auto put) { plain_rows(put, mix + "o", 0, H, s.vd); });
            w.decay_rate = vec_mapped(mix + "A_log", d.heads, [&](size_t i) { return std::log(1.f + static_cast<float>(i % 8)); },
                               [](float v) { return static_cast<float>(-std::exp(static_cast<double>(v)) * 1.4426950408889634074); });
            w.dt_bias = vec(mix + "dt_bias", static_cast<size_t>(d.heads) * d.dim, [](size_t) { return -3.f; });
            w.out_norm = vec(mix + "norm", d.vdim, ones);
            // the three convolutions back to back, [channels, taps]
            std::vector<float> conv(static_cast<size_t>(s.channels) * d.taps, 0.5f);
            if (!random) {
                size_t at = 0;
                for (const auto& [name, ch] : {std::pair<const char*, int>{"q", s.kd}, {"k", s.kd}, {"v", s.vd}}) {
                    const HostMatrix m = matrix(mix + name + ".conv", ch, d.taps);
                    for (uint16_t b : m.v) conv[at++] = bf16_value(b);
                }
            }
            w.conv_w = static_cast<float*>(alloc(conv.size() * 4, mix + "conv"));
            PIE_HIP_CHECK(hipMemcpyAsync(w.conv_w, conv.data(), conv.size() * 4, hipMemcpyHostToDevice, stream));
            PIE_HIP_CHECK(hipStreamSynchronize(stream));
        }
        if (w.spec.has_attn() || w.spec.has_memory()) {
            const MixShape s(w.spec);
            const GroupAttentionSpec& a = w.spec.attn;
            const DecayMemorySpec& d = w.spec.memory;
            const int kd = d.kv_heads * d.dim, vd = d.heads * d.vdim;
            const bool both = w.spec.has_attn() && w.spec.has_memory();
            const std::string left = both ? mix + "left." : mix, mem = both ? mix + "right." : mix;
            const bool ssm = w.spec.has_memory() && d.kind == DecayKind::StateSpace;
            if (w.spec.has_attn()) {
                w.rotary = rotary_of(a.rot);
                auto zeros = [](size_t) { return 0.f; };
                const size_t qd = static_cast<size_t>(a.heads) * a.dim, kd_attn = static_cast<size_t>(a.kv_heads) * a.dim;
                if (a.biases) {
                    w.q_bias = vec(left + "q.b", qd, zeros);
                    w.k_bias = vec(left + "k.b", kd_attn, zeros);
                }
                if (a.norm != QueryKeyNorm::None) {
                    const bool whole = a.norm == QueryKeyNorm::WholeProjection;
                    w.q_norm = vec(left + "q.norm", whole ? qd : a.dim, ones);
                    w.k_norm = vec(left + "k.norm", whole ? kd_attn : a.dim, ones);
                }
            }
            // a state-space checkpoint's one projection: gate | values | keys | queries | step sizes
            HostMatrix in;
            if (ssm && !random) in = matrix(mem + "in", 2 * vd + 2 * kd + d.heads, H);
            linear(w.w_in, mix + "in", s.ld_in, Hp, H, [&](auto put) {
                if (w.spec.has_attn()) {
                    plain_rows(put, left + "q", s.q_off, a.heads * a.dim, H);
                    plain_rows(put, left + "k", s.k_off, a.kv_heads * a.dim, H);
                    if (a.own_values) plain_rows(put, left + "v", s.v_off, a.kv_heads * a.vdim, H);
                    if (a.gate) {
                        const HostMatrix m = matrix(left + "g", a.heads * a.vdim, H);
                        for (int r = 0; r < a.heads * a.vdim; ++r) put(s.attn_gate_off + r / a.vdim * s.dimp + r % a.vdim, 0, m.row(r), H);
                    }
                }
                if (ssm) {
                    for (int r = 0; r < s.channels; ++r) put(s.mv_off + r, 0, in.row(vd + r), H);
                    for (int r = 0; r < vd; ++r) put(s.gate_off + r, 0, in.row(r), H);
                } else if (w.spec.has_memory()) {
                    plain_rows(put, mem + "q", s.mq_off, kd, H);
                    plain_rows(put, mem + "k", s.mk_off, kd, H);
                    plain_rows(put, mem + "v", s.mv_off, vd, H);
                    plain_rows(put, mem + "g", s.gate_off, vd, H);
                }
            });
            if (s.gates) {
                decode_bytes_ += static_cast<size_t>(s.gates) * Hp * 2;
                w.w_gates = device_matrix(mix + "gates", static_cast<size_t>(s.gates) * Hp, H, [&](std::vector<uint16_t>& host) {
                    auto rows = [&](const HostMatrix& m, int from, int to) {
                        for (int r = 0; r < d.heads; ++r)
                            std::memcpy(&host[static_cast<size_t>(to + r) * Hp], m.row(from + r), static_cast<size_t>(H) * 2);
                    };
                    if (ssm) {
                        rows(in, vd + s.channels, 0);
                    } else {
                        rows(matrix(mem + "i", d.heads, H), 0, 0);
                        rows(matrix(mem + "f", d.heads, H), 0, d.heads);
                    }
                });
            }
            auto upload_f32 = [&](const std::string& name, const std::vector<float>& v) {
                float* dst = static_cast<float*>(alloc(v.size() * 4, name));
                PIE_HIP_CHECK(hipMemcpyAsync(dst, v.data(), v.size() * 4, hipMemcpyHostToDevice, stream));
                PIE_HIP_CHECK(hipStreamSynchronize(stream));
                return dst;
            };
            if (w.spec.has_memory() && d.kind == DecayKind::Retention) {
                // (a decay of 0 becomes a power of two that is 0 in fp32)
                std::vector<float> lg;
                for (double v : d.decay) lg.push_back(v > 0.0 ? static_cast<float>(std::max(std::log2(v), -1000.0)) : -1000.f);
                w.decay_log2 = upload_f32("", lg);
            } else if (w.spec.has_memory() && d.kind == DecayKind::MatrixLstm) {
                std::vector<float> b(static_cast<size_t>(2 * d.heads), 0.f);
                if (random) {
                    std::fill(b.begin() + d.heads, b.end(), 3.f);
                } else {
                    size_t at = 0;
                    for (const char* n : {"i.b", "f.b"}) {
                        const StTensor& t = snap->at(mem + n);
                        expect_shape(t, mem + n, d.heads, -1);
                        std::vector<uint16_t> staging;
                        const uint16_t* src = as_bf16(t, staging);
                        for (int h = 0; h < d.heads; ++h) b[at++] = bf16_value(src[h]);
                    }
                }
                w.gate_bias = upload_f32("", b);
                w.out_norm = vec(mem + "norm", vd, ones);
            } else if (ssm) {
                w.decay_log2 = vec_mapped(mem + "A_log", d.heads, [&](size_t i) { return std::log(1.f + static_cast<float>(i % 8)); },
                                          [](float v) { return static_cast<float>(-std::exp(static_cast<double>(v)) * 1.4426950408889634074); });
                w.gate_bias = vec(mem + "dt_bias", d.heads, [](size_t) { return -3.f; });
                w.skip = vec(mem + "D", d.heads, ones);
                w.out_norm = vec(mem + "norm", vd, ones);
                w.conv_b = vec(mem + "conv.b", s.channels, [](size_t) { return 0.f; });
                w.conv_w = vec(mem + "conv", static_cast<size_t>(s.channels) * d.taps, [](size_t) { return 0.5f; });
            }
            linear(w.wo, mix + "o", Hp, s.ld_o, a.heads * a.vdim + vd, [&](auto put) {
                if (w.spec.has_attn()) {
                    const HostMatrix m = matrix(left + "o", H, a.heads * a.vdim);
                    for (int r = 0; r < H; ++r)
                        for (int h = 0; h < a.heads; ++h) put(r, h * s.dimp, m.row(r) + h * a.vdim, a.vdim);
                }
                if (w.spec.has_memory()) {
                    const HostMatrix m = matrix(mem + "o", H, vd);
                    for (int r = 0; r < H; ++r) put(r, s.out_off, m.row(r), vd);
                }
            });
        }
        if (w.spec.moe.experts > 0) {
            const MixtureSpec& e = w.spec.moe;
            const int ff = e.ff, ffp = e.padded_ff(), rows = pad_to(e.router_columns(), 16), parts = e.shared_parts();
            const std::string sh = p + "mlp.shared.";
            decode_bytes_ += static_cast<size_t>(rows) * Hp * 2;
            w.w_router = device_matrix(p + "mlp.router", static_cast<size_t>(rows) * Hp, H, [&](std::vector<uint16_t>& host) {
                const HostMatrix m = matrix(p + "mlp.router", e.experts, H);
                for (int r = 0; r < e.experts; ++r) std::memcpy(&host[static_cast<size_t>(r) * Hp], m.row(r), static_cast<size_t>(H) * 2);
                if (parts) std::memcpy(&host[static_cast<size_t>(e.experts) * Hp], matrix(sh + "sg", 1, H).row(0), static_cast<size_t>(H) * 2);
            });
            if (e.router == RouterKind::CorrectedScores) w.correction = vec(p + "mlp.correction", e.experts, [](size_t) { return 0.f; });
            const bool pair = e.expert == ExpertKind::ClampedPair;
            const int up_rows = (pair ? 2 : 1) * ffp;   // of an expert
            linear(w.w_up, p + "mlp.experts.up", e.all_experts() * up_rows, Hp, H, [&](auto put) {
                if (parts) {   // (part i's rows follow part i - 1's: up_rows is ffp for experts of one matrix)
                    if (pair) throw std::runtime_error("model: shared experts are of one matrix");
                    plain_rows(put, sh + "up", 0, e.shared_ff, H);
                }
                for (int i = 0; i < e.experts; ++i) {
                    const std::string at = p + "mlp.e" + std::to_string(i) + ".";
                    if (pair) paired_rows(put, at, (parts + i) * up_rows, ff);
                    else plain_rows(put, at + "up", (parts + i) * up_rows, ff, H);
                }
            });
            linear(w.w_down, p + "mlp.experts.down", e.all_experts() * Hp, ffp, ff, [&](auto put) {
                if (parts) {
                    const HostMatrix m = matrix(sh + "down", H, e.shared_ff);
                    for (int i = 0; i < parts; ++i)
                        for (int r = 0; r < H; ++r) put(i * Hp + r, 0, m.row(r) + i * ffp, std::min(ffp, e.shared_ff - i * ffp));
                }
                for (int i = 0; i < e.experts; ++i) plain_rows(put, p + "mlp.e" + std::to_string(i) + ".down", (parts + i) * Hp, H, ff);
            });
        } else if (w.spec.ff > 0 && cfg.ff_act == FeedForwardAct::GatedSilu) {
            const int ff = w.spec.ff, ffp = pad_to(ff, 128);
            linear(w.w_up, p + "mlp.up", 2 * ffp, Hp, H, [&](auto put) { paired_rows(put, p + "mlp.", 0, ff); });
            linear(w.w_down, p + "mlp.down", Hp, ffp, ff, [&](auto put) { plain_rows(put, p + "mlp.down", 0, H, ff); });
            if (!cfg.ff_biases) continue;   // (nothing else of the layer is left to load)
            std::vector<float> b(static_cast<size_t>(2 * ffp), 0.f);
            if (!random) {
                int half = 0;
                for (const char* name : {"mlp.gate.b", "mlp.up.b"}) {
                    const StTensor& t = snap->at(p + name);
                    expect_shape(t, p + name, ff, -1);
                    std::vector<uint16_t> staging;
                    const uint16_t* src = as_bf16(t, staging);
                    for (int r = 0; r < ff; ++r) b[static_cast<size_t>(2 * r + half)] = bf16_value(src[r]);
                    ++half;
                }
            }
            w.up_bias = static_cast<float*>(alloc(b.size() * 4, ""));
            PIE_HIP_CHECK(hipMemcpyAsync(w.up_bias, b.data(), b.size() * 4, hipMemcpyHostToDevice, stream));
            PIE_HIP_CHECK(hipStreamSynchronize(stream));
            w.down_bias = vec(p + "mlp.down.b", H, [](size_t) { return 0.f; });
        } else if (w.spec.ff > 0) {
            const int ff = w.spec.ff, ffp = pad_to(ff, 128);
            if (!cfg.shared_norm) w.norm2 = vec(p + post2, H, ones);
            if (cfg.sandwich_norms) w.pre2 = vec(p + "norm2", H, ones);
            linear(w.w_up, p + "mlp.up", ffp, Hp, H, [&](auto put) { plain_rows(put, p + "mlp.up", 0, ff, H); });
            linear(w.w_down, p + "mlp.down", Hp, ffp, ff, [&](auto put) { plain_rows(put, p + "mlp.down", 0, H, ff); });
        }
    }
    PIE_HIP_CHECK(hipStreamSynchronize(stream));
}

}  // namespace pie_hip_driver
