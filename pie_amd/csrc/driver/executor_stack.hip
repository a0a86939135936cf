// Layer stacks in the executor: workspaces, recurrent-state slots, and the forward body of models
// whose layers are listed one by one (ModelConfig::stack).
#include <algorithm>
#include <cmath>
#include <cstring>
#include <set>
#include <stdexcept>
#include <string>

#include "executor.hpp"
#include "pie_hip_kernels.h"

namespace pie_hip_driver {

#define PIE_HIP_CHECK(expr)                                                              \
    do {                                                                                 \
        hipError_t e_ = (expr);                                                          \
        if (e_ != hipSuccess)                                                            \
            throw std::runtime_error(std::string(#expr) + ": " + hipGetErrorString(e_)); \
    } while (0)

#define PIE_KERNEL(expr)                                                                     \
    do {                                                                                     \
        const int st_ = (expr);                                                              \
        if (st_ != PIE_HIP_OK)                                                               \
            throw std::runtime_error(std::string(#expr) + " failed with status " +          \
                                     std::to_string(st_));                                   \
    } while (0)

// Workspaces at their largest over the layers, and the recurrent-state pool.
void Executor::alloc_stack() {
    const ModelConfig& m = model_.cfg();
    const size_t T = static_cast<size_t>(max_tokens_), esize = m.f32() ? 4 : 2;
    const size_t ld_x = static_cast<size_t>(model_.ld_x());
    size_t in = 0, cq = 0, q = 0, q_lat = 0, o_lat = 0, o = 0, act = 0, gate = 0;
    size_t kd = 0, vd = 0, gd = 0, heads = 0, state = 0;
    size_t conv = 0, gates = 0, mem_o = 0, den = 0, head_pad = 0;
    size_t y2 = 0, top = 0, router = 0, experts = 0, glu = 0;
    auto up = [](size_t& v, int n) { v = std::max(v, static_cast<size_t>(n)); };
    auto place = [&](size_t bytes) {
        const size_t at = state;
        state = (state + bytes + 255) / 256 * 256;
        return at;
    };
    for (const LayerRun& run : model_.runs) {
        const StackLayer& l = model_.stack[static_cast<size_t>(run.layer)];
        rs_state_off_.push_back(0);
        rs_conv_off_.push_back(0);
        rs_canon_off_.push_back({0, 0});
        if (m.gated_sublayers)
            for (int n = 0; n < (l.pre2 ? 2 : 1) && m.canon_taps > 1; ++n)
                rs_canon_off_.back()[n] = place(static_cast<size_t>(m.canon_taps - 1) * m.hidden * esize);
        up(act, l.spec.ff > 0 ? pad_to(l.spec.ff, 128) : 0);
        if (m.shared_norm && l.spec.ff > 0) up(y2, model_.ld_x());
        if (m.ff_act == FeedForwardAct::GatedSilu && l.spec.ff > 0) up(glu, 2 * pad_to(l.spec.ff, 128));
        if (l.spec.moe.experts > 0) {
            const MixtureSpec& e = l.spec.moe;
            up(act, e.routes() * e.padded_ff());
            if (e.expert == ExpertKind::ClampedPair) up(glu, 2 * e.routes() * e.padded_ff());
            up(top, e.routes());
            up(router, pad_to(e.router_columns(), 16));
            up(experts, e.all_experts());
        }
        if (l.spec.mixer == MixerKind::LatentAttention) {
            const LatentShape s(l.spec.latent);
            up(in, s.ld_in);
            up(cq, s.ld_cq);
            up(q, s.ld_q);
            up(q_lat, s.heads * s.ld_row);
            up(o_lat, s.heads * s.kvp);
            up(o, s.ld_o);
        } else if (l.spec.mixer == MixerKind::ChannelDelta) {
            const ChannelDeltaSpec& d = l.spec.delta;
            const DeltaShape s(d);
            up(in, s.ld_in);
            up(o, s.ld_o);
            up(gate, s.ld_gate);
            up(kd, s.kd);
            up(vd, s.vd);
            up(gd, d.heads * d.dim);
            up(heads, d.heads);
            rs_state_off_.back() = place(static_cast<size_t>(d.heads) * d.dim * d.vdim * 4);
            rs_conv_off_.back() = place(static_cast<size_t>(d.taps - 1) * s.channels * esize);
        } else {
            const MixShape s(l.spec);
            const DecayMemorySpec& d = l.spec.memory;
            up(in, s.ld_in);
            up(o, s.ld_o);
            if (l.spec.has_attn()) {
                up(q, l.spec.attn.heads * s.dimp);
                up(head_pad, s.dimp);
            }
            if (l.spec.has_memory()) {
                up(conv, s.ld_conv);
                up(gates, s.gates);
                up(mem_o, d.heads * d.vdim);
                up(den, 2 * d.heads);
                const size_t per_head = static_cast<size_t>(d.dim) * d.vdim + (d.kind == DecayKind::MatrixLstm ? d.dim + 1 : 0);
                rs_state_off_.back() = place(d.heads * per_head * 4);
                if (s.channels) rs_conv_off_.back() = place(static_cast<size_t>(d.taps - 1) * s.channels * esize);
            }
        }
    }
    if (m.bigram.buckets > 0 && state == 0) place(4);   // (a request's previous token is state: it needs a slot)
    // Zeroed: columns that pad a row to its product's K are written by nobody.
    auto take = [&](size_t bytes) {
        void* p = nullptr;
        PIE_HIP_CHECK(hipMalloc(&p, std::max<size_t>(bytes, 16)));
        stack_.allocs.push_back(p);
        PIE_HIP_CHECK(hipMemsetAsync(p, 0, std::max<size_t>(bytes, 16), stream_));
        return p;
    };
    auto f32 = [&](size_t n) { return static_cast<float*>(take(n * 4)); };
    auto compute = [&](size_t n) { return take(n * esize); };
    stack_.x = f32(T * ld_x);
    stack_.xa = compute(T * ld_x);
    stack_.in = compute(T * in);
    stack_.y = compute(T * ld_x);
    stack_.cq = compute(T * cq);
    stack_.q = compute(T * q);
    stack_.q_lat = compute(T * q_lat);
    stack_.o_lat = compute(T * o_lat);
    stack_.o = compute(T * o);
    stack_.act = compute(T * act);
    stack_.gate = compute(T * gate);
    stack_.y2 = compute(T * y2);
    if (m.gated_sublayers) {
        stack_.h = compute(T * ld_x);
        stack_.sub_gate = compute(T * ld_x);
    }
    if (top) {
        stack_.routes = compute(T * top * ld_x);
        stack_.router = f32(T * router);
        stack_.route_w = f32(T * top);
        auto i32 = [&](size_t n) { return static_cast<int32_t*>(take(n * 4)); };
        stack_.route_idx = i32(T * top);
        stack_.route_offsets = i32(experts + 1);
        stack_.route_token = i32(T * top);
        stack_.route_pos = i32(T * top);
    }
    if (m.f32()) stack_.glu = f32(T * glu);
    stack_.dq = f32(T * kd);
    stack_.dk = f32(T * kd);
    stack_.dv = f32(T * vd);
    stack_.dg = f32(T * gd);
    stack_.d_beta = f32(T * heads);
    stack_.d_o = f32(T * vd);
    stack_.conv = compute(T * conv);
    stack_.gates = f32(T * gates);
    stack_.mem_o = f32(T * mem_o);
    stack_.den = f32(T * den);
    const size_t srows = std::min<size_t>(T, 2 * static_cast<size_t>(cfg_.batching.max_forward_requests));
    stack_.xs = compute(srows * ld_x);
    stack_.raw_logits = compute(srows * static_cast<size_t>(model_.head.N));
    stack_.logits = f32(srows * static_cast<size_t>(m.vocab));
    for (const RotaryTable& r : model_.rotary) stack_.rotary.push_back(f32(T * static_cast<size_t>(r.spec.dims)));
    for (StackLayer& l : model_.stack)
        for (const Linear* w : {&l.w_in, &l.w_uq, &l.wo, &l.w_gate1, l.spec.moe.experts ? &l.wo : &l.w_up, l.spec.moe.experts ? &l.wo : &l.w_down})
            for (int rows : {64, 128})
                if (!m.f32() && w->data && w->K % 64 == 0)
                    gemm_ws_bytes_ = std::max(gemm_ws_bytes_, pie_hip_gemm_mfma_workspace_bytes(rows, w->N, w->K));
    gemm_ws_bytes_ = std::min<size_t>(gemm_ws_bytes_, size_t(64) << 20);
    if (gemm_ws_bytes_) PIE_HIP_CHECK(hipMalloc(&gemm_ws_, gemm_ws_bytes_));
    // partial results of the attentions' splits: a plan with more than one split has at most 512 (tile,
    // split) blocks of 32 (token, head) pairs (latent) or 16 heads (grouped)
    if (o_lat && !m.f32()) {
        size_t kvp = 0;
        for (const StackLayer& l : model_.stack)
            if (l.spec.mixer == MixerKind::LatentAttention) up(kvp, LatentShape(l.spec.latent).kvp);
        attn_ws_bytes_ = 512 * 32 * (kvp + 2) * sizeof(float);
    }
    if (head_pad && !m.f32()) attn_ws_bytes_ = std::max(attn_ws_bytes_, 512 * 16 * (head_pad + 2) * sizeof(float));
    if (attn_ws_bytes_) PIE_HIP_CHECK(hipMalloc(&attn_ws_, attn_ws_bytes_));
    rs_stride_ = state;
    if (state) {
        rs_slots_ = cfg_.batching.rs_cache_slots;
        cpu_rs_slots_ = cfg_.batching.cpu_rs_slots;
        void* p = nullptr;
        PIE_HIP_CHECK(hipMalloc(&p, state * static_cast<size_t>(rs_slots_)));
        rs_base_ = static_cast<unsigned char*>(p);
        PIE_HIP_CHECK(hipMemsetAsync(rs_base_, 0, state * static_cast<size_t>(rs_slots_), stream_));
        if (cpu_rs_slots_ > 0) {
            PIE_HIP_CHECK(hipHostMalloc(&p, state * static_cast<size_t>(cpu_rs_slots_), hipHostMallocDefault));
            rs_host_ = static_cast<unsigned char*>(p);
            std::memset(rs_host_, 0, state * static_cast<size_t>(cpu_rs_slots_));
        }
        rs_pos_.assign(static_cast<size_t>(rs_slots_), -1);
        rs_host_pos_.assign(static_cast<size_t>(cpu_rs_slots_), -1);
        rs_last_.assign(static_cast<size_t>(rs_slots_), -1);
        rs_host_last_.assign(static_cast<size_t>(cpu_rs_slots_), -1);
    }
    PIE_HIP_CHECK(hipStreamSynchronize(stream_));
}

// Whole slots move, with the number of tokens their state has seen.
void Executor::copy_rs_d2d(const uint32_t* srcs, const uint32_t* dsts, size_t n) {
    for (size_t i = 0; i < n; ++i) {
        if (srcs[i] == dsts[i]) continue;
        PIE_HIP_CHECK(hipMemcpyAsync(rs_base_ + dsts[i] * rs_stride_, rs_base_ + srcs[i] * rs_stride_, rs_stride_,
                                     hipMemcpyDeviceToDevice, stream_));
        rs_pos_[dsts[i]] = rs_pos_[srcs[i]];
        rs_last_[dsts[i]] = rs_last_[srcs[i]];
    }
    PIE_HIP_CHECK(hipStreamSynchronize(stream_));
}
void Executor::copy_rs_d2h(const uint32_t* srcs, const uint32_t* dsts, size_t n) {
    for (size_t i = 0; i < n; ++i) {
        PIE_HIP_CHECK(hipMemcpyAsync(rs_host_ + dsts[i] * rs_stride_, rs_base_ + srcs[i] * rs_stride_, rs_stride_,
                                     hipMemcpyDeviceToHost, stream_));
        rs_host_pos_[dsts[i]] = rs_pos_[srcs[i]];
        rs_host_last_[dsts[i]] = rs_last_[srcs[i]];
    }
    PIE_HIP_CHECK(hipStreamSynchronize(stream_));
}
void Executor::copy_rs_h2d(const uint32_t* srcs, const uint32_t* dsts, size_t n) {
    for (size_t i = 0; i < n; ++i) {
        PIE_HIP_CHECK(hipMemcpyAsync(rs_base_ + dsts[i] * rs_stride_, rs_host_ + srcs[i] * rs_stride_, rs_stride_,
                                     hipMemcpyHostToDevice, stream_));
        rs_pos_[dsts[i]] = rs_host_pos_[srcs[i]];
        rs_last_[dsts[i]] = rs_host_last_[srcs[i]];
    }
    PIE_HIP_CHECK(hipStreamSynchronize(stream_));
}
void Executor::copy_rs_h2h(const uint32_t* srcs, const uint32_t* dsts, size_t n) {
    for (size_t i = 0; i < n; ++i) {
        std::memmove(rs_host_ + dsts[i] * rs_stride_, rs_host_ + srcs[i] * rs_stride_, rs_stride_);
        rs_host_pos_[dsts[i]] = rs_host_pos_[srcs[i]];
        rs_host_last_[dsts[i]] = rs_host_last_[srcs[i]];
    }
}

// What a stack refuses, the state slots of the batch's requests and which of them start from zero.
void Executor::prepare_stack(const BatchPlan& plan, const Inputs& in) {
    if (plan.has_user_masks) throw std::runtime_error("executor: layer stacks take no custom attention masks");
    auto* row_req = reinterpret_cast<int32_t*>(in_host_ + in.off_row_req);
    auto* pair = reinterpret_cast<int32_t*>(in_host_ + in.off_pair);
    const BigramSpec& bigram = model_.cfg().bigram;
    auto pair_row = [&](int32_t before, uint32_t token) {   // (before < 0: a sequence's first token)
        if (bigram.buckets == 0) return 0;
        if (before < 0) return static_cast<int32_t>(bigram.buckets);
        return static_cast<int32_t>((static_cast<uint64_t>(before) * bigram.mul_prev + static_cast<uint64_t>(token) * bigram.mul_cur) % bigram.buckets);
    };
    auto* qo = reinterpret_cast<int32_t*>(in_host_ + in.off_qo);
    auto* slot = reinterpret_cast<int32_t*>(in_host_ + in.off_rs_slot);
    auto* fresh = reinterpret_cast<int32_t*>(in_host_ + in.off_rs_fresh);
    const bool recurrent = rs_slots_ > 0;
    if (recurrent && static_cast<int>(plan.rs_slots.size()) != plan.R)
        throw std::runtime_error("executor: this model needs a recurrent-state slot per request (rs_slot_ids)");
    std::set<uint32_t> seen;   // (a slot's state is read and written by one request of a batch)
    for (int r = 0; r < plan.R; ++r) {
        const int q0 = plan.qo_indptr[r], q1 = plan.qo_indptr[r + 1];
        qo[r] = q0;
        for (int i = q0; i < q1; ++i) {
            row_req[i] = r;
            pair[i] = pair_row(i > q0 ? static_cast<int32_t>(plan.tokens[i - 1]) : -1, plan.tokens[i]);
            if (i > q0 && plan.positions[i] != plan.positions[i - 1] + 1)
                throw std::runtime_error("executor: a request's rows must be consecutive positions");
        }
        slot[r] = 0;
        fresh[r] = 1;
        if (!recurrent) continue;
        const uint32_t s = plan.rs_slots[r];
        if (s >= static_cast<uint32_t>(rs_slots_)) throw std::runtime_error("executor: recurrent-state slot out of range");
        if (!seen.insert(s).second) throw std::runtime_error("executor: two requests of a batch share a recurrent-state slot");
        // state cannot be rolled back to a rejected draft's predecessor
        if (!plan.draft_tokens[r].empty()) throw std::runtime_error("executor: recurrent state cannot verify drafts");
        const bool reset = plan.positions[q0] == 0 || (!plan.rs_flags.empty() && (plan.rs_flags[r] & PIE_RS_RESET));
        if (!reset && rs_pos_[s] != plan.positions[q0])
            throw std::runtime_error("executor: slot " + std::to_string(s) + " holds the state after " +
                                     std::to_string(rs_pos_[s]) + " tokens, the request goes on at position " +
                                     std::to_string(plan.positions[q0]));
        slot[r] = static_cast<int32_t>(s);
        fresh[r] = reset ? 1 : 0;
        if (!reset) pair[q0] = pair_row(rs_last_[s], plan.tokens[q0]);
    }
    qo[plan.R] = plan.N;
    if (recurrent)
        for (int r = 0; r < plan.R; ++r) rs_pos_[plan.rs_slots[r]] = -1;   // (until the pass has succeeded)
    if (!plan.pure_decode) prepare_lists(plan);
    plan_ = &plan;
}

// What the kernels for portions walk: chunks of the recurrences, tiles of the attention.
void Executor::prepare_lists(const BatchPlan& plan) {
    bool delta = false, memory = false;
    tile_lists_.clear();
    std::vector<int32_t> all;
    auto chunk_list = [&](int size) {
        ChunkList l;
        std::vector<int32_t> first(1, 0);
        l.chunks = all.size();
        for (int r = 0; r < plan.R; ++r) {
            for (int i = plan.qo_indptr[r]; i < plan.qo_indptr[r + 1]; i += size) {
                all.push_back(i);
                all.push_back(std::min(size, plan.qo_indptr[r + 1] - i));
                ++l.n;
            }
            first.push_back(l.n);
        }
        l.first = all.size();
        all.insert(all.end(), first.begin(), first.end());
        return l;
    };
    for (const StackLayer& l : model_.stack) {
        delta |= l.spec.mixer == MixerKind::ChannelDelta;
        memory |= l.spec.has_memory();
        if (!l.spec.has_attn() || dt_ != PIE_HIP_DT_BF16 || !pie_hip_group_attn_supported(pad_head(l.spec.attn.widest()))) continue;
        const GroupAttentionSpec& a = l.spec.attn;
        const auto key = std::make_tuple(a.heads, a.kv_heads, pad_head(a.widest()));
        if (tile_lists_.count(key)) continue;
        TileList t;
        std::vector<std::pair<int, int>> tiles;   // (first row, rows)
        // half tiles while whole ones would not give every CU two blocks, and for the widest heads
        for (t.half = std::get<2>(key) > 128 ? 1 : 0;; t.half = 1) {
            const int per = pie_hip_group_attn_tile_rows(a.heads, a.kv_heads, t.half);
            tiles.clear();
            for (int r = 0; r < plan.R; ++r) {
                const int q0 = plan.qo_indptr[r], q1 = plan.qo_indptr[r + 1];
                if (q1 - q0 < 2) continue;
                for (int i = q0; i < q1; i += per) tiles.emplace_back(i, std::min(per, q1 - i));
            }
            if (t.half || tiles.size() * static_cast<size_t>(a.kv_heads) >= 512) break;
        }
        // (the ones that see most keys start first)
        std::stable_sort(tiles.begin(), tiles.end(), [&](const auto& x, const auto& y) {
            return plan.row_kv_len[x.first + x.second - 1] > plan.row_kv_len[y.first + y.second - 1];
        });
        t.n = static_cast<int>(tiles.size());
        t.tiles = all.size();
        for (const auto& [row, n] : tiles) {
            all.push_back(row);
            all.push_back(n);
        }
        tile_lists_[key] = t;
    }
    if (delta) chunks16_ = chunk_list(16);
    if (memory) chunks64_ = chunk_list(64);
    single_rows_ = all.size();
    for (int r = 0; r < plan.R; ++r)
        if (plan.qo_indptr[r + 1] - plan.qo_indptr[r] == 1) all.push_back(plan.qo_indptr[r]);
    n_single_ = static_cast<int>(all.size() - single_rows_);
    if (all.empty()) return;
    list_host_.pinned = true;
    list_host_.ensure(all.size() * 4);
    list_dev_.ensure(all.size() * 4);
    std::memcpy(list_host_.ptr, all.data(), all.size() * 4);
    PIE_HIP_CHECK(hipMemcpyAsync(list_dev_.ptr, list_host_.ptr, all.size() * 4, hipMemcpyHostToDevice, stream_));
}

void Executor::commit_stack(const BatchPlan& plan) {
    plan_ = nullptr;
    if (rs_slots_ == 0) return;
    for (int r = 0; r < plan.R; ++r) {
        const int last = plan.qo_indptr[r + 1] - 1;
        rs_pos_[plan.rs_slots[r]] = plan.positions[last] + 1;
        rs_last_[plan.rs_slots[r]] = static_cast<int32_t>(plan.tokens[last]);
    }
}

void Executor::stack_linear(const Linear& w, const void* act, void* y, int M, int epilogue, const PieHipGlu* glu) {
    if (dt_ == PIE_HIP_DT_F32 && epilogue == PIE_HIP_EPI_SWIGLU) {
        PIE_KERNEL(pie_hip_linear_f32(static_cast<const float*>(act), static_cast<const uint16_t*>(w.data), stack_.glu, M, w.N, w.K,
                                      PIE_HIP_EPI_NONE, stream_));
        PIE_KERNEL(pie_hip_glu_f32(stack_.glu, glu, static_cast<float*>(y), M, w.N / 2, stream_));
    } else if (dt_ == PIE_HIP_DT_F32)
        PIE_KERNEL(pie_hip_linear_f32(static_cast<const float*>(act), static_cast<const uint16_t*>(w.data),
                                      static_cast<float*>(y), M, w.N, w.K, epilogue, stream_));
    else
        linear_fused(w, static_cast<const uint16_t*>(act), nullptr, 0.f, static_cast<uint16_t*>(y), M, 0, epilogue,
                     nullptr, gemm_ws_, gemm_ws_bytes_, stream_, -1, glu);
}

// Each token's row through its experts: routes' rows in stack_.routes, their places and weights beside them.
void Executor::stack_mixture(const StackLayer& w, int N) {
    const MixtureSpec& e = w.spec.moe;
    const int Hp = model_.ld_x(), ffp = w.w_down.K, ld = pad_to(e.router_columns(), 16), E = e.all_experts(), routes = N * e.routes();
    PIE_KERNEL(pie_hip_linear_f32out(dt_, stack_.xa, w.w_router, stack_.router, N, ld, Hp, stream_));
    if (e.router == RouterKind::CorrectedScores)
        PIE_KERNEL(pie_hip_moe_route_corrected(stack_.router, ld, w.correction, stack_.route_idx, stack_.route_w, stack_.route_offsets,
                                               stack_.route_token, stack_.route_pos, N, e.experts, e.top, e.shared_parts(), stream_));
    else
        PIE_KERNEL(pie_hip_moe_route_groups(stack_.router, ld, stack_.route_idx, stack_.route_w, stack_.route_offsets, stack_.route_token,
                                            stack_.route_pos, N, e.experts, e.top, e.groups, e.keep, e.scale, stream_));
    const bool pair = e.expert == ExpertKind::ClampedPair;
    const PieHipGlu glu{nullptr, e.limit, e.alpha, e.shift};
    if (dt_ == PIE_HIP_DT_F32) {
        auto product = [&](const void* act, const int32_t* rows, const Linear& l, float* y, int n, int k, int epilogue) {
            PIE_KERNEL(pie_hip_moe_grouped_linear_f32(static_cast<const float*>(act), rows, stack_.route_offsets, E, N,
                                                      static_cast<const uint16_t*>(l.data), y, n, k, epilogue, stream_));
        };
        if (pair) {
            product(stack_.xa, stack_.route_token, w.w_up, stack_.glu, 2 * ffp, Hp, PIE_HIP_EPI_NONE);
            PIE_KERNEL(pie_hip_glu_f32(stack_.glu, &glu, static_cast<float*>(stack_.act), routes, ffp, stream_));
        } else {
            product(stack_.xa, stack_.route_token, w.w_up, static_cast<float*>(stack_.act), ffp, Hp, PIE_HIP_EPI_RELU2);
        }
        product(stack_.act, nullptr, w.w_down, static_cast<float*>(stack_.routes), Hp, ffp, PIE_HIP_EPI_NONE);
        return;
    }
    const int hint = std::max(1, std::min(N, 2 * ((routes + E - 1) / E)));
    const bool blocks = grouped_in_blocks(routes, E);
    auto grouped = [&](const Linear& l, const void* act, const int32_t* rows, void* y, int epilogue, const PieHipGlu* rule) {
        if (blocks) {
            PIE_KERNEL(pie_hip_moe_grouped_gemm_mfma(static_cast<const uint16_t*>(act), rows, stack_.route_offsets, E, routes,
                                                     l.data_tiled ? l.data_tiled : l.data, l.data_bytes() / E,
                                                     static_cast<uint16_t*>(y), l.N / E, l.K, epilogue, l.data_tiled ? 1 : 0, rule, 0,
                                                     stream_));
            return;
        }
        PIE_KERNEL(pie_hip_moe_grouped_gemm_glu(PIE_HIP_FMT_BF16, static_cast<const uint16_t*>(act), rows, stack_.route_offsets, E,
                                                hint, routes, l.data_tiled ? l.data_tiled : l.data, l.data_bytes() / E, nullptr, 0, 0, 0,
                                                static_cast<uint16_t*>(y), l.N / E, l.K, epilogue, l.data_tiled ? 1 : 0, rule,
                                                stream_));
    };
    grouped(w.w_up, stack_.xa, stack_.route_token, stack_.act, pair ? PIE_HIP_EPI_SWIGLU : PIE_HIP_EPI_RELU2, pair ? &glu : nullptr);
    grouped(w.w_down, stack_.act, nullptr, stack_.routes, PIE_HIP_EPI_NONE, nullptr);
}

void Executor::stack_latent(const StackLayer& w, int layer, int N, int max_kv_len, const Inputs& in) {
    const LatentAttentionSpec& a = w.spec.latent;
    const LatentShape s(a);
    const auto* slots = reinterpret_cast<const int64_t*>(in_dev_ + in.off_slots);
    const auto* row_begin = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_row_begin);
    const auto* row_len = reinterpret_cast<const int32_t*>(in_dev_ + in.off_row_len);
    const auto* pages = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_pages);
    const float* rope = w.rotary >= 0 ? stack_.rotary[static_cast<size_t>(w.rotary)] : nullptr;
    stack_linear(w.w_in, stack_.xa, stack_.in, N);
    const size_t esize = dt_ == PIE_HIP_DT_F32 ? 4 : 2;
    auto rows_of = [&](void* buf, int row, int ld) { return static_cast<unsigned char*>(buf) + static_cast<size_t>(row) * ld * esize; };
    auto gate_of = [&](int row) { return s.gate_cols ? rows_of(stack_.in, row, s.ld_in) + static_cast<size_t>(s.gate_off) * esize : nullptr; };
    PIE_KERNEL(pie_hip_latent_prep(dt_, stack_.in, w.q_norm, w.kv_norm, rope, slots, stack_.cq, run_pool_[layer], N,
                                   s.ld_in, s.kv_off, a.q_rank, s.ld_cq, a.kv_rank, s.kvp, a.rot_dim, a.rot.dims,
                                   s.ld_row, model_.cfg().rms_eps, stream_));
    stack_linear(w.w_uq, stack_.cq, stack_.q, N);

    const bool matrix = dt_ == PIE_HIP_DT_BF16 && pie_hip_latent_attn_rows_supported(s.kvp, s.rotp);
    // rows [r0, r0 + n): through the latent space
    auto rows_form = [&](int r0, int n, int max_len, int max_tokens) {
        if (n <= 0) return;
        PIE_KERNEL(pie_hip_head_linear(dt_, rows_of(stack_.q, r0, s.ld_q), w.w_uk_t, rows_of(stack_.q_lat, r0, s.heads * s.ld_row),
                                       rope ? rope + static_cast<size_t>(r0) * a.rot.dims : nullptr, n, s.heads, s.kvp, s.dimp,
                                       s.ld_q, s.hd, s.heads * s.ld_row, s.ld_row, s.dimp, a.rot_dim, a.rot.dims, s.rotp, nullptr, 0, 0, stream_));
        if (matrix)
            PIE_KERNEL(pie_hip_latent_attn_rows(static_cast<const uint16_t*>(stack_.q_lat),
                                                reinterpret_cast<const uint16_t*>(run_pool_[layer]),
                                                static_cast<uint16_t*>(stack_.o_lat), pages, row_begin, row_len,
                                                reinterpret_cast<const int32_t*>(in_dev_ + in.off_row_req),
                                                reinterpret_cast<const int32_t*>(in_dev_ + in.off_qo), r0, n, s.heads, s.kvp,
                                                s.rotp, page_size_, static_cast<float>(a.scale), w.sinks, max_len, max_tokens, attn_ws_,
                                                attn_ws_bytes_, stream_));
        else
            PIE_KERNEL(pie_hip_latent_attn_rows_plain(dt_, rows_of(stack_.q_lat, r0, s.heads * s.ld_row), run_pool_[layer],
                                                      rows_of(stack_.o_lat, r0, s.heads * s.kvp), pages, row_begin + r0, row_len + r0, n,
                                                      s.heads, s.kvp, s.ld_row, page_size_, static_cast<float>(a.scale), w.sinks, stream_));
        PIE_KERNEL(pie_hip_head_linear(dt_, rows_of(stack_.o_lat, r0, s.heads * s.kvp), w.w_uv, rows_of(stack_.o, r0, s.ld_o), nullptr, n,
                                       s.heads, s.vdp, s.kvp, s.heads * s.kvp, s.kvp, s.ld_o, s.vdp, 0, 0, 0, 0, gate_of(r0), s.ld_in,
                                       s.gate_cols, stream_));
    };
    if (plan_->pure_decode) {
        rows_form(0, N, max_kv_len, 1);
    } else {
        // Portions long enough take the expanded form: projecting `ctx` keys and values costs
        // ctx kv_rank (dim + vdim) per head, what it saves per query and key is
        // 2 kv_rank - (dim + vdim).
        const int per_key = s.dimp + s.vdp, saved = 2 * s.kvp - per_key;
        const bool can_expand = dt_ == PIE_HIP_DT_BF16 && saved > 0 && pie_hip_latent_attn_prefill_supported(s.dimp, s.rotp, s.vdp);
        const int expand_min = can_expand ? std::max(64, static_cast<int>(static_cast<long long>(s.kvp) * per_key / saved)) : 0;
        int run0 = 0, run_len = 0, run_tokens = 1;   // requests of the rows form, launched together
        for (int r = 0; r < plan_->R; ++r) {
            const int q0 = plan_->qo_indptr[r], q1 = plan_->qo_indptr[r + 1];
            if (!can_expand || q1 - q0 < expand_min) {
                run_len = std::max(run_len, plan_->row_kv_len[q1 - 1]);
                run_tokens = std::max(run_tokens, q1 - q0);
                continue;
            }
            rows_form(run0, q0 - run0, run_len, run_tokens);
            run0 = q1;
            run_len = 0;
            run_tokens = 1;
            const int ctx = plan_->row_kv_len[q1 - 1];
            expand_lat_.ensure(static_cast<size_t>(ctx) * s.kvp * 2);
            if (s.rotp) expand_rot_.ensure(static_cast<size_t>(ctx) * s.rotp * 2);
            expand_kv_.ensure(static_cast<size_t>(ctx) * w.w_ukv.N * 2);
            auto* lat = static_cast<uint16_t*>(expand_lat_.ptr);
            auto* rot = s.rotp ? static_cast<uint16_t*>(expand_rot_.ptr) : nullptr;
            auto* kv = static_cast<uint16_t*>(expand_kv_.ptr);
            PIE_KERNEL(pie_hip_latent_gather(reinterpret_cast<const uint16_t*>(run_pool_[layer]),
                                             pages + plan_->row_page_begin[q0], lat, rot, ctx, s.kvp, s.rotp, page_size_, stream_));
            PIE_KERNEL(pie_hip_gemm_mfma(PIE_HIP_FMT_BF16, lat, w.w_ukv.data, nullptr, 0, 0, kv, ctx, w.w_ukv.N, w.w_ukv.K, 0,
                                         PIE_HIP_EPI_NONE, stream_));
            PIE_KERNEL(pie_hip_latent_attn_prefill(static_cast<const uint16_t*>(stack_.q), kv, rot, static_cast<uint16_t*>(stack_.o),
                                                   rope, row_len, q0, q1 - q0, ctx, s.heads, s.dimp, s.rotp, a.rot.dims, s.vdp,
                                                   s.ld_o, static_cast<float>(a.scale), w.sinks, reinterpret_cast<const uint16_t*>(gate_of(0)),
                                                   s.ld_in, s.gate_cols, stream_));
        }
        rows_form(run0, N - run0, run_len, run_tokens);
    }
    stack_linear(w.wo, stack_.o, stack_.y, N);
}

void Executor::stack_delta(const StackLayer& w, int layer, int N, const Inputs& in) {
    const ChannelDeltaSpec& d = w.spec.delta;
    const DeltaShape s(d);
    const auto* row_req = reinterpret_cast<const int32_t*>(in_dev_ + in.off_row_req);
    const auto* qo = reinterpret_cast<const int32_t*>(in_dev_ + in.off_qo);
    const auto* slot = reinterpret_cast<const int32_t*>(in_dev_ + in.off_rs_slot);
    const auto* fresh = reinterpret_cast<const int32_t*>(in_dev_ + in.off_rs_fresh);
    stack_linear(w.w_in, stack_.xa, stack_.in, N);
    PIE_KERNEL(pie_hip_delta_lowrank(dt_, stack_.in, w.w_decay, w.w_gate, w.decay_rate, w.dt_bias, stack_.dg, stack_.gate, N,
                                     s.ld_in, s.decay_off, d.decay_rank, s.ld_a1, s.gate_off, d.gate_rank, s.ld_g1, d.heads,
                                     d.dim, d.vdim, s.ld_gate, stream_));
    const float eps = model_.cfg().rms_eps;
    auto conv_state = [&] {
        PIE_KERNEL(pie_hip_delta_conv_state(dt_, stack_.in, rs_base_, rs_stride_, rs_conv_off_[layer], qo, slot, fresh,
                                            n_requests_, s.ld_in, s.channels, d.taps, stream_));
    };
    if (plan_->pure_decode && pie_hip_delta_step_supported(d.dim, d.vdim)) {
        // (heads that share q / k channels leave the convolution's state to a launch of its own)
        const bool own = d.heads == d.kv_heads;
        PIE_KERNEL(pie_hip_delta_step(dt_, stack_.in, w.conv_w, stack_.dg, stack_.gate, w.out_norm, stack_.o, rs_base_, rs_stride_,
                                      rs_state_off_[layer], rs_conv_off_[layer], slot, fresh, N, s.ld_in, s.ld_gate, s.ld_o,
                                      d.heads, d.kv_heads, d.dim, d.vdim, d.taps, own ? 1 : 0, eps, stream_));
        if (!own) conv_state();
    } else {
        PIE_KERNEL(pie_hip_delta_prep(dt_, stack_.in, w.conv_w, rs_base_, rs_stride_, rs_conv_off_[layer], row_req, qo, slot,
                                      fresh, stack_.dq, stack_.dk, stack_.dv, stack_.d_beta, N, s.ld_in, d.heads, d.kv_heads,
                                      d.dim, d.vdim, d.taps, stream_));
        conv_state();
        if (plan_->pure_decode) {
            PIE_KERNEL(pie_hip_delta_scan(stack_.dq, stack_.dk, stack_.dv, stack_.dg, stack_.d_beta, stack_.d_o, rs_base_,
                                          rs_stride_, rs_state_off_[layer], qo, slot, fresh, n_requests_, d.heads, d.kv_heads,
                                          d.dim, d.vdim, stream_));
        } else {
            record_ws_.ensure(pie_hip_delta_chunked_workspace_bytes(chunks16_.n, d.heads, d.dim));
            PIE_KERNEL(pie_hip_delta_chunked(stack_.dq, stack_.dk, stack_.dv, stack_.dg, stack_.d_beta, stack_.d_o, rs_base_,
                                             rs_stride_, rs_state_off_[layer], list_at(chunks16_.chunks), list_at(chunks16_.first),
                                             qo, slot, fresh, chunks16_.n, n_requests_, d.heads, d.kv_heads, d.dim, d.vdim,
                                             record_ws_.ptr, record_ws_.cap, stream_));
        }
        PIE_KERNEL(pie_hip_delta_out(dt_, stack_.d_o, stack_.gate, w.out_norm, stack_.o, N, s.ld_gate, s.ld_o, d.heads, d.vdim,
                                     eps, stream_));
    }
    stack_linear(w.wo, stack_.o, stack_.y, N);
}

PieHipStateRows Executor::state_rows(int run, int N, const Inputs& in) const {
    PieHipStateRows r{};
    r.row_req = reinterpret_cast<const int32_t*>(in_dev_ + in.off_row_req);
    r.qo_indptr = reinterpret_cast<const int32_t*>(in_dev_ + in.off_qo);
    r.rs_slot = reinterpret_cast<const int32_t*>(in_dev_ + in.off_rs_slot);
    r.rs_fresh = reinterpret_cast<const int32_t*>(in_dev_ + in.off_rs_fresh);
    r.rs_base = rs_base_;
    r.rs_stride = rs_stride_;
    r.state_offset = rs_state_off_[static_cast<size_t>(run)];
    r.conv_offset = rs_conv_off_[static_cast<size_t>(run)];
    r.num_tokens = N;
    r.num_requests = n_requests_;
    return r;
}

// Attention and memory write their columns of the rows that W_o reads, scaled.
void Executor::stack_mix(const StackLayer& w, int run, int N, int max_kv_len, const Inputs& in) {
    const MixShape s(w.spec);
    stack_linear(w.w_in, stack_.xa, stack_.in, N);
    if (s.gates)
        PIE_KERNEL(pie_hip_linear_f32out(dt_, stack_.xa, w.w_gates, stack_.gates, N, s.gates, w.w_in.K, stream_));
    if (w.spec.has_attn()) stack_attention(w, run, N, max_kv_len, in);
    if (w.spec.has_memory()) stack_memory(w, run, N, in);
    stack_linear(w.wo, stack_.o, stack_.y, N);
}

void Executor::stack_attention(const StackLayer& w, int run, int N, int max_kv_len, const Inputs& in) {
    const GroupAttentionSpec& a = w.spec.attn;
    const MixShape s(w.spec);
    const auto* row_begin = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_row_begin);
    const auto* row_len = reinterpret_cast<const int32_t*>(in_dev_ + in.off_row_len);
    const auto* pages = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_pages);
    const float* rope = w.rotary >= 0 ? stack_.rotary[static_cast<size_t>(w.rotary)] : nullptr;
    const float scale = static_cast<float>(a.scale), out_scale = w.spec.attention_scale;
    unsigned char* pool = run_pool_[static_cast<size_t>(run)];
    const size_t esize = dt_ == PIE_HIP_DT_F32 ? 4 : 2;
    const void* gate = a.gate ? static_cast<unsigned char*>(stack_.in) + static_cast<size_t>(s.attn_gate_off) * esize : nullptr;
    const auto* slots = reinterpret_cast<const int64_t*>(in_dev_ + in.off_slots);
    // (the kernel for norms per head rotates half-split vectors and knows biases)
    if (a.norm == QueryKeyNorm::PerHead || a.biases)
        PIE_KERNEL(pie_hip_group_attn_prep(dt_, stack_.in, s.q_off, s.k_off, s.v_off, w.q_bias, w.k_bias, w.q_norm, w.k_norm, rope, a.rot.dims,
                                           slots, stack_.q, pool, N, s.ld_in, a.heads, a.kv_heads, a.dim, s.dimp, model_.cfg().rms_eps, stream_));
    else
        PIE_KERNEL(pie_hip_group_attn_prep_joint(dt_, stack_.in, s.q_off, s.k_off, s.v_off, w.q_norm, w.k_norm, rope, a.rot.dims,
                                                 a.half_split ? PIE_HIP_ROPE_HALF : PIE_HIP_ROPE_ADJACENT, slots, stack_.q, pool, N, s.ld_in,
                                                 a.heads, a.kv_heads, a.dim, a.vdim, s.dimp, model_.cfg().rms_eps, stream_));
    if (dt_ != PIE_HIP_DT_BF16 || !pie_hip_group_attn_supported(s.dimp)) {
        PIE_KERNEL(pie_hip_group_attn_plain(dt_, stack_.q, pool, stack_.o, pages, row_begin, row_len, N, a.heads, a.kv_heads, s.dimp, s.ld_o,
                                            page_size_, scale, a.window, a.sink, out_scale, gate, s.ld_in, stream_));
        return;
    }
    const auto* q = static_cast<const uint16_t*>(stack_.q);
    const auto* kv = reinterpret_cast<const uint16_t*>(pool);
    auto* o = static_cast<uint16_t*>(stack_.o);
    const auto* g = static_cast<const uint16_t*>(gate);
    auto rows_form = [&](const int32_t* rows, int n) {
        PIE_KERNEL(pie_hip_group_attn_rows(q, kv, o, pages, row_begin, row_len, rows, n, a.heads, a.kv_heads, s.dimp, s.ld_o, page_size_,
                                           scale, a.window, a.sink, out_scale, g, s.ld_in, max_kv_len, attn_ws_, attn_ws_bytes_, stream_));
    };
    if (plan_->pure_decode) return rows_form(nullptr, N);
    const TileList& t = tile_lists_.at(std::make_tuple(a.heads, a.kv_heads, s.dimp));
    if (t.n)
        PIE_KERNEL(pie_hip_group_attn_tiles(q, kv, o, pages, row_begin, row_len, list_at(t.tiles), t.n, t.half, a.heads, a.kv_heads, s.dimp,
                                            s.ld_o, page_size_, scale, a.window, a.sink, out_scale, g, s.ld_in, stream_));
    if (n_single_) rows_form(list_at(single_rows_), n_single_);
}

void Executor::stack_memory(const StackLayer& w, int run, int N, const Inputs& in) {
    const DecayMemorySpec& d = w.spec.memory;
    const MixShape s(w.spec);
    const bool ssm = d.kind == DecayKind::StateSpace;
    const float head_scale = static_cast<float>(1.0 / std::sqrt(static_cast<double>(d.dim)));
    PieHipDecayRule rule{};
    rule.kind = d.kind == DecayKind::Retention    ? PIE_HIP_DECAY_FIXED
                : d.kind == DecayKind::MatrixLstm ? PIE_HIP_DECAY_EXP_GATES
                                                  : PIE_HIP_DECAY_STEP;
    rule.heads = d.heads;
    rule.kv_heads = d.kv_heads;
    rule.dim = d.dim;
    rule.vdim = d.vdim;
    rule.q_scale = d.kind == DecayKind::MatrixLstm ? head_scale : 1.f;
    rule.k_scale = d.kind == DecayKind::Retention ? head_scale : 1.f;
    rule.gate_cap = static_cast<float>(d.gate_cap);
    rule.decay = w.decay_log2;
    rule.gate_bias = w.gate_bias;
    const PieHipStateRows rows = state_rows(run, N, in);
    const float eps = model_.cfg().rms_eps;
    const size_t esize = dt_ == PIE_HIP_DT_F32 ? 4 : 2;
    auto at = [&](void* base, int col) { return static_cast<unsigned char*>(base) + static_cast<size_t>(col) * esize; };
    const void* gate = at(stack_.in, s.gate_off);
    void* y = at(stack_.o, s.out_off);
    const int gate_act = d.kind == DecayKind::Retention ? 1 : 0;   // silu, else the logistic function
    const float scale = w.spec.memory_scale;
    auto out = [&] {
        PIE_KERNEL(pie_hip_decay_out(dt_, &rule, &rows, stack_.mem_o, stack_.den, gate, s.ld_in, gate_act, w.out_norm, y, s.ld_o, scale, eps,
                                     stream_));
    };
    auto part_norm = [&](const void* x, const void* conv_fused) {
        PIE_KERNEL(pie_hip_gated_part_norm(dt_, stack_.mem_o, x, s.ld_conv, w.skip, gate, s.ld_in, w.out_norm, y, s.ld_o, d.heads, d.vdim,
                                           d.norm_parts, &rows, conv_fused, s.ld_in, s.channels, d.taps, eps, stream_));
    };
    if (plan_->pure_decode && pie_hip_decay_step_supported(d.dim, d.vdim)) {
        const bool fuse = !ssm && pie_hip_decay_step_fuses(&rule, rows.num_requests);
        // (the heads of a group convolve the same keys and queries again: worth a launch of its own once
        // the batch fills the device)
        const bool conv_first = ssm && rows.num_requests * d.heads >= 1024;
        if (conv_first)
            PIE_KERNEL(pie_hip_conv_silu(dt_, stack_.in, w.conv_w, w.conv_b, &rows, stack_.conv, s.ld_in, s.channels, d.taps, s.ld_conv, 1, stream_));
        const bool conv_in = ssm && !conv_first;
        PIE_KERNEL(pie_hip_decay_step(dt_, &rule, &rows, conv_first ? stack_.conv : stack_.in, s.mq_off, s.mk_off, s.mv_off,
                                      conv_first ? s.ld_conv : s.ld_in, stack_.gates, s.gates, conv_in ? w.conv_w : nullptr,
                                      conv_in ? w.conv_b : nullptr, s.channels, d.taps, ssm ? w.skip : nullptr, stack_.mem_o, stack_.den, gate,
                                      s.ld_in, gate_act, w.out_norm, fuse ? y : nullptr, s.ld_o, scale, eps, stream_));
        if (ssm) part_norm(nullptr, conv_first ? nullptr : stack_.in);
        else if (!fuse) out();
        return;
    }
    const void *q = at(stack_.in, s.mq_off), *k = at(stack_.in, s.mk_off), *v = at(stack_.in, s.mv_off);
    int ld = s.ld_in;
    if (ssm) {
        PIE_KERNEL(pie_hip_conv_silu(dt_, stack_.in, w.conv_w, w.conv_b, &rows, stack_.conv, s.ld_in, s.channels, d.taps, s.ld_conv, 0, stream_));
        PIE_KERNEL(pie_hip_delta_conv_state(dt_, stack_.in, rs_base_, rs_stride_, rows.conv_offset, rows.qo_indptr, rows.rs_slot,
                                            rows.rs_fresh, rows.num_requests, s.ld_in, s.channels, d.taps, stream_));
        q = at(stack_.conv, s.mq_off);
        k = at(stack_.conv, s.mk_off);
        v = at(stack_.conv, s.mv_off);
        ld = s.ld_conv;
    }
    if (dt_ == PIE_HIP_DT_BF16 && !plan_->pure_decode) {
        record_ws_.ensure(pie_hip_decay_chunked_workspace_bytes(&rule, chunks64_.n));
        PIE_KERNEL(pie_hip_decay_chunked(&rule, &rows, static_cast<const uint16_t*>(q), static_cast<const uint16_t*>(k),
                                         static_cast<const uint16_t*>(v), ld, stack_.gates, s.gates, stack_.mem_o, stack_.den,
                                         list_at(chunks64_.chunks), list_at(chunks64_.first), chunks64_.n, record_ws_.ptr, record_ws_.cap,
                                         stream_));
    } else {
        PIE_KERNEL(pie_hip_decay_scan(dt_, &rule, &rows, q, k, v, ld, stack_.gates, s.gates, stack_.mem_o, stack_.den, stream_));
    }
    if (ssm) part_norm(stack_.conv, nullptr);
    else out();
}

void Executor::stack_mixer(const StackLayer& w, int run, int N, int max_kv_len, const Inputs& in) {
    switch (w.spec.mixer) {
        case MixerKind::LatentAttention: stack_latent(w, run, N, max_kv_len, in); break;
        case MixerKind::ChannelDelta: stack_delta(w, run, N, in); break;
        default: stack_mix(w, run, N, max_kv_len, in); break;
    }
}

// A layer's dense feed-forward on stack_.xa (its down projection's bias is left to what adds y).
void Executor::stack_dense(const StackLayer& w, void* y, int N) {
    switch (model_.cfg().ff_act) {
        case FeedForwardAct::GatedSilu: {
            const PieHipGlu glu{w.up_bias, INFINITY, 1.f, 0.f};
            stack_linear(w.w_up, stack_.xa, stack_.act, N, PIE_HIP_EPI_SWIGLU, &glu);
            break;
        }
        case FeedForwardAct::Gelu: stack_linear(w.w_up, stack_.xa, stack_.act, N, PIE_HIP_EPI_GELU); break;
        case FeedForwardAct::SquaredRelu: stack_linear(w.w_up, stack_.xa, stack_.act, N, PIE_HIP_EPI_RELU2); break;
    }
    stack_linear(w.w_down, stack_.act, y, N);
}

// Layers whose mixer and feed-forward read one norm: both outputs join the stream in one kernel, which norms it
// for the next layer.
void Executor::stack_shared_norm(int N, int max_kv_len, const Inputs& in) {
    const ModelConfig& m = model_.cfg();
    const int ld = model_.ld_x();
    const size_t n_runs = model_.runs.size();
    auto layer_of = [&](size_t run) -> const StackLayer& { return model_.stack[static_cast<size_t>(model_.runs[run].layer)]; };
    PIE_KERNEL(pie_hip_residual_join(dt_, nullptr, 0, nullptr, 0, nullptr, nullptr, stack_.x, 0,
                                     reinterpret_cast<const uint32_t*>(in_dev_ + in.off_tokens), model_.embed, m.vocab, m.embed_scale,
                                     layer_of(0).pre1, stack_.xa, N, m.hidden, ld, m.rms_eps, stream_));
    for (size_t r = 0; r < n_runs; ++r) {
        const StackLayer& w = layer_of(r);
        stack_mixer(w, static_cast<int>(r), N, max_kv_len, in);
        const bool dense = w.spec.ff > 0, mixture = w.spec.moe.experts > 0;
        if (dense) stack_dense(w, stack_.y2, N);
        if (mixture) stack_mixture(w, N);
        const PieHipRoutes routes{stack_.routes, stack_.route_pos, stack_.route_w, w.spec.moe.routes(), ld};
        PIE_KERNEL(pie_hip_residual_join(dt_, stack_.y, w.wo.N, dense ? stack_.y2 : nullptr, w.w_down.N, w.down_bias,
                                         mixture ? &routes : nullptr, stack_.x, 1, nullptr, nullptr, 0, 0.f,
                                         r + 1 < n_runs ? layer_of(r + 1).pre1 : nullptr, stack_.xa, N, m.hidden, ld, m.rms_eps, stream_));
    }
}

// Layers of gated sublayers: the kernel that ends one norms the stream for the next, whose input is the normed row
// plus a convolution over it and the rows before it — in the same launch where every request brings one row.
void Executor::stack_gated(int N, int max_kv_len, const Inputs& in) {
    const ModelConfig& m = model_.cfg();
    const int H = m.hidden, ld = model_.ld_x(), taps = m.canon_taps;
    const PieHipEmbedding start{reinterpret_cast<const uint32_t*>(in_dev_ + in.off_tokens),
                                reinterpret_cast<const int32_t*>(in_dev_ + in.off_pair), model_.embed, model_.bigram, model_.embed_norm, m.vocab,
                                m.embed_scale};
    struct Sublayer {
        const float *norm, *gate_bias;
        const uint16_t* canon;
        const Linear* gate;
        size_t state;   // of the convolution
    };
    auto sublayer = [&](size_t run, int n) {
        const StackLayer& w = model_.stack[static_cast<size_t>(model_.runs[run].layer)];
        return n == 0 ? Sublayer{w.pre1, w.gate1_bias, w.canon1, &w.w_gate1, rs_canon_off_[run][0]}
                      : Sublayer{w.pre2, w.gate2_bias, w.canon2, &w.w_gate2, rs_canon_off_[run][1]};
    };
    // the output of `from` (null: the embedding starts the stream) joins the stream, which `to` (null: the last one
    // has ended) reads
    auto join = [&](const Sublayer* from, const void* y, const PieHipRoutes* routes, const Sublayer* to) {
        PieHipStateRows state{};
        if (to) {
            state = state_rows(0, N, in);
            state.conv_offset = to->state;
        }
        const bool fused = to && plan_->pure_decode && taps <= 4;
        PIE_KERNEL(pie_hip_gated_join(dt_, y, ld, routes, from ? stack_.sub_gate : nullptr, ld, from ? from->gate_bias : nullptr, from ? nullptr : &start,
                                      stack_.x,
                                      to ? to->norm : nullptr, stack_.h, stack_.xa, fused ? to->canon : nullptr, taps, &state, N, H, ld,
                                      m.rms_eps, stream_));
        if (!to) return;
        if (!fused) {
            PIE_KERNEL(pie_hip_recent_rows(dt_, stack_.h, to->canon, taps, &state, stack_.xa, H, ld, stream_));
            if (taps > 1)
                PIE_KERNEL(pie_hip_delta_conv_state(dt_, stack_.h, rs_base_, rs_stride_, state.conv_offset, state.qo_indptr, state.rs_slot,
                                                    state.rs_fresh, state.num_requests, ld, H, taps, stream_));
        }
        stack_linear(*to->gate, stack_.h, stack_.sub_gate, N);
    };
    const size_t n_runs = model_.runs.size();
    Sublayer now = sublayer(0, 0);
    join(nullptr, nullptr, nullptr, &now);
    for (size_t r = 0; r < n_runs; ++r) {
        const StackLayer& w = model_.stack[static_cast<size_t>(model_.runs[r].layer)];
        auto finish = [&](const void* y, const PieHipRoutes* routes, bool layer_ends) {
            const bool more = !layer_ends || r + 1 < n_runs;
            const Sublayer next = !more ? Sublayer{} : layer_ends ? sublayer(r + 1, 0) : sublayer(r, 1);
            join(&now, y, routes, more ? &next : nullptr);
            now = next;
        };
        stack_mixer(w, static_cast<int>(r), N, max_kv_len, in);
        const bool dense = w.spec.ff > 0, mixture = w.spec.moe.experts > 0;
        finish(stack_.y, nullptr, !dense && !mixture);
        if (dense) {
            stack_dense(w, stack_.y, N);
            finish(stack_.y, nullptr, true);
        } else if (mixture) {
            stack_mixture(w, N);
            const PieHipRoutes routes{stack_.routes, stack_.route_pos, stack_.route_w, w.spec.moe.routes(), ld};
            finish(nullptr, &routes, true);
        }
    }
}

void Executor::stack_body(int N, int S, int max_kv_len) {
    const Inputs in = input_layout(N, S);
    const ModelConfig& m = model_.cfg();
    const int H = m.hidden, ld = model_.ld_x();
    hipStream_t s = stream_;
    n_requests_ = plan_->R;
    const auto* tokens = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_tokens);
    const size_t n_runs = model_.runs.size();
    auto layer_of = [&](size_t run) -> const StackLayer& { return model_.stack[static_cast<size_t>(model_.runs[run].layer)]; };
    // What the stream takes on ahead of run `run` besides the last sublayer's output (`y` null: nothing yet),
    // and the norm it is read through: a looped pass adds its step vector and, from the second pass on, the
    // embedding again.
    auto enter = [&](size_t run, const void* y, const float* post, int ldy, bool read_x) {
        const bool more = run < n_runs, begins = more && model_.runs[run].begins_pass;
        const int pass = more ? model_.runs[run].pass : 0;
        const bool embed = !read_x || (begins && pass > 0);
        PIE_KERNEL(pie_hip_residual_norm(dt_, y, post, stack_.x, read_x ? 1 : 0, embed ? tokens : nullptr, model_.embed, m.vocab,
                                         begins ? model_.loop_step + static_cast<size_t>(pass) * H : nullptr,
                                         more ? layer_of(run).pre1 : nullptr, stack_.xa, N, H, ldy, ld, m.rms_eps, s));
    };
    if (m.shared_norm || m.gated_sublayers) {
    } else if (m.sandwich_norms) enter(0, nullptr, nullptr, 0, false);
    else PIE_KERNEL(pie_hip_embed_stream(dt_, tokens, model_.embed, stack_.x, stack_.xa, N, H, ld, m.vocab, s));
    for (size_t i = 0; i < model_.rotary.size(); ++i)
        PIE_KERNEL(pie_hip_rotary_table(reinterpret_cast<const int32_t*>(in_dev_ + in.off_positions),
                                        model_.rotary[i].freq, stack_.rotary[i], N, model_.rotary[i].spec.dims,
                                        model_.rotary[i].mscale, s));
    if (m.shared_norm) stack_shared_norm(N, max_kv_len, in);
    else if (m.gated_sublayers) stack_gated(N, max_kv_len, in);
    for (size_t r = 0; r < n_runs && !m.shared_norm && !m.gated_sublayers; ++r) {
        const StackLayer& w = layer_of(r);
        stack_mixer(w, static_cast<int>(r), N, max_kv_len, in);
        // y joins the stream; `last`: the layer's last sublayer
        auto finish = [&](const float* post, int ldy, bool last) {
            if (!m.sandwich_norms)
                PIE_KERNEL(pie_hip_norm_add(dt_, stack_.y, post, stack_.x, stack_.xa, N, H, ldy, ld, m.rms_eps, s));
            else if (last)
                enter(r + 1, stack_.y, post, ldy, true);
            else
                PIE_KERNEL(pie_hip_residual_norm(dt_, stack_.y, post, stack_.x, 1, nullptr, nullptr, 0, nullptr, w.pre2, stack_.xa, N, H,
                                                 ldy, ld, m.rms_eps, s));
        };
        finish(w.norm1, w.wo.N, w.spec.ff == 0);
        if (w.spec.ff > 0) {
            stack_dense(w, stack_.y, N);
            finish(w.norm2, w.w_down.N, true);
        }
    }
    // the output norm and the head on the sampled rows only
    const auto* sample_rows = reinterpret_cast<const uint32_t*>(in_dev_ + in.off_sample_rows);
    const int cap = static_cast<int>(std::min<size_t>(max_tokens_, 2 * static_cast<size_t>(cfg_.batching.max_forward_requests)));
    for (int s0 = 0; s0 < S; s0 += cap) {
        const int n = std::min(cap, S - s0);
        PIE_KERNEL(pie_hip_norm_rows(dt_, stack_.x, sample_rows + s0, model_.stack_norm, stack_.xs, n, H, ld, N, m.rms_eps, s));
        stack_linear(model_.head, stack_.xs, stack_.raw_logits, n);
        PIE_KERNEL(pie_hip_logits_finish(dt_, stack_.raw_logits, stack_.logits, out_tokens_ + s0, n, m.vocab,
                                         model_.head.N, m.logit_scale, m.logit_softcap, s));
        if (samp_gather_in_body_) {   // more sampled rows than one chunk: keep each chunk's rows
            const auto* dev = static_cast<const unsigned char*>(samp_in_dev_.ptr);
            PIE_KERNEL(pie_hip_sample_gather_logits_f32(
                stack_.logits, nullptr, static_cast<float*>(samp_f32_.ptr) + static_cast<size_t>(s0) * m.vocab,
                samp_.n_bounds ? reinterpret_cast<const uint32_t*>(dev + samp_.bounds) : nullptr,
                samp_.n_bounds ? reinterpret_cast<const int32_t*>(dev + samp_.bounds_indptr) + s0 : nullptr, n, m.vocab, s));
        }
    }
}

}  // namespace pie_hip_driver
