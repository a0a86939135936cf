// Linear memories with one decay per head and token, and what surrounds them: retention, mLSTM and
// Mamba-2 differ in how a token's decay and write weight are formed, not in the recurrence
//   S <- d_t S + w_t k_t v_t^T,   o_t = S^T q_t          (S [dim, vdim] in fp32).
// An exponentially gated memory also keeps a running maximum m of its logarithmic weights and a
// vector n, the same recurrence over v = 1; n is carried as one more value column of S.
//
// Three forms: token by token (any compute type), 64 tokens at a time on the matrix cores (portions),
// and one token per request in one launch (decode).
#include "act_type.hip.h"

namespace pie_hip {
namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

constexpr float kLog2e = 1.4426950408889634f;

// The logarithms (base 2) of a token's decay and exponential write weight, and its plain weight.
struct TokenGate {
    float keep, in, weight;
};
__device__ __forceinline__ TokenGate token_gate(const PieHipDecayRule& r, const float* __restrict__ gates, int h) {
    if (r.kind == PIE_HIP_DECAY_EXP_GATES) {
        const float cap = r.gate_cap;
        const float i = cap * tanhf((gates[h] + r.gate_bias[h]) / cap);
        const float f = cap * tanhf((gates[r.heads + h] + r.gate_bias[r.heads + h]) / cap);
        const float log_sigmoid = fminf(f, 0.f) - log1pf(expf(-fabsf(f)));
        return {log_sigmoid * kLog2e, i * kLog2e, r.k_scale};
    }
    if (r.kind == PIE_HIP_DECAY_STEP) {
        const float z = gates[h] + r.gate_bias[h];
        const float dt = fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));   // softplus
        return {r.decay[h] * dt, 0.f, dt * r.k_scale};
    }
    return {r.decay[h], 0.f, r.k_scale};
}
__device__ __forceinline__ bool stabilised(const PieHipDecayRule& r) { return r.kind == PIE_HIP_DECAY_EXP_GATES; }

// A request's state: S, then n and m of the exponentially gated kind.
struct StateOf {
    float *S, *n, *m;
};
__device__ __forceinline__ StateOf state_of(const PieHipDecayRule& r, const PieHipStateRows& rows, int request, int h) {
    float* base = reinterpret_cast<float*>(static_cast<unsigned char*>(rows.rs_base) +
                                           static_cast<size_t>(rows.rs_slot[request]) * rows.rs_stride + rows.state_offset);
    const size_t per_head = static_cast<size_t>(r.dim) * r.vdim;
    float* n = base + r.heads * per_head;
    return {base + h * per_head, n + static_cast<size_t>(h) * r.dim, n + static_cast<size_t>(r.heads) * r.dim + h};
}
template <class T>
__device__ __forceinline__ T* conv_state_of(const PieHipStateRows& rows, int request) {
    return reinterpret_cast<T*>(static_cast<unsigned char*>(rows.rs_base) +
                                static_cast<size_t>(rows.rs_slot[request]) * rows.rs_stride + rows.conv_offset);
}

// ---- the short convolution ahead of a memory ------------------------------------------------------
// A thread takes one channel of a run of rows and walks it with the last four inputs in registers;
// longer convolutions read their window afresh.
template <class T>
__global__ __launch_bounds__(256) void conv_silu_kernel(const T* __restrict__ fused, const float* __restrict__ w,
                                                        const float* __restrict__ bias, const PieHipStateRows rows,
                                                        T* __restrict__ out, int ld, int channels, int taps, int ld_out,
                                                        int run) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= channels) return;
    const int n0 = blockIdx.y * run, n1 = min(n0 + run, rows.num_tokens), keep = taps - 1;
    const float b = bias ? bias[c] : 0.f;
    const bool windowed = taps <= 4;
    float wr[4] = {};
    if (windowed)
#pragma unroll
        for (int j = 0; j < 4; ++j) wr[j] = j >= 4 - taps ? w[static_cast<size_t>(c) * taps + j - (4 - taps)] : 0.f;
    float win[4] = {};
    int row0 = 0, row1 = n0;
    bool fresh = false;
    const T* state = nullptr;
    auto input = [&](int i) {   // the request's input i (negative: from the state)
        if (i >= 0) return act_get<T>(fused[static_cast<size_t>(row0 + i) * ld + c]);
        return fresh ? 0.f : act_get<T>(state[static_cast<size_t>(keep + i) * channels + c]);
    };
    for (int n = n0; n < n1; ++n) {
        const bool enter = n >= row1;
        if (enter) {
            const int r = rows.row_req[n];
            row0 = rows.qo_indptr[r];
            row1 = rows.qo_indptr[r + 1];
            fresh = rows.rs_fresh[r] != 0;
            state = conv_state_of<const T>(rows, r);
        }
        const int i = n - row0;
        float y = b;
        if (windowed) {
            if (enter)
#pragma unroll
                for (int j = 1; j < 4; ++j) win[j] = 4 - j <= keep ? input(i - (4 - j)) : 0.f;
#pragma unroll
            for (int j = 0; j < 3; ++j) win[j] = win[j + 1];
            win[3] = act_get<T>(fused[static_cast<size_t>(n) * ld + c]);
#pragma unroll
            for (int j = 0; j < 4; ++j) y = fmaf(wr[j], win[j], y);
        } else {
            for (int j = 0; j < taps; ++j) y = fmaf(w[static_cast<size_t>(c) * taps + j], input(i - keep + j), y);
        }
        out[static_cast<size_t>(n) * ld_out + c] = act_put<T>(y * sigmoid_f32(y));
    }
}

// ---- token by token -------------------------------------------------------------------------------
struct ScanArgs {
    PieHipDecayRule rule;
    PieHipStateRows rows;
    const void *q, *k, *v;
    const float* gates;
    float *o, *den;
    int ld, ld_gates;
};
// A block takes 32 value columns of one head of one request; a wave's lanes are 8 columns x 8 row
// groups, lane (column, group) holds rows 32 i + 4 group + e of its column.  Queries, keys and gates sit
// in LDS TOK tokens at a time, the next ones requested while the current ones run.
template <class T, int NI, int TOK>   // dim rounded up to 32 NI
__global__ __launch_bounds__(256) void decay_scan_kernel(const ScanArgs a) {
    constexpr int DP = 32 * NI, TPT = 256 / TOK, NV = DP / TPT, COLS = 32, CV = COLS / TPT > 0 ? COLS / TPT : 1;
    __shared__ __attribute__((aligned(16))) float sk[TOK][DP], sq[TOK][DP];
    __shared__ float sv[TOK][COLS], so[TOK][COLS];
    __shared__ TokenGate sg[TOK];
    const PieHipDecayRule& r = a.rule;
    const int req = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * COLS;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const int rg = lane & 7, cl = wv * 8 + (lane >> 3), col = col0 + cl;
    const int row0 = a.rows.qo_indptr[req], T_len = a.rows.qo_indptr[req + 1] - row0;
    const bool fresh = a.rows.rs_fresh[req] != 0, stab = stabilised(r);
    const int kvh = h / (r.heads / r.kv_heads), vd = r.heads * r.vdim;
    const StateOf st = state_of(r, a.rows, req, h);
    const bool is_n = stab && col == r.vdim, live = col < r.vdim || is_n;
    // (column vdim is n: rows one apart instead of vdim)
    float* S = is_n ? st.n : st.S + col;
    const size_t stride = is_n ? 1 : r.vdim;
    f32x4_t s[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int d = 32 * i + 4 * rg + e;
            s[i][e] = live && !fresh && d < r.dim ? S[d * stride] : 0.f;
        }
    float m = stab && !fresh ? *st.m : 0.f;
    const T *q = static_cast<const T*>(a.q), *k = static_cast<const T*>(a.k), *v = static_cast<const T*>(a.v);
    const int tt = tid / TPT, tl = tid % TPT;
    float rk[NV], rq[NV], rv[CV];
    TokenGate rgate{0.f, 0.f, 0.f};
    auto fetch = [&](int t0) {
        const bool in = t0 + tt < T_len;
        const size_t n = static_cast<size_t>(row0) + t0 + tt;
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            const int d = tl + TPT * e;
            const bool ok = in && d < r.dim;
            rk[e] = ok ? act_get<T>(k[n * a.ld + kvh * r.dim + d]) : 0.f;
            rq[e] = ok ? act_get<T>(q[n * a.ld + kvh * r.dim + d]) : 0.f;
        }
#pragma unroll
        for (int e = 0; e < CV; ++e) {
            const int c = col0 + tl + TPT * e;
            rv[e] = in && c < r.vdim ? act_get<T>(v[n * a.ld + h * r.vdim + c]) : stab && c == r.vdim ? 1.f : 0.f;
        }
        if (in && tl == 0) rgate = token_gate(r, a.gates + n * a.ld_gates, h);
    };
    if (T_len > 0) fetch(0);
    for (int t0 = 0; t0 < T_len; t0 += TOK) {
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            sk[tt][tl + TPT * e] = rk[e];
            sq[tt][tl + TPT * e] = rq[e];
        }
#pragma unroll
        for (int e = 0; e < CV; ++e)
            if (tl + TPT * e < COLS) sv[tt][tl + TPT * e] = rv[e];
        if (tl == 0) sg[tt] = rgate;
        if (t0 + TOK < T_len) fetch(t0 + TOK);
        __syncthreads();
        const int nt = min(TOK, T_len - t0);
        for (int t = 0; t < nt; ++t) {
            const TokenGate g = sg[t];
            const float m_new = stab ? fmaxf(g.keep + m, g.in) : 0.f;
            const float keep = exp2f(g.keep + m - m_new);
            const float x = g.weight * exp2f(g.in - m_new) * sv[t][cl];
            m = m_new;
            float o = 0.f;
#pragma unroll
            for (int i = 0; i < NI; ++i) {
                const f32x4_t kk = *reinterpret_cast<const f32x4_t*>(&sk[t][32 * i + 4 * rg]);
                const f32x4_t qq = *reinterpret_cast<const f32x4_t*>(&sq[t][32 * i + 4 * rg]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[i][e] = fmaf(kk[e], x, s[i][e] * keep);
                    o = fmaf(s[i][e], qq[e], o);
                }
            }
            o = dpp_add_f32<0xB1>(o);    // lane ^ 1
            o = dpp_add_f32<0x4E>(o);    // lane ^ 2
            o = dpp_add_f32<0x141>(o);   // the other four of the eight
            if (rg == 0) {
                so[t][cl] = o * r.q_scale;
                if (is_n) {
                    float* den = a.den + (static_cast<size_t>(row0 + t0 + t) * r.heads + h) * 2;
                    den[0] = o * r.q_scale;
                    den[1] = m;
                }
            }
        }
        __syncthreads();
        if (tt < nt)
#pragma unroll
            for (int e = 0; e < CV; ++e) {
                const int c = tl + TPT * e;
                if (c < COLS && col0 + c < r.vdim)
                    a.o[static_cast<size_t>(row0 + t0 + tt) * vd + h * r.vdim + col0 + c] = so[tt][c];
            }
    }
    if (live)
#pragma unroll
        for (int i = 0; i < NI; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = 32 * i + 4 * rg + e;
                if (d < r.dim) S[d * stride] = s[i][e];
            }
}

// ---- portions, 64 tokens at a time ----------------------------------------------------------------
// With F_t the running sum of the chunk's log2 decays, i_s the log2 and u_s the plain write weights,
// M_t = max over s <= t of F_t - F_s + i_s (0 without exponential gates) and m_0, S_0 the state before
// the chunk, m_t = max(F_t + m_0, M_t):
//   P[t, s] = q_t . k_s  u_s 2^(F_t - F_s + i_s - M_t),  s <= t                (nothing of the state in it)
//   o_t     = 2^(F_t + m_0 - m_t) S_0^T q_t + 2^(M_t - m_t) sum_s P[t, s] v_s
//   S       = 2^(F_64 + m_0 - m_64) S_0 + 2^(M_64 - m_64) sum_s k_s (u_s 2^(F_64 - F_s + i_s - M_64) v_s)^T
// All exponents are <= 0.  decay_chunk_kernel forms P and lays everything out in the order the matrix
// instructions' lanes load it, for all chunks at once; decay_walk_kernel carries the state from chunk to
// chunk in registers.  Queries, keys and values are exact bf16; P, the weighted values and the state enter
// their products as hi + lo pairs of bf16 values.
//
// Record of a (chunk, head of keys): Q [4 token tiles][dimp / 32][64 lanes][8], K^T [dimp / 16][2][64][8];
// of a (chunk, head): V^T [cols / 16][2][64][8], P [4][2][hi, lo][64][8], fp32 F, M, weights [64] each.
// The k-slots of every product take a tile pair's rows in the order the accumulators hold them: slot
// (g, e) of lane group g is row 4 g + e of the first tile for e < 4, of the second for e >= 4.
constexpr int kChunk = 64, kWalkCols = 32, kPiece = 64, kPieceStride = kPiece + 8;

struct ChunkLayout {
    int dimp, cols;
    size_t qk_elems, kt_off, vp_elems, p_off, meta_elems;   // bf16 elements, fp32 elements
};
inline int walk_dimp(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 512; }
inline ChunkLayout chunk_layout(const PieHipDecayRule& r) {
    ChunkLayout l;
    l.dimp = walk_dimp(r.dim);
    const int cols = r.vdim + (r.kind == PIE_HIP_DECAY_EXP_GATES ? 1 : 0);
    l.cols = (cols + kWalkCols - 1) / kWalkCols * kWalkCols;
    l.kt_off = static_cast<size_t>(kChunk) * l.dimp;
    l.qk_elems = 2 * l.kt_off;
    l.p_off = static_cast<size_t>(kChunk) * l.cols;
    l.vp_elems = l.p_off + 2 * kChunk * kChunk;
    l.meta_elems = 3 * kChunk;
    return l;
}

struct ChunkArgs {
    PieHipDecayRule rule;
    const uint16_t *q, *k, *v;
    const float* gates;
    const int32_t* chunks;
    uint16_t *qk_rec, *vp_rec;
    float* meta;
    ChunkLayout lay;
    int ld, ld_gates, aligned;   // aligned: 16-byte pieces of q, k, v rows can be loaded whole
};

// 64 columns from c0 on of the chunk's rows into LDS, zeros past the rows and columns that exist; one
// more column of ones at `ones_col` (negative: none)
__device__ __forceinline__ void stage_piece(uint16_t* dst, const uint16_t* __restrict__ src, int ld, int nt, int c0, int n_cols,
                                            bool aligned, int ones_col) {
    const int t = threadIdx.x >> 2, part = (threadIdx.x & 3) * 16;
    uint16_t* d = dst + t * kPieceStride + part;
    if (aligned && c0 + part + 16 <= n_cols) {
        u32x4_t a = {0u, 0u, 0u, 0u}, b = a;
        if (t < nt) {
            const uint16_t* p = src + static_cast<size_t>(t) * ld + c0 + part;
            a = *reinterpret_cast<const u32x4_t*>(p);
            b = *reinterpret_cast<const u32x4_t*>(p + 8);
        }
        *reinterpret_cast<u32x4_t*>(d) = a;
        *reinterpret_cast<u32x4_t*>(d + 8) = b;
        return;
    }
#pragma unroll
    for (int e = 0; e < 16; ++e) {
        const int c = c0 + part + e;
        uint16_t x = 0;
        if (t < nt) {
            if (c < n_cols) x = src[static_cast<size_t>(t) * ld + c];
            else if (c == ones_col) x = 0x3F80;
        }
        d[e] = x;
    }
}
// column `c` of a staged piece, the 8 tokens of k-slot group g of token step ks
__device__ __forceinline__ u32x4_t gather_tokens(const uint16_t* piece, int c, int ks, int g) {
    u32x4_t v;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int t = 32 * ks + (e < 2 ? 4 * g + 2 * e : 16 + 4 * g + 2 * (e - 2));
        v[e] = piece[t * kPieceStride + c] | static_cast<uint32_t>(piece[(t + 1) * kPieceStride + c]) << 16;
    }
    return v;
}

__global__ __launch_bounds__(256) void decay_chunk_kernel(const ChunkArgs a) {
    __shared__ __attribute__((aligned(16))) uint16_t sq[kChunk * kPieceStride], sk[kChunk * kPieceStride];
    __shared__ float s_f[kChunk], s_in[kChunk], s_m[kChunk], s_u[kChunk];
    const PieHipDecayRule& r = a.rule;
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x, lane = tid & (kWave - 1);
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave), l16 = lane & 15, g = lane >> 4;
    const int row0 = a.chunks[2 * ch], nt = a.chunks[2 * ch + 1];
    const int ratio = r.heads / r.kv_heads, kvh = h / ratio;
    const bool lead = h % ratio == 0, stab = stabilised(r);
    const size_t rec = static_cast<size_t>(ch) * r.heads + h;
    uint16_t* qk = a.qk_rec + (static_cast<size_t>(ch) * r.kv_heads + kvh) * a.lay.qk_elems;
    uint16_t* vp = a.vp_rec + rec * a.lay.vp_elems;
    if (wv == 0) {
        TokenGate tg{0.f, stab ? -INFINITY : 0.f, 0.f};   // tokens past the portion: decay 1, weight 0
        if (lane < nt) tg = token_gate(r, a.gates + static_cast<size_t>(row0 + lane) * a.ld_gates, h);
        float F = tg.keep;
#pragma unroll
        for (int off = 1; off < kWave; off <<= 1) {
            const float up = __shfl_up(F, off, kWave);
            if (lane >= off) F += up;
        }
        const float in = tg.in - F;
        float M = 0.f;
        if (stab) {
            float mx = in;
#pragma unroll
            for (int off = 1; off < kWave; off <<= 1) {
                const float up = __shfl_up(mx, off, kWave);
                if (lane >= off) mx = fmaxf(mx, up);
            }
            M = F + mx;
        }
        const float F_end = __shfl(F, kWave - 1, kWave), M_end = __shfl(M, kWave - 1, kWave);
        s_f[lane] = F;
        s_in[lane] = in;
        s_m[lane] = M;
        s_u[lane] = tg.weight;
        float* meta = a.meta + rec * a.lay.meta_elems;
        meta[lane] = F;
        meta[kChunk + lane] = M;
        meta[2 * kChunk + lane] = tg.weight * exp2f(F_end + in - M_end);
    }
    // scores: wave w takes query tile w against key tiles 0 .. w
    f32x4_t acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const uint16_t* qp = a.q + static_cast<size_t>(row0) * a.ld + kvh * r.dim;
    const uint16_t* kp = a.k + static_cast<size_t>(row0) * a.ld + kvh * r.dim;
    const int ksteps = a.lay.dimp / 32;
    for (int d0 = 0; d0 < a.lay.dimp; d0 += kPiece) {
        __syncthreads();
        stage_piece(sq, qp, a.ld, nt, d0, r.dim, a.aligned, -1);
        stage_piece(sk, kp, a.ld, nt, d0, r.dim, a.aligned, -1);
        __syncthreads();
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const bf16x8_t qf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&sq[(16 * wv + l16) * kPieceStride + 32 * j + 8 * g]));
#pragma unroll
            for (int st = 0; st < 4; ++st)
                if (st <= wv) {
                    const bf16x8_t kf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&sk[(16 * st + l16) * kPieceStride + 32 * j + 8 * g]));
                    acc[st] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, acc[st], 0, 0, 0);
                }
        }
        if (!lead) continue;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int ks = d0 / 32 + j;
            if (ks >= ksteps) break;
            const uint16_t* row = &sq[(16 * wv + l16) * kPieceStride + 32 * j + 4 * g];
            const u32x2_t lo = *reinterpret_cast<const u32x2_t*>(row), hi = *reinterpret_cast<const u32x2_t*>(row + 16);
            *reinterpret_cast<u32x4_t*>(qk + ((static_cast<size_t>(wv) * ksteps + ks) * kWave + lane) * 8) = u32x4_t{lo.x, lo.y, hi.x, hi.y};
        }
        const int dt = d0 / 16 + wv;
        if (dt < a.lay.dimp / 16)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
                *reinterpret_cast<u32x4_t*>(qk + a.lay.kt_off + ((static_cast<size_t>(dt) * 2 + ks) * kWave + lane) * 8) =
                    gather_tokens(sk, 16 * wv + l16, ks, g);
    }
    {
        const int t = 16 * wv + l16;
        const float top = s_f[t] - s_m[t];
#pragma unroll
        for (int st = 0; st < 4; ++st)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int s = 16 * st + 4 * g + e;
                acc[st][e] = s <= t ? acc[st][e] * (r.q_scale * s_u[s] * exp2f(top + s_in[s])) : 0.f;
            }
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            u32x4_t hi, lo;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float p0 = acc[2 * ks + (e >> 1)][2 * (e & 1)], p1 = acc[2 * ks + (e >> 1)][2 * (e & 1) + 1];
                const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
                hi[e] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
                lo[e] = pack_bf16x2(p0 - __uint_as_float(u0 & 0xFFFF0000u), p1 - __uint_as_float(u1 & 0xFFFF0000u));
            }
            uint16_t* p = vp + a.lay.p_off + (static_cast<size_t>(wv * 2 + ks) * 2 * kWave + lane) * 8;
            *reinterpret_cast<u32x4_t*>(p) = hi;
            *reinterpret_cast<u32x4_t*>(p + kWave * 8) = lo;
        }
    }
    const uint16_t* vsrc = a.v + static_cast<size_t>(row0) * a.ld + h * r.vdim;
    for (int c0 = 0; c0 < a.lay.cols; c0 += kPiece) {
        __syncthreads();
        stage_piece(sq, vsrc, a.ld, nt, c0, r.vdim, a.aligned, stab ? r.vdim : -1);
        __syncthreads();
        const int ct = c0 / 16 + wv;
        if (ct < a.lay.cols / 16)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
                *reinterpret_cast<u32x4_t*>(vp + ((static_cast<size_t>(ct) * 2 + ks) * kWave + lane) * 8) =
                    gather_tokens(sq, 16 * wv + l16, ks, g);
    }
}

struct WalkArgs {
    PieHipDecayRule rule;
    PieHipStateRows rows;
    const uint16_t *qk_rec, *vp_rec;
    const float* meta;
    const int32_t* req_chunks;
    float *o, *den;
    ChunkLayout lay;
};

// A block takes 32 value columns of one head of one request; wave w keeps rows 32 ND w .. of S as
// accumulator tiles, which are B operands of the read-out as they are (converted to hi + lo).  The
// waves' partial read-outs meet in LDS, one barrier per chunk; wave w finishes token tiles w, w + NW, ..
template <int NW, int ND>
__global__ __launch_bounds__(NW* kWave, 1) void decay_walk_kernel(const WalkArgs a) {
    constexpr int KSTEPS = NW * ND, OWN = 4 / NW;
    __shared__ __attribute__((aligned(16))) float part[NW > 1 ? 2 : 1][NW > 1 ? NW : 1][4][2][NW > 1 ? kWave * 4 : 4];
    const PieHipDecayRule& r = a.rule;
    const int h = blockIdx.x, slice = blockIdx.y, req = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int c_lo = a.req_chunks[req], c_hi = a.req_chunks[req + 1];
    const int req_row0 = a.rows.qo_indptr[req], req_row1 = a.rows.qo_indptr[req + 1];
    const int kvh = h / (r.heads / r.kv_heads), vd = r.heads * r.vdim;
    const bool fresh = a.rows.rs_fresh[req] != 0, stab = stabilised(r);
    const StateOf st = state_of(r, a.rows, req, h);
    const int wrow = 32 * ND * wv;
    f32x4_t s[2 * ND][2];
    int col[2];
    float* S[2];
    size_t stride[2];
    bool live[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        col[c] = slice * kWalkCols + 16 * c + l16;
        const bool is_n = stab && col[c] == r.vdim;   // (column vdim is n: rows one apart instead of vdim)
        live[c] = col[c] < r.vdim || is_n;
        S[c] = is_n ? st.n : st.S + col[c];
        stride[c] = is_n ? 1 : r.vdim;
#pragma unroll
        for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = wrow + 16 * i + 4 * g + e;
                s[i][c][e] = live[c] && !fresh && d < r.dim ? S[c][d * stride[c]] : 0.f;
            }
    }
    float m0 = stab && !fresh ? *st.m : 0.f;
    struct Frags {
        u32x4_t q[4][ND], kt[2 * ND][2], v[2][2], p[OWN][2][2];
        f32x4_t w[2][2], f[OWN], m[OWN];
        float f_end, m_end;
    };
    auto load = [&](Frags& f, int c) {
        const uint16_t* qk = a.qk_rec + (static_cast<size_t>(c) * r.kv_heads + kvh) * a.lay.qk_elems;
        const uint16_t* vp = a.vp_rec + (static_cast<size_t>(c) * r.heads + h) * a.lay.vp_elems;
        const float* meta = a.meta + (static_cast<size_t>(c) * r.heads + h) * a.lay.meta_elems;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int j = 0; j < ND; ++j)
                f.q[t][j] = *reinterpret_cast<const u32x4_t*>(qk + ((t * KSTEPS + wv * ND + j) * kWave + lane) * 8);
#pragma unroll
        for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
                f.kt[i][ks] = *reinterpret_cast<const u32x4_t*>(qk + a.lay.kt_off + (((wv * 2 * ND + i) * 2 + ks) * kWave + lane) * 8);
#pragma unroll
        for (int ct = 0; ct < 2; ++ct)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
                f.v[ct][ks] = *reinterpret_cast<const u32x4_t*>(vp + (((slice * 2 + ct) * 2 + ks) * kWave + lane) * 8);
#pragma unroll
        for (int k = 0; k < OWN; ++k) {
            const int t = wv + NW * k;
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                for (int u = 0; u < 2; ++u)
                    f.p[k][ks][u] = *reinterpret_cast<const u32x4_t*>(vp + a.lay.p_off + (((t * 2 + ks) * 2 + u) * kWave + lane) * 8);
            f.f[k] = *reinterpret_cast<const f32x4_t*>(meta + 16 * t + 4 * g);
            f.m[k] = *reinterpret_cast<const f32x4_t*>(meta + kChunk + 16 * t + 4 * g);
        }
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int u = 0; u < 2; ++u)
                f.w[ks][u] = *reinterpret_cast<const f32x4_t*>(meta + 2 * kChunk + 32 * ks + 16 * u + 4 * g);
        f.f_end = meta[kChunk - 1];
        f.m_end = meta[2 * kChunk - 1];
    };
    auto split = [](const float* x, bf16x8_t& hi, bf16x8_t& lo) {
        u32x4_t a4, b4;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const uint32_t u0 = __float_as_uint(x[2 * e]), u1 = __float_as_uint(x[2 * e + 1]);
            a4[e] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
            b4[e] = pack_bf16x2(x[2 * e] - __uint_as_float(u0 & 0xFFFF0000u), x[2 * e + 1] - __uint_as_float(u1 & 0xFFFF0000u));
        }
        hi = __builtin_bit_cast(bf16x8_t, a4);
        lo = __builtin_bit_cast(bf16x8_t, b4);
    };
    auto run = [&](const Frags& f, int c, int buf) {
        const float m_end = stab ? fmaxf(f.f_end + m0, f.m_end) : 0.f;
        const float keep = exp2f(f.f_end + m0 - m_end), add = exp2f(f.m_end - m_end);
        // the state's part of the read-out, this wave's rows
        f32x4_t inter[4][2];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int ct = 0; ct < 2; ++ct) inter[t][ct] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < ND; ++j)
#pragma unroll
            for (int ct = 0; ct < 2; ++ct) {
                float x[8];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    x[e] = s[2 * j][ct][e];
                    x[4 + e] = s[2 * j + 1][ct][e];
                }
                bf16x8_t hi, lo;
                split(x, hi, lo);
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const bf16x8_t qf = __builtin_bit_cast(bf16x8_t, f.q[t][j]);
                    inter[t][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, hi, inter[t][ct], 0, 0, 0);
                    inter[t][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, lo, inter[t][ct], 0, 0, 0);
                }
            }
        if constexpr (NW > 1) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int ct = 0; ct < 2; ++ct) *reinterpret_cast<f32x4_t*>(&part[buf][wv][t][ct][lane * 4]) = inter[t][ct];
            __syncthreads();   // (the buffer's readers of two chunks ago have passed the last barrier)
        }
        // the state moves on
#pragma unroll
        for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
            for (int ct = 0; ct < 2; ++ct) s[i][ct] *= keep;
#pragma unroll
        for (int ct = 0; ct < 2; ++ct)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                float x[8];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float w0 = f.w[ks][e >> 1][2 * (e & 1)] * add, w1 = f.w[ks][e >> 1][2 * (e & 1) + 1] * add;
                    x[2 * e] = bf16_lo(f.v[ct][ks][e]) * w0;
                    x[2 * e + 1] = bf16_hi(f.v[ct][ks][e]) * w1;
                }
                bf16x8_t hi, lo;
                split(x, hi, lo);
#pragma unroll
                for (int i = 0; i < 2 * ND; ++i) {
                    const bf16x8_t kf = __builtin_bit_cast(bf16x8_t, f.kt[i][ks]);
                    s[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, hi, s[i][ct], 0, 0, 0);
                    s[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, lo, s[i][ct], 0, 0, 0);
                }
            }
        // this wave's token tiles
        const int row0 = req_row0 + (c - c_lo) * kChunk, nt = min(kChunk, req_row1 - row0);
#pragma unroll
        for (int k = 0; k < OWN; ++k) {
            const int t = wv + NW * k;
            if (16 * t >= nt) continue;
            f32x4_t m_t, fi, fa;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                m_t[e] = stab ? fmaxf(f.f[k][e] + m0, f.m[k][e]) : 0.f;
                fi[e] = r.q_scale * exp2f(f.f[k][e] + m0 - m_t[e]);
                fa[e] = exp2f(f.m[k][e] - m_t[e]);
            }
#pragma unroll
            for (int ct = 0; ct < 2; ++ct) {
                f32x4_t pv = {0.f, 0.f, 0.f, 0.f}, x = pv;
#pragma unroll
                for (int ks = 0; ks < 2; ++ks) {
                    const bf16x8_t vf = __builtin_bit_cast(bf16x8_t, f.v[ct][ks]);
                    pv = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, f.p[k][ks][0]), vf, pv, 0, 0, 0);
                    pv = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, f.p[k][ks][1]), vf, pv, 0, 0, 0);
                }
                if constexpr (NW > 1) {
#pragma unroll
                    for (int w = 0; w < NW; ++w) x += *reinterpret_cast<const f32x4_t*>(&part[buf][w][t][ct][lane * 4]);
                } else {
                    x = inter[k][ct];
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int tok = 16 * t + 4 * g + e;
                    if (tok >= nt) continue;
                    const float o = fmaf(x[e], fi[e], pv[e] * fa[e]);
                    if (col[ct] < r.vdim) {
                        a.o[static_cast<size_t>(row0 + tok) * vd + h * r.vdim + col[ct]] = o;
                    } else if (live[ct]) {
                        float* den = a.den + (static_cast<size_t>(row0 + tok) * r.heads + h) * 2;
                        den[0] = o;
                        den[1] = m_t[e];
                    }
                }
            }
        }
        m0 = m_end;
    };
    // (one chunk ahead)
    Frags f[2];
    if (c_lo < c_hi) load(f[0], c_lo);
    for (int c = c_lo; c < c_hi; c += 2) {
        load(f[1], min(c + 1, c_hi - 1));
        __builtin_amdgcn_sched_barrier(0);
        run(f[0], c, 0);
        __builtin_amdgcn_sched_barrier(0);
        if (c + 1 >= c_hi) break;
        load(f[0], min(c + 2, c_hi - 1));
        __builtin_amdgcn_sched_barrier(0);
        run(f[1], c + 1, 1);
        __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int c = 0; c < 2; ++c)
        if (live[c])
#pragma unroll
            for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int d = wrow + 16 * i + 4 * g + e;
                    if (d < r.dim) S[c][d * stride[c]] = s[i][c][e];
                }
}

// ---- read-out: division, norm per head, gate -------------------------------------------------------
__device__ __forceinline__ float gate_value(float z, int act) { return act ? z * sigmoid_f32(z) : sigmoid_f32(z); }
// what o is divided by: max(|n . q|, 2^-m) + 1e-6
__device__ __forceinline__ float exp_gate_divisor(float nq, float m) { return fmaxf(fabsf(nq), exp2f(-m)) + 1e-6f; }

struct OutArgs {
    PieHipDecayRule rule;
    PieHipStateRows rows;
    const float *o, *den, *norm_w;
    const void* gate;
    void* y;
    int ld_gate, ld_y, gate_act;
    float out_scale, eps;
};
// One wave per (row, head).
template <class T>
__global__ __launch_bounds__(256) void decay_out_kernel(const OutArgs a) {
    const PieHipDecayRule& r = a.rule;
    const int unit = blockIdx.x * 4 + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    if (unit >= a.rows.num_tokens * r.heads) return;
    const int n = unit / r.heads, h = unit % r.heads, c0 = h * r.vdim;
    const float* row = a.o + static_cast<size_t>(n) * r.heads * r.vdim + c0;
    float scale = 1.f;
    if (stabilised(r)) {
        const float* den = a.den + static_cast<size_t>(unit) * 2;
        const float m = den[1];
        scale = 1.f / exp_gate_divisor(den[0], m);
        const int req = a.rows.row_req[n];
        if (lane == 0 && n == a.rows.qo_indptr[req + 1] - 1) *state_of(r, a.rows, req, h).m = m;
    }
    constexpr int kCache = 8;   // 512 values in registers
    float v[kCache], local = 0.f;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int c = lane + e * kWave;
        v[e] = c < r.vdim ? row[c] * scale : 0.f;
        local += v[e] * v[e];
    }
    for (int c = lane + kCache * kWave; c < r.vdim; c += kWave) {
        const float x = row[c] * scale;
        local += x * x;
    }
    const float inv = a.out_scale / sqrtf(wave_sum_dpp(local) / static_cast<float>(r.vdim) + a.eps);
    auto store = [&](int c, float x) {
        const float z = act_get<T>(static_cast<const T*>(a.gate)[static_cast<size_t>(n) * a.ld_gate + c0 + c]);
        const float w = a.norm_w ? a.norm_w[c0 + c] : 1.f;
        static_cast<T*>(a.y)[static_cast<size_t>(n) * a.ld_y + c0 + c] = act_put<T>(x * inv * w * gate_value(z, a.gate_act));
    };
#pragma unroll
    for (int e = 0; e < kCache; ++e)
        if (lane + e * kWave < r.vdim) store(lane + e * kWave, v[e]);
    for (int c = lane + kCache * kWave; c < r.vdim; c += kWave) store(c, row[c] * scale);
}

// ---- decode: one token per request -----------------------------------------------------------------
struct StepArgs {
    PieHipDecayRule rule;
    PieHipStateRows rows;
    const void* fused;
    const float *gates, *conv_w, *conv_bias, *skip;
    float *o, *den;
    const void* gate;
    const float* norm_w;
    void* y;
    int q_off, k_off, v_off, ld, ld_gates, channels, taps;
    int ld_gate, ld_y, gate_act;
    int cols, tpr_shift;   // value columns of a block; 1 << tpr_shift threads per state row, four columns each
    float out_scale, eps;
};
// A block per (slice of columns, head, request): its state rows are requested first and travel while
// the token's inputs and gates are formed; thread (row group, four columns) holds its share in registers.
template <class T, int NR>   // state rows per thread
__global__ __launch_bounds__(256) void decay_step_kernel(const StepArgs a) {
    __shared__ float x[512 + 512 + 256];   // q | k | v columns of this block
    __shared__ __attribute__((aligned(16))) float red[4][256];
    __shared__ float s_nq, s_oo[4];
    const PieHipDecayRule& r = a.rule;
    const int slice = blockIdx.x, h = blockIdx.y, req = blockIdx.z, tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const int dim = r.dim, kvh = h / (r.heads / r.kv_heads), col0 = slice * a.cols, cols = min(a.cols, r.vdim - col0);
    const bool fresh = a.rows.rs_fresh[req] != 0, stab = stabilised(r);
    const StateOf st = state_of(r, a.rows, req, h);
    const int tpr = 1 << a.tpr_shift, rg = tid >> a.tpr_shift, ngroups = 256 >> a.tpr_shift;
    const int cl = (tid & (tpr - 1)) * 4;
    const bool live = cl < cols;
    float* S = st.S + col0 + cl;
    f32x4_t s[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = rg + i * ngroups;
        s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (live && !fresh && d < dim) s[i] = *reinterpret_cast<const f32x4_t*>(S + static_cast<size_t>(d) * r.vdim);
    }
    float nv[8];   // n, on the first wave of the first slice
    const bool has_n = stab && slice == 0 && wv == 0;
    if (has_n)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int d = lane + e * kWave;
            nv[e] = !fresh && d < dim ? st.n[d] : 0.f;
        }
    const float m0 = stab && !fresh ? *st.m : 0.f;
    const T* row = static_cast<const T*>(a.fused) + static_cast<size_t>(req) * a.ld;
    const T* conv = a.conv_w ? conv_state_of<const T>(a.rows, req) : nullptr;
    for (int i = tid; i < 2 * dim + cols; i += 256) {
        const int c = i < dim ? a.q_off + kvh * dim + i
                              : i < 2 * dim ? a.k_off + kvh * dim + i - dim : a.v_off + h * r.vdim + col0 + i - 2 * dim;
        float v = act_get<T>(row[c]);
        if (a.conv_w) {
            const float* w = a.conv_w + static_cast<size_t>(c) * a.taps;
            float y = fmaf(w[a.taps - 1], v, a.conv_bias ? a.conv_bias[c] : 0.f);
            if (!fresh)
                for (int j = 0; j < a.taps - 1; ++j) y = fmaf(w[j], act_get<T>(conv[static_cast<size_t>(j) * a.channels + c]), y);
            v = act_get<T>(act_put<T>(y * sigmoid_f32(y)));   // (as the portions' convolution stores it)
        }
        x[i] = v;
    }
    const TokenGate tg = token_gate(r, a.gates + static_cast<size_t>(req) * a.ld_gates, h);
    const float m = stab ? fmaxf(tg.keep + m0, tg.in) : 0.f;
    const float keep = exp2f(tg.keep + m0 - m), weight = tg.weight * exp2f(tg.in - m);
    __syncthreads();
    if (has_n) {
        float nq = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int d = lane + e * kWave;
            if (d < dim) {
                nv[e] = fmaf(x[dim + d], weight, nv[e] * keep);
                nq = fmaf(nv[e], x[d], nq);
                st.n[d] = nv[e];
            }
        }
        nq = wave_sum_dpp(nq) * r.q_scale;
        if (lane == 0) {
            s_nq = nq;
            if (a.y) {
                *st.m = m;   // (the head's only block)
            } else {
                float* den = a.den + (static_cast<size_t>(req) * r.heads + h) * 2;
                den[0] = nq;
                den[1] = m;
            }
        }
    }
    f32x4_t v, dq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = live ? x[2 * dim + min(cl + e, cols - 1)] * weight : 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = rg + i * ngroups;
        if (d >= dim) break;
        const float kk = x[dim + d], qq = x[d];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            s[i][e] = fmaf(kk, v[e], s[i][e] * keep);
            dq[e] = fmaf(s[i][e], qq, dq[e]);
        }
        if (live) *reinterpret_cast<f32x4_t*>(S + static_cast<size_t>(d) * r.vdim) = s[i];
    }
    // over the row groups: inside a wave, then across the waves
    for (int off = tpr; off < kWave; off <<= 1)
#pragma unroll
        for (int e = 0; e < 4; ++e) dq[e] += __shfl_xor(dq[e], off, kWave);
    if (lane < tpr) *reinterpret_cast<f32x4_t*>(&red[wv][cl]) = dq;
    __syncthreads();
    float mine = 0.f;
    if (tid < cols) {
        mine = (red[0][tid] + red[1][tid] + red[2][tid] + red[3][tid]) * r.q_scale;
        if (a.skip) mine = fmaf(a.skip[h], x[2 * dim + tid], mine);
    }
    if (!a.y) {
        if (tid < cols) a.o[(static_cast<size_t>(req) * r.heads + h) * r.vdim + col0 + tid] = mine;
        return;
    }
    if (stab) mine /= exp_gate_divisor(s_nq, m);
    const float part = wave_sum_dpp(mine * mine);
    if (lane == 0) s_oo[wv] = part;
    __syncthreads();
    if (tid < cols) {
        const float inv = a.out_scale / sqrtf((s_oo[0] + s_oo[1] + s_oo[2] + s_oo[3]) / static_cast<float>(r.vdim) + a.eps);
        const int c = h * r.vdim + tid;
        const float z = act_get<T>(static_cast<const T*>(a.gate)[static_cast<size_t>(req) * a.ld_gate + c]);
        const float w = a.norm_w ? a.norm_w[c] : 1.f;
        static_cast<T*>(a.y)[static_cast<size_t>(req) * a.ld_y + c] = act_put<T>(mine * inv * w * gate_value(z, a.gate_act));
    }
}

// ---- gate, then norm over equal parts of the row ---------------------------------------------------
struct PartNormArgs {
    const float *o, *skip, *norm_w;
    const void *x, *z;
    void* y;
    PieHipStateRows rows;
    const void* conv_fused;
    int ld_x, ld_z, ld_y, heads, vdim, parts, ld_fused, channels, taps;
    float eps;
};
template <class T>
__global__ __launch_bounds__(256) void gated_part_norm_kernel(const PartNormArgs a) {
    __shared__ float red[4];
    const int part = blockIdx.x, n = blockIdx.y, inner = a.heads * a.vdim, len = inner / a.parts, c0 = part * len;
    const float* o = a.o + static_cast<size_t>(n) * inner;
    const T* z = static_cast<const T*>(a.z) + static_cast<size_t>(n) * a.ld_z;
    const T* x = a.x ? static_cast<const T*>(a.x) + static_cast<size_t>(n) * a.ld_x : nullptr;
    auto value = [&](int c) {
        float v = o[c];
        if (x) v = fmaf(a.skip[c / a.vdim], act_get<T>(x[c]), v);
        const float zz = act_get<T>(z[c]);
        return v * zz * sigmoid_f32(zz);
    };
    constexpr int kCache = 16;
    float v[kCache], local = 0.f;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int i = threadIdx.x + e * 256;
        v[e] = i < len ? value(c0 + i) : 0.f;
        local += v[e] * v[e];
    }
    for (int i = threadIdx.x + kCache * 256; i < len; i += 256) {
        const float t = value(c0 + i);
        local += t * t;
    }
    const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(len) + a.eps);
    T* y = static_cast<T*>(a.y) + static_cast<size_t>(n) * a.ld_y + c0;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int i = threadIdx.x + e * 256;
        if (i < len) y[i] = act_put<T>(v[e] * inv * a.norm_w[c0 + i]);
    }
    for (int i = threadIdx.x + kCache * 256; i < len; i += 256) y[i] = act_put<T>(value(c0 + i) * inv * a.norm_w[c0 + i]);
    if (!a.conv_fused) return;
    // one row per request: the convolution's state moves on by this row's inputs, a share per part
    const bool fresh = a.rows.rs_fresh[n] != 0;
    T* state = conv_state_of<T>(a.rows, n);
    const T* row = static_cast<const T*>(a.conv_fused) + static_cast<size_t>(n) * a.ld_fused;
    const int keep = a.taps - 1;
    for (int c = part * 256 + threadIdx.x; c < a.channels; c += a.parts * 256) {
        for (int j = 0; j + 1 < keep; ++j)
            state[static_cast<size_t>(j) * a.channels + c] = fresh ? act_put<T>(0.f) : state[static_cast<size_t>(j + 1) * a.channels + c];
        state[static_cast<size_t>(keep - 1) * a.channels + c] = row[c];
    }
}

bool rule_ok(const PieHipDecayRule* r) {
    if (!r || r->heads <= 0 || r->kv_heads <= 0 || r->heads % r->kv_heads != 0 || r->dim <= 0 || r->vdim <= 0) return false;
    if (r->kind == PIE_HIP_DECAY_FIXED) return r->decay != nullptr;
    if (r->kind == PIE_HIP_DECAY_EXP_GATES) return r->gate_bias != nullptr && r->gate_cap > 0.f;
    return r->kind == PIE_HIP_DECAY_STEP && r->decay && r->gate_bias;
}
bool rows_ok(const PieHipStateRows* s) {
    return s && s->row_req && s->qo_indptr && s->rs_slot && s->rs_fresh && s->rs_base && s->num_tokens > 0 && s->num_requests > 0;
}
bool gates_ok(const PieHipDecayRule* r, const float* gates, int ld) {
    if (r->kind == PIE_HIP_DECAY_FIXED) return true;
    return gates && ld >= (r->kind == PIE_HIP_DECAY_EXP_GATES ? 2 : 1) * r->heads;
}

// columns of a step's block: whole heads while the batch alone fills the device, else slices of at least
// 32 columns until it does
int step_cols(const PieHipDecayRule& r, int num_requests) {
    int cols = r.vdim <= 256 ? r.vdim : 256;
    while (cols > 32 && cols % 8 == 0 && static_cast<long long>(num_requests) * r.heads * ((r.vdim + cols - 1) / cols) < 256) cols /= 2;
    return cols;
}
int step_shift(int cols) {
    int sh = 0;
    while ((4 << sh) < cols) ++sh;
    return sh;
}
int step_rows_per_thread(int dim, int cols) {
    const int nr = (dim + (256 >> step_shift(cols)) - 1) / (256 >> step_shift(cols));
    return nr <= 4 ? 4 : nr <= 8 ? 8 : nr <= 16 ? 16 : nr <= 32 ? 32 : nr <= 64 ? 64 : 0;
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_conv_silu(int dtype, const void* fused, const float* conv_w, const float* conv_bias,
                                 const PieHipStateRows* rows, void* out, int ld, int channels, int taps, int ld_out,
                                 void* stream) {
    if (!fused || !conv_w || !rows_ok(rows) || !out || channels <= 0 || taps <= 0 || ld < channels || ld_out < channels)
        return PIE_HIP_ERR_INVALID;
    const int run = rows->num_tokens >= 1024 ? 16 : rows->num_tokens >= 128 ? 4 : 1;
    const dim3 grid((channels + 255) / 256, (rows->num_tokens + run - 1) / run);
    if (grid.y > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(conv_silu_kernel<T>, grid, dim3(256), 0, static_cast<hipStream_t>(stream),
                                                  static_cast<const T*>(fused), conv_w, conv_bias, *rows, static_cast<T*>(out), ld,
                                                  channels, taps, ld_out, run));
    return launch_status();
}

extern "C" int pie_hip_decay_scan(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const void* q,
                                  const void* k, const void* v, int ld, const float* gates, int ld_gates, float* o,
                                  float* den, void* stream) {
    if (!rule_ok(rule) || !rows_ok(rows) || !q || !k || !v || !o || ld < rule->heads * rule->vdim || ld < rule->kv_heads * rule->dim ||
        !gates_ok(rule, gates, ld_gates) || (rule->kind == PIE_HIP_DECAY_EXP_GATES && !den))
        return PIE_HIP_ERR_INVALID;
    const int cols = rule->vdim + (rule->kind == PIE_HIP_DECAY_EXP_GATES ? 1 : 0);
    const dim3 grid(rows->num_requests, rule->heads, (cols + 31) / 32);
    if (rule->dim > 512 || grid.y > 65535 || grid.z > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const ScanArgs a{*rule, *rows, q, k, v, gates, o, den, ld, ld_gates};
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int ni = (rule->dim + 31) / 32;
    PIE_ACT_DISPATCH(dtype, T, {
        if (ni <= 1) hipLaunchKernelGGL((decay_scan_kernel<T, 1, 16>), grid, dim3(256), 0, s, a);
        else if (ni <= 2) hipLaunchKernelGGL((decay_scan_kernel<T, 2, 16>), grid, dim3(256), 0, s, a);
        else if (ni <= 4) hipLaunchKernelGGL((decay_scan_kernel<T, 4, 16>), grid, dim3(256), 0, s, a);
        else if (ni <= 8) hipLaunchKernelGGL((decay_scan_kernel<T, 8, 16>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((decay_scan_kernel<T, 16, 8>), grid, dim3(256), 0, s, a);
    });
    return launch_status();
}

extern "C" size_t pie_hip_decay_chunked_workspace_bytes(const PieHipDecayRule* rule, int num_chunks) {
    if (!rule || rule->heads <= 0 || rule->kv_heads <= 0 || rule->dim <= 0 || rule->dim > 512 || rule->vdim <= 0 || num_chunks <= 0) return 0;
    const ChunkLayout l = chunk_layout(*rule);
    return static_cast<size_t>(num_chunks) * (rule->kv_heads * l.qk_elems * 2 + rule->heads * (l.vp_elems * 2 + l.meta_elems * 4));
}

extern "C" int pie_hip_decay_chunked(const PieHipDecayRule* rule, const PieHipStateRows* rows, const uint16_t* q,
                                     const uint16_t* k, const uint16_t* v, int ld, const float* gates, int ld_gates,
                                     float* o, float* den, const int32_t* chunks, const int32_t* req_chunks, int num_chunks,
                                     void* workspace, size_t workspace_bytes, void* stream) {
    if (!rule_ok(rule) || !rows_ok(rows) || !q || !k || !v || !o || !chunks || !req_chunks || num_chunks <= 0 ||
        ld < rule->heads * rule->vdim || ld < rule->kv_heads * rule->dim || !gates_ok(rule, gates, ld_gates) ||
        (rule->kind == PIE_HIP_DECAY_EXP_GATES && !den))
        return PIE_HIP_ERR_INVALID;
    if (rule->dim > 512 || num_chunks > 65535 || rows->num_requests > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    if (!workspace || workspace_bytes < pie_hip_decay_chunked_workspace_bytes(rule, num_chunks)) return PIE_HIP_ERR_INVALID;
    const ChunkLayout l = chunk_layout(*rule);
    uint16_t* qk = static_cast<uint16_t*>(workspace);
    uint16_t* vp = qk + static_cast<size_t>(num_chunks) * rule->kv_heads * l.qk_elems;
    float* meta = reinterpret_cast<float*>(vp + static_cast<size_t>(num_chunks) * rule->heads * l.vp_elems);
    auto whole = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
    const int aligned = whole(q) && whole(k) && whole(v) && ld % 8 == 0 && rule->dim % 8 == 0 && rule->vdim % 8 == 0;
    const ChunkArgs c{*rule, q, k, v, gates, chunks, qk, vp, meta, l, ld, ld_gates, aligned};
    const WalkArgs w{*rule, *rows, qk, vp, meta, req_chunks, o, den, l};
    hipStream_t s = static_cast<hipStream_t>(stream);
    hipLaunchKernelGGL(decay_chunk_kernel, dim3(rule->heads, num_chunks), dim3(256), 0, s, c);
    const dim3 grid(rule->heads, l.cols / kWalkCols, rows->num_requests);
    if (grid.y > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch (l.dimp) {
        case 32: hipLaunchKernelGGL((decay_walk_kernel<1, 1>), grid, dim3(64), 0, s, w); break;
        case 64: hipLaunchKernelGGL((decay_walk_kernel<2, 1>), grid, dim3(128), 0, s, w); break;
        case 128: hipLaunchKernelGGL((decay_walk_kernel<4, 1>), grid, dim3(256), 0, s, w); break;
        case 256: hipLaunchKernelGGL((decay_walk_kernel<4, 2>), grid, dim3(256), 0, s, w); break;
        default: hipLaunchKernelGGL((decay_walk_kernel<4, 4>), grid, dim3(256), 0, s, w); break;
    }
    return launch_status();
}

extern "C" int pie_hip_decay_out(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const float* o,
                                 const float* den, const void* gate, int ld_gate, int gate_act, const float* norm_w,
                                 void* y, int ld_y, float out_scale, float eps, void* stream) {
    if (!rule_ok(rule) || !rows_ok(rows) || !o || !gate || !y || ld_gate < rule->heads * rule->vdim || ld_y < rule->heads * rule->vdim ||
        (rule->kind == PIE_HIP_DECAY_EXP_GATES && !den))
        return PIE_HIP_ERR_INVALID;
    const OutArgs a{*rule, *rows, o, den, norm_w, gate, y, ld_gate, ld_y, gate_act ? 1 : 0, out_scale, eps};
    const long long units = static_cast<long long>(rows->num_tokens) * rule->heads;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(decay_out_kernel<T>, dim3(static_cast<unsigned>((units + 3) / 4)), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), a));
    return launch_status();
}

extern "C" int pie_hip_decay_step_supported(int dim, int vdim) {
    if (dim <= 0 || vdim <= 0 || dim > 512 || vdim > 1024 || vdim % 4 != 0) return 0;
    return step_rows_per_thread(dim, vdim <= 256 ? vdim : 256) > 0;
}

extern "C" int pie_hip_decay_step_fuses(const PieHipDecayRule* rule, int num_requests) {
    return rule && pie_hip_decay_step_supported(rule->dim, rule->vdim) && step_cols(*rule, num_requests) >= rule->vdim;
}

extern "C" int pie_hip_decay_step(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const void* fused,
                                  int q_off, int k_off, int v_off, int ld, const float* gates, int ld_gates,
                                  const float* conv_w, const float* conv_bias, int channels, int taps, const float* skip,
                                  float* o, float* den, const void* gate, int ld_gate, int gate_act, const float* norm_w,
                                  void* y, int ld_y, float out_scale, float eps, void* stream) {
    if (!rule_ok(rule) || !rows_ok(rows) || !fused || q_off < 0 || k_off < 0 || v_off < 0 || q_off + rule->kv_heads * rule->dim > ld ||
        k_off + rule->kv_heads * rule->dim > ld || v_off + rule->heads * rule->vdim > ld || !gates_ok(rule, gates, ld_gates) ||
        rows->num_tokens != rows->num_requests)
        return PIE_HIP_ERR_INVALID;
    const int width = rule->heads * rule->vdim;
    if (conv_w && (taps <= 0 || channels < q_off + rule->kv_heads * rule->dim || channels < k_off + rule->kv_heads * rule->dim ||
                   channels < v_off + width))
        return PIE_HIP_ERR_INVALID;
    if (y ? !gate || ld_gate < width || ld_y < width : !o || (rule->kind == PIE_HIP_DECAY_EXP_GATES && !den)) return PIE_HIP_ERR_INVALID;
    if (!pie_hip_decay_step_supported(rule->dim, rule->vdim) || rows->num_requests > 65535 || rule->heads > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const int cols = step_cols(*rule, rows->num_requests);
    if (y && cols < rule->vdim) return PIE_HIP_ERR_UNSUPPORTED;
    const StepArgs a{*rule, *rows, fused, gates, conv_w, conv_bias, skip, o, den, gate, norm_w, y, q_off, k_off, v_off, ld, ld_gates,
                     channels, taps, ld_gate, ld_y, gate_act ? 1 : 0, cols, step_shift(cols), out_scale, eps};
    const dim3 grid((rule->vdim + cols - 1) / cols, rule->heads, rows->num_requests);
    hipStream_t s = static_cast<hipStream_t>(stream);
    PIE_ACT_DISPATCH(dtype, T, switch (step_rows_per_thread(rule->dim, cols)) {
        case 4: hipLaunchKernelGGL((decay_step_kernel<T, 4>), grid, dim3(256), 0, s, a); break;
        case 8: hipLaunchKernelGGL((decay_step_kernel<T, 8>), grid, dim3(256), 0, s, a); break;
        case 16: hipLaunchKernelGGL((decay_step_kernel<T, 16>), grid, dim3(256), 0, s, a); break;
        case 32: hipLaunchKernelGGL((decay_step_kernel<T, 32>), grid, dim3(256), 0, s, a); break;
        case 64: hipLaunchKernelGGL((decay_step_kernel<T, 64>), grid, dim3(256), 0, s, a); break;
        default: return PIE_HIP_ERR_UNSUPPORTED;
    });
    return launch_status();
}

extern "C" int pie_hip_gated_part_norm(int dtype, const float* o, const void* x, int ld_x, const float* skip, const void* z,
                                       int ld_z, const float* norm_w, void* y, int ld_y, int heads, int vdim, int parts,
                                       const PieHipStateRows* rows, const void* conv_fused, int ld_fused, int channels,
                                       int taps, float eps, void* stream) {
    if (!o || !z || !norm_w || !y || heads <= 0 || vdim <= 0 || parts <= 0 || (heads * vdim) % parts != 0 || ld_z < heads * vdim ||
        ld_y < heads * vdim || (x && (!skip || ld_x < heads * vdim)) || !rows_ok(rows))
        return PIE_HIP_ERR_INVALID;
    if (taps <= 1) conv_fused = nullptr;
    if (conv_fused && (rows->num_tokens != rows->num_requests || channels <= 0 || ld_fused < channels)) return PIE_HIP_ERR_INVALID;
    if (rows->num_tokens > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const PartNormArgs a{o, skip, norm_w, x, z, y, *rows, conv_fused, ld_x, ld_z, ld_y, heads, vdim, parts, ld_fused, channels, taps, eps};
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(gated_part_norm_kernel<T>, dim3(parts, rows->num_tokens), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), a));
    return launch_status();
}
