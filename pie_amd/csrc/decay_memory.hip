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
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

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
// A thread takes V neighbouring channels of a run of rows and walks it with the last four inputs in
// registers, G rows requested ahead; longer convolutions read their window afresh.
template <class T, int V, int G>
__global__ __launch_bounds__(256) void conv_silu_kernel(const T* __restrict__ fused, const float* __restrict__ w,
                                                        const float* __restrict__ bias, const PieHipStateRows rows,
                                                        T* __restrict__ out, int ld, int channels, int taps, int ld_out,
                                                        int run, int move_state) {
    typedef T vec_t __attribute__((ext_vector_type(V)));
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= channels) return;   // (channels is a multiple of V)
    const int n0 = blockIdx.y * run, n1 = min(n0 + run, rows.num_tokens), keep = taps - 1;
    const bool windowed = taps <= 4;
    float b[V], wr[V][4], win[V][4];
#pragma unroll
    for (int e = 0; e < V; ++e) {
        b[e] = bias ? bias[c + e] : 0.f;
        const float* wc = w + static_cast<size_t>(c + e) * taps;
        f32x4_t w4 = {0.f, 0.f, 0.f, 0.f};
        if (taps == 4) w4 = *reinterpret_cast<const f32x4_t*>(wc);   // (the table starts 16-byte aligned)
        else if (windowed)
#pragma unroll
            for (int j = 1; j < 4; ++j) w4[j] = j >= 4 - taps ? wc[j - (4 - taps)] : 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            wr[e][j] = w4[j];
            win[e][j] = 0.f;
        }
    }
    int row0 = 0, row1 = n0;
    bool fresh = false;
    T* state = nullptr;
    auto input = [&](int i, int e) {   // the request's input i (negative: from the state)
        if (i >= 0) return act_get<T>(fused[static_cast<size_t>(row0 + i) * ld + c + e]);
        return fresh ? 0.f : act_get<T>(state[static_cast<size_t>(keep + i) * channels + c + e]);
    };
    vec_t next[G];
    auto request = [&](int n) {
#pragma unroll
        for (int u = 0; u < G; ++u)
            if (n + u < n1) next[u] = *reinterpret_cast<const vec_t*>(fused + static_cast<size_t>(n + u) * ld + c);
    };
    request(n0);
    for (int nb = n0; nb < n1; nb += G) {
        vec_t group[G];
#pragma unroll
        for (int u = 0; u < G; ++u) group[u] = next[u];
        request(nb + G);
#pragma unroll
        for (int u = 0; u < G; ++u) {
            const int n = nb + u;
            if (n >= n1) break;
            const bool enter = n >= row1;
            if (enter) {
                const int r = rows.row_req[n];
                row0 = rows.qo_indptr[r];
                row1 = rows.qo_indptr[r + 1];
                fresh = rows.rs_fresh[r] != 0;
                state = conv_state_of<T>(rows, r);
            }
            const int i = n - row0;
            vec_t o;
#pragma unroll
            for (int e = 0; e < V; ++e) {
                float y = b[e];
                if (windowed) {
                    if (enter)
#pragma unroll
                        for (int j = 1; j < 4; ++j) win[e][j] = 4 - j <= keep ? input(i - (4 - j), e) : 0.f;
#pragma unroll
                    for (int j = 0; j < 3; ++j) win[e][j] = win[e][j + 1];
                    win[e][3] = act_get<T>(group[u][e]);
#pragma unroll
                    for (int j = 0; j < 4; ++j) y = fmaf(wr[e][j], win[e][j], y);
                } else {
                    for (int j = 0; j < taps; ++j) y = fmaf(w[static_cast<size_t>(c + e) * taps + j], input(i - keep + j, e), y);
                }
                o[e] = act_put<T>(y * sigmoid_f32(y));
            }
            *reinterpret_cast<vec_t*>(out + static_cast<size_t>(n) * ld_out + c) = o;
            if (move_state) {   // one row per request: nobody else reads these channels of its state
                for (int j = 0; j < keep; ++j)
#pragma unroll
                    for (int e = 0; e < V; ++e)
                        state[static_cast<size_t>(j) * channels + c + e] =
                            j + 1 == keep ? group[u][e] : fresh ? act_put<T>(0.f) : state[static_cast<size_t>(j + 1) * channels + c + e];
            }
        }
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
//   P[t, s] = q_t . k_s  u_s 2^(F_t - F_s + i_s - M_t),  s <= t
//   o_t     = 2^(F_t + m_0 - m_t) S_0^T q_t + 2^(M_t - m_t) sum_s P[t, s] v_s
//   S       = 2^(F_64 + m_0 - m_64) S_0 + 2^(M_64 - m_64) sum_s k_s (u_s 2^(F_64 - F_s + i_s - M_64) v_s)^T
// All exponents are <= 0.  What does not need the state — sum_s P v_s, the weighted values — is formed for
// all chunks at once (decay_chunk_kernel) and laid out in the order the matrix instructions' lanes load
// it; decay_walk_kernel carries the state from chunk to chunk in registers.  Queries, keys and values are
// exact bf16; P, the weighted values and the state enter their products as hi + lo pairs of bf16 values.
//
// Record of a (chunk, head of keys): Q [4 token tiles][dimp / 32][64 lanes][8], K^T [dimp / 16][2][64][8];
// of a (chunk, head): weighted V^T [cols / 16][2][hi, lo][64][8], then fp32 sums [4 token tiles][cols / 16]
// [64][4]; fp32 per token F (q_scale 2^F without exponential gates), M, and the chunk's totals.
// The k-slots of every product take a tile pair's rows in the order the accumulators hold them: slot
// (g, e) of lane group g is row 4 g + e of the first tile for e < 4, of the second for e >= 4.
constexpr int kChunk = 64, kPiece = 64, kPieceStride = kPiece + 8;

struct ChunkLayout {
    int dimp, ctiles;                                       // dim rounded up; 16-column tiles, an even number
    size_t qk_elems, kt_off, v_elems, sum_elems, meta_elems;   // bf16, fp32, fp32
};
inline int walk_dimp(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 512; }
inline ChunkLayout chunk_layout(const PieHipDecayRule& r) {
    ChunkLayout l;
    l.dimp = walk_dimp(r.dim);
    const int cols = r.vdim + (r.kind == PIE_HIP_DECAY_EXP_GATES ? 1 : 0);
    l.ctiles = (cols + 31) / 32 * 2;
    l.kt_off = static_cast<size_t>(kChunk) * l.dimp;
    l.qk_elems = 2 * l.kt_off;
    l.v_elems = static_cast<size_t>(kChunk) * l.ctiles * 32;
    l.sum_elems = static_cast<size_t>(kChunk) * l.ctiles * 16;
    l.meta_elems = 2 * kChunk + 8;
    return l;
}

struct ChunkArgs {
    PieHipDecayRule rule;
    const uint16_t *q, *k, *v;
    const float* gates;
    const int32_t* chunks;
    uint16_t *qk_rec, *v_rec;
    float *sum_rec, *meta;
    ChunkLayout lay;
    int ld, ld_gates, aligned;   // aligned: 16-byte pieces of q, k, v rows can be loaded whole
};

// 64 columns from c0 on of the chunk's rows, zeros past the rows and columns that exist, one more column of
// ones at `ones_col` (negative: none): a thread takes 16 columns of a row to registers, then to LDS.
struct Piece {
    u32x4_t a, b;
};
__device__ __forceinline__ Piece fetch_piece(const uint16_t* __restrict__ src, int ld, int nt, int c0, int n_cols, bool aligned, int ones_col) {
    const int t = threadIdx.x >> 2, part = (threadIdx.x & 3) * 16;
    Piece p{{0u, 0u, 0u, 0u}, {0u, 0u, 0u, 0u}};
    if (t >= nt) return p;
    const uint16_t* row = src + static_cast<size_t>(t) * ld + c0 + part;
    if (aligned && c0 + part + 16 <= n_cols) {
        p.a = *reinterpret_cast<const u32x4_t*>(row);
        p.b = *reinterpret_cast<const u32x4_t*>(row + 8);
        return p;
    }
#pragma unroll
    for (int e = 0; e < 16; ++e) {
        const int c = c0 + part + e;
        uint32_t x = 0;
        if (c < n_cols) x = row[e];
        else if (c == ones_col) x = 0x3F80;
        if (e < 8) p.a[e >> 1] |= x << (16 * (e & 1));
        else p.b[(e - 8) >> 1] |= x << (16 * (e & 1));
    }
    return p;
}
__device__ __forceinline__ void put_piece(uint16_t* dst, const Piece& p) {
    uint16_t* d = dst + (threadIdx.x >> 2) * kPieceStride + (threadIdx.x & 3) * 16;
    *reinterpret_cast<u32x4_t*>(d) = p.a;
    *reinterpret_cast<u32x4_t*>(d + 8) = p.b;
}
// column c0 + lane % 16 of a staged piece, the 8 tokens of k-slot group g of token step ks
__device__ __forceinline__ bf16x8_t piece_tokens(const uint16_t* piece, int c0, int ks, int l16, int g) {
    const uint16_t* p = piece + (32 * ks + 4 * g + (l16 >> 2)) * kPieceStride + c0 + 4 * (l16 & 3);
    const bf16x4_t a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(p));
    const bf16x4_t b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(p + 16 * kPieceStride));
    return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}
// eight fp32 values as a hi (truncated) and a lo bf16 value each
__device__ __forceinline__ void split8(const float* x, u32x4_t& hi, u32x4_t& lo) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const uint32_t u0 = __float_as_uint(x[2 * e]), u1 = __float_as_uint(x[2 * e + 1]);
        hi[e] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
        lo[e] = pack_bf16x2(x[2 * e] - __uint_as_float(u0 & 0xFFFF0000u), x[2 * e + 1] - __uint_as_float(u1 & 0xFFFF0000u));
    }
}
__device__ __forceinline__ f32x4_t mfma_bf16(const u32x4_t a, const bf16x8_t b, const f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), b, c, 0, 0, 0);
}

__global__ __launch_bounds__(256) void decay_chunk_kernel(const ChunkArgs a) {
    __shared__ __attribute__((aligned(16))) uint16_t tiles[2][2][kChunk * kPieceStride];   // two steps' queries and keys, or values
    __shared__ __attribute__((aligned(16))) float s_top[kChunk], s_top_lo[kChunk], s_in[kChunk], s_in_lo[kChunk], s_u[kChunk], s_w[kChunk];
    const PieHipDecayRule& r = a.rule;
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x, lane = tid & (kWave - 1);
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave), l16 = lane & 15, g = lane >> 4;
    const int row0 = a.chunks[2 * ch], nt = a.chunks[2 * ch + 1];
    const int ratio = r.heads / r.kv_heads, kvh = h / ratio;
    const bool lead = h % ratio == 0, stab = stabilised(r);
    const size_t rec = static_cast<size_t>(ch) * r.heads + h;
    uint16_t* qk = a.qk_rec + (static_cast<size_t>(ch) * r.kv_heads + kvh) * a.lay.qk_elems;
    if (wv == 0) {
        TokenGate tg{0.f, stab ? -INFINITY : 0.f, 0.f};   // tokens past the portion: decay 1, weight 0
        if (lane < nt) tg = token_gate(r, a.gates + static_cast<size_t>(row0 + lane) * a.ld_gates, h);
        // (running sums in double: differences of two of them stay right to the last bit however fast the
        // head forgets)
        double F = tg.keep;
#pragma unroll
        for (int off = 1; off < kWave; off <<= 1) {
            const double up = __shfl_up(F, off, kWave);
            if (lane >= off) F += up;
        }
        const double in = static_cast<double>(tg.in) - F;
        double M = 0.0;
        if (stab) {
            double mx = in;
#pragma unroll
            for (int off = 1; off < kWave; off <<= 1) {
                const double up = __shfl_up(mx, off, kWave);
                if (lane >= off) mx = fmax(mx, up);
            }
            M = F + mx;
        }
        const double F_end = __shfl(F, kWave - 1, kWave), M_end = __shfl(M, kWave - 1, kWave), top = F - M;
        s_top[lane] = static_cast<float>(top);
        s_top_lo[lane] = static_cast<float>(top - s_top[lane]);
        s_in[lane] = static_cast<float>(in);
        s_in_lo[lane] = lane < nt ? static_cast<float>(in - s_in[lane]) : 0.f;
        s_u[lane] = tg.weight;
        s_w[lane] = tg.weight * exp2f(static_cast<float>(F_end + in - M_end));
        float* meta = a.meta + rec * a.lay.meta_elems;
        meta[lane] = stab ? static_cast<float>(F) : r.q_scale * exp2f(static_cast<float>(F));
        meta[kChunk + lane] = static_cast<float>(M);
        if (lane == 0) {
            meta[2 * kChunk] = stab ? static_cast<float>(F_end) : exp2f(static_cast<float>(F_end));
            meta[2 * kChunk + 1] = static_cast<float>(M_end);
        }
    }
    // scores: wave w takes query tile w against key tiles 0 .. w
    f32x4_t acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const uint16_t* qp = a.q + static_cast<size_t>(row0) * a.ld + kvh * r.dim;
    const uint16_t* kp = a.k + static_cast<size_t>(row0) * a.ld + kvh * r.dim;
    const int ksteps = a.lay.dimp / 32;
    const uint16_t* vsrc = a.v + static_cast<size_t>(row0) * a.ld + h * r.vdim;
    auto fetch_v = [&](int c0) { return fetch_piece(vsrc, a.ld, nt, c0, r.vdim, a.aligned, stab ? r.vdim : -1); };
    // (a step's pieces are requested while the step before is multiplied; tiles alternate, one barrier a step)
    int buf = 0;
    Piece nq = fetch_piece(qp, a.ld, nt, 0, r.dim, a.aligned, -1), nk = fetch_piece(kp, a.ld, nt, 0, r.dim, a.aligned, -1);
    Piece nv = fetch_v(0);
    for (int d0 = 0; d0 < a.lay.dimp; d0 += kPiece, buf ^= 1) {
        uint16_t *sq = tiles[buf][0], *sk = tiles[buf][1];
        put_piece(sq, nq);
        put_piece(sk, nk);
        if (d0 + kPiece < a.lay.dimp) {
            nq = fetch_piece(qp, a.ld, nt, d0 + kPiece, r.dim, a.aligned, -1);
            nk = fetch_piece(kp, a.ld, nt, d0 + kPiece, r.dim, a.aligned, -1);
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const bf16x8_t qf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&sq[(16 * wv + l16) * kPieceStride + 32 * j + 8 * g]));
#pragma unroll
            for (int st = 0; st < 4; ++st)
                if (st <= wv) acc[st] = mfma_bf16(*reinterpret_cast<const u32x4_t*>(&sk[(16 * st + l16) * kPieceStride + 32 * j + 8 * g]), qf, acc[st]);
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
                    __builtin_bit_cast(u32x4_t, piece_tokens(sk, 16 * wv, ks, l16, g));
    }
    // P of this wave's query tile, in the order of the k-slots
    u32x4_t p_hi[2], p_lo[2];
    {
        const int t = 16 * wv + l16;
        const float top = s_top[t], top_lo = s_top_lo[t];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            float x[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int s = 32 * ks + 16 * (e >> 2) + 4 * g + (e & 3);
                x[e] = s <= t ? acc[2 * ks + (e >> 2)][e & 3] * (r.q_scale * s_u[s] * exp2f((top + s_in[s]) + (top_lo + s_in_lo[s]))) : 0.f;
            }
            split8(x, p_hi[ks], p_lo[ks]);
        }
    }
    uint16_t* vr = a.v_rec + rec * a.lay.v_elems;
    float* sums = a.sum_rec + rec * a.lay.sum_elems;
    for (int c0 = 0; c0 < a.lay.ctiles * 16; c0 += kPiece, buf ^= 1) {
        uint16_t* sq = tiles[buf][0];
        put_piece(sq, nv);
        if (c0 + kPiece < a.lay.ctiles * 16) nv = fetch_v(c0 + kPiece);
        __syncthreads();
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) {
            const int tile = c0 / 16 + ct;
            if (tile >= a.lay.ctiles) break;
            f32x4_t pv = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                if (ks == 1 && wv < 2 && ct != wv) continue;   // (keys past this tile's queries)
                const bf16x8_t vf = piece_tokens(sq, 16 * ct, ks, l16, g);
                pv = mfma_bf16(p_hi[ks], vf, pv);
                pv = mfma_bf16(p_lo[ks], vf, pv);
                if (ct == wv) {
                    const u32x4_t raw = __builtin_bit_cast(u32x4_t, vf);
                    const f32x4_t w0 = *reinterpret_cast<const f32x4_t*>(&s_w[32 * ks + 4 * g]), w1 = *reinterpret_cast<const f32x4_t*>(&s_w[32 * ks + 16 + 4 * g]);
                    const float x[8] = {bf16_lo(raw[0]) * w0[0], bf16_hi(raw[0]) * w0[1], bf16_lo(raw[1]) * w0[2], bf16_hi(raw[1]) * w0[3],
                                        bf16_lo(raw[2]) * w1[0], bf16_hi(raw[2]) * w1[1], bf16_lo(raw[3]) * w1[2], bf16_hi(raw[3]) * w1[3]};
                    u32x4_t hi, lo;
                    split8(x, hi, lo);
                    uint16_t* d = vr + (static_cast<size_t>(tile * 2 + ks) * 2 * kWave + lane) * 8;
                    *reinterpret_cast<u32x4_t*>(d) = hi;
                    *reinterpret_cast<u32x4_t*>(d + kWave * 8) = lo;
                }
            }
            *reinterpret_cast<f32x4_t*>(sums + ((static_cast<size_t>(wv) * a.lay.ctiles + tile) * kWave + lane) * 4) = pv;
        }
    }
}

struct WalkArgs {
    PieHipDecayRule rule;
    PieHipStateRows rows;
    const uint16_t *qk_rec, *v_rec;
    const float *sum_rec, *meta;
    const int32_t* req_chunks;
    float *o, *den;
    ChunkLayout lay;
};

// A block takes CT tiles of 16 value columns of one head of one request; wave w keeps rows 32 ND w .. of S
// as accumulator tiles, which are B operands of the read-out as they are (converted to hi + lo).  The
// waves' partial read-outs meet in LDS, one barrier per chunk; wave w finishes token tiles w, w + NW, ..
template <int NW, int ND, int CT, bool STAB>
__global__ __launch_bounds__(NW* kWave, 1) void decay_walk_kernel(const WalkArgs a) {
    constexpr int KSTEPS = NW * ND, OWN = 4 / NW;
    __shared__ __attribute__((aligned(16))) float part[NW > 1 ? 2 : 1][NW > 1 ? NW : 1][4][CT][NW > 1 ? kWave * 4 : 4];
    const PieHipDecayRule& r = a.rule;
    const int h = blockIdx.x, slice = blockIdx.y, req = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int c_lo = a.req_chunks[req], c_hi = a.req_chunks[req + 1];
    const int req_row0 = a.rows.qo_indptr[req], req_row1 = a.rows.qo_indptr[req + 1];
    const int kvh = h / (r.heads / r.kv_heads), vd = r.heads * r.vdim;
    const bool fresh = a.rows.rs_fresh[req] != 0;
    const StateOf st = state_of(r, a.rows, req, h);
    const int wrow = 32 * ND * wv;
    f32x4_t s[2 * ND][CT];
    int col[CT];
    float* S[CT];
    size_t stride[CT];
    bool live[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        col[c] = (slice * CT + c) * 16 + l16;
        const bool is_n = STAB && col[c] == r.vdim;   // (column vdim is n: rows one apart instead of vdim)
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
    const bool whole_cols = (slice + 1) * CT * 16 <= r.vdim;
    float m0 = STAB && !fresh ? *st.m : 0.f;
    // (a zero the compiler takes for a lane's own value: a chunk's totals come through vector loads, since a
    // scalar load on its way holds up every wait for LDS)
    int zero;
    asm("v_mov_b32 %0, 0" : "=v"(zero));
    struct Frags {
        u32x4_t q[4][ND], kt[2 * ND][2], v[CT][2][2];
        f32x4_t sum[OWN][CT], f[OWN], m[STAB ? OWN : 1];
        float f_end, m_end;
    };
    auto load = [&](Frags& f, int c) {
        const uint16_t* qk = a.qk_rec + (static_cast<size_t>(c) * r.kv_heads + kvh) * a.lay.qk_elems + lane * 8;
        const uint16_t* kt = qk + a.lay.kt_off;
        const size_t rec = static_cast<size_t>(c) * r.heads + h;
        const uint16_t* v = a.v_rec + rec * a.lay.v_elems + lane * 8;
        const float* sum = a.sum_rec + rec * a.lay.sum_elems + lane * 4;
        const float* meta = a.meta + rec * a.lay.meta_elems;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int j = 0; j < ND; ++j) f.q[t][j] = *reinterpret_cast<const u32x4_t*>(qk + (t * KSTEPS + wv * ND + j) * kWave * 8);
#pragma unroll
        for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) f.kt[i][ks] = *reinterpret_cast<const u32x4_t*>(kt + ((wv * 2 * ND + i) * 2 + ks) * kWave * 8);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                for (int u = 0; u < 2; ++u)
                    f.v[ct][ks][u] = *reinterpret_cast<const u32x4_t*>(v + (((slice * CT + ct) * 2 + ks) * 2 + u) * kWave * 8);
#pragma unroll
        for (int k = 0; k < OWN; ++k) {
            const int t = wv + NW * k;
#pragma unroll
            for (int ct = 0; ct < CT; ++ct)
                f.sum[k][ct] = *reinterpret_cast<const f32x4_t*>(sum + (t * a.lay.ctiles + slice * CT + ct) * kWave * 4);
            f.f[k] = *reinterpret_cast<const f32x4_t*>(meta + 16 * t + 4 * g);
            if constexpr (STAB) f.m[k] = *reinterpret_cast<const f32x4_t*>(meta + kChunk + 16 * t + 4 * g);
        }
        f.f_end = meta[2 * kChunk + zero];
        if constexpr (STAB) f.m_end = meta[2 * kChunk + 1 + zero];
    };
    auto run = [&](const Frags& f, int c, int buf) {
        // the state's part of the read-out, this wave's rows
        f32x4_t inter[4][CT];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) inter[t][ct] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < ND; ++j)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                const f32x4_t s0 = s[2 * j][ct], s1 = s[2 * j + 1][ct];
                const float x[8] = {s0[0], s0[1], s0[2], s0[3], s1[0], s1[1], s1[2], s1[3]};
                u32x4_t hi, lo;
                split8(x, hi, lo);
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    inter[t][ct] = mfma_bf16(f.q[t][j], __builtin_bit_cast(bf16x8_t, hi), inter[t][ct]);
                    inter[t][ct] = mfma_bf16(f.q[t][j], __builtin_bit_cast(bf16x8_t, lo), inter[t][ct]);
                }
            }
        if constexpr (NW > 1) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int ct = 0; ct < CT; ++ct) *reinterpret_cast<f32x4_t*>(&part[buf][wv][t][ct][lane * 4]) = inter[t][ct];
        }
        // the state moves on
        float keep = f.f_end, add = 1.f, m_end = 0.f;
        if constexpr (STAB) {
            m_end = fmaxf(f.f_end + m0, f.m_end);
            keep = __builtin_amdgcn_exp2f(f.f_end + m0 - m_end);
            add = __builtin_amdgcn_exp2f(f.m_end - m_end);
        }
#pragma unroll
        for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                f32x4_t x = STAB ? f32x4_t{0.f, 0.f, 0.f, 0.f} : s[i][ct] * keep;
#pragma unroll
                for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                    for (int u = 0; u < 2; ++u) x = mfma_bf16(f.kt[i][ks], __builtin_bit_cast(bf16x8_t, f.v[ct][ks][u]), x);
                if constexpr (STAB)
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[i][ct][e] = fmaf(s[i][ct][e], keep, x[e] * add);
                else s[i][ct] = x;
            }
        if constexpr (NW > 1) __syncthreads();   // (the buffer's readers of two chunks ago have passed the last barrier)
        // this wave's token tiles
        const int row0 = req_row0 + (c - c_lo) * kChunk, nt = min(kChunk, req_row1 - row0);
        f32x4_t x[OWN][CT];
#pragma unroll
        for (int k = 0; k < OWN; ++k)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                if constexpr (NW > 1) {
                    f32x4_t y[NW];
#pragma unroll
                    for (int w = 0; w < NW; ++w) y[w] = *reinterpret_cast<const f32x4_t*>(&part[buf][w][wv + NW * k][ct][lane * 4]);
                    x[k][ct] = y[0];
#pragma unroll
                    for (int w = 1; w < NW; ++w) x[k][ct] += y[w];
                } else {
                    x[k][ct] = inter[k][ct];
                }
            }
#pragma unroll
        for (int k = 0; k < OWN; ++k) {
            const int t = wv + NW * k;
            f32x4_t m_t, fi = f.f[k], fa;
            if constexpr (STAB)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    m_t[e] = fmaxf(f.f[k][e] + m0, f.m[k][e]);
                    fi[e] = r.q_scale * __builtin_amdgcn_exp2f(f.f[k][e] + m0 - m_t[e]);
                    fa[e] = __builtin_amdgcn_exp2f(f.m[k][e] - m_t[e]);
                }
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                f32x4_t o;
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] = fmaf(x[k][ct][e], fi[e], STAB ? f.sum[k][ct][e] * fa[e] : f.sum[k][ct][e]);
                const int tok = 16 * t + 4 * g;
                float* dst = a.o + static_cast<size_t>(row0 + tok) * vd + h * r.vdim + col[ct];
                if (whole_cols && nt == kChunk) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) dst[static_cast<size_t>(e) * vd] = o[e];
                    continue;
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (tok + e >= nt) continue;
                    if (col[ct] < r.vdim) {
                        dst[static_cast<size_t>(e) * vd] = o[e];
                    } else if (STAB && live[ct]) {
                        float* den = a.den + (static_cast<size_t>(row0 + tok + e) * r.heads + h) * 2;
                        den[0] = o[e];
                        den[1] = m_t[e];
                    }
                }
            }
        }
        m0 = m_end;
    };
    // (records come from beyond the L2: as many chunks ahead as the registers take)
    constexpr int kBufs = ND == 4 ? 1 : 3;
    Frags f[kBufs];
#pragma unroll
    for (int i = 0; i < kBufs - 1; ++i) load(f[i], min(c_lo + i, c_hi - 1));
    for (int c = c_lo; c < c_hi; c += kBufs) {
#pragma unroll
        for (int i = 0; i < kBufs; ++i) {
            load(f[(i + kBufs - 1) % kBufs], min(c + i + kBufs - 1, c_hi - 1));
            __builtin_amdgcn_sched_barrier(0);
            if (c + i < c_hi) run(f[i], c + i, (c - c_lo + i) & 1);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
#pragma unroll
    for (int c = 0; c < CT; ++c)
        if (live[c])
#pragma unroll
            for (int i = 0; i < 2 * ND; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int d = wrow + 16 * i + 4 * g + e;
                    if (d < r.dim) S[c][d * stride[c]] = s[i][c][e];
                }
}

template <int NW, int ND>
void launch_walk(const WalkArgs& w, int num_requests, hipStream_t s) {
    // (one tile of columns per block while the blocks are all resident: two per CU, one with longer rows)
    const bool one = static_cast<long long>(w.rule.heads) * w.lay.ctiles * num_requests <= (ND == 1 ? 512 : 256);
    const dim3 grid(w.rule.heads, one ? w.lay.ctiles : w.lay.ctiles / 2, num_requests), block(NW * kWave);
    if (w.rule.kind == PIE_HIP_DECAY_EXP_GATES) {
        if (one) hipLaunchKernelGGL((decay_walk_kernel<NW, ND, 1, true>), grid, block, 0, s, w);
        else hipLaunchKernelGGL((decay_walk_kernel<NW, ND, 2, true>), grid, block, 0, s, w);
    } else {
        if (one) hipLaunchKernelGGL((decay_walk_kernel<NW, ND, 1, false>), grid, block, 0, s, w);
        else hipLaunchKernelGGL((decay_walk_kernel<NW, ND, 2, false>), grid, block, 0, s, w);
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
// four consecutive values of an 8- (bf16) or 16-byte (fp32) aligned address
template <class T>
__device__ __forceinline__ f32x4_t load4(const T* p) {
    if constexpr (sizeof(T) == 2) {
        const u32x2_t r = *reinterpret_cast<const u32x2_t*>(p);
        return f32x4_t{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)};
    } else {
        return *reinterpret_cast<const f32x4_t*>(p);
    }
}
template <class T>
__device__ __forceinline__ void store4(T* p, const f32x4_t v) {
    if constexpr (sizeof(T) == 2) *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
    else *reinterpret_cast<f32x4_t*>(p) = v;
}
// One wave per (row, head); V: values per lane and access.
template <class T, int V>
__global__ __launch_bounds__(256) void decay_out_kernel(const OutArgs a) {
    const PieHipDecayRule& r = a.rule;
    const int unit = blockIdx.x * 4 + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    if (unit >= a.rows.num_tokens * r.heads) return;
    const int n = unit / r.heads, h = unit % r.heads, c0 = h * r.vdim;
    const float* row = a.o + static_cast<size_t>(n) * r.heads * r.vdim + c0;
    const T* gate = static_cast<const T*>(a.gate) + static_cast<size_t>(n) * a.ld_gate + c0;
    const float* nw = a.norm_w ? a.norm_w + c0 : nullptr;
    T* y = static_cast<T*>(a.y) + static_cast<size_t>(n) * a.ld_y + c0;
    constexpr int kCache = V == 4 ? 2 : 8;   // 512 values in registers, everything requested at once
    float v[kCache * V], z[kCache * V], w[kCache * V], local = 0.f;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int c = (lane + e * kWave) * V;
        const bool in = c < r.vdim;
        if constexpr (V == 4) {
            const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
            const f32x4_t v4 = in ? load4(row + c) : zero, z4 = in ? load4(gate + c) : zero, w4 = in && nw ? load4(nw + c) : zero;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                v[4 * e + i] = v4[i];
                z[4 * e + i] = z4[i];
                w[4 * e + i] = nw ? w4[i] : 1.f;
            }
        } else {
            v[e] = in ? row[c] : 0.f;
            z[e] = in ? act_get<T>(gate[c]) : 0.f;
            w[e] = in && nw ? nw[c] : 1.f;
        }
    }
    float scale = 1.f;
    if (stabilised(r)) {
        const float* den = a.den + static_cast<size_t>(unit) * 2;
        const float m = den[1];
        scale = 1.f / exp_gate_divisor(den[0], m);
        const int req = a.rows.row_req[n];
        if (lane == 0 && n == a.rows.qo_indptr[req + 1] - 1) *state_of(r, a.rows, req, h).m = m;
    }
#pragma unroll
    for (int e = 0; e < kCache * V; ++e) {
        v[e] *= scale;
        local += v[e] * v[e];
    }
    for (int c = kCache * V * kWave + lane; c < r.vdim; c += kWave) {
        const float x = row[c] * scale;
        local += x * x;
    }
    const float inv = a.out_scale / sqrtf(wave_sum_dpp(local) / static_cast<float>(r.vdim) + a.eps);
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int c = (lane + e * kWave) * V;
        if (c >= r.vdim) continue;
        if constexpr (V == 4) {
            f32x4_t o;
#pragma unroll
            for (int i = 0; i < 4; ++i) o[i] = v[4 * e + i] * inv * w[4 * e + i] * gate_value(z[4 * e + i], a.gate_act);
            store4(y + c, o);
        } else {
            y[c] = act_put<T>(v[e] * inv * w[e] * gate_value(z[e], a.gate_act));
        }
    }
    for (int c = kCache * V * kWave + lane; c < r.vdim; c += kWave)
        y[c] = act_put<T>(row[c] * scale * inv * (nw ? nw[c] : 1.f) * gate_value(act_get<T>(gate[c]), a.gate_act));
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
template <class T, int NR, bool CONV>   // state rows per thread; convolution ahead
__global__ __launch_bounds__(256, NR <= 8 ? 6 : NR <= 16 ? 4 : NR <= 32 ? 2 : 1) void decay_step_kernel(const StepArgs a) {
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
    const T* conv = CONV ? conv_state_of<const T>(a.rows, req) : nullptr;
#pragma unroll 1
    for (int i = tid; i < 2 * dim + cols; i += 256) {
        const int c = i < dim ? a.q_off + kvh * dim + i
                              : i < 2 * dim ? a.k_off + kvh * dim + i - dim : a.v_off + h * r.vdim + col0 + i - 2 * dim;
        float v = act_get<T>(row[c]);
        if constexpr (CONV) {
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
template <class T, int V>   // V: values per thread and access
__global__ __launch_bounds__(256) void gated_part_norm_kernel(const PartNormArgs a) {
    __shared__ float red[4];
    const int part = blockIdx.x, n = blockIdx.y, inner = a.heads * a.vdim, len = inner / a.parts, c0 = part * len;
    const float* o = a.o + static_cast<size_t>(n) * inner + c0;
    const T* z = static_cast<const T*>(a.z) + static_cast<size_t>(n) * a.ld_z + c0;
    const T* x = a.x ? static_cast<const T*>(a.x) + static_cast<size_t>(n) * a.ld_x + c0 : nullptr;
    const float* nw = a.norm_w + c0;
    T* y = static_cast<T*>(a.y) + static_cast<size_t>(n) * a.ld_y + c0;
    auto skip_of = [&](int i) { return x ? a.skip[(c0 + i) / a.vdim] : 0.f; };
    auto value = [&](float ov, float skip, float xv, float zv) { return fmaf(skip, xv, ov) * zv * sigmoid_f32(zv); };
    auto value_at = [&](int i) { return value(o[i], skip_of(i), x ? act_get<T>(x[i]) : 0.f, act_get<T>(z[i])); };
    constexpr int kCache = V == 4 ? 4 : 8;
    float v[kCache * V], local = 0.f;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int i = (threadIdx.x + e * 256) * V;
        const bool in = i < len;
        if constexpr (V == 4) {
            const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
            const f32x4_t o4 = in ? load4(o + i) : zero, z4 = in ? load4(z + i) : zero, x4 = in && x ? load4(x + i) : zero;
            const float skip = in ? skip_of(i) : 0.f;   // (four values share a head)
#pragma unroll
            for (int k = 0; k < 4; ++k) v[4 * e + k] = value(o4[k], skip, x4[k], z4[k]);
        } else {
            v[e] = in ? value_at(i) : 0.f;
        }
    }
#pragma unroll
    for (int e = 0; e < kCache * V; ++e) local += v[e] * v[e];
    for (int i = kCache * V * 256 + threadIdx.x; i < len; i += 256) {
        const float t = value_at(i);
        local += t * t;
    }
    const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(len) + a.eps);
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int i = (threadIdx.x + e * 256) * V;
        if (i >= len) continue;
        if constexpr (V == 4) {
            const f32x4_t w4 = load4(nw + i);
            store4(y + i, f32x4_t{v[4 * e] * inv * w4[0], v[4 * e + 1] * inv * w4[1], v[4 * e + 2] * inv * w4[2], v[4 * e + 3] * inv * w4[3]});
        } else {
            y[i] = act_put<T>(v[e] * inv * nw[i]);
        }
    }
    for (int i = kCache * V * 256 + threadIdx.x; i < len; i += 256) y[i] = act_put<T>(value_at(i) * inv * nw[i]);
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

bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }
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

// columns of a step's block: at most 128 KB of state; whole heads while the batch alone fills the device,
// else slices of at least 32 columns until it does
int step_cols(const PieHipDecayRule& r, int num_requests) {
    int cols = r.vdim <= 256 ? r.vdim : 256;
    if (cols < r.vdim || cols * r.dim > 32768)   // (no whole head anyway: smaller blocks hide more latency)
        while (cols > 32 && cols % 8 == 0 && cols * r.dim > 16384) cols /= 2;
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
                                 int move_state, void* stream) {
    if (move_state && rows && rows->num_tokens != rows->num_requests) return PIE_HIP_ERR_INVALID;
    if (!fused || !conv_w || !rows_ok(rows) || !out || channels <= 0 || taps <= 0 || ld < channels || ld_out < channels)
        return PIE_HIP_ERR_INVALID;
    const int run = rows->num_tokens >= 1024 ? 8 : rows->num_tokens >= 128 ? 4 : 1;
    if (!aligned16(conv_w)) return PIE_HIP_ERR_UNSUPPORTED;
    const bool four = channels % 4 == 0 && ld % 4 == 0 && ld_out % 4 == 0 && aligned16(fused) && aligned16(out) && rows->num_tokens >= 256;
    const dim3 grid((channels / (four ? 4 : 1) + 255) / 256, (rows->num_tokens + run - 1) / run);
    if (grid.y > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    PIE_ACT_DISPATCH(dtype, T, {
        if (four)
            hipLaunchKernelGGL((conv_silu_kernel<T, 4, 4>), grid, dim3(256), 0, s, static_cast<const T*>(fused), conv_w, conv_bias, *rows,
                               static_cast<T*>(out), ld, channels, taps, ld_out, run, move_state);
        else
            hipLaunchKernelGGL((conv_silu_kernel<T, 1, 1>), grid, dim3(256), 0, s, static_cast<const T*>(fused), conv_w, conv_bias, *rows,
                               static_cast<T*>(out), ld, channels, taps, ld_out, run, move_state);
    });
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
    return static_cast<size_t>(num_chunks) * (rule->kv_heads * l.qk_elems * 2 + rule->heads * (l.v_elems * 2 + (l.sum_elems + l.meta_elems) * 4));
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
    uint16_t* vr = qk + static_cast<size_t>(num_chunks) * rule->kv_heads * l.qk_elems;
    float* sums = reinterpret_cast<float*>(vr + static_cast<size_t>(num_chunks) * rule->heads * l.v_elems);
    float* meta = sums + static_cast<size_t>(num_chunks) * rule->heads * l.sum_elems;
    const int aligned = aligned16(q) && aligned16(k) && aligned16(v) && ld % 8 == 0 && rule->dim % 8 == 0 && rule->vdim % 8 == 0;
    const ChunkArgs c{*rule, q, k, v, gates, chunks, qk, vr, sums, meta, l, ld, ld_gates, aligned};
    const WalkArgs w{*rule, *rows, qk, vr, sums, meta, req_chunks, o, den, l};
    if (rule->heads > 65535 || l.ctiles > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    hipLaunchKernelGGL(decay_chunk_kernel, dim3(rule->heads, num_chunks), dim3(256), 0, s, c);
    switch (l.dimp) {
        case 32: launch_walk<1, 1>(w, rows->num_requests, s); break;
        case 64: launch_walk<2, 1>(w, rows->num_requests, s); break;
        case 128: launch_walk<4, 1>(w, rows->num_requests, s); break;
        case 256: launch_walk<4, 2>(w, rows->num_requests, s); break;
        default: launch_walk<4, 4>(w, rows->num_requests, s); break;
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
    const dim3 grid(static_cast<unsigned>((units + 3) / 4));
    const bool four = rule->vdim % 4 == 0 && ld_gate % 4 == 0 && ld_y % 4 == 0 && aligned16(o) && aligned16(gate) && aligned16(y);
    PIE_ACT_DISPATCH(dtype, T, {
        if (four) hipLaunchKernelGGL((decay_out_kernel<T, 4>), grid, dim3(256), 0, static_cast<hipStream_t>(stream), a);
        else hipLaunchKernelGGL((decay_out_kernel<T, 1>), grid, dim3(256), 0, static_cast<hipStream_t>(stream), a);
    });
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
#define PIE_STEP_CASE(NR)                                                                            \
    case NR:                                                                                         \
        if (conv_w) hipLaunchKernelGGL((decay_step_kernel<T, NR, true>), grid, dim3(256), 0, s, a);  \
        else hipLaunchKernelGGL((decay_step_kernel<T, NR, false>), grid, dim3(256), 0, s, a);        \
        break;
    PIE_ACT_DISPATCH(dtype, T, switch (step_rows_per_thread(rule->dim, cols)) {
        PIE_STEP_CASE(4) PIE_STEP_CASE(8) PIE_STEP_CASE(16) PIE_STEP_CASE(32) PIE_STEP_CASE(64)
        default: return PIE_HIP_ERR_UNSUPPORTED;
    });
#undef PIE_STEP_CASE
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
    const dim3 grid(parts, rows->num_tokens);
    const bool four = vdim % 4 == 0 && (heads * vdim / parts) % 4 == 0 && ld_z % 4 == 0 && ld_y % 4 == 0 && (!x || ld_x % 4 == 0) &&
                      aligned16(o) && aligned16(z) && aligned16(y) && aligned16(norm_w) && aligned16(x);
    PIE_ACT_DISPATCH(dtype, T, {
        if (four) hipLaunchKernelGGL((gated_part_norm_kernel<T, 4>), grid, dim3(256), 0, static_cast<hipStream_t>(stream), a);
        else hipLaunchKernelGGL((gated_part_norm_kernel<T, 1>), grid, dim3(256), 0, static_cast<hipStream_t>(stream), a);
    });
    return launch_status();
}
