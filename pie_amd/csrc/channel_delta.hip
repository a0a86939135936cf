// The gated delta rule with one decay per head and key channel, and what surrounds it.
//
// Per head, over a state S [dim, vdim] in fp32:
//   S <- g_t * S (rows), u = beta_t (v_t - S^T k_t), S <- S + k_t u^T, o_t = S^T q_t.
// A request's state lives in a slot of the recurrent-state pool: S per head, then the last
// taps - 1 inputs of the causal convolution ([taps - 1][channels], compute type).  A batch's rows
// belong to requests in order; rs_fresh marks requests that start from zero.
#include "act_type.hip.h"

namespace pie_hip {
namespace {

struct DeltaRows {   // which rows of the batch a request owns, and where its state is
    const int32_t* row_req;     // [N] request of each row
    const int32_t* qo_indptr;   // [R + 1] rows of each request
    const int32_t* rs_slot;     // [R]
    const int32_t* rs_fresh;    // [R] 1: starts from zero
};

// Input of the convolution for channel c of the request's row i (i < 0: earlier tokens, from the
// state; before the sequence's start: 0).
template <class T>
__device__ __forceinline__ float conv_input(const T* __restrict__ fused, const T* __restrict__ conv_state, int ld,
                                            int row0, int i, int c, int keep, int channels, bool fresh) {
    if (i >= 0) return act_get<T>(fused[static_cast<size_t>(row0 + i) * ld + c]);
    if (fresh) return 0.f;
    return act_get<T>(conv_state[static_cast<size_t>(keep + i) * channels + c]);
}

struct DeltaPrepArgs {
    const void* fused;       // [N, ld]: q | k | v | step sizes | ..
    const float* conv_w;     // [channels, taps], channels = q | k | v
    const unsigned char* rs_base;
    size_t rs_stride, conv_offset;   // bytes
    DeltaRows rows;
    float* q;      // [N, kv_heads * dim]
    float* k;
    float* v;      // [N, heads * vdim]
    float* beta;   // [N, heads]
    int num_rows, rows_per_unit, ld, heads, kv_heads, dim, vdim, taps;
};

// One wave per (unit, run of rows).  A unit is a q head, a k head (convolution, silu, unit vector),
// 64 PL channels of v (convolution, silu), or the step sizes.  The wave walks its rows with the
// convolution's window in registers (taps <= 4), so every input is read once; longer convolutions
// read their window afresh.
constexpr int kMaxPerLane = 8;   // q / k heads of up to 512 channels
template <class T, int PL>
__global__ __launch_bounds__(256) void delta_prep_kernel(const DeltaPrepArgs a) {
    const int lane = threadIdx.x & (kWave - 1);
    const int unit = blockIdx.y * 4 + threadIdx.x / kWave;
    const int n0 = blockIdx.x * a.rows_per_unit, n1 = min(n0 + a.rows_per_unit, a.num_rows);
    const int kd = a.kv_heads * a.dim, vd = a.heads * a.vdim;
    constexpr int kVUnit = 64 * PL;
    const int vunits = (vd + kVUnit - 1) / kVUnit;
    const int keep = a.taps - 1, channels = 2 * kd + vd;
    const T* fused = static_cast<const T*>(a.fused);
    if (unit == 2 * a.kv_heads + vunits) {
        for (int n = n0; n < n1; ++n)
            for (int h = lane; h < a.heads; h += kWave)
                a.beta[static_cast<size_t>(n) * a.heads + h] =
                    sigmoid_f32(act_get<T>(fused[static_cast<size_t>(n) * a.ld + channels + h]));
        return;
    }
    if (unit > 2 * a.kv_heads + vunits) return;
    const bool is_v = unit >= 2 * a.kv_heads, is_q = unit < a.kv_heads;
    const int vc = is_v ? (unit - 2 * a.kv_heads) * kVUnit : 0;
    const int c0 = is_v ? 2 * kd + vc : unit * a.dim;              // first channel of the unit
    const int len = is_v ? min(kVUnit, vd - vc) : a.dim;
    float w[PL][4];
    const bool windowed = a.taps <= 4;
    if (windowed)
#pragma unroll
        for (int e = 0; e < PL; ++e)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int d = lane + e * kWave, tap = j - (4 - a.taps);
                w[e][j] = d < len && tap >= 0 ? a.conv_w[static_cast<size_t>(c0 + d) * a.taps + tap] : 0.f;
            }
    float win[PL][4] = {};   // inputs of the last four tokens, oldest first
    const float qk_scale = is_q ? 1.f / sqrtf(static_cast<float>(a.dim)) : 1.f;
    int r = 0, row0 = 0, row1 = n0;   // the request in hand and its rows (re-read where it ends)
    bool fresh = false;
    const T* state = nullptr;
    T now[PL];   // the row's own inputs, requested one row ahead
    auto request = [&](int n) {
#pragma unroll
        for (int e = 0; e < PL; ++e) {
            const int d = lane + e * kWave;
            if (d < len) now[e] = fused[static_cast<size_t>(n) * a.ld + c0 + d];
        }
    };
    request(n0);
    for (int n = n0; n < n1; ++n) {
        const bool enter = n >= row1;
        if (enter) {
            r = a.rows.row_req[n];
            row0 = a.rows.qo_indptr[r];
            row1 = a.rows.qo_indptr[r + 1];
            fresh = a.rows.rs_fresh[r] != 0;
            state = reinterpret_cast<const T*>(a.rs_base + static_cast<size_t>(a.rows.rs_slot[r]) * a.rs_stride + a.conv_offset);
        }
        const int i = n - row0;
        float cur[PL], val[PL];
#pragma unroll
        for (int e = 0; e < PL; ++e) cur[e] = lane + e * kWave < len ? act_get<T>(now[e]) : 0.f;
        if (n + 1 < n1) request(n + 1);
#pragma unroll
        for (int e = 0; e < PL; ++e) {
            const int d = lane + e * kWave;
            val[e] = 0.f;
            if (d >= len) continue;
            auto input = [&](int at) { return conv_input<T>(fused, state, a.ld, row0, at, c0 + d, keep, channels, fresh); };
            float y = 0.f;
            if (windowed) {
                if (enter) {
#pragma unroll
                    for (int j = 1; j < 4; ++j) win[e][j] = 4 - j <= keep ? input(i - (4 - j)) : 0.f;
                }
#pragma unroll
                for (int j = 0; j < 3; ++j) win[e][j] = win[e][j + 1];
                win[e][3] = cur[e];
#pragma unroll
                for (int j = 0; j < 4; ++j) y = fmaf(w[e][j], win[e][j], y);
            } else {
                for (int j = 0; j < a.taps; ++j) y = fmaf(a.conv_w[static_cast<size_t>(c0 + d) * a.taps + j], input(i - keep + j), y);
            }
            val[e] = y * sigmoid_f32(y);
        }
        if (is_v) {
#pragma unroll
            for (int e = 0; e < PL; ++e) {
                const int d = lane + e * kWave;
                if (d < len) a.v[static_cast<size_t>(n) * vd + vc + d] = val[e];
            }
        } else {
            float local = 0.f;
#pragma unroll
            for (int e = 0; e < PL; ++e) local += val[e] * val[e];
            const float inv = qk_scale / sqrtf(wave_sum_dpp(local) + 1e-6f);
            float* dst = (is_q ? a.q : a.k) + static_cast<size_t>(n) * kd + (is_q ? c0 : c0 - kd);
#pragma unroll
            for (int e = 0; e < PL; ++e) {
                const int d = lane + e * kWave;
                if (d < len) dst[d] = val[e] * inv;
            }
        }
    }
}

// The convolution inputs a request's next tokens will need: one thread per channel.  (Entries move
// towards the front: entry j is read no later than it is written.)
template <class T>
__global__ __launch_bounds__(256) void delta_conv_state_kernel(const T* __restrict__ fused, unsigned char* __restrict__ rs_base,
                                                               size_t rs_stride, size_t conv_offset, DeltaRows rows,
                                                               int ld, int channels, int taps) {
    const int r = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x, keep = taps - 1;
    if (c >= channels) return;
    const int row0 = rows.qo_indptr[r], n = rows.qo_indptr[r + 1] - row0;
    const bool fresh = rows.rs_fresh[r] != 0;
    T* state = reinterpret_cast<T*>(rs_base + static_cast<size_t>(rows.rs_slot[r]) * rs_stride + conv_offset);
    for (int j = 0; j < keep; ++j)
        state[static_cast<size_t>(j) * channels + c] = act_put<T>(conv_input<T>(fused, state, ld, row0, n - keep + j, c, keep, channels, fresh));
}

__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// The second factors of the low-rank decay and output gate, straight from the fused projection's
// columns: log2 of the decay, rate[head] softplus(W_a2 a1 + dt_bias), in fp32, and the
// gate's projection in the compute type.  The launch's first blocks along x take the decay's
// outputs, the others the gate's, 64 each; MFMA as in the head-wise linears (weights the A operand).
struct LowRankArgs {
    const void* fused;
    const uint16_t *w_decay, *w_gate;   // [.., ld_a1], [.., ld_g1], zero columns past the rank
    const float *rate, *dt_bias;        // [heads] -exp(A_log) log2(e); [heads * dim]
    float* lg;                          // [M, heads * dim]
    void* gate;                         // [M, ld_gate]
    int M, ld, decay_off, gate_off, decay_rank, gate_rank, ld_a1, ld_g1, dim, decay_n, gate_n, ld_gate, decay_blocks;
};
__device__ __forceinline__ float decay_log2(const LowRankArgs& a, int c, float raw) {
    return a.rate[c / a.dim] * softplus_f32(raw + a.dt_bias[c]);
}
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
template <int MT>
__global__ __launch_bounds__(256) void delta_lowrank_mfma_kernel(const LowRankArgs a) {
    const bool is_gate = static_cast<int>(blockIdx.x) >= a.decay_blocks;
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int l16 = lane & 15, g = lane >> 4;
    const int m0 = blockIdx.y * 16 * MT;
    const int N = is_gate ? a.gate_n : a.decay_n, K = is_gate ? a.ld_g1 : a.ld_a1, rank = is_gate ? a.gate_rank : a.decay_rank;
    const int c0 = ((blockIdx.x - (is_gate ? a.decay_blocks : 0)) * 4 + wv) * 16;
    if (c0 >= N) return;
    const uint16_t* wp = (is_gate ? a.w_gate : a.w_decay) + static_cast<size_t>(min(c0 + l16, N - 1)) * K + 8 * g;
    const uint16_t* ap[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t)
        ap[t] = static_cast<const uint16_t*>(a.fused) + static_cast<size_t>(min(m0 + 16 * t + l16, a.M - 1)) * a.ld +
                (is_gate ? a.gate_off : a.decay_off);
    f32x4_t acc[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < rank; k += 32) {
        const bf16x8_t wf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(wp + k));
#pragma unroll
        for (int t = 0; t < MT; ++t) {
            // (whole 8-value pieces inside the rank's columns; past them zeros, as in the weights)
            u32x4_t v = {0u, 0u, 0u, 0u};
            if (k + 8 * g < rank) v = *reinterpret_cast<const u32x4_t*>(ap[t] + k + 8 * g);
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, __builtin_bit_cast(bf16x8_t, v), acc[t], 0, 0, 0);
        }
    }
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const int m = m0 + 16 * t + l16;
        if (m >= a.M) continue;
        const int c = c0 + 4 * g;
        if (is_gate) {   // (ld_gate is a multiple of 16: whole pieces)
            *reinterpret_cast<u32x2_t*>(static_cast<uint16_t*>(a.gate) + static_cast<size_t>(m) * a.ld_gate + c) =
                u32x2_t{pack_bf16x2(acc[t][0], acc[t][1]), pack_bf16x2(acc[t][2], acc[t][3])};
        } else if (N % 4 == 0 && c + 4 <= N) {
            f32x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = decay_log2(a, c + e, acc[t][e]);
            *reinterpret_cast<f32x4_t*>(a.lg + static_cast<size_t>(m) * N + c) = v;
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (c + e < N) a.lg[static_cast<size_t>(m) * N + c + e] = decay_log2(a, c + e, acc[t][e]);
        }
    }
}
__global__ __launch_bounds__(256) void delta_lowrank_f32_kernel(const LowRankArgs a) {
    const bool is_gate = static_cast<int>(blockIdx.x) >= a.decay_blocks;
    const size_t m = blockIdx.y;
    const int N = is_gate ? a.gate_n : a.decay_n, K = is_gate ? a.ld_g1 : a.ld_a1, rank = is_gate ? a.gate_rank : a.decay_rank;
    const int c = (blockIdx.x - (is_gate ? a.decay_blocks : 0)) * 64 + (threadIdx.x & 63);
    if (threadIdx.x >= 64 || c >= N) return;
    const float* x = static_cast<const float*>(a.fused) + m * a.ld + (is_gate ? a.gate_off : a.decay_off);
    const uint16_t* w = (is_gate ? a.w_gate : a.w_decay) + static_cast<size_t>(c) * K;
    float y = 0.f;
    for (int k = 0; k < rank; ++k) y = fmaf(x[k], bf16_bits_to_f32(w[k]), y);
    if (is_gate) static_cast<float*>(a.gate)[m * a.ld_gate + c] = y;
    else a.lg[m * N + c] = decay_log2(a, c, y);
}

struct DeltaScanArgs {
    const float *q, *k, *v, *lg, *beta;   // lg: log2 of the decays
    float* o;                 // [N, heads * vdim]
    unsigned char* rs_base;
    size_t rs_stride, state_offset;   // bytes
    DeltaRows rows;
    int heads, kv_heads, dim, vdim;
};

// The recurrence, token by token.  A block takes 32 value columns of one head of one request; a
// wave's lanes are 8 columns x 8 row groups, lane (column, group) holding rows 32 i + 4 group + e
// of its column in registers.  The columns are independent, a column's two dot products meet over
// its eight lanes.  With o = (g S)^T q + (q . k) u both are taken from the decayed state at once,
// so a token costs one reduction.  k, q, g (and v, beta) sit in LDS kTok tokens at a time; the next
// ones are requested from memory while the current ones run.
constexpr int kTok = 16, kCols = 32;
template <int NI>   // dim rounded up to 32 NI
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaScanArgs a) {
    constexpr int DP = 32 * NI;
    __shared__ __attribute__((aligned(16))) float sk[kTok][DP], sq[kTok][DP], sg[kTok][DP];
    __shared__ float sv[kTok][kCols], sb[kTok], skq[kTok], so[kTok][kCols];
    const int r = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * kCols;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const int rg = lane & 7, cl = wv * 8 + (lane >> 3), col = col0 + cl;
    const int row0 = a.rows.qo_indptr[r], row1 = a.rows.qo_indptr[r + 1];
    const bool fresh = a.rows.rs_fresh[r] != 0;
    const int kvh = h / (a.heads / a.kv_heads);
    const int kd = a.kv_heads * a.dim, gd = a.heads * a.dim, vd = a.heads * a.vdim;
    float* S = reinterpret_cast<float*>(a.rs_base + static_cast<size_t>(a.rows.rs_slot[r]) * a.rs_stride + a.state_offset) +
               static_cast<size_t>(h) * a.dim * a.vdim;
    const bool live = col < a.vdim;
    f32x4_t s[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int d = 32 * i + 4 * rg + e;
            s[i][e] = live && !fresh && d < a.dim ? S[static_cast<size_t>(d) * a.vdim + col] : 0.f;
        }
    // staging: thread (token tt, lane tl of 16) moves DP / 16 values of each of k, q, g
    const int tt = tid >> 4, tl = tid & 15;
    constexpr int NV = DP / 16;
    float rk[NV], rq[NV], rgv[NV], rv[kCols / 16], rb = 0.f;
    auto fetch = [&](int t0) {
        const int n = row0 + t0 + tt;
        const bool in = n < row1;
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            const int d = tl + 16 * e;
            const bool ok = in && d < a.dim;
            rk[e] = ok ? a.k[static_cast<size_t>(n) * kd + kvh * a.dim + d] : 0.f;
            rq[e] = ok ? a.q[static_cast<size_t>(n) * kd + kvh * a.dim + d] : 0.f;
            rgv[e] = ok ? exp2f(a.lg[static_cast<size_t>(n) * gd + h * a.dim + d]) : 0.f;
        }
#pragma unroll
        for (int e = 0; e < kCols / 16; ++e) {
            const int c = tl + 16 * e;
            rv[e] = in && col0 + c < a.vdim ? a.v[static_cast<size_t>(n) * vd + h * a.vdim + col0 + c] : 0.f;
        }
        if (tl == 0) rb = in ? a.beta[static_cast<size_t>(n) * a.heads + h] : 0.f;
    };
    auto stage = [&]() {
        float kq = 0.f;
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            const int d = tl + 16 * e;
            sk[tt][d] = rk[e];
            sq[tt][d] = rq[e];
            sg[tt][d] = rgv[e];
            kq = fmaf(rk[e], rq[e], kq);
        }
#pragma unroll
        for (int e = 0; e < kCols / 16; ++e) sv[tt][tl + 16 * e] = rv[e];
#pragma unroll
        for (int off = 8; off > 0; off >>= 1) kq += __shfl_xor(kq, off, kWave);
        if (tl == 0) {
            sb[tt] = rb;
            skq[tt] = kq;
        }
    };
    const int T = row1 - row0;
    if (T > 0) fetch(0);
    for (int t0 = 0; t0 < T; t0 += kTok) {
        stage();
        if (t0 + kTok < T) fetch(t0 + kTok);
        __syncthreads();
        const int nt = min(kTok, T - t0);
        for (int t = 0; t < nt; ++t) {
            float dk = 0.f, dq = 0.f;
            f32x4_t kk[NI];
#pragma unroll
            for (int i = 0; i < NI; ++i) {
                const int d = 32 * i + 4 * rg;
                kk[i] = *reinterpret_cast<const f32x4_t*>(&sk[t][d]);
                const f32x4_t qq = *reinterpret_cast<const f32x4_t*>(&sq[t][d]);
                const f32x4_t gg = *reinterpret_cast<const f32x4_t*>(&sg[t][d]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[i][e] *= gg[e];
                    dk = fmaf(s[i][e], kk[i][e], dk);
                    dq = fmaf(s[i][e], qq[e], dq);
                }
            }
            dk = dpp_add_f32<0xB1>(dk);    // lane ^ 1
            dq = dpp_add_f32<0xB1>(dq);
            dk = dpp_add_f32<0x4E>(dk);    // lane ^ 2
            dq = dpp_add_f32<0x4E>(dq);
            dk = dpp_add_f32<0x141>(dk);   // row_half_mirror: the other four of the eight
            dq = dpp_add_f32<0x141>(dq);
            const float u = sb[t] * (sv[t][cl] - dk);
#pragma unroll
            for (int i = 0; i < NI; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) s[i][e] = fmaf(kk[i][e], u, s[i][e]);
            if (rg == 0) so[t][cl] = fmaf(skq[t], u, dq);
        }
        __syncthreads();
        if (tt < nt)
#pragma unroll
            for (int e = 0; e < kCols / 16; ++e) {
                const int c = tl + 16 * e;
                if (col0 + c < a.vdim)
                    a.o[static_cast<size_t>(row0 + t0 + tt) * vd + h * a.vdim + col0 + c] = so[tt][c];
            }
    }
    if (live)
#pragma unroll
        for (int i = 0; i < NI; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = 32 * i + 4 * rg + e;
                if (d < a.dim) S[static_cast<size_t>(d) * a.vdim + col] = s[i][e];
            }
}

// y = o / rms(o) * norm_w * sigmoid(gate) per head; one wave per (row, head).
template <class T>
__global__ __launch_bounds__(256) void delta_out_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                                        const float* __restrict__ norm_w, T* __restrict__ y, int total,
                                                        int heads, int vdim, int ld_gate, int ld_y, float eps) {
    const int unit = blockIdx.x * 4 + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    if (unit >= total) return;
    const size_t n = unit / heads;
    const int c0 = (unit % heads) * vdim;
    const float* row = o + n * heads * vdim + c0;
    constexpr int kCache = 4;   // 256 values in registers
    float v[kCache], local = 0.f;
#pragma unroll
    for (int e = 0; e < kCache; ++e) {
        const int c = lane + e * kWave;
        v[e] = c < vdim ? row[c] : 0.f;
        local += v[e] * v[e];
    }
    for (int c = lane + kCache * kWave; c < vdim; c += kWave) local += row[c] * row[c];
    const float inv = 1.f / sqrtf(wave_sum_dpp(local) / static_cast<float>(vdim) + eps);
    for (int c = lane, e = 0; c < vdim; c += kWave, ++e) {
        const float x = e == 0 ? v[0] : e == 1 ? v[1] : e == 2 ? v[2] : e == 3 ? v[3] : row[c];
        y[n * ld_y + c0 + c] = act_put<T>(x * inv * norm_w[c] * sigmoid_f32(act_get<T>(gate[n * ld_gate + c0 + c])));
    }
}

// One token per request, everything between the projections in one launch: a block per (request,
// head).  Its state rows are requested first and travel while the convolution, the unit vectors and
// the decays are formed; thread (row group, four columns) holds its share of S in registers, so
// the state is read once and written once.
struct DeltaStepArgs {
    const void* fused;
    const float* conv_w;
    const float* lg;
    const void* gate;
    const float* norm_w;
    void* y;
    unsigned char* rs_base;
    size_t rs_stride, state_offset, conv_offset;
    const int32_t *rs_slot, *rs_fresh;
    int ld, ld_gate, ld_y, heads, kv_heads, dim, vdim, taps, tpr_shift;   // 1 << tpr_shift threads per state row
    int write_conv;                                                      // every head has its own q / k channels
    float eps;
};
template <class T, int NR>   // state rows per thread
__global__ __launch_bounds__(256) void delta_step_kernel(const DeltaStepArgs a) {
    __shared__ float x[768];          // q | k | v after the convolution
    __shared__ float dec[256];
    __shared__ __attribute__((aligned(16))) float red[4][2][256];
    __shared__ __attribute__((aligned(16))) float o[256];
    __shared__ float s_qq, s_kk, s_kq, s_oo[4];
    const int r = blockIdx.y, h = blockIdx.x, tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const int dim = a.dim, vdim = a.vdim, kvh = h / (a.heads / a.kv_heads);
    const bool fresh = a.rs_fresh[r] != 0;
    unsigned char* slot = a.rs_base + static_cast<size_t>(a.rs_slot[r]) * a.rs_stride;
    float* S = reinterpret_cast<float*>(slot + a.state_offset) + static_cast<size_t>(h) * dim * vdim;
    const int tpr = 1 << a.tpr_shift, rg = tid >> a.tpr_shift, ngroups = 256 >> a.tpr_shift;
    const int col = (tid & (tpr - 1)) * 4;
    const bool live = col < vdim;
    f32x4_t s[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = rg + i * ngroups;
        s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (live && !fresh && d < dim) s[i] = *reinterpret_cast<const f32x4_t*>(S + static_cast<size_t>(d) * vdim + col);
    }
    // convolution and silu of this head's q, k and v channels; their state moves on by one token
    const int kd = a.kv_heads * dim, vd = a.heads * vdim, channels = 2 * kd + vd, keep = a.taps - 1;
    const T* fused = static_cast<const T*>(a.fused) + static_cast<size_t>(r) * a.ld;
    T* state = reinterpret_cast<T*>(slot + a.conv_offset);
    for (int i = tid; i < 2 * dim + vdim; i += 256) {
        const int c = i < dim ? kvh * dim + i : i < 2 * dim ? kd + kvh * dim + i - dim : 2 * kd + h * vdim + i - 2 * dim;
        const float* w = a.conv_w + static_cast<size_t>(c) * a.taps;
        const T now = fused[c];
        float y = 0.f;
        for (int j = 0; j < keep; ++j) {
            const T old = fresh ? act_put<T>(0.f) : state[static_cast<size_t>(j) * channels + c];
            y = fmaf(w[j], act_get<T>(old), y);
            if (a.write_conv && j > 0) state[static_cast<size_t>(j - 1) * channels + c] = old;
        }
        y = fmaf(w[keep], act_get<T>(now), y);
        if (a.write_conv && keep > 0) state[static_cast<size_t>(keep - 1) * channels + c] = now;
        x[i] = y * sigmoid_f32(y);
    }
    for (int d = tid; d < dim; d += 256) dec[d] = exp2f(a.lg[static_cast<size_t>(r) * a.heads * dim + h * dim + d]);
    const float beta = sigmoid_f32(act_get<T>(fused[channels + h]));
    __syncthreads();
    if (wv < 3) {   // |q|^2, |k|^2, q . k
        const float* p = wv == 1 ? x + dim : x;
        const float* q = wv == 0 ? x : x + dim;
        float v = 0.f;
        for (int d = lane; d < dim; d += kWave) v = fmaf(p[d], q[d], v);
        v = wave_sum_dpp(v);
        if (lane == 0) (wv == 0 ? s_qq : wv == 1 ? s_kk : s_kq) = v;
    }
    __syncthreads();
    const float qs = 1.f / sqrtf(static_cast<float>(dim)) / sqrtf(s_qq + 1e-6f), ks = 1.f / sqrtf(s_kk + 1e-6f);
    f32x4_t dk = {0.f, 0.f, 0.f, 0.f}, dq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = rg + i * ngroups;
        if (d >= dim) break;
        const float g = dec[d], kk = x[dim + d] * ks, qq = x[d] * qs;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            s[i][e] *= g;
            dk[e] = fmaf(s[i][e], kk, dk[e]);
            dq[e] = fmaf(s[i][e], qq, dq[e]);
        }
    }
    // over the row groups: inside a wave, then across the waves
    for (int off = tpr; off < kWave; off <<= 1)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            dk[e] += __shfl_xor(dk[e], off, kWave);
            dq[e] += __shfl_xor(dq[e], off, kWave);
        }
    if (lane < tpr) {
        *reinterpret_cast<f32x4_t*>(&red[wv][0][col]) = dk;
        *reinterpret_cast<f32x4_t*>(&red[wv][1][col]) = dq;
    }
    __syncthreads();
    dk = f32x4_t{0.f, 0.f, 0.f, 0.f};
    dq = dk;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
        dk += *reinterpret_cast<const f32x4_t*>(&red[w][0][col]);
        dq += *reinterpret_cast<const f32x4_t*>(&red[w][1][col]);
    }
    const float kq = s_kq * qs * ks;
    f32x4_t u;
#pragma unroll
    for (int e = 0; e < 4; ++e) u[e] = live ? beta * (x[2 * dim + min(col + e, vdim - 1)] - dk[e]) : 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int d = rg + i * ngroups;
        if (d >= dim) break;
        const float kk = x[dim + d] * ks;
#pragma unroll
        for (int e = 0; e < 4; ++e) s[i][e] = fmaf(kk, u[e], s[i][e]);
        if (live) *reinterpret_cast<f32x4_t*>(S + static_cast<size_t>(d) * vdim + col) = s[i];
    }
    if (rg == 0 && live) {
        f32x4_t ov;
#pragma unroll
        for (int e = 0; e < 4; ++e) ov[e] = fmaf(kq, u[e], dq[e]);
        *reinterpret_cast<f32x4_t*>(&o[col]) = ov;
    }
    __syncthreads();
    const float mine = tid < vdim ? o[tid] : 0.f;
    const float part = wave_sum_dpp(mine * mine);
    if (lane == 0) s_oo[wv] = part;
    __syncthreads();
    if (tid < vdim) {
        const float inv = 1.f / sqrtf((s_oo[0] + s_oo[1] + s_oo[2] + s_oo[3]) / static_cast<float>(vdim) + a.eps);
        const int c = h * vdim + tid;
        static_cast<T*>(a.y)[static_cast<size_t>(r) * a.ld_y + c] = act_put<T>(
            mine * inv * a.norm_w[tid] * sigmoid_f32(act_get<T>(static_cast<const T*>(a.gate)[static_cast<size_t>(r) * a.ld_gate + c])));
    }
}

// ---- portions, sixteen tokens at a time ---------------------------------------------------------
// With L_t the running sum of the chunk's log2 decays, S0 the state before it and per-channel powers
// of two written exp2(.):
//   K~_t = k_t exp2(L_t), Q~_t = q_t exp2(L_t), K^_t = k_t exp2(L_16 - L_t)        (all factors <= 1)
//   A[t, i] = sum_d k_t k_i exp2(L_t - L_i), i < t;   B[t, i] = sum_d q_t k_i exp2(L_t - L_i), i <= t
//   U = Tm (V - K~ S0),  Tm = (1 + diag(beta) A)^-1 diag(beta)
//   O = Q~ S0 + B U,     S = exp2(L_16) S0 + K^^T U
// which is the token recurrence with its within-chunk dependences solved: the same sums in another
// order.  Everything is fp32, the products v_mfma_f32_16x16x4_f32.  What does not depend on the
// state is formed for all chunks at once (delta_chunk_kernel); the walk over a request's chunks
// (delta_walk_kernel) keeps S in registers.
constexpr int kChunkTok = 16;
// record of a (chunk, head): K~ [16][DP], Q~ [16][DP], K^ transposed [DP][16], exp2(L_16) [DP], Tm and
// B [16][16]
template <int DP>
struct ChunkRecord {
    static constexpr int kt = 0, qt = 16 * DP, khat = 32 * DP, gc = 48 * DP, tm = 49 * DP, b = tm + 256, floats = b + 256;
};

struct DeltaChunkArgs {
    const float *q, *k, *lg, *beta;
    const int32_t* chunks;   // [num_chunks][2]: first row, rows
    float* rec;
    int heads, kv_heads, dim;
};
template <int ND>   // dim rounded up to 64 ND
__global__ __launch_bounds__(256) void delta_chunk_kernel(const DeltaChunkArgs a) {
    constexpr int DP = 64 * ND, STR = DP + 4;
    using Rec = ChunkRecord<DP>;
    __shared__ __attribute__((aligned(16))) float sk[16][STR], sq[16][STR], sl[16][STR];
    __shared__ float sa[16][17], sbeta[16];
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x;
    const int row0 = a.chunks[2 * ch], nt = a.chunks[2 * ch + 1];
    const int kvh = h / (a.heads / a.kv_heads), kd = a.kv_heads * a.dim, gd = a.heads * a.dim;
    float* rec = a.rec + (static_cast<size_t>(ch) * a.heads + h) * Rec::floats;
    // tokens past the portion: zero keys and queries, step size 0, decay 1
    for (int i = tid; i < 16 * DP; i += 256) {
        const int t = i / DP, d = i % DP;
        const bool in = t < nt && d < a.dim;
        const size_t n = row0 + t;
        sk[t][d] = in ? a.k[n * kd + kvh * a.dim + d] : 0.f;
        sq[t][d] = in ? a.q[n * kd + kvh * a.dim + d] : 0.f;
        sl[t][d] = in ? a.lg[n * gd + h * a.dim + d] : 0.f;
    }
    if (tid < 16) sbeta[tid] = tid < nt ? a.beta[static_cast<size_t>(row0 + tid) * a.heads + h] : 0.f;
    __syncthreads();
    for (int d = tid; d < DP; d += 256) {
        float l = 0.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            l += sl[t][d];
            sl[t][d] = l;
        }
    }
    __syncthreads();
    {   // thread (t, i): the two products of tokens t and i
        const int t = tid >> 4, i = tid & 15;
        float akk = 0.f, aqk = 0.f;
        if (i <= t)
            for (int d = 0; d < DP; d += 4) {
                const f32x4_t lt = *reinterpret_cast<const f32x4_t*>(&sl[t][d]), li = *reinterpret_cast<const f32x4_t*>(&sl[i][d]);
                const f32x4_t kt = *reinterpret_cast<const f32x4_t*>(&sk[t][d]), ki = *reinterpret_cast<const f32x4_t*>(&sk[i][d]);
                const f32x4_t qt = *reinterpret_cast<const f32x4_t*>(&sq[t][d]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float p = ki[e] * __builtin_amdgcn_exp2f(lt[e] - li[e]);
                    akk = fmaf(kt[e], p, akk);
                    aqk = fmaf(qt[e], p, aqk);
                }
            }
        sa[t][i] = i < t ? sbeta[t] * akk : 0.f;
        rec[Rec::b + tid] = aqk;
    }
    for (int i = tid; i < 16 * DP; i += 256) {
        const int t = i / DP, d = i % DP;
        const float g = __builtin_amdgcn_exp2f(sl[t][d]);
        rec[Rec::kt + i] = sk[t][d] * g;
        rec[Rec::qt + i] = sq[t][d] * g;
        const int tt = i & 15, dd = i >> 4;
        rec[Rec::khat + i] = sk[tt][dd] * __builtin_amdgcn_exp2f(sl[15][dd] - sl[tt][dd]);
    }
    for (int d = tid; d < DP; d += 256) rec[Rec::gc + d] = __builtin_amdgcn_exp2f(sl[15][d]);
    __syncthreads();
    if (tid < 16) {   // column tid of the inverse by forward substitution
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float v = t == tid ? 1.f : 0.f;
#pragma unroll
            for (int i = 0; i < t; ++i) v = fmaf(-sa[t][i], x[i], v);
            x[t] = v;
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) rec[Rec::tm + t * 16 + tid] = x[t] * sbeta[tid];
    }
}

struct DeltaWalkArgs {
    const float* rec;
    const float* v;              // [N, heads * vdim]
    float* o;
    unsigned char* rs_base;
    size_t rs_stride, state_offset;
    const int32_t* req_chunks;   // [R + 1] chunks of each request
    const int32_t* qo_indptr;    // [R + 1] rows of each request
    const int32_t *rs_slot, *rs_fresh;
    int heads, dim, vdim;
};
// A block takes 16 value columns of one head of one request.  Wave w keeps rows 16 ND w .. of S as
// accumulator tiles: lane (l16, g) register r holds row 16 i + 4 g + r, column l16 — which is also a
// B operand for the k-step of rows {4 g + r}, so the state never leaves its registers.  The waves'
// partial products over their rows meet in LDS, one barrier per chunk.  Blocks of one head are
// `heads` apart in launch order: with a multiple of eight heads they share an XCD's L2, from which
// all but the first read the head's records.
template <int ND>
__global__ __launch_bounds__(256) void delta_walk_kernel(const DeltaWalkArgs a) {
    constexpr int DP = 64 * ND;
    using Rec = ChunkRecord<DP>;
    __shared__ __attribute__((aligned(16))) float part[2][4][2][kWave * 4];
    const int h = blockIdx.x, col0 = blockIdx.y * 16, r = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int c_lo = a.req_chunks[r], c_hi = a.req_chunks[r + 1];
    const int req_row0 = a.qo_indptr[r], req_row1 = a.qo_indptr[r + 1];
    const int vd = a.heads * a.vdim, col = col0 + l16;
    const bool live = col < a.vdim, fresh = a.rs_fresh[r] != 0;
    float* S = reinterpret_cast<float*>(a.rs_base + static_cast<size_t>(a.rs_slot[r]) * a.rs_stride + a.state_offset) +
               static_cast<size_t>(h) * a.dim * a.vdim;
    const int wrow = 16 * ND * wv;
    f32x4_t s[ND];
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int d = wrow + 16 * i + 4 * g + e;
            s[i][e] = live && !fresh && d < a.dim ? S[static_cast<size_t>(d) * a.vdim + col] : 0.f;
        }
    struct Frags {
        f32x4_t kt[ND], qt[ND], khat[ND], gc[ND], tm, b, v;
        int row0, nt;
    };
    auto load = [&](Frags& f, int c) {
        const float* rec = a.rec + (static_cast<size_t>(c) * a.heads + h) * Rec::floats;
#pragma unroll
        for (int i = 0; i < ND; ++i) {
            const int d = wrow + 16 * i;
            f.kt[i] = *reinterpret_cast<const f32x4_t*>(rec + Rec::kt + l16 * DP + d + 4 * g);
            f.qt[i] = *reinterpret_cast<const f32x4_t*>(rec + Rec::qt + l16 * DP + d + 4 * g);
            f.khat[i] = *reinterpret_cast<const f32x4_t*>(rec + Rec::khat + (d + l16) * 16 + 4 * g);
            f.gc[i] = *reinterpret_cast<const f32x4_t*>(rec + Rec::gc + d + 4 * g);
        }
        f.tm = *reinterpret_cast<const f32x4_t*>(rec + Rec::tm + l16 * 16 + 4 * g);
        f.b = *reinterpret_cast<const f32x4_t*>(rec + Rec::b + l16 * 16 + 4 * g);
        f.row0 = req_row0 + (c - c_lo) * kChunkTok;
        f.nt = min(kChunkTok, req_row1 - f.row0);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int t = 4 * g + e;
            // (columns and tokens past the end repeat the last one: they are not stored, their step size is 0)
            f.v[e] = a.v[static_cast<size_t>(f.row0 + min(t, f.nt - 1)) * vd + h * a.vdim + min(col, a.vdim - 1)];
        }
    };
    auto run = [&](const Frags& f, int buf) {
        f32x4_t pk = {0.f, 0.f, 0.f, 0.f}, pq = pk;
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                pk = __builtin_amdgcn_mfma_f32_16x16x4f32(f.kt[i][e], s[i][e], pk, 0, 0, 0);
                pq = __builtin_amdgcn_mfma_f32_16x16x4f32(f.qt[i][e], s[i][e], pq, 0, 0, 0);
            }
        *reinterpret_cast<f32x4_t*>(&part[buf][wv][0][lane * 4]) = pk;
        *reinterpret_cast<f32x4_t*>(&part[buf][wv][1][lane * 4]) = pq;
        __syncthreads();   // (the buffer's readers of two chunks ago have passed the last barrier)
        f32x4_t x = f.v;
#pragma unroll
        for (int w = 0; w < 4; ++w) x -= *reinterpret_cast<const f32x4_t*>(&part[buf][w][0][lane * 4]);
        f32x4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) u = __builtin_amdgcn_mfma_f32_16x16x4f32(f.tm[e], x[e], u, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < ND; ++i) {
#pragma unroll
            for (int e = 0; e < 4; ++e) s[i][e] *= f.gc[i][e];
#pragma unroll
            for (int e = 0; e < 4; ++e) s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.khat[i][e], u[e], s[i], 0, 0, 0);
        }
        if (wv == 0) {
            f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int w = 0; w < 4; ++w) o += *reinterpret_cast<const f32x4_t*>(&part[buf][w][1][lane * 4]);
#pragma unroll
            for (int e = 0; e < 4; ++e) o = __builtin_amdgcn_mfma_f32_16x16x4f32(f.b[e], u[e], o, 0, 0, 0);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = 4 * g + e;
                if (live && t < f.nt) a.o[static_cast<size_t>(f.row0 + t) * vd + h * a.vdim + col] = o[e];
            }
        }
    };
    // (three chunks ahead: the records come from beyond the L2, a chunk's arithmetic is shorter than
    // that takes)
    constexpr int kAhead = 4;
    Frags f[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead - 1; ++i) load(f[i], min(c_lo + i, c_hi - 1));
    for (int c = c_lo; c < c_hi; c += kAhead) {
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            load(f[(i + kAhead - 1) % kAhead], min(c + i + kAhead - 1, c_hi - 1));
            __builtin_amdgcn_sched_barrier(0);
            if (c + i < c_hi) run(f[i], i & 1);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    if (live)
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = wrow + 16 * i + 4 * g + e;
                if (d < a.dim) S[static_cast<size_t>(d) * a.vdim + col] = s[i][e];
            }
}

template <int ND>
int launch_chunked(const DeltaChunkArgs& c, const DeltaWalkArgs& w, int num_chunks, int num_requests, hipStream_t s) {
    hipLaunchKernelGGL(delta_chunk_kernel<ND>, dim3(c.heads, num_chunks), dim3(256), 0, s, c);
    hipLaunchKernelGGL(delta_walk_kernel<ND>, dim3(w.heads, (w.vdim + 15) / 16, num_requests), dim3(256), 0, s, w);
    return launch_status();
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_delta_prep(int dtype, const void* fused, const float* conv_w, const void* rs_base,
                                  size_t rs_stride, size_t conv_offset, const int32_t* row_req,
                                  const int32_t* qo_indptr, const int32_t* rs_slot, const int32_t* rs_fresh, float* q,
                                  float* k, float* v, float* beta, int num_tokens, int ld, int heads, int kv_heads,
                                  int dim, int vdim, int taps, void* stream) {
    if (!fused || !conv_w || !rs_base || !row_req || !qo_indptr || !rs_slot || !rs_fresh || !q || !k || !v || !beta ||
        num_tokens <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || vdim <= 0 || taps <= 0 ||
        2 * kv_heads * dim + heads * vdim + heads > ld)
        return PIE_HIP_ERR_INVALID;
    if (dim > kMaxPerLane * kWave) return PIE_HIP_ERR_UNSUPPORTED;
    // (runs of rows share the convolution's window; few rows: one each, more waves)
    const int run = num_tokens >= 512 ? 16 : num_tokens >= 128 ? 4 : 1;
    const DeltaPrepArgs a{fused, conv_w, static_cast<const unsigned char*>(rs_base), rs_stride, conv_offset,
                          {row_req, qo_indptr, rs_slot, rs_fresh}, q, k, v, beta, num_tokens, run, ld, heads, kv_heads,
                          dim, vdim, taps};
    const int pl = dim <= 64 ? 1 : dim <= 128 ? 2 : dim <= 256 ? 4 : 8;
    const int units = 2 * kv_heads + (heads * vdim + 64 * pl - 1) / (64 * pl) + 1;
    const dim3 grid((num_tokens + run - 1) / run, (units + 3) / 4);
    if (grid.y > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    PIE_ACT_DISPATCH(dtype, T, switch (pl) {
        case 1: hipLaunchKernelGGL((delta_prep_kernel<T, 1>), grid, dim3(256), 0, s, a); break;
        case 2: hipLaunchKernelGGL((delta_prep_kernel<T, 2>), grid, dim3(256), 0, s, a); break;
        case 4: hipLaunchKernelGGL((delta_prep_kernel<T, 4>), grid, dim3(256), 0, s, a); break;
        default: hipLaunchKernelGGL((delta_prep_kernel<T, 8>), grid, dim3(256), 0, s, a); break;
    });
    return launch_status();
}

extern "C" int pie_hip_delta_conv_state(int dtype, const void* fused, void* rs_base, size_t rs_stride,
                                        size_t conv_offset, const int32_t* qo_indptr, const int32_t* rs_slot,
                                        const int32_t* rs_fresh, int num_requests, int ld, int channels, int taps,
                                        void* stream) {
    if (!fused || !rs_base || !qo_indptr || !rs_slot || !rs_fresh || num_requests <= 0 || channels <= 0 || ld < channels || taps <= 0)
        return PIE_HIP_ERR_INVALID;
    if (num_requests > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    if (taps == 1) return PIE_HIP_OK;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(delta_conv_state_kernel<T>, dim3((channels + 255) / 256, num_requests), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), static_cast<const T*>(fused),
                                                  static_cast<unsigned char*>(rs_base), rs_stride, conv_offset,
                                                  DeltaRows{nullptr, qo_indptr, rs_slot, rs_fresh}, ld, channels, taps));
    return launch_status();
}

extern "C" int pie_hip_delta_lowrank(int dtype, const void* fused, const uint16_t* w_decay, const uint16_t* w_gate,
                                     const float* rate, const float* dt_bias, float* log2_decay, void* gate,
                                     int num_tokens, int ld, int decay_off, int decay_rank, int ld_a1, int gate_off,
                                     int gate_rank, int ld_g1, int heads, int dim, int vdim, int ld_gate, void* stream) {
    if (!fused || !w_decay || !w_gate || !rate || !dt_bias || !log2_decay || !gate || num_tokens <= 0 || heads <= 0 ||
        dim <= 0 || vdim <= 0 || decay_rank <= 0 || gate_rank <= 0 || ld_a1 < decay_rank || ld_g1 < gate_rank ||
        decay_off + decay_rank > ld || gate_off + gate_rank > ld || ld_gate < heads * vdim)
        return PIE_HIP_ERR_INVALID;
    // whole 16-byte pieces of the low-rank columns must lie inside a row
    if (ld % 8 != 0 || ld_gate % 16 != 0 || decay_off % 8 != 0 || gate_off % 8 != 0 || ld_a1 % 32 != 0 || ld_g1 % 32 != 0 ||
        decay_off + (decay_rank + 7) / 8 * 8 > ld || gate_off + (gate_rank + 7) / 8 * 8 > ld)
        return PIE_HIP_ERR_UNSUPPORTED;
    const LowRankArgs a{fused, w_decay, w_gate, rate, dt_bias, log2_decay, gate, num_tokens, ld, decay_off, gate_off,
                        decay_rank, gate_rank, ld_a1, ld_g1, dim, heads * dim, heads * vdim, ld_gate, (heads * dim + 63) / 64};
    const int gx = a.decay_blocks + (heads * vdim + 63) / 64;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == PIE_HIP_DT_F32) {
        if (num_tokens > 65535) return PIE_HIP_ERR_UNSUPPORTED;
        hipLaunchKernelGGL(delta_lowrank_f32_kernel, dim3(gx, num_tokens), dim3(64), 0, s, a);
        return launch_status();
    }
    if (dtype != PIE_HIP_DT_BF16) return PIE_HIP_ERR_INVALID;
    const int mt = num_tokens <= 16 ? 1 : num_tokens <= 32 ? 2 : 4, gy = (num_tokens + 16 * mt - 1) / (16 * mt);
    if (gy > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch (mt) {
        case 1: hipLaunchKernelGGL(delta_lowrank_mfma_kernel<1>, dim3(gx, gy), dim3(256), 0, s, a); break;
        case 2: hipLaunchKernelGGL(delta_lowrank_mfma_kernel<2>, dim3(gx, gy), dim3(256), 0, s, a); break;
        default: hipLaunchKernelGGL(delta_lowrank_mfma_kernel<4>, dim3(gx, gy), dim3(256), 0, s, a); break;
    }
    return launch_status();
}

extern "C" int pie_hip_delta_scan(const float* q, const float* k, const float* v, const float* log2_decay,
                                  const float* beta, float* o, void* rs_base, size_t rs_stride, size_t state_offset,
                                  const int32_t* qo_indptr, const int32_t* rs_slot, const int32_t* rs_fresh,
                                  int num_requests, int heads, int kv_heads, int dim, int vdim, void* stream) {
    if (!q || !k || !v || !log2_decay || !beta || !o || !rs_base || !qo_indptr || !rs_slot || !rs_fresh || num_requests <= 0 ||
        heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || vdim <= 0)
        return PIE_HIP_ERR_INVALID;
    const DeltaScanArgs a{q, k, v, log2_decay, beta, o, static_cast<unsigned char*>(rs_base), rs_stride, state_offset,
                          {nullptr, qo_indptr, rs_slot, rs_fresh}, heads, kv_heads, dim, vdim};
    const dim3 grid(num_requests, heads, (vdim + kCols - 1) / kCols);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (heads > 65535 || grid.z > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch ((dim + 31) / 32) {
        case 1: hipLaunchKernelGGL(delta_scan_kernel<1>, grid, dim3(256), 0, s, a); break;
        case 2: hipLaunchKernelGGL(delta_scan_kernel<2>, grid, dim3(256), 0, s, a); break;
        case 3: case 4: hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(256), 0, s, a); break;
        case 5: case 6: hipLaunchKernelGGL(delta_scan_kernel<6>, grid, dim3(256), 0, s, a); break;
        case 7: case 8: hipLaunchKernelGGL(delta_scan_kernel<8>, grid, dim3(256), 0, s, a); break;
        default: return PIE_HIP_ERR_UNSUPPORTED;
    }
    return launch_status();
}

extern "C" size_t pie_hip_delta_chunked_workspace_bytes(int num_chunks, int heads, int dim) {
    if (num_chunks <= 0 || heads <= 0 || dim <= 0 || dim > 256) return 0;
    const size_t dp = static_cast<size_t>((dim + 63) / 64) * 64;
    return static_cast<size_t>(num_chunks) * heads * (49 * dp + 512) * sizeof(float);
}

extern "C" int pie_hip_delta_chunked(const float* q, const float* k, const float* v, const float* log2_decay,
                                     const float* beta, float* o, void* rs_base, size_t rs_stride, size_t state_offset,
                                     const int32_t* chunks, const int32_t* req_chunks, const int32_t* qo_indptr,
                                     const int32_t* rs_slot, const int32_t* rs_fresh, int num_chunks, int num_requests, int heads, int kv_heads,
                                     int dim, int vdim, void* workspace, size_t workspace_bytes, void* stream) {
    if (!q || !k || !v || !log2_decay || !beta || !o || !rs_base || !chunks || !req_chunks || !qo_indptr || !rs_slot || !rs_fresh ||
        num_chunks <= 0 || num_requests <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || vdim <= 0)
        return PIE_HIP_ERR_INVALID;
    if (dim > 256 || num_chunks > 65535 || num_requests > 65535 || (vdim + 15) / 16 > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    if (!workspace || workspace_bytes < pie_hip_delta_chunked_workspace_bytes(num_chunks, heads, dim)) return PIE_HIP_ERR_INVALID;
    float* rec = static_cast<float*>(workspace);
    const DeltaChunkArgs c{q, k, log2_decay, beta, chunks, rec, heads, kv_heads, dim};
    const DeltaWalkArgs w{rec, v, o, static_cast<unsigned char*>(rs_base), rs_stride, state_offset, req_chunks, qo_indptr,
                          rs_slot, rs_fresh, heads, dim, vdim};
    hipStream_t s = static_cast<hipStream_t>(stream);
    switch ((dim + 63) / 64) {
        case 1: return launch_chunked<1>(c, w, num_chunks, num_requests, s);
        case 2: return launch_chunked<2>(c, w, num_chunks, num_requests, s);
        case 3: return launch_chunked<3>(c, w, num_chunks, num_requests, s);
        default: return launch_chunked<4>(c, w, num_chunks, num_requests, s);
    }
}

extern "C" int pie_hip_delta_out(int dtype, const float* o, const void* gate, const float* norm_w, void* y,
                                 int num_tokens, int ld_gate, int ld_y, int heads, int vdim, float eps, void* stream) {
    if (!o || !gate || !norm_w || !y || num_tokens <= 0 || heads <= 0 || vdim <= 0 || ld_gate < heads * vdim || ld_y < heads * vdim)
        return PIE_HIP_ERR_INVALID;
    const int total = num_tokens * heads;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(delta_out_kernel<T>, dim3((total + 3) / 4), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), o, static_cast<const T*>(gate), norm_w,
                                                  static_cast<T*>(y), total, heads, vdim, ld_gate, ld_y, eps));
    return launch_status();
}

namespace {
// threads per state row (four columns each) and rows per thread of the one-token kernel; 0: not taken
int step_rows(int dim, int vdim, int* tpr_shift) {
    if (dim <= 0 || vdim <= 0 || dim > 256 || vdim > 256 || vdim % 4 != 0) return 0;
    int sh = 0;
    while ((4 << sh) < vdim) ++sh;
    *tpr_shift = sh;
    const int nr = (dim + (256 >> sh) - 1) / (256 >> sh);
    return nr <= 4 ? 4 : nr <= 8 ? 8 : nr <= 16 ? 16 : nr <= 32 ? 32 : 0;
}
}  // namespace

extern "C" int pie_hip_delta_step_supported(int dim, int vdim) {
    int sh = 0;
    return step_rows(dim, vdim, &sh) > 0;
}

extern "C" int pie_hip_delta_step(int dtype, const void* fused, const float* conv_w, const float* log2_decay,
                                  const void* gate, const float* norm_w, void* y, void* rs_base, size_t rs_stride,
                                  size_t state_offset, size_t conv_offset, const int32_t* rs_slot,
                                  const int32_t* rs_fresh, int num_requests, int ld, int ld_gate, int ld_y, int heads,
                                  int kv_heads, int dim, int vdim, int taps, int write_conv, float eps, void* stream) {
    if (!fused || !conv_w || !log2_decay || !gate || !norm_w || !y || !rs_base || !rs_slot || !rs_fresh || num_requests <= 0 ||
        heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || taps <= 0 || ld < 2 * kv_heads * dim + heads * vdim + heads ||
        ld_gate < heads * vdim || ld_y < heads * vdim)
        return PIE_HIP_ERR_INVALID;
    if (write_conv && heads != kv_heads) return PIE_HIP_ERR_INVALID;   // (heads that share channels would race)
    DeltaStepArgs a{fused, conv_w, log2_decay, gate, norm_w, y, static_cast<unsigned char*>(rs_base), rs_stride, state_offset,
                    conv_offset, rs_slot, rs_fresh, ld, ld_gate, ld_y, heads, kv_heads, dim, vdim, taps, 0, write_conv ? 1 : 0, eps};
    const int nr = step_rows(dim, vdim, &a.tpr_shift);
    if (nr == 0 || num_requests > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const dim3 grid(heads, num_requests);
    hipStream_t s = static_cast<hipStream_t>(stream);
    PIE_ACT_DISPATCH(dtype, T, switch (nr) {
        case 4: hipLaunchKernelGGL((delta_step_kernel<T, 4>), grid, dim3(256), 0, s, a); break;
        case 8: hipLaunchKernelGGL((delta_step_kernel<T, 8>), grid, dim3(256), 0, s, a); break;
        case 16: hipLaunchKernelGGL((delta_step_kernel<T, 16>), grid, dim3(256), 0, s, a); break;
        default: hipLaunchKernelGGL((delta_step_kernel<T, 32>), grid, dim3(256), 0, s, a); break;
    });
    return launch_status();
}
