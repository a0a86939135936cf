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
    const void* fused;       // [N, ld]: q | k | v | b | (decay_off) a1 | (gate_off) g1
    const float* conv_w;     // [channels, taps], channels = q | k | v
    const unsigned char* rs_base;
    size_t rs_stride, conv_offset;   // bytes
    DeltaRows rows;
    float* q;      // [N, kv_heads * dim]
    float* k;
    float* v;      // [N, heads * vdim]
    float* beta;   // [N, heads]
    void* a1;      // [N, ld_a1]
    void* g1;      // [N, ld_g1]
    int ld, heads, kv_heads, dim, vdim, taps, decay_off, decay_rank, ld_a1, gate_off, gate_rank, ld_g1;
};

// One wave per unit of a row: a q head, a k head (convolution, silu, unit vector), 256 channels of
// v (convolution, silu), or the row's step sizes and low-rank inputs.
constexpr int kVUnit = 256, kMaxPerLane = 8;   // q / k heads of up to 512 channels
template <class T>
__global__ __launch_bounds__(256) void delta_prep_kernel(const DeltaPrepArgs a) {
    const int n = blockIdx.x, lane = threadIdx.x & (kWave - 1);
    const int unit = blockIdx.y * 4 + threadIdx.x / kWave;
    const int kd = a.kv_heads * a.dim, vd = a.heads * a.vdim;
    const int vunits = (vd + kVUnit - 1) / kVUnit;
    const int r = a.rows.row_req[n];
    const int row0 = a.rows.qo_indptr[r], i = n - row0;
    const bool fresh = a.rows.rs_fresh[r] != 0;
    const int keep = a.taps - 1, channels = 2 * kd + vd;
    const T* fused = static_cast<const T*>(a.fused);
    const T* state = reinterpret_cast<const T*>(a.rs_base + static_cast<size_t>(a.rows.rs_slot[r]) * a.rs_stride + a.conv_offset);
    auto conv_silu = [&](int c) {
        const float* w = a.conv_w + static_cast<size_t>(c) * a.taps;
        float y = 0.f;
        for (int j = 0; j < a.taps; ++j)
            y = fmaf(w[j], conv_input<T>(fused, state, a.ld, row0, i - keep + j, c, keep, channels, fresh), y);
        return y * sigmoid_f32(y);
    };
    if (unit < 2 * a.kv_heads) {
        const bool is_q = unit < a.kv_heads;
        const int h = is_q ? unit : unit - a.kv_heads;
        const int c0 = (is_q ? 0 : kd) + h * a.dim;
        float val[kMaxPerLane];
        float local = 0.f;
#pragma unroll
        for (int e = 0; e < kMaxPerLane; ++e) {
            const int d = lane + e * kWave;
            val[e] = d < a.dim ? conv_silu(c0 + d) : 0.f;
            local += val[e] * val[e];
        }
        const float inv = (is_q ? 1.f / sqrtf(static_cast<float>(a.dim)) : 1.f) / sqrtf(wave_sum(local) + 1e-6f);
        float* dst = (is_q ? a.q : a.k) + static_cast<size_t>(n) * kd + h * a.dim;
#pragma unroll
        for (int e = 0; e < kMaxPerLane; ++e) {
            const int d = lane + e * kWave;
            if (d < a.dim) dst[d] = val[e] * inv;
        }
    } else if (unit < 2 * a.kv_heads + vunits) {
        const int c0 = (unit - 2 * a.kv_heads) * kVUnit;
        for (int c = c0 + lane; c < min(c0 + kVUnit, vd); c += kWave)
            a.v[static_cast<size_t>(n) * vd + c] = conv_silu(2 * kd + c);
    } else if (unit == 2 * a.kv_heads + vunits) {
        const T* row = fused + static_cast<size_t>(n) * a.ld;
        for (int h = lane; h < a.heads; h += kWave)
            a.beta[static_cast<size_t>(n) * a.heads + h] = sigmoid_f32(act_get<T>(row[channels + h]));
        T* a1 = static_cast<T*>(a.a1) + static_cast<size_t>(n) * a.ld_a1;
        T* g1 = static_cast<T*>(a.g1) + static_cast<size_t>(n) * a.ld_g1;
        for (int c = lane; c < a.ld_a1; c += kWave) a1[c] = c < a.decay_rank ? row[a.decay_off + c] : act_put<T>(0.f);
        for (int c = lane; c < a.ld_g1; c += kWave) g1[c] = c < a.gate_rank ? row[a.gate_off + c] : act_put<T>(0.f);
    }
}

__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// g = exp(-exp(A_log[head]) * softplus(raw + dt_bias)), four elements per thread
template <class T>
__global__ __launch_bounds__(256) void delta_decay_kernel(const T* __restrict__ raw, const float* __restrict__ a_log,
                                                          const float* __restrict__ dt_bias, float* __restrict__ g,
                                                          int ld_raw, int dim, int width) {
    const size_t n = blockIdx.y;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < width; c += gridDim.x * 256)
        g[n * width + c] = expf(-expf(a_log[c / dim]) * softplus_f32(act_get<T>(raw[n * ld_raw + c]) + dt_bias[c]));
}

struct DeltaScanArgs {
    const float *q, *k, *v, *g, *beta;
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
            rgv[e] = ok ? a.g[static_cast<size_t>(n) * gd + h * a.dim + d] : 0.f;
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

struct DeltaOutArgs {
    const float* o;        // [N, heads * vdim]
    const void* gate;      // [N, ld_gate] projected gate
    const float* norm_w;   // [vdim]
    void* y;               // [N, ld_y]
    const void* fused;     // the convolution's inputs (this step's rows)
    unsigned char* rs_base;
    size_t rs_stride, conv_offset;
    DeltaRows rows;
    int ld_gate, ld_y, ld_fused, heads, vdim, taps, channels;
    float eps;
};

// y = o / rms(o) * norm_w * sigmoid(gate) per head, and, on each request's last row, the
// convolution inputs its next tokens will need.  One block per row, a wave per head in turn.
template <class T>
__global__ __launch_bounds__(256) void delta_out_kernel(const DeltaOutArgs a) {
    const int n = blockIdx.x, lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int vd = a.heads * a.vdim;
    const T* gate = static_cast<const T*>(a.gate) + static_cast<size_t>(n) * a.ld_gate;
    T* y = static_cast<T*>(a.y) + static_cast<size_t>(n) * a.ld_y;
    for (int h = wv; h < a.heads; h += 4) {
        const float* o = a.o + static_cast<size_t>(n) * vd + h * a.vdim;
        float local = 0.f;
        for (int c = lane; c < a.vdim; c += kWave) local += o[c] * o[c];
        const float inv = 1.f / sqrtf(wave_sum(local) / static_cast<float>(a.vdim) + a.eps);
        for (int c = lane; c < a.vdim; c += kWave)
            y[h * a.vdim + c] = act_put<T>(o[c] * inv * a.norm_w[c] * sigmoid_f32(act_get<T>(gate[h * a.vdim + c])));
    }
    const int r = a.rows.row_req[n];
    const int row0 = a.rows.qo_indptr[r], T_ = a.rows.qo_indptr[r + 1] - row0;
    if (n != row0 + T_ - 1) return;
    const int keep = a.taps - 1;
    const bool fresh = a.rows.rs_fresh[r] != 0;
    const T* fused = static_cast<const T*>(a.fused);
    T* state = reinterpret_cast<T*>(a.rs_base + static_cast<size_t>(a.rows.rs_slot[r]) * a.rs_stride + a.conv_offset);
    // (a channel's entries move towards the front: entry j is read no later than it is written)
    for (int c = threadIdx.x; c < a.channels; c += 256)
        for (int j = 0; j < keep; ++j)
            state[static_cast<size_t>(j) * a.channels + c] =
                act_put<T>(conv_input<T>(fused, state, a.ld_fused, row0, T_ - keep + j, c, keep, a.channels, fresh));
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_delta_prep(int dtype, const void* fused, const float* conv_w, const void* rs_base,
                                  size_t rs_stride, size_t conv_offset, const int32_t* row_req,
                                  const int32_t* qo_indptr, const int32_t* rs_slot, const int32_t* rs_fresh, float* q,
                                  float* k, float* v, float* beta, void* a1, void* g1, int num_tokens, int ld,
                                  int heads, int kv_heads, int dim, int vdim, int taps, int decay_off, int decay_rank,
                                  int ld_a1, int gate_off, int gate_rank, int ld_g1, void* stream) {
    if (!fused || !conv_w || !rs_base || !row_req || !qo_indptr || !rs_slot || !rs_fresh || !q || !k || !v || !beta ||
        !a1 || !g1 || num_tokens <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 ||
        vdim <= 0 || taps <= 0)
        return PIE_HIP_ERR_INVALID;
    const int channels = 2 * kv_heads * dim + heads * vdim;
    if (decay_off < channels + heads || gate_off < channels + heads || decay_off + decay_rank > ld ||
        gate_off + gate_rank > ld || ld_a1 < decay_rank || ld_g1 < gate_rank)
        return PIE_HIP_ERR_INVALID;
    if (dim > kMaxPerLane * kWave) return PIE_HIP_ERR_UNSUPPORTED;
    const DeltaPrepArgs a{fused, conv_w, static_cast<const unsigned char*>(rs_base), rs_stride, conv_offset,
                          {row_req, qo_indptr, rs_slot, rs_fresh}, q, k, v, beta, a1, g1, ld, heads, kv_heads, dim, vdim,
                          taps, decay_off, decay_rank, ld_a1, gate_off, gate_rank, ld_g1};
    const int units = 2 * kv_heads + (heads * vdim + kVUnit - 1) / kVUnit + 1;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(delta_prep_kernel<T>, dim3(num_tokens, (units + 3) / 4), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), a));
    return launch_status();
}

extern "C" int pie_hip_delta_decay(int dtype, const void* raw, const float* a_log, const float* dt_bias, float* g,
                                   int num_tokens, int ld_raw, int heads, int dim, void* stream) {
    if (!raw || !a_log || !dt_bias || !g || num_tokens <= 0 || heads <= 0 || dim <= 0 || ld_raw < heads * dim)
        return PIE_HIP_ERR_INVALID;
    if (num_tokens > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(delta_decay_kernel<T>, dim3((heads * dim + 255) / 256, num_tokens),
                                                  dim3(256), 0, static_cast<hipStream_t>(stream),
                                                  static_cast<const T*>(raw), a_log, dt_bias, g, ld_raw, dim, heads * dim));
    return launch_status();
}

extern "C" int pie_hip_delta_scan(const float* q, const float* k, const float* v, const float* g, const float* beta,
                                  float* o, void* rs_base, size_t rs_stride, size_t state_offset,
                                  const int32_t* qo_indptr, const int32_t* rs_slot, const int32_t* rs_fresh,
                                  int num_requests, int heads, int kv_heads, int dim, int vdim, void* stream) {
    if (!q || !k || !v || !g || !beta || !o || !rs_base || !qo_indptr || !rs_slot || !rs_fresh || num_requests <= 0 ||
        heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || vdim <= 0)
        return PIE_HIP_ERR_INVALID;
    const DeltaScanArgs a{q, k, v, g, beta, o, static_cast<unsigned char*>(rs_base), rs_stride, state_offset,
                          {nullptr, qo_indptr, rs_slot, rs_fresh}, heads, kv_heads, dim, vdim};
    const dim3 grid(num_requests, heads, (vdim + kCols - 1) / kCols);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (heads > 65535 || grid.z > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch ((dim + 31) / 32) {
        case 1: hipLaunchKernelGGL(delta_scan_kernel<1>, grid, dim3(256), 0, s, a); break;
        case 2: hipLaunchKernelGGL(delta_scan_kernel<2>, grid, dim3(256), 0, s, a); break;
        case 3: hipLaunchKernelGGL(delta_scan_kernel<3>, grid, dim3(256), 0, s, a); break;
        case 4: hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(256), 0, s, a); break;
        case 5: case 6: hipLaunchKernelGGL(delta_scan_kernel<6>, grid, dim3(256), 0, s, a); break;
        case 7: case 8: hipLaunchKernelGGL(delta_scan_kernel<8>, grid, dim3(256), 0, s, a); break;
        default: return PIE_HIP_ERR_UNSUPPORTED;
    }
    return launch_status();
}

extern "C" int pie_hip_delta_out(int dtype, const float* o, const void* gate, const float* norm_w, void* y,
                                 const void* fused, void* rs_base, size_t rs_stride, size_t conv_offset,
                                 const int32_t* row_req, const int32_t* qo_indptr, const int32_t* rs_slot,
                                 const int32_t* rs_fresh, int num_tokens, int ld_gate, int ld_y, int ld_fused,
                                 int heads, int kv_heads, int dim, int vdim, int taps, float eps, void* stream) {
    if (!o || !gate || !norm_w || !y || !fused || !rs_base || !row_req || !qo_indptr || !rs_slot || !rs_fresh ||
        num_tokens <= 0 || heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || taps <= 0 ||
        ld_gate < heads * vdim || ld_y < heads * vdim || ld_fused < 2 * kv_heads * dim + heads * vdim)
        return PIE_HIP_ERR_INVALID;
    const DeltaOutArgs a{o, gate, norm_w, y, fused, static_cast<unsigned char*>(rs_base), rs_stride, conv_offset,
                         {row_req, qo_indptr, rs_slot, rs_fresh}, ld_gate, ld_y, ld_fused, heads, vdim, taps,
                         2 * kv_heads * dim + heads * vdim, eps};
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(delta_out_kernel<T>, dim3(num_tokens), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), a));
    return launch_status();
}
