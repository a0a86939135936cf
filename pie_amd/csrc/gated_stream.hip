// The residual stream of layers whose sublayers' outputs pass a logistic gate and whose sublayers read a short
// convolution of the normed stream:
//   h = norm(x),  x += sublayer(h + conv(h)) * sigmoid(W h + b)
//   gated_join     what ends a sublayer: the gated output joins the fp32 stream, which is normed for the next one;
//                  with one row per request the convolution and the move of its state ride along.  The stream's
//                  start is the same kernel: the normed sum of up to two embedding rows instead of a stream
//   recent_rows    the convolution of portions, over the requests' rows and states
// The normed row is rounded to the compute type before anything reads it, so that the convolution of a row
// does not depend on which of the two kernels formed it.
#include "act_type.hip.h"

namespace pie_hip {
namespace {

struct GatedJoinArgs {
    const void *y, *gate;
    const float *gate_bias, *next_w;
    const uint16_t* conv_w;
    PieHipRoutes routes;
    PieHipEmbedding start;
    float* x;
    void *h, *recent;
    PieHipStateRows state;
    int ldy, ld_gate, width, ld;
    float eps;
};
// One block per row: a thread has eight neighbouring columns, and whatever it reads for them is requested before
// the row's sum is formed.  Columns past 8 BLOCK, and rows whose width is no multiple of eight, one by one.
// TAPS > 0: row n is request n's only one, and its convolution follows.
template <class T, int BLOCK, int TAPS>
__global__ __launch_bounds__(BLOCK) void gated_join_kernel(const GatedJoinArgs a) {
    __shared__ float red[BLOCK / kWave];
    __shared__ int pos[kJoinRoutes];
    __shared__ float weight[kJoinRoutes];
    constexpr int KEEP = TAPS > 0 ? TAPS - 1 : 0;
    const size_t n = blockIdx.x;
    const T* yr = a.y ? static_cast<const T*>(a.y) + n * a.ldy : nullptr;
    const T* gr = a.gate ? static_cast<const T*>(a.gate) + n * a.ld_gate : nullptr;
    const T* ry = static_cast<const T*>(a.routes.y);
    const int K = ry ? a.routes.top_k : 0;
    const bool joins = yr || K, starts = a.start.token_ids != nullptr;
    const uint16_t *er = nullptr, *pr = nullptr;
    if (starts) {
        const uint32_t t = a.start.token_ids[n];
        er = a.start.table + static_cast<size_t>(t < static_cast<uint32_t>(a.start.vocab) ? t : 0) * a.width;
        if (a.start.pair_table) pr = a.start.pair_table + static_cast<size_t>(a.start.pair_rows[n]) * a.width;
    }
    float* xr = a.x + n * a.ld;
    T* hr = static_cast<T*>(a.h) + n * a.ld;
    T* rr = static_cast<T*>(a.recent) + n * a.ld;
    T* st = nullptr;
    bool fresh = true;
    if constexpr (KEEP > 0) {
        fresh = a.state.rs_fresh[n] != 0;
        st = reinterpret_cast<T*>(static_cast<unsigned char*>(a.state.rs_base) + static_cast<size_t>(a.state.rs_slot[n]) * a.state.rs_stride +
                                  a.state.conv_offset);
    }
    if (K) {
        if (threadIdx.x < static_cast<unsigned>(K)) {
            pos[threadIdx.x] = a.routes.pos[n * K + threadIdx.x];
            weight[threadIdx.x] = a.routes.weight[n * K + threadIdx.x];
        }
        __syncthreads();
    }
    const int n8 = a.width % 8 == 0 ? min(a.width / 8, BLOCK) : 0;
    const int done = 8 * n8, i8 = 8 * threadIdx.x;
    const bool mine = static_cast<int>(threadIdx.x) < n8;
    float v[8], local = 0.f;
    Eight<float> nw;
    Eight<uint16_t> cw[TAPS > 0 ? TAPS : 1];
    Eight<T> past[KEEP > 0 ? KEEP : 1];
    Eight<float> sw;
    if (mine) {
        Eight<uint16_t> ge, gp;
        if (starts) {
            ge.load(er + i8);
            if (pr) gp.load(pr + i8);
            sw.load(a.start.norm_weight + i8);
        }
        Eight<T> gy, gz;
        Eight<float> gb, gx;
        if (yr) gy.load(yr + i8);
        if (joins) {
            gz.load(gr + i8);
            gb.load(a.gate_bias + i8);
        }
        if (!starts) gx.load(xr + i8);
        if (a.next_w) nw.load(a.next_w + i8);
        if constexpr (TAPS > 0) {
#pragma unroll
            for (int j = 0; j < TAPS; ++j) cw[j].load(a.conv_w + static_cast<size_t>(j) * a.width + i8);
#pragma unroll
            for (int j = 0; j < KEEP; ++j)
                if (!fresh) past[j].load(st + static_cast<size_t>(j) * a.width + i8);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = yr ? gy.get(e) : 0.f;
        for (int k0 = 0; k0 < K; k0 += 8) {
            Eight<T> r[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) r[u].load(ry + static_cast<size_t>(pos[min(k0 + u, K - 1)]) * a.routes.ld + i8);
#pragma unroll
            for (int u = 0; u < 8; ++u)
                if (k0 + u < K) {
                    const float w = weight[k0 + u];
#pragma unroll
                    for (int e = 0; e < 8; ++e) v[e] = fmaf(r[u].get(e), w, v[e]);
                }
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            if (!starts) v[e] = joins ? fmaf(v[e], sigmoid_f32(gz.get(e) + gb.get(e)), gx.get(e)) : gx.get(e);
            else v[e] = ge.get(e) * a.start.scale + (pr ? gp.get(e) : 0.f);
            local += v[e] * v[e];
        }
    }
    if (starts) {   // (uniform: the whole block)
        for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {
            const float o = bf16_bits_to_f32(er[i]) * a.start.scale + (pr ? bf16_bits_to_f32(pr[i]) : 0.f);
            xr[i] = o;
            local += o * o;
        }
        const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(a.width) + a.eps);
        local = 0.f;
        if (mine)
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                v[e] *= inv * sw.get(e);
                local += v[e] * v[e];
            }
        for (int i = done + threadIdx.x; i < a.width; i += BLOCK) xr[i] *= inv * a.start.norm_weight[i];
    }
    if (mine && (joins || starts))
#pragma unroll
        for (int p = 0; p < 2; ++p)
            *reinterpret_cast<f32x4_t*>(xr + i8 + 4 * p) = f32x4_t{v[4 * p], v[4 * p + 1], v[4 * p + 2], v[4 * p + 3]};
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {
        float s = yr ? act_get<T>(yr[i]) : 0.f;
        for (int k = 0; k < K; ++k) s = fmaf(act_get<T>(ry[static_cast<size_t>(pos[k]) * a.routes.ld + i]), weight[k], s);
        const float o = joins ? fmaf(s, sigmoid_f32(act_get<T>(gr[i]) + a.gate_bias[i]), xr[i]) : xr[i];
        if (joins) xr[i] = o;
        local += o * o;
    }
    if (!a.next_w) return;
    const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(a.width) + a.eps);
    auto store = [&](T* to, const T (&o)[8]) {
        if constexpr (sizeof(T) == 2) {
            *reinterpret_cast<u32x4_t*>(to) = u32x4_t{o[0] | static_cast<uint32_t>(o[1]) << 16, o[2] | static_cast<uint32_t>(o[3]) << 16,
                                                      o[4] | static_cast<uint32_t>(o[5]) << 16, o[6] | static_cast<uint32_t>(o[7]) << 16};
        } else {
#pragma unroll
            for (int p = 0; p < 2; ++p) *reinterpret_cast<f32x4_t*>(to + 4 * p) = f32x4_t{o[4 * p], o[4 * p + 1], o[4 * p + 2], o[4 * p + 3]};
        }
    };
    if (mine) {
        T h[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) h[e] = act_put<T>(v[e] * inv * nw.get(e));
        store(hr + i8, h);
        if constexpr (TAPS > 0) {
            T o[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float now = act_get<T>(h[e]);
                float s = 0.f;
#pragma unroll
                for (int j = 0; j < KEEP; ++j) s = fmaf(cw[j].get(e), fresh ? 0.f : past[j].get(e), s);
                o[e] = act_put<T>(now + fmaf(cw[TAPS - 1].get(e), now, s));
            }
            store(rr + i8, o);
#pragma unroll
            for (int j = 0; j + 1 < KEEP; ++j) {
                T moved[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) moved[e] = act_put<T>(fresh ? 0.f : past[j + 1].get(e));
                store(st + static_cast<size_t>(j) * a.width + i8, moved);
            }
            if constexpr (KEEP > 0) store(st + static_cast<size_t>(KEEP - 1) * a.width + i8, h);
        }
    }
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {   // (a thread reads what it wrote)
        const T h = act_put<T>(xr[i] * inv * a.next_w[i]);
        hr[i] = h;
        if constexpr (TAPS > 0) {
            const float now = act_get<T>(h);
            float s = 0.f;
#pragma unroll
            for (int j = 0; j < KEEP; ++j) {
                T* at = st + static_cast<size_t>(j) * a.width + i;
                s = fmaf(bf16_bits_to_f32(a.conv_w[static_cast<size_t>(j) * a.width + i]), fresh ? 0.f : act_get<T>(*at), s);
                *at = j + 1 < KEEP ? (fresh ? act_put<T>(0.f) : at[a.width]) : h;
            }
            rr[i] = act_put<T>(now + fmaf(bf16_bits_to_f32(a.conv_w[static_cast<size_t>(KEEP) * a.width + i]), now, s));
        }
    }
}

// V columns per thread, RUN consecutive rows per block.  TAPS > 0: the window of earlier rows stays in registers
// and moves with the rows; 0: any number of taps, the window read afresh for every row.
template <class T, int V, int RUN, int TAPS>
__global__ __launch_bounds__(256) void recent_rows_kernel(const T* __restrict__ h, const uint16_t* __restrict__ w, int taps,
                                                          const PieHipStateRows rows, T* __restrict__ out, int width, int ld) {
    typedef T vec_t __attribute__((ext_vector_type(V)));
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= width) return;   // (width is a multiple of V)
    const int n0 = blockIdx.y * RUN, n1 = min(n0 + RUN, rows.num_tokens), keep = (TAPS > 0 ? TAPS : taps) - 1;
    vec_t now[RUN];
#pragma unroll
    for (int u = 0; u < RUN; ++u)
        if (n0 + u < n1) now[u] = *reinterpret_cast<const vec_t*>(h + static_cast<size_t>(n0 + u) * ld + c);
    int r = -1, row0 = 0;
    bool fresh = true;
    const T* state = nullptr;
    auto earlier = [&](int i, int e) {   // the request's row i (negative: from its state)
        if (i >= 0) return act_get<T>(h[static_cast<size_t>(row0 + i) * ld + c + e]);
        return fresh ? 0.f : act_get<T>(state[static_cast<size_t>(keep + i) * width + c + e]);
    };
    constexpr int KEEP = TAPS > 1 ? TAPS - 1 : 1;
    typedef uint16_t weights_t __attribute__((ext_vector_type(V)));
    float win[KEEP][V];
    weights_t wr[TAPS > 0 ? TAPS : 1];
    if constexpr (TAPS > 0)
#pragma unroll
        for (int j = 0; j < TAPS; ++j) wr[j] = *reinterpret_cast<const weights_t*>(w + static_cast<size_t>(j) * width + c);
#pragma unroll
    for (int u = 0; u < RUN; ++u) {
        const int n = n0 + u;
        if (n >= n1) break;
        const int req = rows.row_req[n];
        if (req != r) {
            r = req;
            row0 = rows.qo_indptr[r];
            fresh = rows.rs_fresh[r] != 0;
            state = reinterpret_cast<const T*>(static_cast<const unsigned char*>(rows.rs_base) +
                                               static_cast<size_t>(rows.rs_slot[r]) * rows.rs_stride + rows.conv_offset);
            if constexpr (TAPS > 1)
#pragma unroll
                for (int j = 0; j < KEEP; ++j)
#pragma unroll
                    for (int e = 0; e < V; ++e) win[j][e] = earlier(n - row0 - KEEP + j, e);
        }
        vec_t o;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            const float x = act_get<T>(now[u][e]);
            float s = 0.f;
            if constexpr (TAPS > 0) {
                if constexpr (TAPS > 1) {
#pragma unroll
                    for (int j = 0; j < KEEP; ++j) s = fmaf(bf16_bits_to_f32(wr[j][e]), win[j][e], s);
#pragma unroll
                    for (int j = 0; j < KEEP; ++j) win[j][e] = j + 1 < KEEP ? win[j + 1 < KEEP ? j + 1 : j][e] : x;
                }
                s = fmaf(bf16_bits_to_f32(wr[TAPS - 1][e]), x, s);
            } else {
                for (int j = 0; j < keep; ++j) s = fmaf(bf16_bits_to_f32(w[static_cast<size_t>(j) * width + c + e]), earlier(n - row0 - keep + j, e), s);
                s = fmaf(bf16_bits_to_f32(w[static_cast<size_t>(keep) * width + c + e]), x, s);
            }
            o[e] = act_put<T>(x + s);
        }
        *reinterpret_cast<vec_t*>(out + static_cast<size_t>(n) * ld + c) = o;
    }
}

bool state_ok(const PieHipStateRows* r) {
    return r && r->row_req && r->qo_indptr && r->rs_slot && r->rs_fresh && r->num_tokens > 0 && r->num_requests > 0;
}

template <class T, int BLOCK>
int launch_gated_join(const GatedJoinArgs& a, int rows, int taps, hipStream_t s) {
    switch (a.conv_w ? taps : 0) {
        case 0: hipLaunchKernelGGL((gated_join_kernel<T, BLOCK, 0>), dim3(rows), dim3(BLOCK), 0, s, a); break;
        case 1: hipLaunchKernelGGL((gated_join_kernel<T, BLOCK, 1>), dim3(rows), dim3(BLOCK), 0, s, a); break;
        case 2: hipLaunchKernelGGL((gated_join_kernel<T, BLOCK, 2>), dim3(rows), dim3(BLOCK), 0, s, a); break;
        case 3: hipLaunchKernelGGL((gated_join_kernel<T, BLOCK, 3>), dim3(rows), dim3(BLOCK), 0, s, a); break;
        case 4: hipLaunchKernelGGL((gated_join_kernel<T, BLOCK, 4>), dim3(rows), dim3(BLOCK), 0, s, a); break;
        default: return PIE_HIP_ERR_UNSUPPORTED;
    }
    return launch_status();
}

template <class T, int V, int RUN>
int launch_recent_rows(const T* h, const uint16_t* w, int taps, const PieHipStateRows& rows, T* out, int width, int ld, hipStream_t s) {
    const dim3 grid((width / V + 255) / 256, (rows.num_tokens + RUN - 1) / RUN);
    if (grid.y > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch (taps <= 4 ? taps : 0) {
        case 1: hipLaunchKernelGGL((recent_rows_kernel<T, V, RUN, 1>), grid, dim3(256), 0, s, h, w, taps, rows, out, width, ld); break;
        case 2: hipLaunchKernelGGL((recent_rows_kernel<T, V, RUN, 2>), grid, dim3(256), 0, s, h, w, taps, rows, out, width, ld); break;
        case 3: hipLaunchKernelGGL((recent_rows_kernel<T, V, RUN, 3>), grid, dim3(256), 0, s, h, w, taps, rows, out, width, ld); break;
        case 4: hipLaunchKernelGGL((recent_rows_kernel<T, V, RUN, 4>), grid, dim3(256), 0, s, h, w, taps, rows, out, width, ld); break;
        default: hipLaunchKernelGGL((recent_rows_kernel<T, V, RUN, 0>), grid, dim3(256), 0, s, h, w, taps, rows, out, width, ld); break;
    }
    return launch_status();
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_gated_join(int dtype, const void* y, int ldy, const PieHipRoutes* routes, const void* gate, int ld_gate,
                                  const float* gate_bias, const PieHipEmbedding* start, float* x, const float* next_weight,
                                  void* h, void* recent, const uint16_t* conv_w, int taps, const PieHipStateRows* state, int rows, int width, int ld,
                                  float eps, void* stream) {
    if (!x || rows <= 0 || width <= 0 || ld < width || (y && (routes || ldy < width)) || (next_weight && !h) ||
        ((y || routes) && (start || !gate || !gate_bias || ld_gate < width)) || (!y && !routes && !start && !next_weight) ||
        (start && (!start->token_ids || !start->table || !start->norm_weight || start->vocab <= 0 || (start->pair_table && !start->pair_rows))) ||
        (routes && (!routes->y || !routes->pos || !routes->weight || routes->top_k <= 0 || routes->ld < width)))
        return PIE_HIP_ERR_INVALID;
    if (conv_w && (!next_weight || !recent || taps <= 0 || !state_ok(state) || state->num_tokens != rows || state->num_requests != rows ||
                   (taps > 1 && !state->rs_base)))
        return PIE_HIP_ERR_INVALID;
    if ((y && ldy % 8 != 0) || ((y || routes) && ld_gate % 8 != 0) || (routes && (routes->ld % 8 != 0 || routes->top_k > kJoinRoutes)) ||
        ld % 8 != 0 || (conv_w && taps > 4))
        return PIE_HIP_ERR_UNSUPPORTED;
    const GatedJoinArgs a{y, gate, gate_bias, next_weight, conv_w, routes ? *routes : PieHipRoutes{}, start ? *start : PieHipEmbedding{}, x, h, recent,
                          conv_w ? *state : PieHipStateRows{}, ldy, ld_gate, width, ld, eps};
    hipStream_t s = static_cast<hipStream_t>(stream);
    PIE_ACT_DISPATCH(dtype, T, {
        if (width <= 2048) return launch_gated_join<T, 256>(a, rows, taps, s);
        if (width <= 4096) return launch_gated_join<T, 512>(a, rows, taps, s);
        return launch_gated_join<T, 1024>(a, rows, taps, s);
    });
}

extern "C" int pie_hip_recent_rows(int dtype, const void* h, const uint16_t* conv_w, int taps, const PieHipStateRows* state, void* recent,
                                   int width, int ld, void* stream) {
    if (!h || !conv_w || taps <= 0 || !state_ok(state) || (taps > 1 && !state->rs_base) || !recent || width <= 0 || ld < width)
        return PIE_HIP_ERR_INVALID;
    if (ld % 8 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const bool many = state->num_tokens >= 1024;
    PIE_ACT_DISPATCH(dtype, T, {
        // (many rows: 4-byte columns, 2048 rows of 4096 in 11.3 us against 13.1 of 16-byte ones; a copy of them takes 8.4)
        constexpr int V = 16 / sizeof(T), VMANY = sizeof(T) == 2 ? 2 : 4;
        const T* x = static_cast<const T*>(h);
        T* o = static_cast<T*>(recent);
        if (width % V != 0) return many ? launch_recent_rows<T, 1, 8>(x, conv_w, taps, *state, o, width, ld, s)
                                        : launch_recent_rows<T, 1, 1>(x, conv_w, taps, *state, o, width, ld, s);
        return many ? launch_recent_rows<T, VMANY, 8>(x, conv_w, taps, *state, o, width, ld, s)
                    : launch_recent_rows<T, V, 1>(x, conv_w, taps, *state, o, width, ld, s);
    });
}
