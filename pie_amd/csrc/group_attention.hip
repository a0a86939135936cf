// Grouped-query attention of the layer stacks: any head size, any number of query heads per key head, an
// optional sliding window, an optional sink (a constant added to the sum of exponentials), an optional gate
// on the output.
//   o[n, h, :] = sum_j p_j v_j,  p_j = exp(s_j) / (sink + sum exp(s)),  s_j = q[n, h, :] . k_j * scale,
//   len - window <= j < len = row_kv_len[n]
// A cache row holds, per key head, the key and the value next to each other: [kv_heads][dimp | dimp].
#include "act_type.hip.h"

#include <type_traits>

namespace pie_hip {
namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kStep = 32, kBlock = 256, kWaves = kBlock / kWave;

// ---- biases, norms per head, rotation, cache write -------------------------------------------------
struct PrepArgs {
    const void* fused;
    const float *q_bias, *k_bias, *q_norm, *k_norm, *rope;
    const int64_t* slots;
    void *q, *pool;
    int q_off, k_off, v_off, rot_dims, num_tokens, ld, heads, kv_heads, dim, dimp;
    float eps;
};
// One wave per (row, head): the query heads first, then the key heads (key and value).
constexpr int kPrepPerLane = 16;   // heads of up to 1024 values
template <class T, int PL>
__global__ __launch_bounds__(256) void group_prep_kernel(const PrepArgs a) {
    __shared__ float sh[4][PL * kWave];
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int units = a.heads + a.kv_heads;
    const long long unit = static_cast<long long>(blockIdx.x) * 4 + wv;
    const bool on = unit < static_cast<long long>(a.num_tokens) * units;
    const size_t n = on ? unit / units : 0;
    const int u = on ? static_cast<int>(unit % units) : 0;
    const bool is_q = u < a.heads;
    const int h = is_q ? u : u - a.heads;
    const T* row = static_cast<const T*>(a.fused) + n * a.ld;
    const T* src = row + (is_q ? a.q_off : a.k_off) + h * a.dim;
    const float* bias = is_q ? a.q_bias : a.k_bias;
    const float* norm = is_q ? a.q_norm : a.k_norm;
    float x[PL], raw[PL], local = 0.f;
#pragma unroll
    for (int e = 0; e < PL; ++e) {
        const int d = lane + e * kWave;
        x[e] = d < a.dim ? act_get<T>(src[d]) + (bias ? bias[h * a.dim + d] : 0.f) : 0.f;
        raw[e] = x[e];
        local += x[e] * x[e];
    }
    if (norm) {
        const float inv = 1.f / sqrtf(wave_sum_dpp(local) / static_cast<float>(a.dim) + a.eps);
#pragma unroll
        for (int e = 0; e < PL; ++e) {
            const int d = lane + e * kWave;
            if (d < a.dim) x[e] *= inv * norm[d];
        }
    }
#pragma unroll
    for (int e = 0; e < PL; ++e) sh[wv][lane + e * kWave] = x[e];
    __syncthreads();
    if (!on) return;
    const int half = a.rot_dims / 2;
    const float* tab = a.rope + n * a.rot_dims;
#pragma unroll
    for (int e = 0; e < PL; ++e) {
        const int d = lane + e * kWave;
        if (d < half) x[e] = x[e] * tab[d] - sh[wv][d + half] * tab[half + d];
        else if (d < a.rot_dims) x[e] = x[e] * tab[d - half] + sh[wv][d - half] * tab[d];
    }
    if (is_q) {
        T* q = static_cast<T*>(a.q) + (n * a.heads + h) * a.dimp;
#pragma unroll
        for (int e = 0; e < PL; ++e)
            if (lane + e * kWave < a.dimp) q[lane + e * kWave] = act_put<T>(x[e]);
        return;
    }
    const int64_t slot = a.slots[n];
    if (slot < 0) return;
    T* k = static_cast<T*>(a.pool) + (static_cast<size_t>(slot) * a.kv_heads + h) * 2 * a.dimp;
#pragma unroll
    for (int e = 0; e < PL; ++e) {
        const int d = lane + e * kWave;
        if (d >= a.dimp) continue;
        k[d] = act_put<T>(x[e]);
        k[a.dimp + d] = a.v_off < 0 ? act_put<T>(raw[e]) : d < a.dim ? row[a.v_off + h * a.dim + d] : act_put<T>(0.f);
    }
}

// The same for heads of whole 8-value pieces: a lane takes eight neighbouring values, LPH lanes a head, 64 / LPH
// heads a wave; a rotated value's partner is half / 8 lanes away.
template <class T>
__device__ __forceinline__ void load8(const T* p, float* f) {
    if constexpr (sizeof(T) == 2) {
        ActVec<T>::load(p, f);
    } else {
        ActVec<T>::load(p, f);
        ActVec<T>::load(p + 4, f + 4);
    }
}
template <class T>
__device__ __forceinline__ void store8(T* p, const float* f) {
    if constexpr (sizeof(T) == 2) {
        *reinterpret_cast<u32x4_t*>(p) = u32x4_t{pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]), pack_bf16x2(f[4], f[5]), pack_bf16x2(f[6], f[7])};
    } else {
        *reinterpret_cast<f32x4_t*>(p) = f32x4_t{f[0], f[1], f[2], f[3]};
        *reinterpret_cast<f32x4_t*>(p + 4) = f32x4_t{f[4], f[5], f[6], f[7]};
    }
}
template <class T, int LPH>
__global__ __launch_bounds__(256) void group_prep_vec_kernel(const PrepArgs a) {
    const int units = a.heads + a.kv_heads, lane = threadIdx.x & (kWave - 1);
    const long long unit = static_cast<long long>(blockIdx.x) * (256 / LPH) + threadIdx.x / LPH;
    const bool on = unit < static_cast<long long>(a.num_tokens) * units;   // (every lane takes part in the exchanges)
    const size_t n = on ? unit / units : 0;
    const int u = on ? static_cast<int>(unit % units) : 0;
    const bool is_q = u < a.heads;
    const int h = is_q ? u : u - a.heads, d = 8 * (lane & (LPH - 1));
    const bool in = on && d < a.dim, rotated = in && d < a.rot_dims;
    const T* row = static_cast<const T*>(a.fused) + n * a.ld;
    const int half = a.rot_dims / 2, t = d < half ? d : d - half;
    const float* bias = is_q ? a.q_bias : a.k_bias;
    const float* norm = is_q ? a.q_norm : a.k_norm;
    float x[8] = {}, raw[8], b[8] = {}, w[8] = {}, c[8] = {}, s[8] = {}, v[8] = {}, local = 0.f;
    const int64_t slot = on && !is_q ? a.slots[n] : -1;
    if (in) {
        load8(row + (is_q ? a.q_off : a.k_off) + h * a.dim + d, x);
        if (bias) load8(bias + h * a.dim + d, b);
        if (norm) load8(norm + d, w);
        if (!is_q && a.v_off >= 0) load8(row + a.v_off + h * a.dim + d, v);
    }
    if (rotated) {
        load8(a.rope + n * a.rot_dims + t, c);
        load8(a.rope + n * a.rot_dims + half + t, s);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        x[e] += b[e];
        raw[e] = x[e];
        local += x[e] * x[e];
    }
    if (norm) {
#pragma unroll
        for (int off = 1; off < LPH; off <<= 1) local += __shfl_xor(local, off, kWave);
        const float inv = 1.f / sqrtf(local / static_cast<float>(a.dim) + a.eps);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= inv * w[e];
    }
    if (a.rot_dims > 0) {
        const int from = lane + (d < half ? half / 8 : -half / 8);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float other = __shfl(x[e], from, kWave);
            if (rotated) x[e] = d < half ? x[e] * c[e] - other * s[e] : x[e] * c[e] + other * s[e];
        }
    }
    if (!on || d >= a.dimp) return;
    if (is_q) {
        store8(static_cast<T*>(a.q) + (n * a.heads + h) * a.dimp + d, x);
    } else if (slot >= 0) {
        T* k = static_cast<T*>(a.pool) + (static_cast<size_t>(slot) * a.kv_heads + h) * 2 * a.dimp + d;
        store8(k, x);
        store8(k + a.dimp, a.v_off < 0 ? raw : v);
    }
}

// One norm over a row's whole query projection and one over its whole key projection, values of their own
// size, either pairing of the rotated entries.  One block per row.
struct JointPrepArgs {
    const void* fused;
    const float *q_norm, *k_norm, *rope;
    const int64_t* slots;
    void *q, *pool;
    int q_off, k_off, v_off, rot_dims, adjacent, ld, heads, kv_heads, dim, vdim, dimp;
    float eps;
};
// Eight neighbouring values per thread and unit (pairs of neighbours rotate inside one): the first kCache units
// of a thread stay in registers between the sums and the stores.
template <class T>
__global__ __launch_bounds__(256) void group_prep_joint_vec_kernel(const JointPrepArgs a) {
    __shared__ float red[2][256 / kWave];
    constexpr int kCache = 4;
    const size_t n = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const T* row = static_cast<const T*>(a.fused) + n * a.ld;
    const int per = a.dimp / 8, nq = a.heads * per, nk = a.kv_heads * per, total = nq + 2 * nk;   // q | k | v
    const int64_t slot = a.slots[n];
    // where unit u's values are (null: padding), and its place
    auto source = [&](int u, int& h, int& d) -> const T* {
        const int part = u < nq ? 0 : u < nq + nk ? 1 : 2;
        const int w = u - (part == 0 ? 0 : part == 1 ? nq : nq + nk);
        h = w / per;
        d = 8 * (w - h * per);
        if (d >= (part == 2 ? a.vdim : a.dim)) return nullptr;
        if (part == 0) return row + a.q_off + h * a.dim + d;
        if (part == 1 || a.v_off < 0) return row + a.k_off + h * a.dim + d;   // (values that are the keys as projected)
        return row + a.v_off + h * a.vdim + d;
    };
    float x[kCache][8], sq = 0.f, sk = 0.f;
    auto add_up = [&](int u, const float* f) {
        float s = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) s += f[e] * f[e];
        if (u < nq) sq += s;
        else if (u < nq + nk) sk += s;
    };
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int u = tid + 256 * c;
        int h, d;
        const T* p = u < total ? source(u, h, d) : nullptr;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[c][e] = 0.f;
        if (p) load8(p, x[c]);
    }
    float inv_q = 1.f, inv_k = 1.f;
    if (a.q_norm || a.k_norm) {
#pragma unroll
        for (int c = 0; c < kCache; ++c)
            if (tid + 256 * c < nq + nk) add_up(tid + 256 * c, x[c]);
        for (int u = tid + 256 * kCache; u < nq + nk; u += 256) {
            int h, d;
            float f[8];
            if (const T* p = source(u, h, d)) {
                load8(p, f);
                add_up(u, f);
            }
        }
        sq = wave_sum(sq);
        sk = wave_sum(sk);
        if (lane == 0) {
            red[0][wv] = sq;
            red[1][wv] = sk;
        }
        __syncthreads();
        sq = sk = 0.f;
#pragma unroll
        for (int w = 0; w < 256 / kWave; ++w) {
            sq += red[0][w];
            sk += red[1][w];
        }
        if (a.q_norm) inv_q = 1.f / sqrtf(sq / static_cast<float>(a.heads * a.dim) + a.eps);
        if (a.k_norm) inv_k = 1.f / sqrtf(sk / static_cast<float>(a.kv_heads * a.dim) + a.eps);
    }
    const float* tab = a.rope + n * a.rot_dims;
    const int half = a.rot_dims / 2;
    auto finish = [&](int u, float* f) {
        int h, d;
        const bool in = source(u, h, d) != nullptr;
        if (u < nq + nk && in) {
            const float* norm = u < nq ? a.q_norm : a.k_norm;
            const float inv = u < nq ? inv_q : inv_k;
            if (norm) {
                float w[8];
                load8(norm + h * a.dim + d, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) f[e] *= inv * w[e];
            }
#pragma unroll
            for (int e = 0; e < 8; e += 2)
                if (d + e < a.rot_dims) {
                    const float c = tab[(d + e) >> 1], s = tab[half + ((d + e) >> 1)], u0 = f[e], u1 = f[e + 1];
                    f[e] = u0 * c - u1 * s;
                    f[e + 1] = u1 * c + u0 * s;
                }
        }
        if (u < nq) {
            store8(static_cast<T*>(a.q) + (n * a.heads + h) * a.dimp + d, f);
        } else if (slot >= 0) {
            T* k = static_cast<T*>(a.pool) + (static_cast<size_t>(slot) * a.kv_heads + h) * 2 * a.dimp + d;
            store8(u < nq + nk ? k : k + a.dimp, f);
        }
    };
#pragma unroll
    for (int c = 0; c < kCache; ++c)
        if (tid + 256 * c < total) finish(tid + 256 * c, x[c]);
    for (int u = tid + 256 * kCache; u < total; u += 256) {
        int h, d;
        float f[8] = {};
        if (const T* p = source(u, h, d)) load8(p, f);
        finish(u, f);
    }
}
// Any size and pairing, a value per thread.
template <class T>
__global__ __launch_bounds__(256) void group_prep_joint_kernel(const JointPrepArgs a) {
    __shared__ float red[256 / kWave];
    const size_t n = blockIdx.x;
    const T *row = static_cast<const T*>(a.fused) + n * a.ld, *q = row + a.q_off, *k = row + a.k_off;
    const int Q = a.heads * a.dim, K = a.kv_heads * a.dim;
    auto inverse = [&](const T* p, int len) {
        float s = 0.f;
        for (int i = threadIdx.x; i < len; i += 256) {
            const float v = act_get<T>(p[i]);
            s += v * v;
        }
        return 1.f / sqrtf(block_total(s, red) / static_cast<float>(len) + a.eps);
    };
    const float inv_q = a.q_norm ? inverse(q, Q) : 1.f, inv_k = a.k_norm ? inverse(k, K) : 1.f;
    const int64_t slot = a.slots[n];
    const float* tab = a.rope + n * a.rot_dims;
    const int half = a.rot_dims / 2;
    auto rotated = [&](const T* p, const float* norm, float inv, int h, int d) {
        auto value = [&](int i) { return act_get<T>(p[h * a.dim + i]) * (norm ? inv * norm[h * a.dim + i] : 1.f); };
        if (d >= a.rot_dims) return value(d);
        const bool first = a.adjacent ? (d & 1) == 0 : d < half;
        const int t = a.adjacent ? d >> 1 : first ? d : d - half, other = a.adjacent ? d ^ 1 : first ? d + half : d - half;
        return first ? value(d) * tab[t] - value(other) * tab[half + t] : value(d) * tab[t] + value(other) * tab[half + t];
    };
    for (int i = threadIdx.x; i < a.heads * a.dimp; i += 256) {
        const int h = i / a.dimp, d = i % a.dimp;
        static_cast<T*>(a.q)[n * a.heads * a.dimp + i] = act_put<T>(d < a.dim ? rotated(q, a.q_norm, inv_q, h, d) : 0.f);
    }
    if (slot < 0) return;
    T* pool = static_cast<T*>(a.pool) + static_cast<size_t>(slot) * a.kv_heads * 2 * a.dimp;
    for (int i = threadIdx.x; i < a.kv_heads * a.dimp; i += 256) {
        const int h = i / a.dimp, d = i % a.dimp;
        const T zero = act_put<T>(0.f);
        pool[h * 2 * a.dimp + d] = d < a.dim ? act_put<T>(rotated(k, a.k_norm, inv_k, h, d)) : zero;
        pool[(h * 2 + 1) * a.dimp + d] = d >= a.vdim ? zero : a.v_off < 0 ? k[h * a.dim + d] : row[a.v_off + h * a.vdim + d];
    }
}

// ---- any size, any compute type --------------------------------------------------------------------
struct PlainArgs {
    const void *q, *pool;
    void* o;
    const uint32_t *pages, *row_begin;
    const int32_t* row_len;
    int heads, kv_heads, dimp, ld_o, ps, window;
    float scale, sink, out_scale;
    const void* gate;   // null: none
    int ld_gate;
};
// One block per (row, head): 64 keys at a time, a wave per key for the scores, a thread per column for the
// sums.
template <class T>
__global__ __launch_bounds__(256) void group_attn_plain_kernel(const PlainArgs a) {
    __shared__ float sq[1024], sp[64], s_stat[2];
    __shared__ size_t s_row[64];
    const size_t n = blockIdx.x;
    const int h = blockIdx.y, tid = threadIdx.x, lane = tid & (kWave - 1), wv = tid / kWave;
    const int kvh = h / (a.heads / a.kv_heads), D = a.dimp;
    const int len = a.row_len[n], begin = a.window > 0 ? max(0, len - a.window) : 0;
    const uint32_t* pages = a.pages + a.row_begin[n];
    const T *q = static_cast<const T*>(a.q) + (n * a.heads + h) * D, *pool = static_cast<const T*>(a.pool);
    for (int d = tid; d < D; d += 256) sq[d] = act_get<T>(q[d]);
    float mx = -INFINITY, sum = 0.f, acc[4] = {0.f, 0.f, 0.f, 0.f};   // (columns tid + 256 c)
    for (int j0 = begin; j0 < len; j0 += 64) {
        const int cnt = min(64, len - j0);
        __syncthreads();
        if (tid < cnt)
            s_row[tid] = ((static_cast<size_t>(pages[(j0 + tid) / a.ps]) * a.ps + (j0 + tid) % a.ps) * a.kv_heads + kvh) * 2 * D;
        __syncthreads();
        for (int j = wv; j < cnt; j += 4) {
            const T* k = pool + s_row[j];
            float dot = 0.f;
            for (int d = lane; d < D; d += kWave) dot = fmaf(sq[d], act_get<T>(k[d]), dot);
            dot = wave_sum(dot);
            if (lane == 0) sp[j] = dot * a.scale;
        }
        __syncthreads();
        if (wv == 0) {
            const float s = lane < cnt ? sp[lane] : -INFINITY;
            const float m_new = fmaxf(mx, wave_max(s));
            const float p = lane < cnt ? expf(s - m_new) : 0.f, alpha = expf(mx - m_new);
            sum = sum * alpha + wave_sum(p);
            mx = m_new;
            sp[lane] = p;
            if (lane == 0) {
                s_stat[0] = alpha;
                s_stat[1] = m_new;
            }
        }
        __syncthreads();
        const float alpha = s_stat[0];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int d = tid + 256 * c;
            if (d >= D) break;
            float v = acc[c] * alpha;
            for (int j = 0; j < cnt; ++j) v = fmaf(sp[j], act_get<T>(pool[s_row[j] + D + d]), v);
            acc[c] = v;
        }
    }
    if (tid == 0) {   // exp(s) / (sink + sum): relative to the larger of the maximum and 0
        float f = 0.f;
        if (len > begin) {
            const float top = a.sink > 0.f ? fmaxf(mx, 0.f) : mx;
            f = expf(mx - top) / (sum * expf(mx - top) + a.sink * expf(-top));
        }
        s_stat[0] = f * a.out_scale;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < 4; ++c) {
        const int d = tid + 256 * c;
        if (d >= D) break;
        const float f = a.gate ? s_stat[0] / (1.f + expf(-act_get<T>(static_cast<const T*>(a.gate)[n * a.ld_gate + h * D + d]))) : s_stat[0];
        static_cast<T*>(a.o)[n * a.ld_o + h * D + d] = act_put<T>(acc[c] * f);
    }
}

// ---- the matrix-core forms ---------------------------------------------------------------------------
struct AttnArgs {
    const uint16_t *q, *pool;
    uint16_t* o;               // null: partial results
    float *part_o, *part_ml;   // [row of the launch, head, nsplit, dimp], [.., 2] (max in units of log 2, sum)
    const uint32_t *pages, *row_begin;
    const int32_t *row_len, *list;   // rows of the rows form (null: 0, 1, ..); (first row, rows) of the tiles form
    int heads, kv_heads, ratio, heads_per_tile, head_groups, ld_o, ps, ps_shift, window, nsplit;
    float scale_log2e, sink, out_scale;
    const uint16_t* gate;      // logistic gates of the outputs, null: none
    int ld_gate;
};
// Four neighbouring outputs, times the logistic function of their gates.
__device__ __forceinline__ void store_gated(uint16_t* o, f32x4_t v, const uint16_t* gate) {
    if (gate) {
        const u32x2_t r = *reinterpret_cast<const u32x2_t*>(gate);
        v *= f32x4_t{sigmoid_f32(bf16_lo(r.x)), sigmoid_f32(bf16_hi(r.x)), sigmoid_f32(bf16_lo(r.y)), sigmoid_f32(bf16_hi(r.y))};
    }
    *reinterpret_cast<u32x2_t*>(o) = u32x2_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
}
__device__ __forceinline__ void split_weights(const float* s, float off, float c, float& sum, bf16x8_t& hi_out, bf16x8_t& lo_out) {
    uint32_t hi[4], lo[4];
#pragma unroll
    for (int e = 0; e < 8; e += 2) {
        const float p0 = __builtin_amdgcn_exp2f(fmaf(s[e], c, off)), p1 = __builtin_amdgcn_exp2f(fmaf(s[e + 1], c, off));
        sum += p0 + p1;
        const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
        hi[e >> 1] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
        lo[e >> 1] = pack_bf16x2(p0 - __uint_as_float(u0 & 0xFFFF0000u), p1 - __uint_as_float(u1 & 0xFFFF0000u));
    }
    hi_out = __builtin_bit_cast(bf16x8_t, u32x4_t{hi[0], hi[1], hi[2], hi[3]});
    lo_out = __builtin_bit_cast(bf16x8_t, u32x4_t{lo[0], lo[1], lo[2], lo[3]});
}
__device__ __forceinline__ bf16x8_t transposed_values(const uint16_t* tile, int stride, int d0, int l16, int g) {
    const uint16_t* va = tile + (4 * g + (l16 >> 2)) * stride + d0 + 4 * (l16 & 3);
    const bf16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va));
    const bf16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va + 16 * stride));
    return __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
}
// 1 / (sum + sink) for a running maximum mx in units of log 2: sums are relative to 2^mx
__device__ __forceinline__ float normaliser(float sum, float mx, float sink) {
    if (mx == -INFINITY) return 0.f;
    return sink > 0.f && mx < -126.f ? 0.f : 1.f / (sum + (sink > 0.f ? sink * exp2f(-mx) : 0.f));
}

// Rows form: a block takes up to 16 query heads of one key head of one row, its waves take the 32-key
// steps of the block's share of the keys in turn, each with a softmax state of its own; they meet in LDS
// at the end.  Keys go from memory to the score's operand registers as they are (lane = key, 16-byte
// pieces), values through a tile in LDS that only their wave touches.
template <int KS>
__global__ __launch_bounds__(kBlock, 2) void group_rows_kernel(const AttnArgs a) {
    constexpr int D = 32 * KS, DT = 2 * KS, VSTRIDE = D + 16, PPR = D / 8, NP = kStep * PPR / kWave;
    constexpr int kTileBytes = kWaves * kStep * VSTRIDE * 2, kMergeBytes = kWaves * 16 * D * 4;
    __shared__ __attribute__((aligned(16))) unsigned char mem[kTileBytes > kMergeBytes ? kTileBytes : kMergeBytes];
    __shared__ float s_m[kWaves][16], s_l[kWaves][16];
    const int tid = threadIdx.x, lane = tid & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    uint16_t* tile = reinterpret_cast<uint16_t*>(mem) + wv * kStep * VSTRIDE;
    const int per_row = a.kv_heads * a.head_groups;
    const int idx = blockIdx.x / per_row, sub = blockIdx.x % per_row;
    const int n = a.list ? a.list[idx] : idx;
    const int kvh = sub / a.head_groups, h0 = kvh * a.ratio + (sub % a.head_groups) * 16;
    const int nh = min(16, (kvh + 1) * a.ratio - h0);
    const int len = a.row_len[n], begin = a.window > 0 ? max(0, len - a.window) : 0;
    const int steps = (len - begin + kStep - 1) / kStep, per = max(1, (steps + a.nsplit - 1) / a.nsplit);
    const int s_lo = blockIdx.y * per, s_hi = min(steps, s_lo + per);
    if (s_lo >= steps && blockIdx.y > 0) return;
    const uint32_t* pages = a.pages + a.row_begin[n];
    bf16x8_t qf[KS];
    {
        const uint16_t* qp = a.q + (static_cast<size_t>(n) * a.heads + h0 + min(l16, nh - 1)) * D + 8 * g;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) qf[ks] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(qp + 32 * ks));
    }
    // Places of this lane's rows of a step: two keys and a value row.  Their pages are asked for one step of
    // this wave ahead of the rows, so that the two requests do not stand in line.
    uint32_t pid[3];
    int in_page[3];
    auto fetch_pages = [&](int step) {
        const int j0 = begin + step * kStep;
#pragma unroll
        for (int i = 0; i < 3; ++i) {   // (keys past the end repeat the last: their weights are zero)
            const int j = min(j0 + (i < 2 ? 16 * i + l16 : lane >> 1), len - 1);
            const int page = a.ps_shift >= 0 ? j >> a.ps_shift : j / a.ps;
            pid[i] = pages[page];
            in_page[i] = j - page * a.ps;
        }
    };
    u32x4_t kr[2][KS], vr[NP];
    auto issue = [&](int step) {
        const uint16_t* row[3];
#pragma unroll
        for (int i = 0; i < 3; ++i) row[i] = a.pool + ((static_cast<size_t>(pid[i]) * a.ps + in_page[i]) * a.kv_heads + kvh) * 2 * D;
        fetch_pages(step + kWaves);
#pragma unroll
        for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) kr[nt][ks] = *reinterpret_cast<const u32x4_t*>(row[nt] + 8 * g + 32 * ks);
        // values: two lanes per key, NP pieces each
#pragma unroll
        for (int u = 0; u < NP; ++u) vr[u] = *reinterpret_cast<const u32x4_t*>(row[2] + D + (lane & 1) * 8 + 16 * u);
    };
    f32x4_t acc[DT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) acc[dt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    float mx = -INFINITY, lsum = 0.f;   // (raw score units)
    if (s_lo + wv < s_hi) {
        fetch_pages(s_lo + wv);
        issue(s_lo + wv);
    }
    for (int st = s_lo + wv; st < s_hi; st += kWaves) {
        const int j0 = begin + st * kStep;
        f32x4_t sc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int nt = 0; nt < 2; ++nt)
                sc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kr[nt][ks]), qf[ks], sc[nt], 0, 0, 0);
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");   // (the tile's last reads come first)
#pragma unroll
        for (int u = 0; u < NP; ++u) *reinterpret_cast<u32x4_t*>(&tile[(lane >> 1) * VSTRIDE + (lane & 1) * 8 + 16 * u]) = vr[u];
        if (st + kWaves < s_hi) issue(st + kWaves);
        float s[8], m_new = mx;
#pragma unroll
        for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float v = j0 + 16 * nt + 4 * g + e < len ? sc[nt][e] : -INFINITY;
                s[4 * nt + e] = v;
                m_new = fmaxf(m_new, v);
            }
        m_new = rows_max(m_new);
        const float off = -m_new * a.scale_log2e;   // (every step holds a key: finite)
        const float alpha = __builtin_amdgcn_exp2f(fmaf(mx, a.scale_log2e, off));
        mx = m_new;
        float sum = 0.f;
        bf16x8_t hi, lo;
        split_weights(s, off, a.scale_log2e, sum, hi, lo);
        lsum = lsum * alpha + sum;
        if (__any(alpha != 1.f))
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) acc[dt] *= alpha;
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");   // (the wave's LDS operations are in order)
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            const bf16x8_t vf = transposed_values(tile, VSTRIDE, 16 * dt, l16, g);
            acc[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, hi, acc[dt], 0, 0, 0);
            acc[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, lo, acc[dt], 0, 0, 0);
        }
    }
    lsum += __shfl_xor(lsum, 16, kWave);
    lsum += __shfl_xor(lsum, 32, kWave);
    if (g == 0) {
        s_m[wv][l16] = mx * a.scale_log2e;
        s_l[wv][l16] = lsum;
    }
    __syncthreads();   // (the tiles have been read: their memory takes the sums)
    float* sums = reinterpret_cast<float*>(mem);
    float top = -INFINITY;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) top = fmaxf(top, s_m[w][l16]);
    const float f = top == -INFINITY ? 0.f : exp2f(mx * a.scale_log2e - top);
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) *reinterpret_cast<f32x4_t*>(&sums[(wv * 16 + l16) * D + 16 * dt + 4 * g]) = acc[dt] * f;
    __syncthreads();
    // thread -> (head hd, columns)
    constexpr int TPH = kBlock / 16;
    const int hd = tid / TPH;
    if (hd >= nh) return;
    float t2 = -INFINITY, l = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) t2 = fmaxf(t2, s_m[w][hd]);
#pragma unroll
    for (int w = 0; w < kWaves; ++w) l += t2 == -INFINITY ? 0.f : s_l[w][hd] * exp2f(s_m[w][hd] - t2);
    const size_t out = static_cast<size_t>(idx) * a.heads + h0 + hd;
    const float inv = a.out_scale * normaliser(l, t2, a.sink);
    for (int d = (tid % TPH) * 4; d < D; d += TPH * 4) {
        f32x4_t v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < kWaves; ++w) v += *reinterpret_cast<const f32x4_t*>(&sums[(w * 16 + hd) * D + d]);
        if (a.o)
            store_gated(a.o + static_cast<size_t>(n) * a.ld_o + (h0 + hd) * D + d, v * inv,
                        a.gate ? a.gate + static_cast<size_t>(n) * a.ld_gate + (h0 + hd) * D + d : nullptr);
        else
            *reinterpret_cast<f32x4_t*>(a.part_o + (out * a.nsplit + blockIdx.y) * D + d) = v;
    }
    if (!a.o && tid % TPH == 0) {
        a.part_ml[(out * a.nsplit + blockIdx.y) * 2] = t2;
        a.part_ml[(out * a.nsplit + blockIdx.y) * 2 + 1] = l;
    }
}

// One block per (row, head), four columns per thread.
__global__ void group_merge_kernel(const AttnArgs a, uint16_t* __restrict__ o, int D) {
    const int idx = blockIdx.x / a.heads, h = blockIdx.x % a.heads;
    const int n = a.list ? a.list[idx] : idx;
    const size_t out = static_cast<size_t>(idx) * a.heads + h;
    const int len = a.row_len[n], begin = a.window > 0 ? max(0, len - a.window) : 0;
    const int steps = (len - begin + kStep - 1) / kStep, per = max(1, (steps + a.nsplit - 1) / a.nsplit);
    const int ns = min(a.nsplit, (steps + per - 1) / per);
    const float* ml = a.part_ml + out * a.nsplit * 2;
    float mx = -INFINITY, l = 0.f;
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    const float* po = a.part_o + out * a.nsplit * D + 4 * threadIdx.x;
    constexpr int kAhead = 8;   // splits requested together (those behind the last read it again and weigh nothing)
    for (int s0 = 0; s0 < ns; s0 += kAhead) {
        float m[kAhead];
#pragma unroll
        for (int u = 0; u < kAhead; ++u) m[u] = ml[2 * min(s0 + u, ns - 1)];
#pragma unroll
        for (int u = 0; u < kAhead; ++u) mx = fmaxf(mx, m[u]);
    }
    for (int s0 = 0; s0 < ns; s0 += kAhead) {
        f32x4_t p[kAhead];
        float w[kAhead], sum[kAhead];
#pragma unroll
        for (int u = 0; u < kAhead; ++u) {
            const int s = min(s0 + u, ns - 1);
            p[u] = *reinterpret_cast<const f32x4_t*>(po + static_cast<size_t>(s) * D);
            w[u] = ml[2 * s];
            sum[u] = ml[2 * s + 1];
        }
#pragma unroll
        for (int u = 0; u < kAhead; ++u) {
            const float e = mx == -INFINITY || s0 + u >= ns ? 0.f : exp2f(w[u] - mx);
            l = fmaf(sum[u], e, l);
            v += p[u] * e;
        }
    }
    const float inv = a.out_scale * normaliser(l, mx, a.sink);
    store_gated(o + static_cast<size_t>(n) * a.ld_o + h * D + 4 * threadIdx.x, v * inv,
                a.gate ? a.gate + static_cast<size_t>(n) * a.ld_gate + h * D + 4 * threadIdx.x : nullptr);
}

// Tiles form: a block takes 64 QT (token, head) pairs of one key head — pair m is token m / heads_per_tile,
// head m % heads_per_tile of the tile — a wave 16 QT of them.  Keys advance 32 at a time through
// double-buffered LDS tiles, one barrier per step, two steps requested ahead in registers; the block
// starts at its first token's window, a wave skips the steps outside all of its windows.
template <int KS, int QT>
__global__ __launch_bounds__(kBlock, KS > 4 ? 1 : 2) void group_tiles_kernel(const AttnArgs a) {
    constexpr int D = 32 * KS, DT = 2 * KS, KSTRIDE = D + 8, VSTRIDE = D + 16;
    constexpr int NP = D / 4 / 8;   // 16-byte pieces of a (key | value) row per thread, eight threads a row
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    uint16_t* k_tile[2] = {lds, lds + kStep * KSTRIDE};
    uint16_t* v_tile[2] = {lds + 2 * kStep * KSTRIDE, lds + 2 * kStep * KSTRIDE + kStep * VSTRIDE};
    const int per_tile = a.kv_heads * a.head_groups;
    const int ti = blockIdx.x / per_tile, sub = blockIdx.x % per_tile;
    const int n0 = a.list[2 * ti], rows = a.list[2 * ti + 1];
    const int kvh = sub / a.head_groups, h0 = kvh * a.ratio + (sub % a.head_groups) * a.heads_per_tile;
    const int nh = min(a.heads_per_tile, (kvh + 1) * a.ratio - h0);
    const int tid = threadIdx.x, lane = tid & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const uint32_t* pages = a.pages + a.row_begin[n0];
    const int kmax = a.row_len[n0 + rows - 1];   // (rows of a request are consecutive positions)
    const int first = a.window > 0 ? max(0, a.row_len[n0] - a.window) : 0;

    int my_len[QT], my_lo[QT], my_row[QT], my_head[QT];
    bf16x8_t qf[QT][KS];
    int lo_all = kmax, len_lo = kmax, len_hi = 0, lo_hi = 0;
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int m = wv * 16 * QT + t * 16 + l16, tok = m / a.heads_per_tile, hd = m % a.heads_per_tile;
        const bool valid = tok < rows && hd < nh;
        my_row[t] = n0 + (valid ? tok : 0);
        my_head[t] = valid ? h0 + hd : -1;
        my_len[t] = valid ? a.row_len[my_row[t]] : 0;
        my_lo[t] = a.window > 0 ? max(0, my_len[t] - a.window) : 0;
        if (valid) {
            lo_all = min(lo_all, my_lo[t]);
            lo_hi = max(lo_hi, my_lo[t]);
            len_hi = max(len_hi, my_len[t]);
        }
        len_lo = min(len_lo, my_len[t]);
        const uint16_t* qp = a.q + (static_cast<size_t>(my_row[t]) * a.heads + (valid ? my_head[t] : h0)) * D + 8 * g;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) qf[t][ks] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(qp + 32 * ks));
    }
#pragma unroll
    for (int sh = 1; sh < 16; sh <<= 1) {   // (the four lane groups hold the same pairs)
        lo_all = min(lo_all, __shfl_xor(lo_all, sh, kWave));
        lo_hi = max(lo_hi, __shfl_xor(lo_hi, sh, kWave));
        len_lo = min(len_lo, __shfl_xor(len_lo, sh, kWave));
        len_hi = max(len_hi, __shfl_xor(len_hi, sh, kWave));
    }
    const int w_lo = __builtin_amdgcn_readfirstlane(lo_all), w_hi = __builtin_amdgcn_readfirstlane(len_hi);
    const int w_all_lo = __builtin_amdgcn_readfirstlane(lo_hi), w_all_hi = __builtin_amdgcn_readfirstlane(len_lo);

    const int key = tid >> 3, piece0 = tid & 7;
    u32x4_t reg[2][NP];
    auto issue = [&](int slot, int j0) {
        const int j = min(j0 + key, kmax - 1);   // (keys past the extent repeat the last: their weights are zero)
        const int page = a.ps_shift >= 0 ? j >> a.ps_shift : j / a.ps;
        const uint16_t* p = a.pool + ((static_cast<size_t>(pages[page]) * a.ps + (j - page * a.ps)) * a.kv_heads + kvh) * 2 * D + piece0 * 8;
#pragma unroll
        for (int u = 0; u < NP; ++u) reg[slot][u] = *reinterpret_cast<const u32x4_t*>(p + 64 * u);
    };
    auto stage = [&](int slot) {
#pragma unroll
        for (int u = 0; u < NP; ++u) {
            const int e = (piece0 + 8 * u) * 8;
            uint16_t* dst = e < D ? &k_tile[slot][key * KSTRIDE + e] : &v_tile[slot][key * VSTRIDE + e - D];
            *reinterpret_cast<u32x4_t*>(dst) = reg[slot][u];
        }
    };
    f32x4_t acc[QT][DT];
    float mx[QT], lsum[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        mx[t] = -INFINITY;
        lsum[t] = 0.f;
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) acc[t][dt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    auto compute = [&](int slot, int j0) {
        const uint16_t* kt = k_tile[slot];
        f32x4_t st[QT][2];
#pragma unroll
        for (int t = 0; t < QT; ++t)
#pragma unroll
            for (int nt = 0; nt < 2; ++nt) st[t][nt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int nt = 0; nt < 2; ++nt) {
                const bf16x8_t kf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&kt[(16 * nt + l16) * KSTRIDE + 32 * ks + 8 * g]));
#pragma unroll
                for (int t = 0; t < QT; ++t) st[t][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[t][ks], st[t][nt], 0, 0, 0);
            }
        bf16x8_t p_hi[QT], p_lo[QT];
        auto softmax = [&](auto masked_tag) {
            constexpr bool kMask = decltype(masked_tag)::value;
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                float s[8], m_new = mx[t];
#pragma unroll
                for (int nt = 0; nt < 2; ++nt)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        float v = st[t][nt][e];
                        const int j = j0 + 16 * nt + 4 * g + e;
                        if constexpr (kMask) v = j < my_len[t] && j >= my_lo[t] ? v : -INFINITY;
                        s[4 * nt + e] = v;
                        m_new = fmaxf(m_new, v);
                    }
                m_new = rows_max(m_new);
                const float safe = m_new == -INFINITY ? 0.f : m_new, off = -safe * a.scale_log2e;
                const float alpha = __builtin_amdgcn_exp2f(fmaf(mx[t], a.scale_log2e, off));
                mx[t] = m_new;
                float sum = 0.f;
                split_weights(s, off, a.scale_log2e, sum, p_hi[t], p_lo[t]);
                lsum[t] = lsum[t] * alpha + sum;
                if (__any(alpha != 1.f))
#pragma unroll
                    for (int dt = 0; dt < DT; ++dt) acc[t][dt] *= alpha;
            }
        };
        if (j0 >= w_all_lo && j0 + kStep <= w_all_hi) softmax(std::false_type{});
        else softmax(std::true_type{});
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            const bf16x8_t vf = transposed_values(v_tile[slot], VSTRIDE, 16 * dt, l16, g);
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_hi[t], acc[t][dt], 0, 0, 0);
                acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_lo[t], acc[t][dt], 0, 0, 0);
            }
        }
    };
    auto step = [&](int slot, int j0) {
        if (j0 + kStep < kmax) stage(slot ^ 1);
        if (j0 + 3 * kStep < kmax) issue(slot ^ 1, j0 + 3 * kStep);
        if (j0 < w_hi && j0 + kStep > w_lo) compute(slot, j0);
        __syncthreads();
    };
    if (first < kmax) issue(0, first);
    if (first + kStep < kmax) issue(1, first + kStep);
    if (first < kmax) stage(0);
    if (first + 2 * kStep < kmax) issue(0, first + 2 * kStep);
    __syncthreads();
    for (int j0 = first; j0 < kmax; j0 += 2 * kStep) {
        step(0, j0);
        if (j0 + kStep < kmax) step(1, j0 + kStep);
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        float l = lsum[t];
        l += __shfl_xor(l, 16, kWave);
        l += __shfl_xor(l, 32, kWave);
        if (my_head[t] < 0) continue;
        const float inv = a.out_scale * normaliser(l, mx[t] * a.scale_log2e, a.sink);
        uint16_t* op = a.o + static_cast<size_t>(my_row[t]) * a.ld_o + my_head[t] * D + 4 * g;
#pragma unroll
        for (int dt = 0; dt < DT; ++dt)
            store_gated(op + 16 * dt, acc[t][dt] * inv,
                        a.gate ? a.gate + static_cast<size_t>(my_row[t]) * a.ld_gate + my_head[t] * D + 4 * g + 16 * dt : nullptr);
    }
}

template <int KS, int QT>
int launch_group_tiles(const AttnArgs& a, int num_tiles, hipStream_t s) {
    constexpr size_t smem = 2 * kStep * (2 * 32 * KS + 24) * sizeof(uint16_t);
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&group_tiles_kernel<KS, QT>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(smem));
    if (attr != hipSuccess) return PIE_HIP_ERR_LAUNCH;
    hipLaunchKernelGGL((group_tiles_kernel<KS, QT>), dim3(num_tiles * a.kv_heads * a.head_groups), dim3(kBlock), smem, s, a);
    return launch_status();
}

// Splits of the rows form: about two blocks per CU over the batch, at least four steps (one per wave) each.
int rows_splits(int num_rows, int heads, int kv_heads, int max_kv_len, int window) {
    const int ratio = heads / kv_heads, keys = window > 0 && window < max_kv_len ? window : max_kv_len;
    const long long blocks = static_cast<long long>(num_rows) * kv_heads * ((ratio + 15) / 16);
    const int steps = (keys + kStep - 1) / kStep;
    long long ns = 512 / blocks;
    if (ns > steps / kWaves) ns = steps / kWaves;
    return ns < 1 ? 1 : static_cast<int>(ns);
}
int shift_of(int ps) { return (ps & (ps - 1)) == 0 ? __builtin_ctz(static_cast<unsigned>(ps)) : -1; }
// gates: none, or rows of all heads; eight-byte pieces where four outputs are stored together
bool gate_ok(const void* gate, int ld_gate, int heads, int dimp, bool pieces) {
    return !gate || (ld_gate >= heads * dimp && (!pieces || (ld_gate % 4 == 0 && reinterpret_cast<uintptr_t>(gate) % 8 == 0)));
}
bool sizes_ok(int heads, int kv_heads, int dimp, int ld_o, int ps, int window, float sink) {
    return heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dimp > 0 && ld_o >= heads * dimp && ps > 0 && window >= 0 && sink >= 0.f;
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_group_attn_prep(int dtype, const void* fused, int q_off, int k_off, int v_off, const float* q_bias,
                                       const float* k_bias, const float* q_norm, const float* k_norm,
                                       const float* rope_table, int rot_dims, const int64_t* kv_slots, void* q_out, void* pool,
                                       int num_tokens, int ld_fused, int heads, int kv_heads, int dim, int dimp, float eps,
                                       void* stream) {
    if (!fused || !kv_slots || !q_out || !pool || num_tokens <= 0 || heads <= 0 || kv_heads <= 0 || dim <= 0 || dimp < dim || q_off < 0 ||
        k_off < 0 || q_off + heads * dim > ld_fused || k_off + kv_heads * dim > ld_fused || v_off + kv_heads * dim > ld_fused ||
        rot_dims < 0 || rot_dims % 2 != 0 || rot_dims > dim || (rot_dims > 0 && !rope_table))
        return PIE_HIP_ERR_INVALID;
    if (dimp > kPrepPerLane * kWave) return PIE_HIP_ERR_UNSUPPORTED;
    const PrepArgs a{fused, q_bias, k_bias, q_norm, k_norm, rope_table, kv_slots, q_out, pool, q_off, k_off, v_off, rot_dims,
                     num_tokens, ld_fused, heads, kv_heads, dim, dimp, eps};
    const long long units = static_cast<long long>(num_tokens) * (heads + kv_heads);
    const dim3 grid(static_cast<unsigned>((units + 3) / 4));
    hipStream_t s = static_cast<hipStream_t>(stream);
    auto whole = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
    if (dim % 8 == 0 && dimp % 8 == 0 && rot_dims % 16 == 0 && q_off % 8 == 0 && k_off % 8 == 0 && (v_off < 0 || v_off % 8 == 0) &&
        ld_fused % 8 == 0 && dimp <= 512 && whole(fused) && whole(q_out) && whole(pool) && whole(rope_table) && whole(q_bias) &&
        whole(k_bias) && whole(q_norm) && whole(k_norm)) {
        const int pieces = dimp / 8, lph = pieces <= 4 ? 4 : pieces <= 8 ? 8 : pieces <= 16 ? 16 : pieces <= 32 ? 32 : 64;
        const dim3 vgrid(static_cast<unsigned>((units + 256 / lph - 1) / (256 / lph)));
        PIE_ACT_DISPATCH(dtype, T, switch (lph) {
            case 4: hipLaunchKernelGGL((group_prep_vec_kernel<T, 4>), vgrid, dim3(256), 0, s, a); break;
            case 8: hipLaunchKernelGGL((group_prep_vec_kernel<T, 8>), vgrid, dim3(256), 0, s, a); break;
            case 16: hipLaunchKernelGGL((group_prep_vec_kernel<T, 16>), vgrid, dim3(256), 0, s, a); break;
            case 32: hipLaunchKernelGGL((group_prep_vec_kernel<T, 32>), vgrid, dim3(256), 0, s, a); break;
            default: hipLaunchKernelGGL((group_prep_vec_kernel<T, 64>), vgrid, dim3(256), 0, s, a); break;
        });
        return launch_status();
    }
    PIE_ACT_DISPATCH(dtype, T, {
        if (dimp <= 64) hipLaunchKernelGGL((group_prep_kernel<T, 1>), grid, dim3(256), 0, s, a);
        else if (dimp <= 128) hipLaunchKernelGGL((group_prep_kernel<T, 2>), grid, dim3(256), 0, s, a);
        else if (dimp <= 256) hipLaunchKernelGGL((group_prep_kernel<T, 4>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((group_prep_kernel<T, 16>), grid, dim3(256), 0, s, a);
    });
    return launch_status();
}

extern "C" int pie_hip_group_attn_prep_joint(int dtype, const void* fused, int q_off, int k_off, int v_off, const float* q_norm,
                                             const float* k_norm, const float* rope_table, int rot_dims, int pairing,
                                             const int64_t* kv_slots, void* q_out, void* pool, int num_tokens,
                                             int ld_fused, int heads, int kv_heads, int dim, int vdim, int dimp,
                                             float eps, void* stream) {
    if (!fused || !kv_slots || !q_out || !pool || num_tokens <= 0 || heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || dimp < dim ||
        dimp < vdim || q_off < 0 || k_off < 0 || q_off + heads * dim > ld_fused || k_off + kv_heads * dim > ld_fused ||
        (v_off < 0 && vdim != dim) || v_off + kv_heads * vdim > ld_fused || rot_dims < 0 || rot_dims % 2 != 0 || rot_dims > dim ||
        (rot_dims > 0 && !rope_table) || (pairing != PIE_HIP_ROPE_HALF && pairing != PIE_HIP_ROPE_ADJACENT))
        return PIE_HIP_ERR_INVALID;
    const bool adjacent = pairing == PIE_HIP_ROPE_ADJACENT;
    const JointPrepArgs a{fused, q_norm, k_norm, rope_table, kv_slots, q_out, pool, q_off, k_off, v_off, rot_dims, adjacent ? 1 : 0,
                          ld_fused, heads, kv_heads, dim, vdim, dimp, eps};
    hipStream_t s = static_cast<hipStream_t>(stream);
    auto whole = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
    if (dim % 8 == 0 && vdim % 8 == 0 && dimp % 8 == 0 && (adjacent || rot_dims == 0) && q_off % 8 == 0 && k_off % 8 == 0 &&
        (v_off < 0 || v_off % 8 == 0) && ld_fused % 8 == 0 && whole(fused) && whole(q_out) && whole(pool) && whole(q_norm) && whole(k_norm))
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(group_prep_joint_vec_kernel<T>, dim3(num_tokens), dim3(256), 0, s, a));
    else
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(group_prep_joint_kernel<T>, dim3(num_tokens), dim3(256), 0, s, a));
    return launch_status();
}

extern "C" int pie_hip_group_attn_supported(int dimp) {
    return dimp == 32 || dimp == 64 || dimp == 96 || dimp == 128 || dimp == 192 || dimp == 256;
}

extern "C" size_t pie_hip_group_attn_rows_workspace_bytes(int num_rows, int heads, int kv_heads, int dimp, int max_kv_len, int window) {
    if (num_rows <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dimp <= 0) return 0;
    const int ns = rows_splits(num_rows, heads, kv_heads, max_kv_len, window);
    return ns > 1 ? static_cast<size_t>(num_rows) * heads * ns * (dimp + 2) * sizeof(float) : 0;
}

#define PIE_GROUP_CASES(X) X(1) X(2) X(3) X(4) X(6) X(8)

extern "C" int pie_hip_group_attn_rows(const uint16_t* q, const uint16_t* pool, uint16_t* o, const uint32_t* kv_page_indices,
                                       const uint32_t* row_page_begin, const int32_t* row_kv_len, const int32_t* rows,
                                       int num_rows, int heads, int kv_heads, int dimp, int ld_o, int page_size, float scale,
                                       int window, float sink, float out_scale, const uint16_t* gate, int ld_gate,
                                       int max_kv_len, void* workspace, size_t workspace_bytes, void* stream) {
    if (!q || !pool || !o || !kv_page_indices || !row_page_begin || !row_kv_len || num_rows <= 0 || max_kv_len <= 0 ||
        !sizes_ok(heads, kv_heads, dimp, ld_o, page_size, window, sink) || !gate_ok(gate, ld_gate, heads, dimp, true))
        return PIE_HIP_ERR_INVALID;
    if (!pie_hip_group_attn_supported(dimp) || ld_o % 4 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const int ratio = heads / kv_heads, ns = rows_splits(num_rows, heads, kv_heads, max_kv_len, window);
    AttnArgs a{q, pool, o, nullptr, nullptr, kv_page_indices, row_page_begin, row_kv_len, rows, heads, kv_heads, ratio, 16,
               (ratio + 15) / 16, ld_o, page_size, shift_of(page_size), window, ns, scale * kLog2e, sink, out_scale, gate, ld_gate};
    if (ns > 1) {
        if (!workspace || workspace_bytes < pie_hip_group_attn_rows_workspace_bytes(num_rows, heads, kv_heads, dimp, max_kv_len, window))
            return PIE_HIP_ERR_INVALID;
        a.o = nullptr;
        a.part_o = static_cast<float*>(workspace);
        a.part_ml = a.part_o + static_cast<size_t>(num_rows) * heads * ns * dimp;
    }
    const long long blocks = static_cast<long long>(num_rows) * kv_heads * a.head_groups;
    if (blocks > 0x7FFFFFFF) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const dim3 grid(static_cast<unsigned>(blocks), a.nsplit);
    switch (dimp / 32) {
#define PIE_GROUP_ROWS(KS) \
    case KS: hipLaunchKernelGGL(group_rows_kernel<KS>, grid, dim3(kBlock), 0, s, a); break;
        PIE_GROUP_CASES(PIE_GROUP_ROWS)
#undef PIE_GROUP_ROWS
        default: return PIE_HIP_ERR_UNSUPPORTED;
    }
    if (!a.o) hipLaunchKernelGGL(group_merge_kernel, dim3(num_rows * heads), dim3(dimp / 4), 0, s, a, o, dimp);
    return launch_status();
}

extern "C" int pie_hip_group_attn_tile_rows(int heads, int kv_heads, int half) {
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0) return 0;
    const int pairs = half ? 64 : 128, ratio = heads / kv_heads;
    return ratio >= 64 ? pairs / 64 : pairs / ratio;
}

extern "C" int pie_hip_group_attn_tiles(const uint16_t* q, const uint16_t* pool, uint16_t* o, const uint32_t* kv_page_indices,
                                        const uint32_t* row_page_begin, const int32_t* row_kv_len, const int32_t* tiles,
                                        int num_tiles, int half, int heads, int kv_heads, int dimp, int ld_o, int page_size,
                                        float scale, int window, float sink, float out_scale, const uint16_t* gate,
                                        int ld_gate, void* stream) {
    if (!q || !pool || !o || !kv_page_indices || !row_page_begin || !row_kv_len || !tiles || num_tiles <= 0 ||
        !sizes_ok(heads, kv_heads, dimp, ld_o, page_size, window, sink) || !gate_ok(gate, ld_gate, heads, dimp, true))
        return PIE_HIP_ERR_INVALID;
    if (!pie_hip_group_attn_supported(dimp) || ld_o % 4 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const int ratio = heads / kv_heads, hpt = ratio >= 64 ? 64 : ratio;
    const AttnArgs a{q, pool, o, nullptr, nullptr, kv_page_indices, row_page_begin, row_kv_len, tiles, heads, kv_heads, ratio, hpt,
                     (ratio + hpt - 1) / hpt, ld_o, page_size, shift_of(page_size), window, 1, scale * kLog2e, sink, out_scale,
                     gate, ld_gate};
    if (static_cast<long long>(num_tiles) * kv_heads * a.head_groups > 0x7FFFFFFF) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    switch (dimp / 32) {
#define PIE_GROUP_TILES(KS) \
    case KS: return half ? launch_group_tiles<KS, 1>(a, num_tiles, s) : launch_group_tiles<KS, 2>(a, num_tiles, s);
        PIE_GROUP_TILES(1) PIE_GROUP_TILES(2) PIE_GROUP_TILES(3) PIE_GROUP_TILES(4)
#undef PIE_GROUP_TILES
        // (wider heads: the accumulators of two tiles per wave do not fit the registers)
        case 6: return half ? launch_group_tiles<6, 1>(a, num_tiles, s) : PIE_HIP_ERR_UNSUPPORTED;
        case 8: return half ? launch_group_tiles<8, 1>(a, num_tiles, s) : PIE_HIP_ERR_UNSUPPORTED;
        default: return PIE_HIP_ERR_UNSUPPORTED;
    }
}

extern "C" int pie_hip_group_attn_plain(int dtype, const void* q, const void* pool, void* o, const uint32_t* kv_page_indices,
                                        const uint32_t* row_page_begin, const int32_t* row_kv_len, int num_rows, int heads,
                                        int kv_heads, int dimp, int ld_o, int page_size, float scale, int window, float sink,
                                        float out_scale, const void* gate, int ld_gate, void* stream) {
    if (!q || !pool || !o || !kv_page_indices || !row_page_begin || !row_kv_len || num_rows <= 0 ||
        !sizes_ok(heads, kv_heads, dimp, ld_o, page_size, window, sink) || !gate_ok(gate, ld_gate, heads, dimp, false))
        return PIE_HIP_ERR_INVALID;
    if (dimp > 1024 || heads > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const PlainArgs a{q, pool, o, kv_page_indices, row_page_begin, row_kv_len, heads, kv_heads, dimp, ld_o, page_size, window, scale, sink, out_scale, gate, ld_gate};
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(group_attn_plain_kernel<T>, dim3(num_rows, heads), dim3(256), 0,
                                                  static_cast<hipStream_t>(stream), a));
    return launch_status();
}
