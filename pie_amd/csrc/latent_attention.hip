// Attention over a cached low-rank latent: the kernels around the attention itself.
//
// A token's cache row is [kvp latent values | rotp rotated key values] in the compute type, kvp
// and rotp the latent rank and the rotated size rounded up (zeros between), shared by all heads.
// Two forms of the same function read it:
//   rows form      the key projection is moved to the query side, q~ = W_uk^T q: the scores are
//                  q~ . row and the weighted sum of the rows' latent parts goes through W_uv once
//                  per query (latent_attention_mfma.hip, any sizes here).  Reads each cached row once per (token, head group); decode and
//                  short portions.
//   expanded form  keys and values of all cached tokens are projected out of the latents first,
//                  then ordinary attention runs on them (latent_attention_prefill.hip); long
//                  portions, where it needs a third of the arithmetic.
#include "act_type.hip.h"

#include <type_traits>

namespace pie_hip {
namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

// Adjacent-pair rotation of entry i of a vector; tab = this token's cos | sin row.  Entries past
// `dims` pass unchanged.
template <class Get>
__device__ __forceinline__ float rotated_entry(int i, int dims, const float* tab, const Get& get) {
    if (i >= dims) return get(i);
    const float c = tab[i >> 1], s = tab[(dims >> 1) + (i >> 1)];
    return (i & 1) ? get(i) * c + get(i - 1) * s : get(i) * c - get(i + 1) * s;
}

// The fused down projection's row -> the normed query latent (compact, padded with zeros) and the
// token's cache row: normed latent, rotated key part (`kv_norm` null: only the query latent, the cache rows
// are another layer's).  One block per token.
template <class T>
__global__ __launch_bounds__(256) void latent_prep_kernel(
    const T* __restrict__ fused, const float* __restrict__ q_norm, const float* __restrict__ kv_norm,
    const float* __restrict__ rope_table, const int64_t* __restrict__ kv_slots, T* __restrict__ cq,
    T* __restrict__ pool, int ld_fused, int kv_off, int q_rank, int ld_cq, int kv_rank, int kvp, int rot_dim,
    int rot_dims, int ld_row, float eps) {
    __shared__ float red[4];
    const size_t n = blockIdx.x;
    const T* fq = fused + n * ld_fused;
    const T* fk = fq + kv_off;
    // both sums of squares: waves 0-1 the query latent, waves 2-3 the key/value latent
    const int half = threadIdx.x >> 7, t = threadIdx.x & 127;
    const T* src = half ? fk : fq;
    const float* wgt = half ? kv_norm : q_norm;
    const int len = half ? (kv_norm ? kv_rank : 0) : q_rank, padded = half ? (kv_norm ? kvp : 0) : ld_cq;
    const int64_t slot = kv_norm ? kv_slots[n] : -1;
    // eight values at a time, up to two groups per thread in registers with their weights (the groups' starts are
    // multiples of 16 bytes where a row is read or written; longer latents, and a length's last values, one by one)
    const bool whole = kv_off % 8 == 0 && ld_fused % 8 == 0 && ld_cq % 8 == 0 && kvp % 8 == 0 && ld_row % 8 == 0;
    const int groups = whole ? min(len / 8, 256) : 0, done = 8 * groups;
    Eight<T> x[2];
    Eight<float> w[2];
    float local = 0.f;
#pragma unroll
    for (int c = 0; c < 2; ++c)
        if (t + 128 * c < groups) {
            x[c].load(src + 8 * (t + 128 * c));
            w[c].load(wgt + 8 * (t + 128 * c));
        }
#pragma unroll
    for (int c = 0; c < 2; ++c)
        if (t + 128 * c < groups)
#pragma unroll
            for (int e = 0; e < 8; ++e) local += x[c].get(e) * x[c].get(e);
    for (int i = done + t; i < len; i += 128) {
        const float v = act_get<T>(src[i]);
        local += v * v;
    }
    local = wave_sum(local);
    if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x / kWave] = local;
    __syncthreads();
    const float inv = 1.f / sqrtf((red[2 * half] + red[2 * half + 1]) / static_cast<float>(half ? kv_rank : q_rank) + eps);
    if (half && slot < 0) return;
    T* dst = half ? pool + static_cast<size_t>(slot) * ld_row : cq + n * ld_cq;
#pragma unroll
    for (int c = 0; c < 2; ++c)
        if (t + 128 * c < groups) {
            float o[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = x[c].get(e) * inv * w[c].get(e);
            store_eight<T>(dst + 8 * (t + 128 * c), o);
        }
    for (int i = done + t; i < padded; i += 128) dst[i] = act_put<T>(i < len ? act_get<T>(src[i]) * inv * wgt[i] : 0.f);
    if (!half) return;   // (the rotated key part: waves 2-3)
    T* row = dst;
    const float* tab = rope_table + n * rot_dims;
    for (int i = t; i < ld_row - kvp; i += 128) {
        float v = 0.f;
        if (i < rot_dim)
            v = rotated_entry(i, rot_dims, tab, [&](int e) { return act_get<T>(fk[kv_rank + e]); });
        row[kvp + i] = act_put<T>(v);
    }
}

// y[n, h, :] = W[h] . act[n, h, :] for per-head matrices W [heads, C, K] bf16 (C, K multiples of
// 16 and 32; act rows of `ld_act`, heads `act_stride` apart): the query's way into the latent
// space and the latent sum's way out of it.  With rotp > 0 the launch's last blocks along x write the
// rotated part of the query: y[n, h, C + i] = rotated(act[n, h, rot_off + i]), zeros past rot_dim.
struct HeadArgs {
    const void* act;
    const uint16_t* w;
    void* y;
    const float* rope_table;   // (used when rotp > 0 and rot_dims > 0)
    int M, heads, C, K, ld_act, act_stride, ld_y, y_stride;
    int rot_off, rot_dim, rot_dims, rotp;
    const void* gate;          // logistic gates of the outputs [M, ld_gate] (null: none)
    int ld_gate, gate_cols;    // per head C (one per output) or 1
};

template <class T>
__device__ __forceinline__ void head_rotated_part(const HeadArgs& a, int h, int m_begin, int m_end, int part, int parts) {
    for (int idx = part * blockDim.x + threadIdx.x; idx < (m_end - m_begin) * a.rotp; idx += parts * blockDim.x) {
        const int m = m_begin + idx / a.rotp, i = idx % a.rotp;
        const T* src = static_cast<const T*>(a.act) + static_cast<size_t>(m) * a.ld_act +
                       static_cast<size_t>(h) * a.act_stride + a.rot_off;
        float v = 0.f;
        if (i < a.rot_dim)
            v = rotated_entry(i, a.rot_dims, a.rope_table + static_cast<size_t>(m) * a.rot_dims,
                              [&](int e) { return act_get<T>(src[e]); });
        static_cast<T*>(a.y)[static_cast<size_t>(m) * a.ld_y + static_cast<size_t>(h) * a.y_stride + a.C + i] = act_put<T>(v);
    }
}

// Matrix-core form: a wave (a block of its own: with few rows these launches are small, and single
// waves spread over the most CUs) takes 16 outputs of one head for MT tiles of 16 rows; the weight
// fragment (A operand: output on lane%16, k in the lane) is read once for all of them, the rows
// are the B operand, so a lane ends with four consecutive outputs of one row.
template <int MT>
__global__ __launch_bounds__(kWave) void head_linear_mfma_kernel(const HeadArgs a) {
    const int h = blockIdx.y, m0 = blockIdx.z * 16 * MT;
    const int lane = threadIdx.x;
    const int l16 = lane & 15, g = lane >> 4;
    const int cblocks = a.C / 16;
    if (static_cast<int>(blockIdx.x) >= cblocks) {
        head_rotated_part<uint16_t>(a, h, m0, min(m0 + 16 * MT, a.M), blockIdx.x - cblocks, gridDim.x - cblocks);
        return;
    }
    const int c0 = blockIdx.x * 16;
    const uint16_t* wp = a.w + (static_cast<size_t>(h) * a.C + c0 + l16) * a.K + 8 * g;
    const uint16_t* ap[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t)
        ap[t] = static_cast<const uint16_t*>(a.act) + static_cast<size_t>(min(m0 + 16 * t + l16, a.M - 1)) * a.ld_act +
                static_cast<size_t>(h) * a.act_stride + 8 * g;
    // (requested ahead of the products; without a gate infinities, whose logistic function is 1)
    u32x2_t gates[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const uint16_t* gp = static_cast<const uint16_t*>(a.gate) + static_cast<size_t>(min(m0 + 16 * t + l16, a.M - 1)) * a.ld_gate;
        gates[t] = u32x2_t{0x7F807F80u, 0x7F807F80u};
        if (a.gate && a.gate_cols == 1) gates[t].x = gates[t].y = gp[h] * 0x10001u;
        else if (a.gate) gates[t] = *reinterpret_cast<const u32x2_t*>(gp + h * a.C + c0 + 4 * g);
    }
    f32x4_t acc[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    // (eight k-steps requested together, four with many rows; past K a request repeats the last step and is not multiplied)
    constexpr int U = MT == 1 ? 8 : 4;
    for (int k0 = 0; k0 < a.K; k0 += 32 * U) {
        u32x4_t wf[U], af[U][MT];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = min(k0 + 32 * u, a.K - 32);
            wf[u] = *reinterpret_cast<const u32x4_t*>(wp + k);
#pragma unroll
            for (int t = 0; t < MT; ++t) af[u][t] = *reinterpret_cast<const u32x4_t*>(ap[t] + k);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (k0 + 32 * u >= a.K) break;
#pragma unroll
            for (int t = 0; t < MT; ++t)
                acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, wf[u]),
                                                                 __builtin_bit_cast(bf16x8_t, af[u][t]), acc[t], 0, 0, 0);
        }
    }
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const int m = m0 + 16 * t + l16;
        if (m >= a.M) continue;
        uint16_t* yp = static_cast<uint16_t*>(a.y) + static_cast<size_t>(m) * a.ld_y + static_cast<size_t>(h) * a.y_stride + c0 + 4 * g;
        const u32x2_t r = gates[t];
        const f32x4_t v = acc[t] * f32x4_t{sigmoid_f32(bf16_lo(r.x)), sigmoid_f32(bf16_hi(r.x)), sigmoid_f32(bf16_lo(r.y)), sigmoid_f32(bf16_hi(r.y))};
        *reinterpret_cast<u32x2_t*>(yp) = u32x2_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
    }
}

// fp32 form: one block per (row, head), the row in LDS, a thread per output.
__global__ __launch_bounds__(256) void head_linear_f32_kernel(const HeadArgs a) {
    extern __shared__ float row[];
    const int m = blockIdx.x, h = blockIdx.y;
    const float* src = static_cast<const float*>(a.act) + static_cast<size_t>(m) * a.ld_act + static_cast<size_t>(h) * a.act_stride;
    for (int i = threadIdx.x; i < a.K; i += blockDim.x) row[i] = src[i];
    __syncthreads();
    float* dst = static_cast<float*>(a.y) + static_cast<size_t>(m) * a.ld_y + static_cast<size_t>(h) * a.y_stride;
    for (int c = threadIdx.x; c < a.C; c += blockDim.x) {
        const uint16_t* wp = a.w + (static_cast<size_t>(h) * a.C + c) * a.K;
        float acc = 0.f;
        for (int k = 0; k < a.K; k += 8) {
            float w[8];
            ActVec<uint16_t>::load(wp + k, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = fmaf(row[k + e], w[e], acc);
        }
        if (a.gate)
            acc /= 1.f + expf(-static_cast<const float*>(a.gate)[static_cast<size_t>(m) * a.ld_gate + (a.gate_cols == 1 ? h : h * a.C + c)]);
        dst[c] = acc;
    }
    if (a.rotp > 0) head_rotated_part<float>(a, h, m, m + 1, 0, 1);
}

// The rows form of the attention, any sizes and either compute type: one block per (head, row),
// 256 keys at a time — a thread per key for the scores, a thread per latent column for the sum.
constexpr int kPlainThreads = 256, kPlainCols = 8;   // columns per thread: latents up to 2048
template <class T>
__global__ __launch_bounds__(kPlainThreads) void latent_rows_plain_kernel(
    const T* __restrict__ q, const T* __restrict__ pool, T* __restrict__ o, const uint32_t* __restrict__ page_indices,
    const uint32_t* __restrict__ row_begin, const int32_t* __restrict__ row_len, int heads, int kvp, int ld_row, int ps,
    float scale, const float* __restrict__ sinks) {
    extern __shared__ float sm[];
    float* qrow = sm;                      // ld_row
    float* prob = sm + ld_row;             // kPlainThreads
    uint32_t* slot = reinterpret_cast<uint32_t*>(prob + kPlainThreads);
    __shared__ float red[kPlainThreads / kWave];
    const int h = blockIdx.x, n = blockIdx.y;
    const int len = row_len[n];
    const uint32_t* pages = page_indices + row_begin[n];
    const T* qp = q + (static_cast<size_t>(n) * heads + h) * ld_row;
    for (int i = threadIdx.x; i < ld_row; i += kPlainThreads) qrow[i] = act_get<T>(qp[i]);
    float acc[kPlainCols];
#pragma unroll
    for (int c = 0; c < kPlainCols; ++c) acc[c] = 0.f;
    float mx = -INFINITY, sum = 0.f;
    constexpr int VN = ActVec<T>::kN;
    for (int j0 = 0; j0 < len; j0 += kPlainThreads) {
        const int nk = min(kPlainThreads, len - j0);
        __syncthreads();   // (the query row is staged; the previous keys' weights have been read)
        const int j = j0 + static_cast<int>(threadIdx.x);
        float s = -INFINITY;
        if (static_cast<int>(threadIdx.x) < nk) {
            const uint32_t sl = pages[j / ps] * ps + j % ps;
            slot[threadIdx.x] = sl;
            const T* kp = pool + static_cast<size_t>(sl) * ld_row;
            float d = 0.f;
            for (int i = 0; i < ld_row; i += VN) {
                float kv[VN];
                ActVec<T>::load(kp + i, kv);
#pragma unroll
                for (int e = 0; e < VN; ++e) d = fmaf(qrow[i + e], kv[e], d);
            }
            s = d * scale;
        }
        const float wmax = wave_max(s);
        if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x / kWave] = wmax;
        __syncthreads();
        float m_new = mx;
#pragma unroll
        for (int w = 0; w < kPlainThreads / kWave; ++w) m_new = fmaxf(m_new, red[w]);
        const float alpha = expf(mx - m_new);   // (a first step: exp(-inf) = 0)
        mx = m_new;
        const float p = static_cast<int>(threadIdx.x) < nk ? expf(s - m_new) : 0.f;
        prob[threadIdx.x] = p;
        sum = sum * alpha + block_total(p, red);   // (its barriers also publish the weights)
#pragma unroll
        for (int c = 0; c < kPlainCols; ++c) {
            const int col = threadIdx.x + c * kPlainThreads;
            if (col >= kvp) break;
            float a = acc[c] * alpha;
            for (int k = 0; k < nk; ++k) a = fmaf(prob[k], act_get<T>(pool[static_cast<size_t>(slot[k]) * ld_row + col]), a);
            acc[c] = a;
        }
    }
    float inv = sum > 0.f ? 1.f / sum : 0.f;
    if (sinks) {   // (in the units of the larger of the two)
        const float top = fmaxf(mx, sinks[h]), w = expf(mx - top);
        inv = w / (sum * w + expf(sinks[h] - top));
    }
    T* op = o + (static_cast<size_t>(n) * heads + h) * kvp;
#pragma unroll
    for (int c = 0; c < kPlainCols; ++c) {
        const int col = threadIdx.x + c * kPlainThreads;
        if (col < kvp) op[col] = act_put<T>(acc[c] * inv);
    }
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_latent_prep(int dtype, const void* fused, const float* q_norm, const float* kv_norm,
                                   const float* rope_table, const int64_t* kv_slots, void* cq, void* pool,
                                   int num_tokens, int ld_fused, int kv_off, int q_rank, int ld_cq, int kv_rank,
                                   int kvp, int rot_dim, int rot_dims, int ld_row, float eps, void* stream) {
    if (!fused || !q_norm || !cq || num_tokens <= 0 || q_rank <= 0 || kv_rank <= 0 ||
        (kv_norm && (!kv_slots || !pool || (rot_dims > 0 && !rope_table))))
        return PIE_HIP_ERR_INVALID;
    if (kv_off < q_rank || q_rank > ld_fused || (kv_norm && kv_off + kv_rank + rot_dim > ld_fused) || ld_cq < q_rank || kvp < kv_rank ||
        ld_row < kvp + rot_dim || rot_dims > rot_dim || rot_dims % 2 != 0)
        return PIE_HIP_ERR_INVALID;
    PIE_ACT_DISPATCH(dtype, T,
                     hipLaunchKernelGGL(latent_prep_kernel<T>, dim3(num_tokens), dim3(256), 0,
                                        static_cast<hipStream_t>(stream), static_cast<const T*>(fused), q_norm, kv_norm,
                                        rope_table, kv_slots, static_cast<T*>(cq), static_cast<T*>(pool), ld_fused,
                                        kv_off, q_rank, ld_cq, kv_rank, kvp, rot_dim, rot_dims, ld_row, eps));
    return launch_status();
}

extern "C" int pie_hip_head_linear(int dtype, const void* act, const uint16_t* w_bf16, void* y,
                                   const float* rope_table, int M, int heads, int C, int K, int ld_act,
                                   int act_stride, int ld_y, int y_stride, int rot_off, int rot_dim, int rot_dims,
                                   int rotp, const void* gate, int ld_gate, int gate_cols, void* stream) {
    if (!act || !w_bf16 || !y || M <= 0 || heads <= 0 || C <= 0 || K <= 0) return PIE_HIP_ERR_INVALID;
    if (C % 16 != 0 || K % 32 != 0 || ld_act % 8 != 0 || act_stride % 8 != 0 || ld_y % 8 != 0 || y_stride % 8 != 0)
        return PIE_HIP_ERR_UNSUPPORTED;
    if (ld_act < (heads - 1) * act_stride + K || ld_y < (heads - 1) * y_stride + C) return PIE_HIP_ERR_INVALID;
    if (rotp > 0 && ((rot_dims > 0 && !rope_table) || rot_dims > rot_dim || rot_dims % 2 != 0 || rotp < rot_dim || y_stride < C + rotp ||
                       act_stride < rot_off + rot_dim))
        return PIE_HIP_ERR_INVALID;
    if (gate && ((gate_cols != 1 && gate_cols != C) || ld_gate < heads * gate_cols)) return PIE_HIP_ERR_INVALID;
    if (gate && gate_cols == C && (ld_gate % 4 != 0 || reinterpret_cast<uintptr_t>(gate) % 8 != 0)) return PIE_HIP_ERR_INVALID;
    const HeadArgs a{act, w_bf16, y, rope_table, M, heads, C, K, ld_act, act_stride, ld_y, y_stride, rot_off, rot_dim,
                     rot_dims, rotp, gate, ld_gate, gate_cols};
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (heads > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    if (dtype == PIE_HIP_DT_F32) {
        hipLaunchKernelGGL(head_linear_f32_kernel, dim3(M, heads), dim3(256), K * sizeof(float), s, a);
        return launch_status();
    }
    if (dtype != PIE_HIP_DT_BF16) return PIE_HIP_ERR_INVALID;
    const int mt = M <= 16 ? 1 : M <= 32 ? 2 : 4;
    const int gx = C / 16 + (rotp > 0 ? mt : 0);
    const int gz = (M + 16 * mt - 1) / (16 * mt);
    if (gz > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    switch (mt) {
        case 1: hipLaunchKernelGGL(head_linear_mfma_kernel<1>, dim3(gx, heads, gz), dim3(64), 0, s, a); break;
        case 2: hipLaunchKernelGGL(head_linear_mfma_kernel<2>, dim3(gx, heads, gz), dim3(64), 0, s, a); break;
        default: hipLaunchKernelGGL(head_linear_mfma_kernel<4>, dim3(gx, heads, gz), dim3(64), 0, s, a); break;
    }
    return launch_status();
}

extern "C" int pie_hip_latent_attn_rows_plain(int dtype, const void* q, const void* pool, void* o,
                                              const uint32_t* kv_page_indices, const uint32_t* row_page_begin,
                                              const int32_t* row_kv_len, int num_rows, int heads, int kvp, int ld_row,
                                              int page_size, float scale, const float* sinks, void* stream) {
    if (!q || !pool || !o || !kv_page_indices || !row_page_begin || !row_kv_len || num_rows <= 0 || heads <= 0 ||
        kvp <= 0 || ld_row < kvp || page_size <= 0)
        return PIE_HIP_ERR_INVALID;
    if (ld_row % 8 != 0 || kvp > kPlainCols * kPlainThreads || num_rows > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const size_t smem = (static_cast<size_t>(ld_row) + 2 * kPlainThreads) * sizeof(float);
    if (smem > 60 * 1024) return PIE_HIP_ERR_UNSUPPORTED;
    PIE_ACT_DISPATCH(dtype, T,
                     hipLaunchKernelGGL(latent_rows_plain_kernel<T>, dim3(heads, num_rows), dim3(kPlainThreads), smem,
                                        static_cast<hipStream_t>(stream), static_cast<const T*>(q),
                                        static_cast<const T*>(pool), static_cast<T*>(o), kv_page_indices,
                                        row_page_begin, row_kv_len, heads, kvp, ld_row, page_size, scale, sinks));
    return launch_status();
}
