// The rows form of latent attention on the matrix cores (gfx950, v_mfma_f32_16x16x32_bf16):
//   o[n, h, :] = softmax_j( q[n, h, :] . row_j * scale ) . row_j[:kvp],  j < row_kv_len[n]
// over the bf16 latent pool.  All heads of a token share the rows, so a block takes 16 or 32 (token,
// head) pairs of one request — the heads of a token, or a few tokens' when there are fewer heads —
// and reads every row once for both products.
//
// A block is four waves and advances 32 keys at a time:
//   stage    the step's rows go from registers (requested one step ahead) to one LDS tile
//   scores   S^T[key, pair] = K . Q^T: wave w takes 16 keys and, of 32 pairs, one half (of 16 pairs:
//            one half of the row's length); the fragments of Q stay in registers
//   softmax  eight (sixteen) threads per pair over the score tile in LDS; weights leave as a hi + lo
//            pair of bf16 values (16 significant bits), the normaliser sums the unrounded ones
//   sum      O^T[column, pair] += V^T . P^T: wave w takes a quarter of the latent columns, V^T read
//            from the same tile by the transposing LDS read
// so a row is read from LDS once per product whatever the number of heads.  Tile rows are padded
// by eight values: the 16-byte row reads and the 8-byte transposing reads both fall on distinct
// banks.  Keys are cut into splits over grid.y; more than one leaves fp32 partial results for the
// merge kernel.
#include "common.hip.h"

namespace pie_hip {
namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

constexpr int kStep = 32, kBlock = 256;

struct LatentRowsArgs {
    const uint16_t* q;        // [rows, heads, LD]
    const uint16_t* pool;
    uint16_t* o;              // [rows, heads, kvp], null: partial results
    float* part_o;            // [rows, heads, nsplit, kvp]
    float* part_ml;           // [rows, heads, nsplit, 2] (max in units of scale * log2 e, sum)
    const uint32_t* page_indices;
    const uint32_t* row_begin;
    const int32_t* row_len;
    const int32_t* row_req;   // request of each row, qo_indptr its rows (null: every row its own request)
    const int32_t* qo_indptr;
    int row0, num_rows, heads, head_groups, heads_per_tile, tokens_per_tile, ps, ps_shift, steps_per_split, nsplit;
    float scale_log2e;
    const float* sinks;       // [heads] (null: none); with partial results the merge adds them
};

// What the weighted sum is multiplied by: its sum of exponentials l, taken at m (in powers of two), and a sink's
// join in the units of the larger of m and the sink.
__device__ __forceinline__ float sink_inverse(float m, float l, float sink_log2) {
    const float top = fmaxf(m, sink_log2), w = exp2f(m - top);
    return w / (l * w + exp2f(sink_log2 - top));
}

// Keys of one split: a decode row cuts its own keys evenly (steps_per_split 0), whatever the bound
// the launch was planned with; portions take the planned length.
__device__ __forceinline__ int split_keys(int keys, int nsplit, int steps_per_split) {
    if (steps_per_split > 0) return steps_per_split * kStep;
    const int steps = (keys + kStep - 1) / kStep;
    return max(1, (steps + nsplit - 1) / nsplit) * kStep;
}

// C: latent columns / 64; R: rotated columns / 32 (0: the rows are latents only); MT: 16-pair tiles per block
template <int C, int R, int MT>
__global__ __launch_bounds__(kBlock, 2) void latent_rows_kernel(const LatentRowsArgs a) {
    constexpr int LD = 64 * C + 32 * R, STRIDE = LD + 8, KS = 2 * C + R;
    constexpr int PPR = LD / 8;                                     // 16-byte pieces per row
    constexpr int NP = (PPR + 7) / 8;                               // pieces per thread and step: eight threads per row
    constexpr int PAIRS = 16 * MT, SSTR = kStep + 4, PSTR = kStep + 8;
    constexpr int KSW = MT == 2 ? KS : (KS + 1) / 2;                // k-steps of a wave's score tile
    constexpr int TPP = kBlock / PAIRS, KPT = kStep / TPP;          // softmax: threads per pair, keys per thread
    __shared__ __attribute__((aligned(16))) uint16_t tile[kStep * STRIDE];
    __shared__ __attribute__((aligned(16))) float sc[MT == 2 ? 1 : 2][PAIRS * SSTR];
    __shared__ __attribute__((aligned(16))) uint16_t p_hi[PAIRS * PSTR], p_lo[PAIRS * PSTR];
    __shared__ float s_alpha[PAIRS], s_l[PAIRS], s_m[PAIRS];
    const int tid = threadIdx.x, lane = tid & (kWave - 1);
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int l16 = lane & 15, g = lane >> 4;

    // the tile: tokens n .. n + nt - 1 of one request, heads h0 .. h0 + heads_per_tile - 1
    const int n = a.row0 + blockIdx.x / a.head_groups, h0 = (blockIdx.x % a.head_groups) * a.heads_per_tile;
    int nt = 1;
    if (a.row_req && a.tokens_per_tile > 1) {
        const int r = a.row_req[n];
        if ((n - a.qo_indptr[r]) % a.tokens_per_tile != 0) return;
        nt = min(a.tokens_per_tile, a.qo_indptr[r + 1] - n);
    }
    const int kmax = a.row_len[n + nt - 1];   // (rows of a request are consecutive positions)
    const int keys_per_split = split_keys(kmax, a.nsplit, a.steps_per_split);
    const int k_begin = blockIdx.y * keys_per_split;
    const int k_end = min(kmax, k_begin + keys_per_split);
    if (k_begin >= kmax && !(a.nsplit == 1 && kmax == 0)) return;
    const uint32_t* pages = a.page_indices + a.row_begin[n];
    // pair m of the tile -> token, head, visible keys
    auto pair_valid = [&](int m) { return m / a.heads_per_tile < nt && h0 + m % a.heads_per_tile < a.heads; };
    auto pair_out = [&](int m) {
        return static_cast<size_t>(n + m / a.heads_per_tile) * a.heads + h0 + m % a.heads_per_tile;
    };

    // Q fragments of this wave: pair l16 of tile `rt`, k-steps ks0 ..
    const int kh = wv & 1, rt = MT == 2 ? wv >> 1 : 0, ks0 = MT == 2 ? 0 : (wv >> 1) * KSW;
    bf16x8_t qf[KSW];
    {
        const int m = rt * 16 + l16;
        const bool valid = pair_valid(m);
        const uint16_t* qp = a.q + (valid ? pair_out(m) : pair_out(0)) * LD + 8 * g;
#pragma unroll
        for (int ks = 0; ks < KSW; ++ks) {
            u32x4_t v = {0u, 0u, 0u, 0u};
            if (valid && ks0 + ks < KS) v = *reinterpret_cast<const u32x4_t*>(qp + 32 * (ks0 + ks));
            qf[ks] = __builtin_bit_cast(bf16x8_t, v);
        }
    }
    // softmax role: pair sp, keys sk0 .. sk0 + KPT - 1 of the step
    const int sp = tid / TPP, sk0 = (tid % TPP) * KPT;
    const int my_len = pair_valid(sp) ? a.row_len[n + sp / a.heads_per_tile] : 0;
    float mx = -INFINITY, lsum = 0.f;

    const int key = tid >> 3, piece0 = tid & 7;
    u32x4_t reg[NP];
    // the page of this thread's key, requested a step ahead of the key itself: the two requests
    // depend on each other and would otherwise stand in line in every step
    uint32_t pid = 0;
    int in_page = 0;
    auto fetch_page = [&](int j0) {
        const int j = min(j0 + key, kmax - 1);   // (keys past the extent repeat the last: their weights are zero)
        const int page = a.ps_shift >= 0 ? j >> a.ps_shift : j / a.ps;
        pid = pages[page];
        in_page = j - page * a.ps;
    };
    auto issue = [&](int j0) {
        const uint16_t* row = a.pool + (static_cast<size_t>(pid) * a.ps + in_page) * LD + piece0 * 8;
#pragma unroll
        for (int u = 0; u < NP; ++u)
            if (PPR % 8 == 0 || piece0 + 8 * u < PPR) reg[u] = *reinterpret_cast<const u32x4_t*>(row + 64 * u);
        fetch_page(j0 + kStep);
    };
    auto stage = [&]() {
        uint16_t* row = &tile[key * STRIDE + piece0 * 8];
#pragma unroll
        for (int u = 0; u < NP; ++u)
            if (PPR % 8 == 0 || piece0 + 8 * u < PPR) *reinterpret_cast<u32x4_t*>(row + 64 * u) = reg[u];
    };

    f32x4_t acc[C][MT];
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
        for (int t = 0; t < MT; ++t) acc[c][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};

    if (k_begin < k_end) {
        fetch_page(k_begin);
        issue(k_begin);
    }
    for (int j0 = k_begin; j0 < k_end; j0 += kStep) {
        stage();
        if (j0 + kStep < k_end) issue(j0 + kStep);
        __syncthreads();
        // scores
        {
            // (fragments requested KG at a time ahead of their products, two accumulator chains)
            f32x4_t st = {0.f, 0.f, 0.f, 0.f}, st1 = st;
            const uint16_t* kp = &tile[(16 * kh + l16) * STRIDE + 8 * g];
            constexpr int KG = 6;
#pragma unroll
            for (int k0 = 0; k0 < KSW; k0 += KG) {
                u32x4_t kf[KG];
#pragma unroll
                for (int u = 0; u < KG; ++u)
                    if (k0 + u < KSW) kf[u] = *reinterpret_cast<const u32x4_t*>(kp + 32 * min(ks0 + k0 + u, KS - 1));
#pragma unroll
                for (int u = 0; u < KG; ++u)
                    if (k0 + u < KSW) {   // (a k-step past the row meets a zero query fragment)
                        if (u & 1) st1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[u]), qf[k0 + u], st1, 0, 0, 0);
                        else st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[u]), qf[k0 + u], st, 0, 0, 0);
                    }
            }
            st += st1;
            *reinterpret_cast<f32x4_t*>(&sc[MT == 2 ? 0 : wv >> 1][(rt * 16 + l16) * SSTR + 16 * kh + 4 * g]) = st;
        }
        __syncthreads();
        // softmax
        {
            float s[KPT], m_new = mx;
#pragma unroll
            for (int e = 0; e < KPT; ++e) {
                float v = sc[0][sp * SSTR + sk0 + e];
                if (MT == 1) v += sc[MT == 2 ? 0 : 1][sp * SSTR + sk0 + e];
                v = j0 + sk0 + e < min(my_len, k_end) ? v * a.scale_log2e : -INFINITY;
                s[e] = v;
                m_new = fmaxf(m_new, v);
            }
#pragma unroll
            for (int off = 1; off < TPP; off <<= 1) m_new = fmaxf(m_new, __shfl_xor(m_new, off, kWave));
            const float safe = m_new == -INFINITY ? 0.f : m_new;
            const float alpha = exp2f(mx - safe);
            mx = m_new;
            float sum = 0.f;
            uint32_t hi[KPT / 2], lo[KPT / 2];
#pragma unroll
            for (int e = 0; e < KPT; e += 2) {
                const float p0 = exp2f(s[e] - safe), p1 = exp2f(s[e + 1] - safe);
                sum += p0 + p1;
                const uint32_t b0 = __float_as_uint(p0) & 0xFFFF0000u, b1 = __float_as_uint(p1) & 0xFFFF0000u;
                hi[e / 2] = (b0 >> 16) | b1;
                lo[e / 2] = pack_bf16x2(p0 - __uint_as_float(b0), p1 - __uint_as_float(b1));
            }
            lsum = lsum * alpha + sum;
#pragma unroll
            for (int e = 0; e < KPT / 2; ++e) {
                *reinterpret_cast<uint32_t*>(&p_hi[sp * PSTR + sk0 + 2 * e]) = hi[e];
                *reinterpret_cast<uint32_t*>(&p_lo[sp * PSTR + sk0 + 2 * e]) = lo[e];
            }
            if (tid % TPP == 0) s_alpha[sp] = alpha;
        }
        __syncthreads();
        // weighted sum: this wave's columns 16 (C wv + c) ..
        {
            bf16x8_t ph[MT], pl[MT];
#pragma unroll
            for (int t = 0; t < MT; ++t) {
                const int at = (16 * t + l16) * PSTR + 4 * g;
                const u32x2_t h0v = *reinterpret_cast<const u32x2_t*>(&p_hi[at]), h1v = *reinterpret_cast<const u32x2_t*>(&p_hi[at + 16]);
                const u32x2_t l0v = *reinterpret_cast<const u32x2_t*>(&p_lo[at]), l1v = *reinterpret_cast<const u32x2_t*>(&p_lo[at + 16]);
                ph[t] = __builtin_bit_cast(bf16x8_t, u32x4_t{h0v.x, h0v.y, h1v.x, h1v.y});
                pl[t] = __builtin_bit_cast(bf16x8_t, u32x4_t{l0v.x, l0v.y, l1v.x, l1v.y});
                const float alpha = s_alpha[16 * t + l16];
                if (__any(alpha != 1.0f)) {
#pragma unroll
                    for (int c = 0; c < C; ++c) acc[c][t] *= alpha;
                }
            }
#pragma unroll
            for (int c = 0; c < C; ++c) {
                const uint16_t* va = &tile[(4 * g + (l16 >> 2)) * STRIDE + 16 * (C * wv + c) + 4 * (l16 & 3)];
                const bf16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va));
                const bf16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va + 16 * STRIDE));
                const bf16x8_t vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                for (int t = 0; t < MT; ++t) {
                    acc[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[t], acc[c][t], 0, 0, 0);
                    acc[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[t], acc[c][t], 0, 0, 0);
                }
            }
        }
        __syncthreads();   // the tile has been read
    }

    // the pairs' normalisers meet in LDS
#pragma unroll
    for (int off = 1; off < TPP; off <<= 1) lsum += __shfl_xor(lsum, off, kWave);
    if (tid % TPP == 0) {
        s_l[sp] = lsum;
        s_m[sp] = mx;
    }
    __syncthreads();
    constexpr int KVP = 64 * C;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const int m = 16 * t + l16;
        if (!pair_valid(m)) continue;
        const size_t out = pair_out(m);
        const float l = s_l[m];
        if (a.o) {
            const float inv = a.sinks ? sink_inverse(s_m[m], l, a.sinks[h0 + m % a.heads_per_tile] * 1.4426950408889634f)
                              : l > 0.f ? 1.f / l : 0.f;
#pragma unroll
            for (int c = 0; c < C; ++c) {
                const f32x4_t v = acc[c][t];
                *reinterpret_cast<u32x2_t*>(a.o + out * KVP + 16 * (C * wv + c) + 4 * g) =
                    u32x2_t{pack_bf16x2(v[0] * inv, v[1] * inv), pack_bf16x2(v[2] * inv, v[3] * inv)};
            }
        } else {
            const size_t slot = out * a.nsplit + blockIdx.y;
#pragma unroll
            for (int c = 0; c < C; ++c)
                *reinterpret_cast<f32x4_t*>(a.part_o + slot * KVP + 16 * (C * wv + c) + 4 * g) = acc[c][t];
            if (wv == 0 && g == 0) {
                a.part_ml[slot * 2] = s_m[m];
                a.part_ml[slot * 2 + 1] = l;
            }
        }
    }
}

// o[n, h, :] = the merged, normalised partial results; one block per (row, head), four columns per
// thread.  A row has as many pieces as splits start before its last key.
__global__ void latent_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                    const int32_t* __restrict__ row_len, uint16_t* __restrict__ o, int row0, int heads,
                                    int kvp, int nsplit, int steps_per_split, const float* __restrict__ sinks) {
    const size_t out = static_cast<size_t>(row0) * heads + blockIdx.x;
    const int len = row_len[out / heads], keys_per_split = split_keys(len, nsplit, steps_per_split);
    const int ns = min(nsplit, (len + keys_per_split - 1) / keys_per_split);
    const float* ml = part_ml + out * nsplit * 2;
    float mx = -INFINITY;
    for (int s = 0; s < ns; ++s) mx = fmaxf(mx, ml[2 * s]);
    const float sink = sinks ? sinks[out % heads] * 1.4426950408889634f : -INFINITY;
    mx = fmaxf(mx, sink);
    const float safe = mx == -INFINITY ? 0.f : mx;
    float l = exp2f(sink - safe);
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    const float* po = part_o + out * nsplit * kvp + 4 * threadIdx.x;
#pragma unroll 4
    for (int s = 0; s < ns; ++s) {
        const float w = exp2f(ml[2 * s] - safe);
        const f32x4_t p = *reinterpret_cast<const f32x4_t*>(po + static_cast<size_t>(s) * kvp);
        l = fmaf(ml[2 * s + 1], w, l);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = fmaf(p[e], w, v[e]);
    }
    const float inv = l > 0.f ? 1.f / l : 0.f;
    *reinterpret_cast<u32x2_t*>(o + out * kvp + 4 * threadIdx.x) =
        u32x2_t{pack_bf16x2(v[0] * inv, v[1] * inv), pack_bf16x2(v[2] * inv, v[3] * inv)};
}

struct LatentPlan {
    int mt, heads_per_tile, head_groups, tokens_per_tile, steps_per_split, nsplit;
};
// Splits: about two blocks per CU over the batch, at least 128 keys each.
LatentPlan latent_plan(int num_rows, int heads, int max_kv_len, int max_tokens_per_req) {
    LatentPlan p;
    p.mt = heads > 16 || max_tokens_per_req > 1 ? 2 : 1;
    p.heads_per_tile = heads < 16 * p.mt ? heads : 16 * p.mt;
    p.head_groups = (heads + p.heads_per_tile - 1) / p.heads_per_tile;
    p.tokens_per_tile = max_tokens_per_req > 1 ? 16 * p.mt / p.heads_per_tile : 1;
    const long long tiles = static_cast<long long>((num_rows + p.tokens_per_tile - 1) / p.tokens_per_tile) * p.head_groups;
    const int steps = max_kv_len > 0 ? (max_kv_len + kStep - 1) / kStep : 1;
    long long ns = 512 / tiles;
    if (ns > (steps + 3) / 4) ns = (steps + 3) / 4;
    if (ns < 1) ns = 1;
    p.steps_per_split = static_cast<int>((steps + ns - 1) / ns);
    p.nsplit = (steps + p.steps_per_split - 1) / p.steps_per_split;
    if (max_tokens_per_req == 1) p.steps_per_split = 0;
    return p;
}

template <int C, int R>
int launch_latent_rows(const LatentRowsArgs& a, const LatentPlan& p, hipStream_t s) {
    const dim3 grid(a.num_rows * p.head_groups, p.nsplit);
    if (p.mt == 2) hipLaunchKernelGGL((latent_rows_kernel<C, R, 2>), grid, dim3(kBlock), 0, s, a);
    else hipLaunchKernelGGL((latent_rows_kernel<C, R, 1>), grid, dim3(kBlock), 0, s, a);
    return launch_status();
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_latent_attn_rows_supported(int kvp, int rotp) {
    if (rotp != 0 && rotp != 32 && rotp != 64) return 0;
    return kvp == 64 || kvp == 128 || kvp == 192 || kvp == 256 || kvp == 384 || kvp == 512;
}

extern "C" size_t pie_hip_latent_attn_rows_workspace_bytes(int num_rows, int heads, int kvp, int max_kv_len,
                                                           int max_tokens_per_req) {
    if (num_rows <= 0 || heads <= 0 || kvp <= 0) return 0;
    const LatentPlan p = latent_plan(num_rows, heads, max_kv_len, max_tokens_per_req);
    return p.nsplit > 1 ? static_cast<size_t>(num_rows) * heads * p.nsplit * (kvp + 2) * sizeof(float) : 0;
}

extern "C" int pie_hip_latent_attn_rows(const uint16_t* q, const uint16_t* pool, uint16_t* o,
                                        const uint32_t* kv_page_indices, const uint32_t* row_page_begin,
                                        const int32_t* row_kv_len, const int32_t* row_req, const int32_t* qo_indptr,
                                        int row0, int num_rows, int heads, int kvp, int rotp, int page_size,
                                        float scale, const float* sinks, int max_kv_len, int max_tokens_per_req,
                                        void* workspace, size_t workspace_bytes, void* stream) {
    if (!q || !pool || !o || !kv_page_indices || !row_page_begin || !row_kv_len || row0 < 0 || num_rows <= 0 ||
        heads <= 0 || page_size <= 0 || max_tokens_per_req <= 0)
        return PIE_HIP_ERR_INVALID;
    if (max_tokens_per_req > 1 && (!row_req || !qo_indptr)) return PIE_HIP_ERR_INVALID;
    if (!pie_hip_latent_attn_rows_supported(kvp, rotp) || page_size % 16 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const LatentPlan p = latent_plan(num_rows, heads, max_kv_len, max_tokens_per_req);
    if (p.nsplit > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    LatentRowsArgs a{q, pool, o, nullptr, nullptr, kv_page_indices, row_page_begin, row_kv_len,
                     max_tokens_per_req > 1 ? row_req : nullptr, qo_indptr, row0, num_rows, heads, p.head_groups,
                     p.heads_per_tile, p.tokens_per_tile, page_size,
                     (page_size & (page_size - 1)) == 0 ? __builtin_ctz(static_cast<unsigned>(page_size)) : -1, p.steps_per_split, p.nsplit,
                     scale * 1.4426950408889634f, sinks};
    if (p.nsplit > 1) {
        if (!workspace || workspace_bytes < pie_hip_latent_attn_rows_workspace_bytes(num_rows, heads, kvp, max_kv_len, max_tokens_per_req))
            return PIE_HIP_ERR_INVALID;
        // (row `row0` sits at the front of the workspace)
        const size_t pairs = static_cast<size_t>(num_rows) * heads * p.nsplit, skip = static_cast<size_t>(row0) * heads * p.nsplit;
        a.o = nullptr;
        a.part_o = static_cast<float*>(workspace) - skip * kvp;
        a.part_ml = static_cast<float*>(workspace) + pairs * kvp - skip * 2;
    }
    hipStream_t s = static_cast<hipStream_t>(stream);
    int st = PIE_HIP_ERR_UNSUPPORTED;
#define PIE_LATENT_CASE(CC, RR) \
    if (kvp == 64 * CC && rotp == 32 * RR) st = launch_latent_rows<CC, RR>(a, p, s);
    PIE_LATENT_CASE(1, 0) PIE_LATENT_CASE(2, 0) PIE_LATENT_CASE(3, 0) PIE_LATENT_CASE(4, 0) PIE_LATENT_CASE(6, 0) PIE_LATENT_CASE(8, 0)
    PIE_LATENT_CASE(1, 1) PIE_LATENT_CASE(2, 1) PIE_LATENT_CASE(3, 1) PIE_LATENT_CASE(4, 1) PIE_LATENT_CASE(6, 1) PIE_LATENT_CASE(8, 1)
    PIE_LATENT_CASE(1, 2) PIE_LATENT_CASE(2, 2) PIE_LATENT_CASE(3, 2) PIE_LATENT_CASE(4, 2) PIE_LATENT_CASE(6, 2) PIE_LATENT_CASE(8, 2)
#undef PIE_LATENT_CASE
    if (st != PIE_HIP_OK || p.nsplit == 1) return st;
    hipLaunchKernelGGL(latent_merge_kernel, dim3(num_rows * heads), dim3(kvp / 4), 0, s, a.part_o, a.part_ml, row_kv_len, o,
                       row0, heads, kvp, p.nsplit, p.steps_per_split, sinks);
    return launch_status();
}
