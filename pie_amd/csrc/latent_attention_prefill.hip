// The expanded form of latent attention, for portions long enough that projecting keys and values
// out of the cached latents once costs less than carrying every query through the latent space.
//
//   latent_gather   the cached rows of a request as compact matrices (latents, rotated key parts)
//   (a GEMM)        keys and values of every head, kv [keys, heads, dimp | vdp]
//   latent_prefill  o[n, h, :] = softmax_j( (q . k_j + q_rot . rot_j) * scale ) . v_j,  j < row_kv_len[n]
//
// The attention kernel has the shape of the uniform models' prefill kernel: a block of four waves
// takes 64 QT query tokens of one head, a wave 16 QT of them; keys advance 32 at a time through
// double-buffered LDS tiles, one barrier per step, two steps requested ahead in registers.
//   S^T[key, query] = K . Q^T     Q fragments in registers, the rotated part rotated as it is loaded
//   O^T[d, query]  += V^T . P^T   V^T by the transposing LDS read; P as a hi + lo pair of bf16 values
// Queries sit on the lane%16 axis of both products, so the softmax state is per lane.  A wave skips
// the steps past its own last query.  Blocks of one head follow each other eight apart in launch
// order, so a head's keys stay in one XCD's L2; the longest tiles start first.
#include "act_type.hip.h"

#include <type_traits>

namespace pie_hip {
namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

constexpr int kStep = 32, kBlock = 256;

__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ pool,
                                                            const uint32_t* __restrict__ pages,
                                                            uint16_t* __restrict__ lat, uint16_t* __restrict__ rot,
                                                            int num_keys, int kvp, int rotp, int ps) {
    const int ld = kvp + rotp, ppr = ld / 8;
    const size_t total = static_cast<size_t>(num_keys) * ppr;
    for (size_t i = blockIdx.x * 256ull + threadIdx.x; i < total; i += gridDim.x * 256ull) {
        const int j = static_cast<int>(i / ppr), piece = static_cast<int>(i % ppr);
        const size_t slot = static_cast<size_t>(pages[j / ps]) * ps + j % ps;
        const u32x4_t v = *reinterpret_cast<const u32x4_t*>(pool + slot * ld + piece * 8);
        uint16_t* dst = piece * 8 < kvp ? lat + static_cast<size_t>(j) * kvp + piece * 8
                                        : rot + static_cast<size_t>(j) * rotp + (piece * 8 - kvp);
        *reinterpret_cast<u32x4_t*>(dst) = v;
    }
}

struct LatentPrefillArgs {
    const uint16_t *q, *kv, *rot;
    uint16_t* o;
    const float* rope_table;
    const int32_t* row_len;
    int row0, num_rows, heads, dimp, rotp, rot_dims, ld_o;
    float scale_log2e;
    const float* sinks;     // [heads] (null: none)
    const uint16_t* gate;   // logistic gates of the outputs [rows, ld_gate] (null: none)
    int ld_gate, gate_cols;   // per head DV or 1
};

template <int KS, int VT, int QT>
__global__ __launch_bounds__(kBlock, 2) void latent_prefill_kernel(const LatentPrefillArgs a) {
    constexpr int D = 32 * KS, DV = 32 * VT, DT = 2 * VT;
    constexpr int KSTRIDE = D + 8, VSTRIDE = DV + 16;
    constexpr int PPK = 4 * KS, PPR = 4 * (KS + VT), NP = (PPR + 7) / 8;   // 16-byte pieces per key, eight threads a key
    __shared__ __attribute__((aligned(16))) uint16_t k_tile[2][kStep * KSTRIDE];
    __shared__ __attribute__((aligned(16))) uint16_t v_tile[2][kStep * VSTRIDE];
    const int h = blockIdx.x, t0 = (gridDim.y - 1 - blockIdx.y) * 64 * QT;
    const int tid = threadIdx.x, lane = tid & (kWave - 1);
    const int wv = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int l16 = lane & 15, g = lane >> 4;
    const int rows = min(64 * QT, a.num_rows - t0);
    const int kmax = a.row_len[a.row0 + t0 + rows - 1];
    const int per_head = a.dimp + DV;
    const size_t ld_kv = static_cast<size_t>(a.heads) * per_head;

    // this lane's queries and their fragments
    int my_len[QT];
    bf16x8_t qf[QT][KS];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int m = wv * 16 * QT + t * 16 + l16;
        const bool valid = m < rows;
        const size_t n = a.row0 + t0 + (valid ? m : 0);
        my_len[t] = valid ? a.row_len[n] : 0;
        const uint16_t* qp = a.q + (n * a.heads + h) * D + 8 * g;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            u32x4_t v = *reinterpret_cast<const u32x4_t*>(qp + 32 * ks);
            const int r0 = 32 * ks - a.dimp + 8 * g;   // place in the rotated part
            if (r0 >= 0 && r0 < a.rot_dims) {
                const float* tab = a.rope_table + n * a.rot_dims;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int i = r0 + 2 * e;
                    if (i < a.rot_dims) {
                        const float c = tab[i >> 1], s = tab[(a.rot_dims >> 1) + (i >> 1)];
                        const float x = bf16_lo(v[e]), y = bf16_hi(v[e]);
                        v[e] = pack_bf16x2(x * c - y * s, y * c + x * s);
                    }
                }
            }
            if (!valid) v = u32x4_t{0u, 0u, 0u, 0u};
            qf[t][ks] = __builtin_bit_cast(bf16x8_t, v);
        }
    }
    int lo_len = my_len[0], hi_len = my_len[0];
#pragma unroll
    for (int t = 1; t < QT; ++t) {
        lo_len = min(lo_len, my_len[t]);
        hi_len = max(hi_len, my_len[t]);
    }
#pragma unroll
    for (int sh = 1; sh < kWave; sh <<= 1) {
        lo_len = min(lo_len, __shfl_xor(lo_len, sh, kWave));
        hi_len = max(hi_len, __shfl_xor(hi_len, sh, kWave));
    }
    const int wave_min = __builtin_amdgcn_readfirstlane(lo_len), wave_max = __builtin_amdgcn_readfirstlane(hi_len);

    // staging: thread -> key tid / 8, pieces tid % 8 + 8 u of (unrotated key | rotated key | value)
    const int key = tid >> 3, piece0 = tid & 7;
    const uint16_t* src[NP];
    int step_elems[NP];
#pragma unroll
    for (int u = 0; u < NP; ++u) {
        const int p = min(piece0 + 8 * u, PPR - 1), e = p * 8;
        if (e < a.dimp) src[u] = a.kv + static_cast<size_t>(h) * per_head + e;
        else if (p < PPK) src[u] = a.rot + (e - a.dimp);   // (rotp 0: no such piece)
        else src[u] = a.kv + static_cast<size_t>(h) * per_head + a.dimp + (e - D);
        step_elems[u] = e >= a.dimp && p < PPK ? a.rotp : static_cast<int>(ld_kv);
    }
    u32x4_t reg[2][NP];
    auto issue = [&](int slot, int j0) {
        const size_t j = min(j0 + key, kmax - 1);   // (keys past the extent repeat the last: their weights are zero)
#pragma unroll
        for (int u = 0; u < NP; ++u)
            reg[slot][u] = *reinterpret_cast<const u32x4_t*>(src[u] + j * step_elems[u]);
    };
    auto stage = [&](int slot) {
#pragma unroll
        for (int u = 0; u < NP; ++u) {
            const int p = piece0 + 8 * u;
            if (PPR % 8 != 0 && p >= PPR) continue;
            uint16_t* dst = p < PPK ? &k_tile[slot][key * KSTRIDE + p * 8] : &v_tile[slot][key * VSTRIDE + (p - PPK) * 8];
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
        const uint16_t* vt = v_tile[slot];
        f32x4_t st[QT][2];
#pragma unroll
        for (int t = 0; t < QT; ++t)
#pragma unroll
            for (int nt = 0; nt < 2; ++nt) st[t][nt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int nt = 0; nt < 2; ++nt) {
                const bf16x8_t kf = __builtin_bit_cast(
                    bf16x8_t, *reinterpret_cast<const u32x4_t*>(&kt[(16 * nt + l16) * KSTRIDE + 32 * ks + 8 * g]));
#pragma unroll
                for (int t = 0; t < QT; ++t)
                    st[t][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[t][ks], st[t][nt], 0, 0, 0);
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
                    for (int r = 0; r < 4; ++r) {
                        float v = st[t][nt][r];
                        if constexpr (kMask) v = j0 + 16 * nt + 4 * g + r < my_len[t] ? v : -INFINITY;
                        s[4 * nt + r] = v;
                        m_new = fmaxf(m_new, v);
                    }
                m_new = rows_max(m_new);
                const float safe = m_new == -INFINITY ? 0.f : m_new;
                const float off = -safe * a.scale_log2e;
                const float alpha = __builtin_amdgcn_exp2f(fmaf(mx[t], a.scale_log2e, off));
                mx[t] = m_new;
                float sum = 0.f;
                uint32_t hi[4], lo[4];
#pragma unroll
                for (int e = 0; e < 8; e += 2) {
                    const float p0 = __builtin_amdgcn_exp2f(fmaf(s[e], a.scale_log2e, off));
                    const float p1 = __builtin_amdgcn_exp2f(fmaf(s[e + 1], a.scale_log2e, off));
                    sum += p0 + p1;
                    const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
                    hi[e >> 1] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
                    lo[e >> 1] = pack_bf16x2(p0 - __uint_as_float(u0 & 0xFFFF0000u), p1 - __uint_as_float(u1 & 0xFFFF0000u));
                }
                p_hi[t] = __builtin_bit_cast(bf16x8_t, u32x4_t{hi[0], hi[1], hi[2], hi[3]});
                p_lo[t] = __builtin_bit_cast(bf16x8_t, u32x4_t{lo[0], lo[1], lo[2], lo[3]});
                lsum[t] = lsum[t] * alpha + sum;
                if (__any(alpha != 1.0f)) {
#pragma unroll
                    for (int dt = 0; dt < DT; ++dt) acc[t][dt] *= alpha;
                }
            }
        };
        if (j0 + kStep <= wave_min) softmax(std::false_type{});
        else softmax(std::true_type{});
        // (the score accumulator holds keys 4g.. and 16 + 4g..: the order the two transposing reads give)
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            const uint16_t* va = &vt[(4 * g + (l16 >> 2)) * VSTRIDE + 16 * dt + 4 * (l16 & 3)];
            const bf16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va));
            const bf16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4_t*)(va + 16 * VSTRIDE));
            const bf16x8_t vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_hi[t], acc[t][dt], 0, 0, 0);
                acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p_lo[t], acc[t][dt], 0, 0, 0);
            }
        }
    };
    // Step j reads buffer j % 2; it first stages step j + 1 (whose buffer's readers passed the last
    // barrier) and refills that register slot with step j + 3.
    auto step = [&](int slot, int j0) {
        if (j0 + kStep < kmax) stage(slot ^ 1);
        if (j0 + 3 * kStep < kmax) issue(slot ^ 1, j0 + 3 * kStep);
        if (j0 < wave_max) compute(slot, j0);
        __syncthreads();
    };
    if (kmax > 0) issue(0, 0);
    if (kmax > kStep) issue(1, kStep);
    if (kmax > 0) stage(0);
    if (kmax > 2 * kStep) issue(0, 2 * kStep);
    __syncthreads();
    for (int j0 = 0; j0 < kmax; j0 += 2 * kStep) {
        step(0, j0);
        if (j0 + kStep < kmax) step(1, j0 + kStep);
    }

#pragma unroll
    for (int t = 0; t < QT; ++t) {
        float l = lsum[t];
        l += __shfl_xor(l, 16, kWave);
        l += __shfl_xor(l, 32, kWave);
        const int m = wv * 16 * QT + t * 16 + l16;
        if (m >= rows) continue;
        float inv = l > 0.f ? 1.f / l : 0.f;
        if (a.sinks) {   // (in the units of the larger of the two)
            const float m2 = mx[t] * a.scale_log2e, sink = a.sinks[h] * 1.4426950408889634f;
            const float top = fmaxf(m2, sink), w = exp2f(m2 - top);
            inv = w / (l * w + exp2f(sink - top));
        }
        if (a.gate && a.gate_cols == 1)
            inv *= sigmoid_f32(bf16_bits_to_f32(a.gate[static_cast<size_t>(a.row0 + t0 + m) * a.ld_gate + h]));
        uint16_t* op = a.o + static_cast<size_t>(a.row0 + t0 + m) * a.ld_o + h * DV + 4 * g;
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            f32x4_t v = acc[t][dt] * inv;
            if (a.gate && a.gate_cols != 1) {
                const u32x2_t r = *reinterpret_cast<const u32x2_t*>(a.gate + static_cast<size_t>(a.row0 + t0 + m) * a.ld_gate + h * DV + 4 * g + 16 * dt);
                v *= f32x4_t{sigmoid_f32(bf16_lo(r.x)), sigmoid_f32(bf16_hi(r.x)), sigmoid_f32(bf16_lo(r.y)), sigmoid_f32(bf16_hi(r.y))};
            }
            *reinterpret_cast<u32x2_t*>(op + 16 * dt) = u32x2_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
        }
    }
}

template <int KS, int VT>
int launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t s) {
    // (fewer than two 128-token blocks per CU: 64-token blocks)
    const int t2 = (a.num_rows + 127) / 128, t1 = (a.num_rows + 63) / 64;
    if (static_cast<long long>(t2) * a.heads >= 512)
        hipLaunchKernelGGL((latent_prefill_kernel<KS, VT, 2>), dim3(a.heads, t2), dim3(kBlock), 0, s, a);
    else
        hipLaunchKernelGGL((latent_prefill_kernel<KS, VT, 1>), dim3(a.heads, t1), dim3(kBlock), 0, s, a);
    return launch_status();
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_latent_gather(const uint16_t* pool, const uint32_t* pages, uint16_t* lat, uint16_t* rot,
                                     int num_keys, int kvp, int rotp, int page_size, void* stream) {
    if (!pool || !pages || !lat || (!rot && rotp > 0) || num_keys <= 0 || kvp <= 0 || rotp < 0 || page_size <= 0) return PIE_HIP_ERR_INVALID;
    if (kvp % 8 != 0 || rotp % 8 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const size_t pieces = static_cast<size_t>(num_keys) * ((kvp + rotp) / 8);
    const size_t blocks = (pieces + 255) / 256;
    hipLaunchKernelGGL(latent_gather_kernel, dim3(static_cast<unsigned>(blocks < 4096 ? blocks : 4096)), dim3(256), 0,
                       static_cast<hipStream_t>(stream), pool, pages, lat, rot, num_keys, kvp, rotp, page_size);
    return launch_status();
}

extern "C" int pie_hip_latent_attn_prefill_supported(int dimp, int rotp, int vdp) {
    const int ks = (dimp + rotp) / 32, vt = vdp / 32;
    return dimp > 0 && rotp >= 0 && dimp % 32 == 0 && rotp % 32 == 0 && vdp % 32 == 0 && ks >= 1 && ks <= 6 && vt >= 1 && vt <= 4;
}

extern "C" int pie_hip_latent_attn_prefill(const uint16_t* q, const uint16_t* kv, const uint16_t* rot, uint16_t* o,
                                           const float* rope_table, const int32_t* row_kv_len, int row0, int num_rows,
                                           int num_keys, int heads, int dimp, int rotp, int rot_dims, int vdp, int ld_o,
                                           float scale, const float* sinks, const uint16_t* gate, int ld_gate, int gate_cols,
                                           void* stream) {
    if (!q || !kv || (!rot && rotp > 0) || !o || !row_kv_len || row0 < 0 || num_rows <= 0 || num_keys <= 0 || heads <= 0 ||
        (rot_dims > 0 && !rope_table) || rot_dims > rotp || rot_dims % 2 != 0 || ld_o < heads * vdp ||
        (gate && ((gate_cols != 1 && gate_cols != vdp) || ld_gate < heads * gate_cols)) ||
        (gate && gate_cols == vdp && (ld_gate % 4 != 0 || reinterpret_cast<uintptr_t>(gate) % 8 != 0)))
        return PIE_HIP_ERR_INVALID;
    if (!pie_hip_latent_attn_prefill_supported(dimp, rotp, vdp) || ld_o % 8 != 0 || num_rows > 64 * 65535) return PIE_HIP_ERR_UNSUPPORTED;
    const LatentPrefillArgs a{q, kv, rot, o, rope_table, row_kv_len, row0, num_rows, heads, dimp, rotp, rot_dims, ld_o,
                              scale * 1.4426950408889634f, sinks, gate, ld_gate, gate_cols};
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int ks = (dimp + rotp) / 32, vt = vdp / 32;
#define PIE_PREFILL_CASE(KK, VV) \
    if (ks == KK && vt == VV) return launch_latent_prefill<KK, VV>(a, s);
#define PIE_PREFILL_ROW(KK) PIE_PREFILL_CASE(KK, 1) PIE_PREFILL_CASE(KK, 2) PIE_PREFILL_CASE(KK, 3) PIE_PREFILL_CASE(KK, 4)
    PIE_PREFILL_ROW(1) PIE_PREFILL_ROW(2) PIE_PREFILL_ROW(3) PIE_PREFILL_ROW(4) PIE_PREFILL_ROW(5) PIE_PREFILL_ROW(6)
#undef PIE_PREFILL_ROW
#undef PIE_PREFILL_CASE
    return PIE_HIP_ERR_UNSUPPORTED;
}
