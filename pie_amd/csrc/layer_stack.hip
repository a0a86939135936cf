// The kernels every layer of a layer-stack model shares: embedding into an fp32 residual stream,
// the norm-and-add that ends a sublayer, the join of sublayers that share a norm, the output norm, the
// logit finish (scale, soft cap, argmax), the rotation table, and the fp32 linears of the 32-bit compute
// type.
//
// The residual stream x is fp32 [rows, ld]; the activations the products read are a copy of it in
// the compute type, written by the kernel that last changed x, so no product starts with a
// conversion.  Columns from the width to ld are zero in both.
#include "act_type.hip.h"

namespace pie_hip {
namespace {

template <class T>
__global__ __launch_bounds__(1024) void embed_stream_kernel(const uint32_t* __restrict__ tokens,
                                                            const uint16_t* __restrict__ table,
                                                            float* __restrict__ x, T* __restrict__ xa, int width,
                                                            int ld, int vocab) {
    const int n = blockIdx.x;
    const uint32_t t = tokens[n];
    const size_t row = t < static_cast<uint32_t>(vocab) ? t : 0;
    for (int i = 4 * threadIdx.x; i < ld; i += 4 * blockDim.x) {   // (ld is a multiple of 4)
        f32x4_t v = {0.f, 0.f, 0.f, 0.f};
        if (i + 4 <= width && width % 4 == 0) {
            const u32x2_t r = *reinterpret_cast<const u32x2_t*>(table + row * width + i);
            v = f32x4_t{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)};
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (i + e < width) v[e] = bf16_bits_to_f32(table[row * width + i + e]);
        }
        *reinterpret_cast<f32x4_t*>(x + static_cast<size_t>(n) * ld + i) = v;
#pragma unroll
        for (int e = 0; e < 4; ++e) xa[static_cast<size_t>(n) * ld + i + e] = act_put<T>(v[e]);
    }
}

// x += y / sqrt(mean(y^2) + eps) * w, and the compute-type copy of the new x.  One block per row;
// a thread keeps the first kCache of its elements in registers between the two passes, requested
// together with x and w so that the row waits for memory once.
template <class T, int BLOCK>
__global__ __launch_bounds__(BLOCK) void norm_add_kernel(const T* __restrict__ y, const float* __restrict__ w,
                                                       float* __restrict__ x, T* __restrict__ xa, int width, int ldy,
                                                       int ld, float eps) {
    __shared__ float red[BLOCK / kWave];
    const size_t n = blockIdx.x;
    const T* yr = y + n * ldy;
    float* xr = x + n * ld;
    T* ar = xa + n * ld;
    constexpr int kCache = 8;   // groups of four
    f32x4_t yv[kCache], xv[kCache], wv[kCache];
    float local = 0.f;
    const int n4 = width / 4;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * BLOCK;
        if (i < n4) {
            if constexpr (sizeof(T) == 2) {
                const u32x2_t r = *reinterpret_cast<const u32x2_t*>(yr + 4 * i);
                yv[c] = f32x4_t{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)};
            } else {
                yv[c] = *reinterpret_cast<const f32x4_t*>(yr + 4 * i);
            }
            xv[c] = *reinterpret_cast<const f32x4_t*>(xr + 4 * i);
            wv[c] = *reinterpret_cast<const f32x4_t*>(w + 4 * i);
        }
    }
#pragma unroll
    for (int c = 0; c < kCache; ++c)
        if (threadIdx.x + c * BLOCK < n4)
#pragma unroll
            for (int e = 0; e < 4; ++e) local += yv[c][e] * yv[c][e];
    const int done = min(n4, kCache * BLOCK) * 4;   // the rest: wider rows and a width's last one to three
    for (int i = done + threadIdx.x; i < width; i += BLOCK) {
        const float v = act_get<T>(yr[i]);
        local += v * v;
    }
    const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(width) + eps);
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * BLOCK;
        if (i < n4) {
            f32x4_t o;
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = xv[c][e] + yv[c][e] * inv * wv[c][e];
            *reinterpret_cast<f32x4_t*>(xr + 4 * i) = o;
            if constexpr (sizeof(T) == 2)
                *reinterpret_cast<u32x2_t*>(ar + 4 * i) = u32x2_t{pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
            else *reinterpret_cast<f32x4_t*>(ar + 4 * i) = o;
        }
    }
    for (int i = done + threadIdx.x; i < width; i += BLOCK) {
        const float v = xr[i] + act_get<T>(yr[i]) * inv * w[i];
        xr[i] = v;
        ar[i] = act_put<T>(v);
    }
}

// Layers with norms ahead of and after their sublayers: x takes a sublayer's normed output and whatever
// else enters the stream (a row of the embedding table, a vector), and its compute-type copy is normed
// for the next sublayer.  One block per row, up to 8192 values of the row in registers between the
// passes; wider rows go through memory again.
struct ResidualArgs {
    const void* y;
    const float *post_w, *add, *next_w;
    float* x;
    const uint32_t* tokens;
    const uint16_t* table;
    void* xa;
    int read_x, vocab, width, ldy, ld;
    float eps;
};
template <class T, int BLOCK>
__global__ __launch_bounds__(BLOCK) void residual_norm_kernel(const ResidualArgs a) {
    __shared__ float red[BLOCK / kWave];
    const size_t n = blockIdx.x;
    const T* yr = a.y ? static_cast<const T*>(a.y) + n * a.ldy : nullptr;
    float* xr = a.x + n * a.ld;
    T* ar = static_cast<T*>(a.xa) + n * a.ld;
    const uint16_t* er = nullptr;
    if (a.tokens) {
        const uint32_t t = a.tokens[n];
        er = a.table + static_cast<size_t>(t < static_cast<uint32_t>(a.vocab) ? t : 0) * a.width;
    }
    constexpr int kCache = 2048 / BLOCK;   // groups of four
    const int n4 = a.width % 4 == 0 ? a.width / 4 : 0;   // (a table row of another width is not aligned)
    const int done = min(n4, kCache * BLOCK) * 4;
    f32x4_t yv[kCache], xv[kCache], wv[kCache], nv[kCache];
    const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
    float local = 0.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * BLOCK;
        if (i >= n4) break;
        yv[c] = wv[c] = zero;
        if (yr) {
            if constexpr (sizeof(T) == 2) {
                const u32x2_t r = *reinterpret_cast<const u32x2_t*>(yr + 4 * i);
                yv[c] = f32x4_t{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)};
            } else {
                yv[c] = *reinterpret_cast<const f32x4_t*>(yr + 4 * i);
            }
            wv[c] = *reinterpret_cast<const f32x4_t*>(a.post_w + 4 * i);
        }
        xv[c] = a.read_x ? *reinterpret_cast<const f32x4_t*>(xr + 4 * i) : zero;
        if (er) {
            const u32x2_t r = *reinterpret_cast<const u32x2_t*>(er + 4 * i);
            xv[c] += f32x4_t{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)};
        }
        if (a.next_w) nv[c] = *reinterpret_cast<const f32x4_t*>(a.next_w + 4 * i);
    }
    auto other = [&](int i) {   // what joins x besides the sublayer's output, beyond the cached part
        return (a.read_x ? xr[i] : 0.f) + (er ? bf16_bits_to_f32(er[i]) : 0.f) + (a.add ? a.add[i] : 0.f);
    };
    float inv = 0.f;
    if (yr) {
#pragma unroll
        for (int c = 0; c < kCache; ++c)
            if (threadIdx.x + c * BLOCK < n4)
#pragma unroll
                for (int e = 0; e < 4; ++e) local += yv[c][e] * yv[c][e];
        for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {
            const float v = act_get<T>(yr[i]);
            local += v * v;
        }
        inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(a.width) + a.eps);
    }
    local = 0.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * BLOCK;
        if (i >= n4) break;
        if (a.add) xv[c] += *reinterpret_cast<const f32x4_t*>(a.add + 4 * i);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            xv[c][e] += yv[c][e] * inv * wv[c][e];
            local += xv[c][e] * xv[c][e];
        }
        *reinterpret_cast<f32x4_t*>(xr + 4 * i) = xv[c];
    }
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {
        const float v = other(i) + (yr ? act_get<T>(yr[i]) * inv * a.post_w[i] : 0.f);
        xr[i] = v;
        local += v * v;
    }
    const float scale = a.next_w ? 1.f / sqrtf(block_total(local, red) / static_cast<float>(a.width) + a.eps) : 1.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * BLOCK;
        if (i >= n4) break;
        f32x4_t o = xv[c];
        if (a.next_w)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] *= scale * nv[c][e];
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<u32x2_t*>(ar + 4 * i) = u32x2_t{pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
        else *reinterpret_cast<f32x4_t*>(ar + 4 * i) = o;
    }
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK)   // (a thread reads what it wrote)
        ar[i] = act_put<T>(a.next_w ? xr[i] * scale * a.next_w[i] : xr[i]);
}

// Layers whose sublayers read one norm: x takes what they give together — up to two rows, a vector, a
// token's routes through a mixture, a row of the embedding table — and its compute-type copy is normed for
// the next layer.  One block per row, as above.
struct JoinArgs {
    const void *y, *y2;
    const float *add, *next_w;
    PieHipRoutes routes;
    float* x;
    const uint32_t* tokens;
    const uint16_t* table;
    void* xa;
    int ldy, ldy2, read_x, vocab, width, ld;
    float table_scale, eps;
};
template <class T, int BLOCK>
__global__ __launch_bounds__(BLOCK) void residual_join_kernel(const JoinArgs a) {
    __shared__ float red[BLOCK / kWave];
    __shared__ int pos[kJoinRoutes];
    __shared__ float weight[kJoinRoutes];
    const size_t n = blockIdx.x;
    const T* yr = a.y ? static_cast<const T*>(a.y) + n * a.ldy : nullptr;
    const T* y2r = a.y2 ? static_cast<const T*>(a.y2) + n * a.ldy2 : nullptr;
    float* xr = a.x + n * a.ld;
    T* ar = static_cast<T*>(a.xa) + n * a.ld;
    const uint16_t* er = nullptr;
    if (a.tokens) {
        const uint32_t t = a.tokens[n];
        er = a.table + static_cast<size_t>(t < static_cast<uint32_t>(a.vocab) ? t : 0) * a.width;
    }
    const int K = a.routes.y ? a.routes.top_k : 0;
    const T* ry = static_cast<const T*>(a.routes.y);
    if (K) {
        if (threadIdx.x < static_cast<unsigned>(K)) {
            pos[threadIdx.x] = a.routes.pos[n * K + threadIdx.x];
            weight[threadIdx.x] = a.routes.weight[n * K + threadIdx.x];
        }
        __syncthreads();
    }
    constexpr int kCache = 8192 / (8 * BLOCK);   // groups of eight
    const int n8 = a.width % 8 == 0 ? a.width / 8 : 0;
    const int done = min(n8, kCache * BLOCK) * 8;
    float v[kCache][8];
    float local = 0.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = 8 * (threadIdx.x + c * BLOCK);
        if (i >= 8 * n8) break;
        // (what a group reads is requested before any of it is used; the sublayers' sum first, then the stream)
        Eight<T> g1, g2;
        Eight<uint16_t> ge;
        Eight<float> gx, gadd;
        if (yr) g1.load(yr + i);
        if (y2r) g2.load(y2r + i);
        if (er) ge.load(er + i);
        if (a.read_x) gx.load(xr + i);
        if (a.add) gadd.load(a.add + i);
        float (&s)[8] = v[c];
#pragma unroll
        for (int e = 0; e < 8; ++e) s[e] = 0.f;
        if (yr)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e] += g1.get(e);
        if (y2r)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e] += g2.get(e);
        if (a.add)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e] += gadd.get(e);
        for (int k0 = 0; k0 < K; k0 += 8) {
            Eight<T> r[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) r[u].load(ry + static_cast<size_t>(pos[min(k0 + u, K - 1)]) * a.routes.ld + i);
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                const float w = k0 + u < K ? weight[min(k0 + u, K - 1)] : 0.f;
                if (k0 + u < K)
#pragma unroll
                    for (int e = 0; e < 8; ++e) s[e] = fmaf(r[u].get(e), w, s[e]);
            }
        }
        if (er)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e] = fmaf(ge.get(e), a.table_scale, s[e]);
        if (a.read_x)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e] += gx.get(e);
#pragma unroll
        for (int e = 0; e < 8; ++e) local += s[e] * s[e];
#pragma unroll
        for (int h = 0; h < 2; ++h)
            *reinterpret_cast<f32x4_t*>(xr + i + 4 * h) = f32x4_t{s[4 * h], s[4 * h + 1], s[4 * h + 2], s[4 * h + 3]};
    }
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK) {
        float s = 0.f;
        if (yr) s += act_get<T>(yr[i]);
        if (y2r) s += act_get<T>(y2r[i]);
        if (a.add) s += a.add[i];
        for (int k = 0; k < K; ++k) s += act_get<T>(ry[static_cast<size_t>(pos[k]) * a.routes.ld + i]) * weight[k];
        if (er) s += bf16_bits_to_f32(er[i]) * a.table_scale;
        if (a.read_x) s += xr[i];
        xr[i] = s;
        local += s * s;
    }
    const float scale = a.next_w ? 1.f / sqrtf(block_total(local, red) / static_cast<float>(a.width) + a.eps) : 1.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = 8 * (threadIdx.x + c * BLOCK);
        if (i >= 8 * n8) break;
        float (&o)[8] = v[c];
        if (a.next_w) {
            Eight<float> w;
            w.load(a.next_w + i);
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] *= w.get(e) * scale;
        }
        store_eight<T>(ar + i, o);
    }
    for (int i = done + threadIdx.x; i < a.width; i += BLOCK)   // (a thread reads what it wrote)
        ar[i] = act_put<T>(a.next_w ? xr[i] * (scale * a.next_w[i]) : xr[i]);
}

// y = act . W^T with fp32 outputs: the waves of a block share the K of a row tile and NT column tiles, each
// requesting U of its k-steps at once.
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
template <int WAVES, int NT, int U>
__global__ __launch_bounds__(WAVES* kWave) void linear_f32out_kernel(const uint16_t* __restrict__ act,
                                                                     const uint16_t* __restrict__ w, float* __restrict__ y,
                                                                     int M, int N, int K) {
    __shared__ __attribute__((aligned(16))) float part[NT][WAVES][kWave * 4];
    const int n0 = blockIdx.x * 16 * NT, m0 = blockIdx.y * 16, lane = threadIdx.x & (kWave - 1), l16 = lane & 15, g = lane >> 4;
    const int wv = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
    const uint16_t* ap = act + static_cast<size_t>(min(m0 + l16, M - 1)) * K + 8 * g;
    const uint16_t* wp[NT];
    f32x4_t acc[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        wp[t] = w + static_cast<size_t>(min(n0 + 16 * t, N - 16) + l16) * K + 8 * g;   // (a tile past N repeats the last one)
        acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    const int steps = K / 32;
    for (int s0 = wv; s0 < steps; s0 += U * WAVES) {
        u32x4_t a[U], b[NT][U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = 32 * min(s0 + u * WAVES, steps - 1);
            a[u] = *reinterpret_cast<const u32x4_t*>(ap + k);
#pragma unroll
            for (int t = 0; t < NT; ++t) b[t][u] = *reinterpret_cast<const u32x4_t*>(wp[t] + k);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (s0 + u * WAVES < steps)
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, b[t][u]), __builtin_bit_cast(bf16x8_t, a[u]), acc[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4_t*>(&part[t][wv][lane * 4]) = acc[t];
    __syncthreads();
    if (wv >= NT || n0 + 16 * wv >= N) return;   // wave t adds tile t up
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < WAVES; ++i) v += *reinterpret_cast<const f32x4_t*>(&part[wv][i][lane * 4]);
    if (m0 + l16 < M) *reinterpret_cast<f32x4_t*>(y + static_cast<size_t>(m0 + l16) * N + n0 + 16 * wv + 4 * g) = v;
}

// out[s] = rmsnorm(x[rows[s]]) * w in the compute type; columns past the width are zero
template <class T>
__global__ __launch_bounds__(1024) void norm_rows_kernel(const float* __restrict__ x, const uint32_t* __restrict__ rows,
                                                         const float* __restrict__ w, T* __restrict__ out, int width,
                                                         int ld, int num_rows, float eps) {
    __shared__ float red[16];
    const size_t s = blockIdx.x;
    const uint32_t r = rows[s];
    const float* xr = x + static_cast<size_t>(r < static_cast<uint32_t>(num_rows) ? r : 0) * ld;
    constexpr int kCache = 8;
    float xv[kCache], wv[kCache], local = 0.f;
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * 1024;
        xv[c] = i < width ? xr[i] : 0.f;
        wv[c] = i < width ? w[i] : 0.f;
    }
#pragma unroll
    for (int c = 0; c < kCache; ++c) local += xv[c] * xv[c];
    for (int i = threadIdx.x + kCache * 1024; i < width; i += 1024) local += xr[i] * xr[i];
    const float inv = 1.f / sqrtf(block_total(local, red) / static_cast<float>(width) + eps);
#pragma unroll
    for (int c = 0; c < kCache; ++c) {
        const int i = threadIdx.x + c * 1024;
        if (i < ld) out[s * ld + i] = act_put<T>(xv[c] * inv * wv[c]);
    }
    for (int i = threadIdx.x + kCache * 1024; i < ld; i += 1024)
        out[s * ld + i] = i < width ? act_put<T>(xr[i] * inv * w[i]) : act_put<T>(0.f);
}

// logits f32 = cap * tanh(y * scale / cap) (cap 0: y * scale), and their argmax (the lowest index
// among equals, NaN never wins).  One block per row.
template <class T>
__global__ __launch_bounds__(1024) void logits_finish_kernel(const T* __restrict__ y, float* __restrict__ logits,
                                                             uint32_t* __restrict__ tokens, int vocab, int ldy,
                                                             float scale, float cap) {
    __shared__ float sv[16];
    __shared__ int si[16];
    const size_t s = blockIdx.x;
    float bv = -INFINITY;
    int bi = 0;
    constexpr int U = 8;   // values requested together
    for (int i0 = threadIdx.x; i0 < vocab; i0 += U * 1024) {
        T raw[U];
#pragma unroll
        for (int u = 0; u < U; ++u) raw[u] = y[s * ldy + min(i0 + u * 1024, vocab - 1)];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = i0 + u * 1024;
            if (i >= vocab) break;
            float v = act_get<T>(raw[u]) * scale;
            if (cap > 0.f) v = cap * tanhf(v / cap);
            logits[s * vocab + i] = v;
            if (v > bv) {   // (indices ascend inside a thread)
                bv = v;
                bi = i;
            }
        }
    }
    auto better = [&](float ov, int oi) {
        if (ov > bv || (ov == bv && oi < bi)) {
            bv = ov;
            bi = oi;
        }
    };
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) better(__shfl_xor(bv, off, kWave), __shfl_xor(bi, off, kWave));
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    if (lane == 0) {
        sv[wv] = bv;
        si[wv] = bi;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int i = 1; i < static_cast<int>(blockDim.x) / kWave; ++i) better(sv[i], si[i]);
        tokens[s] = static_cast<uint32_t>(bi);
    }
}

// table[n, i] = cos(a) * mscale, table[n, half + i] = sin(a) * mscale, a = position * f_i.  The
// angle is formed and reduced in double so that its fp32 value is right to the last bit at any
// position.
__global__ void rotary_table_kernel(const int32_t* __restrict__ positions, const double* __restrict__ freq,
                                    float* __restrict__ table, int half, float mscale) {
    const int n = blockIdx.x;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
        constexpr double kTwoPi = 6.283185307179586476925;
        double a = static_cast<double>(positions[n]) * freq[i];
        a -= rint(a / kTwoPi) * kTwoPi;
        float s, c;
        sincosf(static_cast<float>(a), &s, &c);
        table[static_cast<size_t>(n) * 2 * half + i] = c * mscale;
        table[static_cast<size_t>(n) * 2 * half + half + i] = s * mscale;
    }
}

// y[M, N] = epilogue(act[M, K] fp32 . W[N, K]^T bf16), fp32 products and sums: 64 x 64 tiles of
// 16-wide K steps through LDS, 4 x 4 outputs per thread.
constexpr int kFT = 64, kFK = 16;
// With `offsets` one of several problems (blockIdx.z): rows offsets[z] .. offsets[z + 1] of y, its weights
// N * K further, its rows of act as `act_rows` lists them.
__global__ __launch_bounds__(256) void linear_f32_kernel(const float* __restrict__ act, const uint16_t* __restrict__ w,
                                                         float* __restrict__ y, int M, int N, int K, int pointwise,
                                                         const int32_t* __restrict__ offsets, const int32_t* __restrict__ act_rows) {
    __shared__ float as[kFK][kFT + 4];
    __shared__ float ws[kFK][kFT + 4];
    const int n0 = blockIdx.x * kFT, m0 = blockIdx.y * kFT + (offsets ? offsets[blockIdx.z] : 0);
    if (offsets) {
        M = offsets[blockIdx.z + 1];
        if (m0 >= M) return;
        w += static_cast<size_t>(blockIdx.z) * N * K;
    }
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    const int lr = tid >> 2, lk = (tid & 3) * 4;   // the row and the four k-values this thread stages
    const size_t arow = m0 + lr >= M ? 0 : act_rows ? act_rows[m0 + lr] : m0 + lr;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += kFK) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int k = k0 + lk + e;
            const bool kin = k < K;
            as[lk + e][lr] = kin && m0 + lr < M ? act[arow * K + k] : 0.f;
            ws[lk + e][lr] = kin && n0 + lr < N ? bf16_bits_to_f32(w[static_cast<size_t>(n0 + lr) * K + k]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < kFK; ++k) {
            float a[4], b[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                a[i] = as[k][ty * 4 + i];
                b[i] = ws[k][tx * 4 + i];
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int m = m0 + ty * 4 + i, n = n0 + tx * 4 + j;
            if (m >= M || n >= N) continue;
            float v = acc[i][j];
            if (pointwise == PIE_HIP_EPI_GELU) v = 0.5f * v * (1.f + erff(v * 0.70710678118654752f));
            else v = epilogue_pointwise<false>(v, pointwise);
            y[static_cast<size_t>(m) * N + n] = v;
        }
}

// y[m, i] = the gated rule on columns (2i, 2i + 1) of x
__global__ __launch_bounds__(256) void glu_f32_kernel(const float* __restrict__ x, const PieHipGlu glu, float* __restrict__ y,
                                                      size_t total, int n) {
    const size_t idx = static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x;
    if (idx >= total) return;
    const size_t m = idx / n, i = idx % n;
    float g = x[m * 2 * n + 2 * i], u = x[m * 2 * n + 2 * i + 1];
    if (glu.bias) {
        g += glu.bias[2 * i];
        u += glu.bias[2 * i + 1];
    }
    y[idx] = glu_value(g, u, glu);
}

}  // namespace
}  // namespace pie_hip

using namespace pie_hip;

extern "C" int pie_hip_embed_stream(int dtype, const uint32_t* token_ids, const uint16_t* table_bf16, float* x,
                                    void* x_act, int num_tokens, int width, int ld, int vocab, void* stream) {
    if (!token_ids || !table_bf16 || !x || !x_act || num_tokens <= 0 || width <= 0 || ld < width || vocab <= 0)
        return PIE_HIP_ERR_INVALID;
    if (ld % 4 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const int threads = ld >= 4096 ? 1024 : 256;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(embed_stream_kernel<T>, dim3(num_tokens), dim3(threads), 0,
                                                  static_cast<hipStream_t>(stream), token_ids, table_bf16, x,
                                                  static_cast<T*>(x_act), width, ld, vocab));
    return launch_status();
}

extern "C" int pie_hip_norm_add(int dtype, const void* y, const float* weight, float* x, void* x_act, int rows,
                                int width, int ldy, int ld, float eps, void* stream) {
    if (!y || !weight || !x || !x_act || rows <= 0 || width <= 0 || ldy < width || ld < width) return PIE_HIP_ERR_INVALID;
    if (ldy % 8 != 0 || ld % 8 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    // (few wide rows: wider blocks, so that a row's traffic is in flight at once)
    if (width >= 2048 && rows < 512)
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((norm_add_kernel<T, 1024>), dim3(rows), dim3(1024), 0,
                                                      static_cast<hipStream_t>(stream), static_cast<const T*>(y),
                                                      weight, x, static_cast<T*>(x_act), width, ldy, ld, eps));
    else
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((norm_add_kernel<T, 256>), dim3(rows), dim3(256), 0,
                                                      static_cast<hipStream_t>(stream), static_cast<const T*>(y),
                                                      weight, x, static_cast<T*>(x_act), width, ldy, ld, eps));
    return launch_status();
}

extern "C" int pie_hip_residual_norm(int dtype, const void* y, const float* post_weight, float* x, int read_x,
                                     const uint32_t* token_ids, const uint16_t* table_bf16, int vocab, const float* add,
                                     const float* next_weight, void* x_act, int rows, int width, int ldy, int ld,
                                     float eps, void* stream) {
    if (!x || !x_act || rows <= 0 || width <= 0 || ld < width || (y && (!post_weight || ldy < width)) ||
        (token_ids && (!table_bf16 || vocab <= 0)))
        return PIE_HIP_ERR_INVALID;
    if ((y && ldy % 8 != 0) || ld % 8 != 0) return PIE_HIP_ERR_UNSUPPORTED;
    const ResidualArgs a{y, post_weight, add, next_weight, x, token_ids, table_bf16, x_act, read_x ? 1 : 0, vocab, width, ldy, ld, eps};
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (width >= 2048 && rows < 512)
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((residual_norm_kernel<T, 1024>), dim3(rows), dim3(1024), 0, s, a));
    else
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((residual_norm_kernel<T, 256>), dim3(rows), dim3(256), 0, s, a));
    return launch_status();
}

extern "C" int pie_hip_residual_join(int dtype, const void* y, int ldy, const void* y2, int ldy2, const float* add,
                                     const PieHipRoutes* routes, float* x, int read_x, const uint32_t* token_ids,
                                     const uint16_t* table_bf16, int vocab, float table_scale, const float* next_weight,
                                     void* x_act, int rows, int width, int ld, float eps, void* stream) {
    if (!x || !x_act || rows <= 0 || width <= 0 || ld < width || (y && ldy < width) || (y2 && ldy2 < width) ||
        (token_ids && (!table_bf16 || vocab <= 0)) ||
        (routes && (!routes->y || !routes->pos || !routes->weight || routes->top_k <= 0 || routes->ld < width)))
        return PIE_HIP_ERR_INVALID;
    if ((y && ldy % 8 != 0) || (y2 && ldy2 % 8 != 0) || (routes && (routes->ld % 8 != 0 || routes->top_k > kJoinRoutes)) || ld % 8 != 0)
        return PIE_HIP_ERR_UNSUPPORTED;
    const JoinArgs a{y, y2, add, next_weight, routes ? *routes : PieHipRoutes{}, x, token_ids, table_bf16, x_act, ldy, ldy2,
                     read_x ? 1 : 0, vocab, width, ld, table_scale, eps};
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (width > 2048 && rows < 512)
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((residual_join_kernel<T, 512>), dim3(rows), dim3(512), 0, s, a));
    else
        PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL((residual_join_kernel<T, 256>), dim3(rows), dim3(256), 0, s, a));
    return launch_status();
}

extern "C" int pie_hip_linear_f32out(int dtype, const void* act, const uint16_t* w_bf16, float* y, int M, int N, int K,
                                     void* stream) {
    if (dtype == PIE_HIP_DT_F32)
        return pie_hip_linear_f32(static_cast<const float*>(act), w_bf16, y, M, N, K, PIE_HIP_EPI_NONE, stream);
    if (dtype != PIE_HIP_DT_BF16 || !act || !w_bf16 || !y || M <= 0 || N <= 0 || K <= 0) return PIE_HIP_ERR_INVALID;
    const int gy = (M + 15) / 16;
    if (K % 32 != 0 || N % 16 != 0 || gy > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const auto* x = static_cast<const uint16_t*>(act);
    if (M >= 512 && N > 16)   // (row tiles fill the device: column tiles share their activations)
        hipLaunchKernelGGL((linear_f32out_kernel<8, 4, 8>), dim3((N + 63) / 64, gy), dim3(512), 0, s, x, w_bf16, y, M, N, K);
    else
        hipLaunchKernelGGL((linear_f32out_kernel<16, 1, 8>), dim3(N / 16, gy), dim3(1024), 0, s, x, w_bf16, y, M, N, K);
    return launch_status();
}

extern "C" int pie_hip_norm_rows(int dtype, const float* x, const uint32_t* rows, const float* weight, void* out,
                                 int num_out, int width, int ld, int num_rows, float eps, void* stream) {
    if (!x || !rows || !weight || !out || num_out <= 0 || width <= 0 || ld < width || num_rows <= 0)
        return PIE_HIP_ERR_INVALID;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(norm_rows_kernel<T>, dim3(num_out), dim3(1024), 0,
                                                  static_cast<hipStream_t>(stream), x, rows, weight,
                                                  static_cast<T*>(out), width, ld, num_rows, eps));
    return launch_status();
}

extern "C" int pie_hip_logits_finish(int dtype, const void* y, float* logits, uint32_t* tokens, int rows, int vocab,
                                     int ldy, float scale, float cap, void* stream) {
    if (!y || !logits || !tokens || rows <= 0 || vocab <= 0 || ldy < vocab) return PIE_HIP_ERR_INVALID;
    PIE_ACT_DISPATCH(dtype, T, hipLaunchKernelGGL(logits_finish_kernel<T>, dim3(rows), dim3(1024), 0,
                                                  static_cast<hipStream_t>(stream), static_cast<const T*>(y), logits,
                                                  tokens, vocab, ldy, scale, cap));
    return launch_status();
}

extern "C" int pie_hip_rotary_table(const int32_t* positions, const double* freq, float* table, int num_tokens,
                                    int dims, float mscale, void* stream) {
    if (!positions || !freq || !table || num_tokens <= 0 || dims <= 0 || dims % 2 != 0) return PIE_HIP_ERR_INVALID;
    hipLaunchKernelGGL(rotary_table_kernel, dim3(num_tokens), dim3(64), 0, static_cast<hipStream_t>(stream), positions,
                       freq, table, dims / 2, mscale);
    return launch_status();
}

extern "C" int pie_hip_linear_f32(const float* act, const uint16_t* w_bf16, float* y, int M, int N, int K,
                                  int epilogue, void* stream) {
    if (!act || !w_bf16 || !y || M <= 0 || N <= 0 || K <= 0) return PIE_HIP_ERR_INVALID;
    if (epilogue != PIE_HIP_EPI_NONE && epilogue != PIE_HIP_EPI_RELU2 && epilogue != PIE_HIP_EPI_GELU) return PIE_HIP_ERR_UNSUPPORTED;
    const int gy = (M + kFT - 1) / kFT;
    if (gy > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(linear_f32_kernel, dim3((N + kFT - 1) / kFT, gy), dim3(256), 0, static_cast<hipStream_t>(stream),
                       act, w_bf16, y, M, N, K, pointwise_code(epilogue), nullptr, nullptr);
    return launch_status();
}

extern "C" int pie_hip_moe_grouped_linear_f32(const float* act, const int32_t* route_act_rows, const int32_t* expert_offsets,
                                              int num_experts, int max_rows, const uint16_t* w_bf16, float* y, int N,
                                              int K, int epilogue, void* stream) {
    if (!act || !expert_offsets || !w_bf16 || !y || num_experts <= 0 || max_rows <= 0 || N <= 0 || K <= 0) return PIE_HIP_ERR_INVALID;
    if (epilogue != PIE_HIP_EPI_NONE && epilogue != PIE_HIP_EPI_RELU2 && epilogue != PIE_HIP_EPI_GELU) return PIE_HIP_ERR_UNSUPPORTED;
    const int gy = (max_rows + kFT - 1) / kFT;
    if (gy > 65535 || num_experts > 65535) return PIE_HIP_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(linear_f32_kernel, dim3((N + kFT - 1) / kFT, gy, num_experts), dim3(256), 0, static_cast<hipStream_t>(stream),
                       act, w_bf16, y, 0, N, K, pointwise_code(epilogue), expert_offsets, route_act_rows);
    return launch_status();
}

extern "C" int pie_hip_glu_f32(const float* x, const PieHipGlu* glu, float* y, int M, int n, void* stream) {
    if (!x || !y || M <= 0 || n <= 0 || !glu_ok(glu, PIE_HIP_EPI_SWIGLU)) return PIE_HIP_ERR_INVALID;
    const size_t total = static_cast<size_t>(M) * n;
    if ((total + 255) / 256 > 0x7FFFFFFFull) return PIE_HIP_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(glu_f32_kernel, dim3(static_cast<unsigned>((total + 255) / 256)), dim3(256), 0,
                       static_cast<hipStream_t>(stream), x, glu ? *glu : kPlainGlu, y, total, n);
    return launch_status();
}
