// Activation storage of the layer-stack kernels: bf16 bits or fp32, fp32 maths either way.
#pragma once

#include "common.hip.h"

namespace pie_hip {

template <class T>
struct ActType;
template <>
struct ActType<uint16_t> {
    static __device__ __forceinline__ float get(uint16_t v) { return bf16_bits_to_f32(v); }
    static __device__ __forceinline__ uint16_t put(float v) { return f32_to_bf16_bits(v); }
};
template <>
struct ActType<float> {
    static __device__ __forceinline__ float get(float v) { return v; }
    static __device__ __forceinline__ float put(float v) { return v; }
};
template <class T>
__device__ __forceinline__ float act_get(T v) {
    return ActType<T>::get(v);
}
template <class T>
__device__ __forceinline__ T act_put(float v) {
    return ActType<T>::put(v);
}

// eight (bf16) or four (fp32) consecutive elements of a 16-byte aligned address
template <class T>
struct ActVec;
template <>
struct ActVec<uint16_t> {
    static constexpr int kN = 8;
    static __device__ __forceinline__ void load(const uint16_t* p, float* f) {
        const u32x4_t r = *reinterpret_cast<const u32x4_t*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            f[2 * i] = bf16_lo(r[i]);
            f[2 * i + 1] = bf16_hi(r[i]);
        }
    }
};
template <>
struct ActVec<float> {
    static constexpr int kN = 4;
    static __device__ __forceinline__ void load(const float* p, float* f) {
        const f32x4_t r = *reinterpret_cast<const f32x4_t*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) f[i] = r[i];
    }
};

// Eight values at a time, still in the compute type.
template <class T>
struct Eight {
    u32x4_t r[sizeof(T) / 2];
    __device__ __forceinline__ void load(const T* p) {
#pragma unroll
        for (int h = 0; h < static_cast<int>(sizeof(T)) / 2; ++h) r[h] = reinterpret_cast<const u32x4_t*>(p)[h];
    }
    __device__ __forceinline__ float get(int e) const {
        if constexpr (sizeof(T) == 2) return e & 1 ? bf16_hi(r[0][e / 2]) : bf16_lo(r[0][e / 2]);
        else return __uint_as_float(r[e / 4][e % 4]);
    }
};
// (rounded to the compute type; p 16-byte aligned)
template <class T>
__device__ __forceinline__ void store_eight(T* p, const float (&v)[8]) {
    if constexpr (sizeof(T) == 2) {
        *reinterpret_cast<u32x4_t*>(p) = u32x4_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7])};
    } else {
#pragma unroll
        for (int h = 0; h < 2; ++h) *reinterpret_cast<f32x4_t*>(p + 4 * h) = f32x4_t{v[4 * h], v[4 * h + 1], v[4 * h + 2], v[4 * h + 3]};
    }
}
constexpr int kJoinRoutes = 64;   // places and weights of a token's routes through a mixture wait in LDS

// (the bare exponential and reciprocal: a few units in the last place)
__device__ __forceinline__ float sigmoid_f32(float z) {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

// Sum over a block of up to 1024 threads (a multiple of 64); every thread gets the total.
// `smem`: one float per wave.
__device__ __forceinline__ float block_total(float v, float* smem) {
    v = wave_sum(v);
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int nw = blockDim.x / kWave;
    __syncthreads();
    if (lane == 0) smem[wv] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < nw; ++i) t += smem[i];
    return t;
}

// dtype argument of the C entry points -> a call of F<T>::run
#define PIE_ACT_DISPATCH(dtype, T, ...)                     \
    do {                                                    \
        if ((dtype) == PIE_HIP_DT_BF16) {                   \
            using T = uint16_t;                             \
            __VA_ARGS__;                                    \
        } else if ((dtype) == PIE_HIP_DT_F32) {             \
            using T = float;                                \
            __VA_ARGS__;                                    \
        } else {                                            \
            return PIE_HIP_ERR_INVALID;                     \
        }                                                   \
    } while (0)

}  // namespace pie_hip
