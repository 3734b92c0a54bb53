// Register rows shared by the block-level kernels: V consecutive elements of a row as floats, reductions over the
// threads of a row, and the activations in the accuracy the element type asks for.
#pragma once
#include "pa_common.h"

template <int V> __device__ __forceinline__ void row_fill(float *f, float v) {
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] = v;
}
template <int V> __device__ __forceinline__ void row_zero(float *f) { row_fill<V>(f, 0.f); }

// V elements from memory (one load of V * sizeof(T) bytes for V = 4 and 8; the caller guarantees the alignment).
template <typename T, int V> __device__ __forceinline__ void row_load(const T *p, float *f) {
    if constexpr (V == 1) {
        f[0] = pa_scalar<T>::load(p);
    } else if constexpr (sizeof(T) == 4) {
#pragma unroll
        for (int i = 0; i < V / 4; ++i) pa_vec16<T>::unpack(reinterpret_cast<const uint4 *>(p)[i], f + 4 * i);
    } else if constexpr (V == 8) {
        pa_vec16<T>::unpack(*reinterpret_cast<const uint4 *>(p), f);
    } else {
        static_assert(V == 4, "four or eight 16-bit elements");
        const uint2 r = *reinterpret_cast<const uint2 *>(p);
        f[0] = __builtin_bit_cast(float, r.x << 16);
        f[1] = __builtin_bit_cast(float, r.x & 0xffff0000u);
        f[2] = __builtin_bit_cast(float, r.y << 16);
        f[3] = __builtin_bit_cast(float, r.y & 0xffff0000u);
    }
}

__device__ __forceinline__ uint32_t row_pack_bf16(float lo, float hi) {
    typedef __bf16 bf2 __attribute__((ext_vector_type(2)));
    const bf2 pair = {(__bf16)lo, (__bf16)hi};
    return __builtin_bit_cast(uint32_t, pair);
}

template <typename T, int V> __device__ __forceinline__ void row_store(T *p, const float *f) {
    if constexpr (V == 1) {
        pa_scalar<T>::store(p, f[0]);
    } else if constexpr (sizeof(T) == 4) {
#pragma unroll
        for (int i = 0; i < V / 4; ++i)
            reinterpret_cast<float4 *>(p)[i] = make_float4(f[4 * i], f[4 * i + 1], f[4 * i + 2], f[4 * i + 3]);
    } else if constexpr (V == 8) {
        *reinterpret_cast<uint4 *>(p) = make_uint4(row_pack_bf16(f[0], f[1]), row_pack_bf16(f[2], f[3]),
                                                   row_pack_bf16(f[4], f[5]), row_pack_bf16(f[6], f[7]));
    } else {
        *reinterpret_cast<uint2 *>(p) = make_uint2(row_pack_bf16(f[0], f[1]), row_pack_bf16(f[2], f[3]));
    }
}

// Sum over the TPR threads of a row (part of a wave, a wave, or the whole workgroup of 256 through `red`, 8 floats of LDS).
template <int TPR> __device__ __forceinline__ float row_sum(float x, float *red) {
    x = pa_group_sum<(TPR < 64 ? TPR : 64)>(x);
    if constexpr (TPR > 64) {
        __syncthreads();  // the previous sum has been read
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
        __syncthreads();
        x = red[0] + red[1] + red[2] + red[3];
    }
    return x;
}

// 1 / (1 + exp(-x)): to float accuracy for 32-bit tensors, with the hardware's exponential and reciprocal for 16-bit.
template <typename T> __device__ __forceinline__ float row_sigmoid(float x) {
    if constexpr (sizeof(T) == 4) return 1.f / (1.f + expf(-x));
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}
template <typename T> __device__ __forceinline__ float row_silu(float x) { return x * row_sigmoid<T>(x); }
// 0.5 x (1 + tanh(a)) = x * sigmoid(2 a), a = sqrt(2/pi) (x + 0.044715 x^3)
template <typename T> __device__ __forceinline__ float row_gelu_tanh(float x) {
    const float a = 0.7978845608028654f * fmaf(0.044715f * x * x, x, x);
    return x * row_sigmoid<T>(2.f * a);
}
