// Element-type helpers of the kernels that exist for bf16 and for fp32 tensors.
#pragma once

#include "nva_common.h"

namespace nva {

template <typename T> struct Elem;
template <> struct Elem<bf16_t> {
    static __device__ __forceinline__ float to_f32(bf16_t v) { return bf16_to_f32(v); }
    static __device__ __forceinline__ bf16_t from_f32(float v) { return f32_to_bf16(v); }
};
template <> struct Elem<float> {
    static __device__ __forceinline__ float to_f32(float v) { return v; }
    static __device__ __forceinline__ float from_f32(float v) { return v; }
};

// V consecutive elements as floats; V is 1 or 8, and 8 elements go in 16-byte pieces
template <typename T, int V>
__device__ __forceinline__ void load_f32(const T *p, float (&f)[V]) {
    if constexpr (V == 8 && sizeof(T) == 2) {
        unpack8(*reinterpret_cast<const uint4 *>(p), f);
    } else if constexpr (V == 8) {
        const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
        f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
        f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) f[i] = Elem<T>::to_f32(p[i]);
    }
}

template <typename T, int V>
__device__ __forceinline__ void store_f32(T *p, const float (&f)[V]) {
    if constexpr (V == 8 && sizeof(T) == 2) {
        uint4 o;
        o.x = pack_bf16x2(f[0], f[1]); o.y = pack_bf16x2(f[2], f[3]);
        o.z = pack_bf16x2(f[4], f[5]); o.w = pack_bf16x2(f[6], f[7]);
        *reinterpret_cast<uint4 *>(p) = o;
    } else if constexpr (V == 8) {
        reinterpret_cast<float4 *>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
        reinterpret_cast<float4 *>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) p[i] = Elem<T>::from_f32(f[i]);
    }
}

// exp, logistic and tanh: the hardware's base-2 exponential and reciprocal (one ulp each) in the bf16
// kernels, the accurate library functions in the fp32 ones
template <typename T> __device__ __forceinline__ float exp_of(float x) {
    if constexpr (sizeof(T) == 2) return __builtin_amdgcn_exp2f(1.4426950408889634f * x);
    else return expf(x);
}
template <typename T> __device__ __forceinline__ float sigmoid_of(float x) {
    if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
    else return 1.0f / (1.0f + expf(-x));
}
template <typename T> __device__ __forceinline__ float tanh_of(float x) {
    if constexpr (sizeof(T) == 2) {
        // 1 - 2 / (1 + e^{2x}); e^{2x} = inf gives 1, e^{2x} = 0 gives -1
        return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.8853900817779268f * x));
    } else {
        return tanhf(x);
    }
}

// ln(1 + x): the hardware's base-2 logarithm of the rounded sum in the bf16 kernels
template <typename T> __device__ __forceinline__ float log1p_of(float x) {
    if constexpr (sizeof(T) == 2) return 0.6931471805599453f * __builtin_amdgcn_logf(1.0f + x);
    else return log1pf(x);
}

inline bool known_dtype(int32_t dtype) { return dtype == NVA_DTYPE_BF16 || dtype == NVA_DTYPE_F32; }
inline int elem_bytes(int32_t dtype) { return dtype == NVA_DTYPE_F32 ? 4 : 2; }

}  // namespace nva
