// Matrix-core helpers of the mixers' bf16 kernels: v_mfma_f32_16x16x32_bf16 operands and LDS pointers.
// Operand A: lane l holds row l % 16, inner indices 8 (l / 16) + [0, 8); B the same for columns; C: lane l holds
// column l % 16, rows 4 (l / 16) + [0, 4).  Any order of the inner indices will do that A and B share.
#pragma once

#include "nva_common.h"

namespace nva {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));
typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef short s16x8_t __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) char *lds_char_ptr;
typedef __attribute__((address_space(3))) u32x4_t *lds_u32x4_ptr;
typedef __attribute__((address_space(3))) s16x4_t *lds_s16x4_ptr;

__device__ __forceinline__ bf16x8_t as_bf16x8(const u32x4_t &u) { return __builtin_bit_cast(bf16x8_t, u); }
__device__ __forceinline__ f32x4_t mfma16(const u32x4_t &x, const u32x4_t &y, const f32x4_t &c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(x), as_bf16x8(y), c, 0, 0, 0);
}
// a pair of floats as the sum of two bf16 pairs
__device__ __forceinline__ void split_pair(float a, float b, uint32_t &hi, uint32_t &lo) {
    hi = pack_bf16x2(a, b);
    lo = pack_bf16x2(a - bf16lo_to_f32(hi), b - bf16hi_to_f32(hi));
}
// value rounded to bf16 pieces of eight: v = hi + lo to 16 bits of mantissa
__device__ __forceinline__ void split8(const float (&v)[8], u32x4_t &hi, u32x4_t &lo) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        uint32_t h, l;
        split_pair(v[2 * i], v[2 * i + 1], h, l);
        hi[i] = h;
        lo[i] = l;
    }
}

}  // namespace nva
