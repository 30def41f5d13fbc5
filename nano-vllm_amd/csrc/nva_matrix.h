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

// global -> LDS without a register in between: lane l's 16 bytes at base + voff land at LDS byte
// address lds_addr + 16 l.  Written as inline assembly on purpose: the compiler would make every
// LDS read that follows its own builtin wait for the load (it cannot tell the two LDS buffers
// apart), which would serialise the prefetch of the next tile with the arithmetic of this one.
// The caller waits with s_waitcnt vmcnt(0) before the barrier that publishes the tile.
// (s_nop 0: the load needs one wait state after the write of m0, which the compiler cannot provide
// for an instruction it does not see.  Its scalar operands are always results of scalar
// arithmetic; one written by a vector instruction -- v_readfirstlane -- would need five.)
__device__ __forceinline__ void load_to_lds_16(const void *base, uint32_t &voff, uint32_t lds_addr) {
    // Not volatile, and the offset register is declared as written although it keeps its value: the
    // statement is then an ordinary instruction that the scheduler may place anywhere between the
    // computation of its operands and the next use of the offset (a volatile statement is a fence
    // for every LDS read and cuts the block into separately scheduled pieces).  The loads of one
    // tensor form a chain through the offset; loads_issued() ends the chains before the wait.
    asm("s_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, %1"
        : "+v"(voff) : "s"(base), "s"(lds_addr) : "m0");
}
__device__ __forceinline__ void loads_issued(uint32_t koff, uint32_t voff) { asm volatile("" :: "v"(koff), "v"(voff)); }

}  // namespace nva
