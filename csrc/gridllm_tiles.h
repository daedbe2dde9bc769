// Helpers of the kernels that move 16-bit tiles through LDS into MFMA operands:
// rotation by tables, packing, transposed LDS reads, direct loads into LDS,
// and a barrier that leaves such loads in flight.
#pragma once

#include "gridllm_common.h"

#define PAGE 64
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(2))) unsigned int u32x2;
typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;

// cos and sin of a position times each pair's frequency: rows of R / 2 values
// (1 and 0 for pairs that are not rotated)
struct Rotation {
    const float* cos_;
    const float* sin_;
    int half, rows;
};

// Rotate the neighbouring pairs of 8 coordinates by 4 cosines and sines.
DEV_INLINE void rotate_by(float* f, const float* cos_, const float* sin_) {
    float co[4], si[4];
    ld4(cos_, co);
    ld4(sin_, si);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float u = f[2 * i], v = f[2 * i + 1];
        f[2 * i] = u * co[i] - v * si[i];
        f[2 * i + 1] = v * co[i] + u * si[i];
    }
}

// The same by the tables; the first is coordinate c of the rotated part.
DEV_INLINE void rotate8(float* f, int c, int p, const Rotation rot) {
    const long at = (long)min(p, rot.rows - 1) * rot.half + c / 2;
    rotate_by(f, rot.cos_ + at, rot.sin_ + at);
}

DEV_INLINE bf16x8 to_bf16x8(const float* f) {
    bf16x8 o;
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = (__bf16)f[i];
    return o;
}

DEV_INLINE u32 pack2(float a, float b) {
    typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
    bf16x2 v = {(__bf16)a, (__bf16)b};
    return __builtin_bit_cast(u32, v);
}

// max over the lanes that differ in bit 5, or bits 4 and 5, of the lane number
DEV_INLINE float max_across32(float x) {
    const u32x2 r = __builtin_amdgcn_permlane32_swap(
        __float_as_uint(x), __float_as_uint(x), false, false);
    return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
DEV_INLINE float max_across16(float x) {
    const u32x2 r = __builtin_amdgcn_permlane16_swap(
        __float_as_uint(x), __float_as_uint(x), false, false);
    return max_across32(fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1])));
}

// 2^x by the hardware instruction (tiny results become 0)
DEV_INLINE float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

// 4 x 16 block of 16-bit elements in LDS, read transposed by 16 lanes: lane l
// passes the address of row l / 4, columns 4 (l % 4) .. + 3, and gets column l,
// rows 0 .. 3.
DEV_INLINE bf16x4 read_transposed(const bf16_t* p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)p);
}

DEV_INLINE void load_lds16(const bf16_t* src, bf16_t* dst) {
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) unsigned int*)src,
        (__attribute__((address_space(3))) unsigned int*)dst, 16, 0, 0);
}

// Barrier that orders LDS accesses alone: loads into LDS stay in flight.
DEV_INLINE void lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
