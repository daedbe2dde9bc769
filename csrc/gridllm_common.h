// Helpers shared by the gfx950 kernel sources: bf16 packing, wave
// reductions, MFMA fragment types, and the gated-linear-unit activation.
#pragma once

#include <hip/hip_runtime.h>
#include <math.h>
#include <float.h>

typedef unsigned short bf16_t;
typedef unsigned int u32;

#define WAVE 64
#define DEV_INLINE __device__ __forceinline__

DEV_INLINE float bf2f(bf16_t v) {
    u32 u = ((u32)v) << 16;
    return __uint_as_float(u);
}

DEV_INLINE bf16_t f2bf(float f) {
    u32 u = __float_as_uint(f);
    // round-to-nearest-even; NaN-safe (quiet the NaN)
    if ((u & 0x7fffffffu) > 0x7f800000u) return (bf16_t)0x7fc0;
    u32 r = (u + 0x7fffu + ((u >> 16) & 1u)) >> 16;
    return (bf16_t)r;
}

// unpack 8 bf16 from a uint4 into f32[8]
DEV_INLINE void unpack8(const uint4 v, float* f) {
    const u32 w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        f[2 * i]     = __uint_as_float((w[i] & 0xffffu) << 16);
        f[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}

// pack f32[8] -> uint4 of 8 bf16
DEV_INLINE uint4 pack8(const float* f) {
    uint4 v;
    u32* w = (u32*)&v;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        u32 lo = (u32)f2bf(f[2 * i]);
        u32 hi = (u32)f2bf(f[2 * i + 1]);
        w[i] = lo | (hi << 16);
    }
    return v;
}

DEV_INLINE float wave_reduce_sum(float x) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) x += __shfl_xor(x, off, WAVE);
    return x;
}

DEV_INLINE float wave_reduce_max(float x) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) x = fmaxf(x, __shfl_xor(x, off, WAVE));
    return x;
}

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(16))) float f32x16;

// Gated linear unit, by its constants:
//   g' = min(g, limit), u' = clamp(u, -limit, limit)
//   y  = g' * sigmoid(alpha * g') * (u' + shift)
// SwiGLU is {alpha 1, limit inf, shift 0}.
struct GluParams { float alpha, limit, shift; };

DEV_INLINE float glu_act(float g, float u, const GluParams p) {
    g = fminf(g, p.limit);
    u = fminf(fmaxf(u, -p.limit), p.limit);
    return g * (1.f / (1.f + __expf(-p.alpha * g))) * (u + p.shift);
}

#define LAUNCH_CHECK() do { hipError_t e = hipGetLastError(); \
    if (e != hipSuccess) return (int)e; } while (0)
