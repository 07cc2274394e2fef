// Shared device helpers for the gfx950 kernels: storage types, wave/block reductions, checks.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

#define TM_WAVE 64

// dtype codes of the C interface
#define TM_F32 0
#define TM_BF16 1
#define TM_NONE (-1)

// error codes of the C interface (0 = ok)
#define TM_OK 0
#define TM_ERR_ARG 1        // an argument the kernel cannot run with
#define TM_ERR_LAUNCH 2     // the runtime refused the launch
#define TM_ERR_UNSUPPORTED 3 // a library has no routine for the request: use another path

typedef uint16_t bf16_t;    // bfloat16 bits

__device__ __forceinline__ float bf16_to_f32(bf16_t v) {
    return __uint_as_float(((uint32_t)v) << 16);
}

// round to nearest even; NaN stays NaN
__device__ __forceinline__ bf16_t f32_to_bf16(float f) {
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (bf16_t)((u >> 16) | 0x0040u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (bf16_t)(u >> 16);
}

template <typename T> struct Elem;
template <> struct Elem<float> {
    static __device__ __forceinline__ float load(const float* p) { return *p; }
    static __device__ __forceinline__ void store(float* p, float v) { *p = v; }
    static __device__ __forceinline__ float round(float v) { return v; }
};
template <> struct Elem<bf16_t> {
    static __device__ __forceinline__ float load(const bf16_t* p) { return bf16_to_f32(*p); }
    static __device__ __forceinline__ void store(bf16_t* p, float v) { *p = f32_to_bf16(v); }
    static __device__ __forceinline__ float round(float v) { return bf16_to_f32(f32_to_bf16(v)); }
};

// Sixteen bytes of a row as 32-bit floats: 4 float32 values or 8 bfloat16 values.
template <typename T> struct Piece;
template <> struct Piece<float> {
    static constexpr int N = 4;
    static __device__ __forceinline__ void unpack(const uint4& u, float* f) {
        f[0] = __uint_as_float(u.x); f[1] = __uint_as_float(u.y); f[2] = __uint_as_float(u.z); f[3] = __uint_as_float(u.w);
    }
};
template <> struct Piece<bf16_t> {
    static constexpr int N = 8;
    static __device__ __forceinline__ void unpack(const uint4& u, float* f) {
        f[0] = __uint_as_float(u.x << 16); f[1] = __uint_as_float(u.x & 0xffff0000u);
        f[2] = __uint_as_float(u.y << 16); f[3] = __uint_as_float(u.y & 0xffff0000u);
        f[4] = __uint_as_float(u.z << 16); f[5] = __uint_as_float(u.z & 0xffff0000u);
        f[6] = __uint_as_float(u.w << 16); f[7] = __uint_as_float(u.w & 0xffff0000u);
    }
};

// The rotation of a pair (x1, x2) by the angle whose cosine and sine are c and s (reference
// src/infer/model/layers.py:60-64). Every product and each sum is rounded to 32-bit on its own, as a tensor
// library's x1 * cos - x2 * sin is: left to itself the compiler fuses a product into the sum, and which one it
// picks differs from one kernel (or one instantiation of a kernel) to the next, so that the same token would get
// other last bits from the kernel for 8 rows than from the kernel for 40.
__device__ __forceinline__ void rotate_pair(float x1, float x2, float c, float s, float& y1, float& y2) {
#pragma clang fp contract(off)
    const float a = x1 * c, b = x2 * s, d = x2 * c, e = x1 * s;
    y1 = a - b;
    y2 = d + e;
}

// sigmoid from the hardware's exponential
__device__ __forceinline__ float sigmoid_fast(float x) { return 1.0f / (1.0f + __expf(-x)); }

// the clamped gated activation g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = up held to +-limit
__device__ __forceinline__ float clamped_glu_f32(float g, float u, float alpha, float limit) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.0f + expf(-alpha * g)) * (u + 1.0f);
}

// tanh from the hardware's exp2 and reciprocal: 1 - 2 / (e^(2x) + 1), exact at both ends (e^(2x) = inf or 0); its absolute
// error of about 1e-7 is far below a bfloat16 score's own
__device__ __forceinline__ float tanh_fast(float x) {
    return 1.f - 2.f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(x * 2.8853900817779268f) + 1.f);
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = TM_WAVE / 2; off > 0; off >>= 1) v += __shfl_xor(v, off, TM_WAVE);
    return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int off = TM_WAVE / 2; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, TM_WAVE));
    return v;
}

// Sum over a block of NT threads (NT a multiple of 64, at most 1024). Every thread gets the result.
// The order of the additions is fixed by the thread layout, never by the data.
template <int NT>
__device__ __forceinline__ float block_sum(float v, float* smem /* NT/64 floats */) {
    v = wave_sum(v);
    const int wave = threadIdx.x / TM_WAVE, lane = threadIdx.x % TM_WAVE;
    __syncthreads();
    if (lane == 0) smem[wave] = v;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < NT / TM_WAVE; ++w) total += smem[w];
    return total;
}

#define TM_CHECK_LAUNCH()                                        \
    do {                                                         \
        hipError_t e_ = hipGetLastError();                       \
        if (e_ != hipSuccess) return TM_ERR_LAUNCH;              \
    } while (0)
