// What the two bfloat16 prefill attention kernels share: operand fragments, the softmax state of a
// wavefront's heads, and what a wavefront knows about the tile of query tokens it works on.
#pragma once
#include "common.h"

#define PF_SLACK 8.f        // how far (log2 units) a score may exceed the running reference before it moves

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));

union PFrag {
    u32x4_t u;
    bf16x8_t b;
};

typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
typedef float f32x2_t __attribute__((ext_vector_type(2)));

// two floats -> packed bfloat16 (round to nearest even, one instruction on gfx950)
__device__ __forceinline__ uint32_t pk_bf16(float a, float b) {
    const bf16x2_t v = __builtin_convertvector(f32x2_t{a, b}, bf16x2_t);
    return *(const uint32_t*)&v;
}

// max(a, b, c) in the nesting the compiler turns into one three-operand maximum. A two-operand
// maximum of values whose origin it cannot see (matrix-unit results, lane swaps) costs it an extra
// instruction per operand (it first makes signalling NaNs quiet); the three-operand form does not,
// so the reductions below are chains of these, started from a constant.
__device__ __forceinline__ float max3(float a, float b, float c) { return fmaxf(fmaxf(a, b), c); }

// maximum over the four lanes (r, 0..3) that hold one query column
__device__ __forceinline__ float column_max(float v) {
    const uint32_t u = __float_as_uint(v);
    const auto a = __builtin_amdgcn_permlane32_swap(u, u, false, false);     // lanes l and l ^ 32
    const float m32 = max3(-INFINITY, __uint_as_float(a[0]), __uint_as_float(a[1]));
    const uint32_t w = __float_as_uint(m32);
    const auto b = __builtin_amdgcn_permlane16_swap(w, w, false, false);     // lanes l and l ^ 16
    return max3(-INFINITY, __uint_as_float(b[0]), __uint_as_float(b[1]));
}

// Running softmax state of the query heads a wavefront works on.
//   m: running maximum of (score * scale * log2 e) of this lane's column; l: this lane's share of
//   the running sum (its 8 keys of every block), reduced over the lanes of a column at the end
template <int D, int HPW>
struct HeadState {
    float m[HPW], l[HPW];
    f32x4_t o[HPW][D / 16];
};

// What a wavefront knows about the tile it works on (all wave-uniform but my_pos and my_lo).
struct TileView {
    int pos0;               // position of the tile's first query
    int last_key;           // newest key any query of the tile sees
    int first_key;          // oldest key of the windows of the tile's queries (0 without a window, or where the kept keys reach up to it)
    int last_lo;            // oldest key of the window of the tile's last query (0 without a window)
    int keep;               // with a window: the first keys of the request, which every query sees too
    int my_pos, my_lo;      // this lane's query column: its position and the oldest key of its window

    // does this lane's query see key k?
    __device__ __forceinline__ bool mine(int k) const { return k <= my_pos && (k >= my_lo || k < keep); }
    // does any query of the tile?
    __device__ __forceinline__ bool seen(int k) const { return k <= last_key && (k >= first_key || k < keep); }
};

__device__ __forceinline__ TileView tile_view(int pos0, int valid, int r, int window, int keep) {
    TileView tv;
    tv.pos0 = pos0;
    tv.last_key = pos0 + valid - 1;
    tv.my_pos = pos0 + r < tv.last_key ? pos0 + r : tv.last_key;
    tv.my_lo = (window > 0 && tv.my_pos - window + 1 > 0) ? tv.my_pos - window + 1 : 0;
    tv.last_lo = (window > 0 && tv.last_key - window + 1 > 0) ? tv.last_key - window + 1 : 0;
    tv.first_key = (window > 0 && pos0 - window + 1 > 0) ? pos0 - window + 1 : 0;
    tv.keep = window > 0 ? keep : 0;
    if (tv.first_key <= tv.keep) tv.first_key = 0;          // no gap between the kept keys and the windows
    return tv;
}
