// Several results on their way into the residual stream at once (sublayers side by side), and the RMS norm of the sum:
//
//   v = resid[r] + (s0 y0[r] + s1 y1[r] + s2 y2[r])          (y1 and y2 may be null)
//   resid[r] = v;  out[r] = v / sqrt(mean(v^2) + eps) * w     (out null: the add alone)
//   out2[r] = v / sqrt(mean(v^2) + eps) * w2                  (w2 and out2 null: one norm; y0 may be null too: nothing to add)
//
// rows == nullptr: every row, the residual updated in place. rows != nullptr: row rows[r] is read, nothing is written back, out
// row r (the rows whose logits are wanted). Everything is 32-bit; a bfloat16 result is rounded once, where it is stored. A
// block a row; the sum of squares has one order per width.
#include "common.h"
#include "api.h"

#define SN_THREADS 256
#define SN_PIECES 4             // a thread's 4-element pieces of a row that stays in registers

typedef float sn_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ sn_f32x4 sn_load(const float* p) { return *(const sn_f32x4*)p; }
__device__ __forceinline__ sn_f32x4 sn_load(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return sn_f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                    __uint_as_float(u.y & 0xffff0000u)};
}
__device__ __forceinline__ void sn_store(float* p, sn_f32x4 v) { *(sn_f32x4*)p = v; }
__device__ __forceinline__ void sn_store(bf16_t* p, sn_f32x4 v) {
    uint2 u;
    u.x = (uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
    u.y = (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
    *(uint2*)p = u;
}

// Rows of up to 4 * 256 * 4 elements in whole pieces of four: everything a block needs is asked for at once and the row stays in
// registers.
template <typename T, typename WT>
__global__ __launch_bounds__(SN_THREADS) void sum_norm_reg_kernel(float* __restrict__ resid, const T* __restrict__ y0, float s0,
                                                                  const T* __restrict__ y1, float s1, const T* __restrict__ y2, float s2,
                                                                  const int* __restrict__ rows, const WT* __restrict__ w,
                                                                  const WT* __restrict__ w2, T* __restrict__ out, T* __restrict__ out2, int hidden, float eps) {
    __shared__ float red[SN_THREADS / TM_WAVE];
    const int r = blockIdx.x;
    const size_t at = (rows ? (size_t)rows[r] : (size_t)r) * hidden;
    const int pieces = hidden / 4;
    sn_f32x4 x[SN_PIECES], a[SN_PIECES], b[SN_PIECES], c[SN_PIECES], wv[SN_PIECES], wu[SN_PIECES];
#pragma unroll
    for (int i = 0; i < SN_PIECES; ++i) {
        const int p = threadIdx.x + i * SN_THREADS;
        x[i] = a[i] = b[i] = c[i] = wv[i] = wu[i] = sn_f32x4{0.f, 0.f, 0.f, 0.f};
        if (p < pieces) {
            x[i] = sn_load(resid + at + 4 * p);
            if (y0) a[i] = sn_load(y0 + at + 4 * p);
            if (y1) b[i] = sn_load(y1 + at + 4 * p);
            if (y2) c[i] = sn_load(y2 + at + 4 * p);
            if (out) wv[i] = sn_load(w + 4 * p);
            if (out2) wu[i] = sn_load(w2 + 4 * p);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < SN_PIECES; ++i) {
        const int p = threadIdx.x + i * SN_THREADS;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            x[i][k] += s0 * a[i][k] + s1 * b[i][k] + s2 * c[i][k];
            ss += x[i][k] * x[i][k];
        }
        if (!rows && y0 && p < pieces) sn_store(resid + at + 4 * p, x[i]);
    }
    if (!out) return;
    const float scale = 1.0f / sqrtf(block_sum<SN_THREADS>(ss, red) / (float)hidden + eps);
    T* o = out + (size_t)r * hidden;
#pragma unroll
    for (int i = 0; i < SN_PIECES; ++i) {
        const int p = threadIdx.x + i * SN_THREADS;
        if (p >= pieces) continue;
        sn_f32x4 v;
#pragma unroll
        for (int k = 0; k < 4; ++k) v[k] = wv[i][k] * (x[i][k] * scale);
        sn_store(o + 4 * p, v);
        if (out2) {
#pragma unroll
            for (int k = 0; k < 4; ++k) v[k] = wu[i][k] * (x[i][k] * scale);
            sn_store(out2 + (size_t)r * hidden + 4 * p, v);
        }
    }
}

// Any width up to 16,128: the row in LDS.
template <typename T, typename WT>
__global__ __launch_bounds__(SN_THREADS) void sum_norm_kernel(float* __restrict__ resid, const T* __restrict__ y0, float s0,
                                                              const T* __restrict__ y1, float s1, const T* __restrict__ y2, float s2,
                                                              const int* __restrict__ rows, const WT* __restrict__ w,
                                                              const WT* __restrict__ w2, T* __restrict__ out, T* __restrict__ out2, int hidden, float eps) {
    extern __shared__ float xs[];                           // [hidden]
    __shared__ float red[SN_THREADS / TM_WAVE];
    const int r = blockIdx.x;
    const size_t at = (rows ? (size_t)rows[r] : (size_t)r) * hidden;
    float ss = 0.f;
#pragma unroll 4
    for (int c = threadIdx.x; c < hidden; c += SN_THREADS) {
        float d = y0 ? s0 * Elem<T>::load(y0 + at + c) : 0.f;
        if (y1) d += s1 * Elem<T>::load(y1 + at + c);
        if (y2) d += s2 * Elem<T>::load(y2 + at + c);
        const float v = resid[at + c] + d;
        if (!rows && y0) resid[at + c] = v;
        xs[c] = v;                                          // read by the same thread only
        ss += v * v;
    }
    if (!out) return;
    const float scale = 1.0f / sqrtf(block_sum<SN_THREADS>(ss, red) / (float)hidden + eps);
    T* o = out + (size_t)r * hidden;
    for (int c = threadIdx.x; c < hidden; c += SN_THREADS) {
        Elem<T>::store(o + c, Elem<WT>::load(w + c) * (xs[c] * scale));
        if (out2) Elem<T>::store(out2 + (size_t)r * hidden + c, Elem<WT>::load(w2 + c) * (xs[c] * scale));
    }
}

template <typename T, typename WT>
static void launch_sum_norm(float* resid, const void* y0, float s0, const void* y1, float s1, const void* y2, float s2, const int* rows,
                            const void* w, const void* w2, void* out, void* out2, int R, int hidden, float eps, hipStream_t stream) {
    auto ok = [](const void* p, int bytes) { return ((uintptr_t)p % bytes) == 0; };
    const int e = 4 * (int)sizeof(T);
    if (hidden % 4 == 0 && hidden <= 4 * SN_THREADS * SN_PIECES && ok(resid, 16) && ok(y0, e) && ok(y1, e) && ok(y2, e) && ok(out, e) &&
        ok(w, 4 * (int)sizeof(WT)) && ok(w2, 4 * (int)sizeof(WT)) && ok(out2, e))
        sum_norm_reg_kernel<T, WT><<<R, SN_THREADS, 0, stream>>>(resid, (const T*)y0, s0, (const T*)y1, s1, (const T*)y2, s2, rows,
                                                                 (const WT*)w, (const WT*)w2, (T*)out, (T*)out2, hidden, eps);
    else
        sum_norm_kernel<T, WT><<<R, SN_THREADS, (size_t)hidden * sizeof(float), stream>>>(
            resid, (const T*)y0, s0, (const T*)y1, s1, (const T*)y2, s2, rows, (const WT*)w, (const WT*)w2, (T*)out, (T*)out2, hidden, eps);
}

// A second norm of the same sum with weights of its own (w2, out2; both or neither), for sublayers side by side; y0 null: nothing is
// added and resid stays as it is.
extern "C" int tm_sum_norm2(float* resid, const void* y0, float s0, const void* y1, float s1, const void* y2, float s2, const int* rows,
                            const void* w, const void* w2, int w_dtype, void* out, void* out2, int dtype, int R, int hidden, float eps,
                            hipStream_t stream) {
    if (R <= 0) return TM_OK;
    if (!resid || (!y0 && (y1 || y2 || !out)) || hidden <= 0 || (size_t)hidden * sizeof(float) > 63 * 1024 ||
        (out && (!w || !(eps > 0.f))) || (rows && !out) || (out2 && (!out || !w2)) || (w2 && !out2))
        return TM_ERR_ARG;
    if (!out) w_dtype = dtype;
    if (dtype == TM_F32 && w_dtype == TM_F32)
        launch_sum_norm<float, float>(resid, y0, s0, y1, s1, y2, s2, rows, w, w2, out, out2, R, hidden, eps, stream);
    else if (dtype == TM_BF16 && w_dtype == TM_BF16)
        launch_sum_norm<bf16_t, bf16_t>(resid, y0, s0, y1, s1, y2, s2, rows, w, w2, out, out2, R, hidden, eps, stream);
    else if (dtype == TM_BF16 && w_dtype == TM_F32)
        launch_sum_norm<bf16_t, float>(resid, y0, s0, y1, s1, y2, s2, rows, w, w2, out, out2, R, hidden, eps, stream);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

extern "C" int tm_sum_norm(float* resid, const void* y0, float s0, const void* y1, float s1, const void* y2, float s2, const int* rows,
                           const void* w, int w_dtype, void* out, int dtype, int R, int hidden, float eps, hipStream_t stream) {
    if (R > 0 && !y0) return TM_ERR_ARG;
    return tm_sum_norm2(resid, y0, s0, y1, s1, y2, s2, rows, w, nullptr, w_dtype, out, nullptr, dtype, R, hidden, eps, stream);
}
