// Row-wise kernels: embedding rows, residual add + RMSNorm, rotary position encoding fused with
// the cache write, SiLU(gate)*up, type conversion.
//
// Exactness: the residual stream is 32-bit; sums of squares, the reciprocal root and the rotation
// are 32-bit; a bfloat16 result is rounded once, where the tensor is stored.
#include "common.h"
#include "api.h"

// ------------------------------------------------------------------------------------------
// embedding rows -> 32-bit residual stream           (reference src/infer/model/qwen2.py:46)
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ void embed_gather_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                    float* __restrict__ out, int hidden, int vocab) {
    const int t = blockIdx.x;
    int id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);       // the host rejects such ids; never read outside
    const T* row = table + (size_t)id * hidden;
    float* o = out + (size_t)t * hidden;
    for (int c = threadIdx.x; c < hidden; c += blockDim.x) o[c] = Elem<T>::load(row + c);
}

extern "C" int tm_embed_gather(const void* table, int dtype, const int* ids, float* out, int T,
                               int hidden, int vocab, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (hidden <= 0 || vocab <= 0) return TM_ERR_ARG;
    if (dtype == TM_F32)
        embed_gather_kernel<float><<<T, 256, 0, stream>>>((const float*)table, ids, out, hidden, vocab);
    else if (dtype == TM_BF16)
        embed_gather_kernel<bf16_t><<<T, 256, 0, stream>>>((const bf16_t*)table, ids, out, hidden, vocab);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// out[t] = table[ids[t]] * scale: a model that multiplies its embedding rows by a constant on their way into the stream (the
// product in 32-bit)
template <typename T>
__global__ void embed_gather_scaled_kernel(const T* __restrict__ table, const int* __restrict__ ids, float* __restrict__ out,
                                           int hidden, int vocab, float scale) {
    const int t = blockIdx.x;
    int id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);       // the host rejects such ids; never read outside
    const T* row = table + (size_t)id * hidden;
    float* o = out + (size_t)t * hidden;
    for (int c = threadIdx.x; c < hidden; c += blockDim.x) o[c] = Elem<T>::load(row + c) * scale;
}

extern "C" int tm_embed_gather_scaled(const void* table, int dtype, const int* ids, float* out, int T, int hidden, int vocab,
                                      float scale, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (hidden <= 0 || vocab <= 0 || !table || !ids || !out) return TM_ERR_ARG;
    if (dtype == TM_F32)
        embed_gather_scaled_kernel<float><<<T, 256, 0, stream>>>((const float*)table, ids, out, hidden, vocab, scale);
    else if (dtype == TM_BF16)
        embed_gather_scaled_kernel<bf16_t><<<T, 256, 0, stream>>>((const bf16_t*)table, ids, out, hidden, vocab, scale);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// embedding rows plus learned position rows -> 32-bit residual stream: out[t] = table[ids[t]] + places[positions[t]]
// (the sum in 32-bit; no scaling of either)
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ void embed_gather_pos_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                        const T* __restrict__ places, const int* __restrict__ positions,
                                        float* __restrict__ out, int hidden, int vocab, int max_pos) {
    const int t = blockIdx.x;
    int id = ids[t], p = positions[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);       // the host rejects such ids and positions; never read outside
    p = p < 0 ? 0 : (p >= max_pos ? max_pos - 1 : p);
    const T* row = table + (size_t)id * hidden;
    const T* prow = places + (size_t)p * hidden;
    float* o = out + (size_t)t * hidden;
    for (int c = threadIdx.x; c < hidden; c += blockDim.x) o[c] = Elem<T>::load(row + c) + Elem<T>::load(prow + c);
}

extern "C" int tm_embed_gather_pos(const void* table, const void* places, int dtype, const int* ids, const int* positions,
                                   float* out, int T, int hidden, int vocab, int max_pos, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (hidden <= 0 || vocab <= 0 || max_pos <= 0 || !places || !positions) return TM_ERR_ARG;
    if (dtype == TM_F32)
        embed_gather_pos_kernel<float><<<T, 256, 0, stream>>>((const float*)table, ids, (const float*)places, positions, out,
                                                             hidden, vocab, max_pos);
    else if (dtype == TM_BF16)
        embed_gather_pos_kernel<bf16_t><<<T, 256, 0, stream>>>((const bf16_t*)table, ids, (const bf16_t*)places, positions,
                                                              out, hidden, vocab, max_pos);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// residual += delta ; out = weight * round(residual * rsqrt(mean(residual^2) + eps))
//                                                    (reference src/infer/model/layers.py:41-44,
//                                                     src/infer/model/qwen2.py:22-23)
// rows == nullptr: row r of the residual is updated in place.
// rows != nullptr: row rows[r] is read (residual + delta), nothing is written back, out row r.
// ------------------------------------------------------------------------------------------
// What is still to be added to the residual stream: a tensor of the model's type, or the partial sums of a product
// whose K was split over blocks (32-bit, `parts` of them, `stride` elements apart), which are added in their
// order and rounded to the model's type first, as the product's own epilogue would have stored them.
template <typename T>
struct Pending {
    const T* delta;
    const float* parts;
    int n_parts;
    size_t stride;
    __device__ __forceinline__ bool any() const { return delta || parts; }
    __device__ __forceinline__ float at(size_t i) const {
        if (delta) return Elem<T>::load(delta + i);
        float s = parts[i];
        for (int p = 1; p < n_parts; ++p) s += parts[p * stride + i];
        return Elem<T>::round(s);
    }
};

template <typename T, typename WT>
__global__ void add_rmsnorm_kernel(float* __restrict__ resid, const Pending<T> pending,
                                   const int* __restrict__ rows, const WT* __restrict__ weight,
                                   T* __restrict__ out, int hidden, float eps) {
    __shared__ float red[4];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* x = resid + src * hidden;
    const bool d = pending.any();
    T* o = out + (size_t)r * hidden;
    float ss = 0.f;
    for (int c = threadIdx.x; c < hidden; c += 256) {
        float v = x[c];
        if (d) v += pending.at(src * hidden + c);
        if (d && !rows) x[c] = v;
        ss += v * v;
    }
    ss = block_sum<256>(ss, red);
    const float rs = rsqrtf(ss / (float)hidden + eps);
    for (int c = threadIdx.x; c < hidden; c += 256) {
        float v = x[c];
        if (d && rows) v += pending.at(src * hidden + c);   // in-place rows already hold the sum
        const float n = Elem<T>::round(v * rs);            // rounded BEFORE the weight multiplies
        Elem<T>::store(o + c, Elem<WT>::load(weight + c) * n);
    }
}

// The same for widths that are a multiple of 4 and at most 16,384: every thread (256, 512 or 1,024 of them) keeps
// its (up to four) 4-element groups of the row in registers, so the row is read once.
typedef float ew_f32x4 __attribute__((ext_vector_type(4)));

template <typename T> struct Vec4;
template <> struct Vec4<float> {
    static __device__ __forceinline__ ew_f32x4 load(const float* p) { return *(const ew_f32x4*)p; }
    static __device__ __forceinline__ void store(float* p, ew_f32x4 v) { *(ew_f32x4*)p = v; }
};
template <> struct Vec4<bf16_t> {
    static __device__ __forceinline__ ew_f32x4 load(const bf16_t* p) {
        const uint2 u = *(const uint2*)p;
        return ew_f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                        __uint_as_float(u.y & 0xffff0000u)};
    }
    static __device__ __forceinline__ void store(bf16_t* p, ew_f32x4 v) {
        uint2 u;
        u.x = (uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
        u.y = (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
        *(uint2*)p = u;
    }
};

#define ADD_NORM_MAX_PARTS 8       // most partial sums the vector kernel adds (more: the plain kernel)

template <typename T, typename WT, int THREADS>
__global__ __launch_bounds__(THREADS) void add_rmsnorm_vec_kernel(float* __restrict__ resid, const Pending<T> pending,
                                                              const int* __restrict__ rows,
                                                              const WT* __restrict__ weight, T* __restrict__ out,
                                                              int hidden, float eps) {
    __shared__ float red[THREADS / 64];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* x = resid + src * hidden;
    const T* d = pending.delta ? pending.delta + src * hidden : nullptr;
    const float* ps = pending.parts ? pending.parts + src * hidden : nullptr;
    T* o = out + (size_t)r * hidden;
    const int groups = hidden / 4;
    ew_f32x4 v[4];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int gidx = threadIdx.x + i * THREADS;
        v[i] = ew_f32x4{0.f, 0.f, 0.f, 0.f};
        if (gidx < groups) {
            v[i] = Vec4<float>::load(x + 4 * gidx);
            if (d) {
                v[i] += Vec4<T>::load(d + 4 * gidx);
                if (!rows) Vec4<float>::store(x + 4 * gidx, v[i]);
            } else if (ps) {
                // all parts asked for at once (a part that does not exist: part 0 again, not counted), then added in order
                ew_f32x4 part[ADD_NORM_MAX_PARTS];
#pragma unroll
                for (int p = 0; p < ADD_NORM_MAX_PARTS; ++p)
                    part[p] = Vec4<float>::load(ps + (size_t)(p < pending.n_parts ? p : 0) * pending.stride + 4 * gidx);
                ew_f32x4 sum = part[0];
#pragma unroll
                for (int p = 1; p < ADD_NORM_MAX_PARTS; ++p)
                    if (p < pending.n_parts) sum += part[p];
#pragma unroll
                for (int k = 0; k < 4; ++k) v[i][k] += Elem<T>::round(sum[k]);
                if (!rows) Vec4<float>::store(x + 4 * gidx, v[i]);
            }
            ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
        }
    }
    ss = block_sum<THREADS>(ss, red);
    const float rs = rsqrtf(ss / (float)hidden + eps);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int gidx = threadIdx.x + i * THREADS;
        if (gidx < groups) {
            const ew_f32x4 w = Vec4<WT>::load(weight + 4 * gidx);
            ew_f32x4 y;
#pragma unroll
            for (int k = 0; k < 4; ++k) y[k] = w[k] * Elem<T>::round(v[i][k] * rs);   // rounded BEFORE the weight multiplies
            Vec4<T>::store(o + 4 * gidx, y);
        }
    }
}

template <typename T, typename WT>
static void launch_add_rmsnorm(float* resid, const void* delta, const float* parts, int n_parts, size_t stride,
                               const int* rows, const void* weight, void* out, int R, int hidden, float eps,
                               hipStream_t stream) {
    const bool vec = hidden % 4 == 0 && hidden <= 16384 && ((uintptr_t)resid % 16) == 0 && ((uintptr_t)weight % 16) == 0 &&
                     ((uintptr_t)out % 16) == 0 && (!delta || ((uintptr_t)delta % 16) == 0) &&
                     (!parts || (((uintptr_t)parts % 16) == 0 && stride % 4 == 0 && n_parts <= ADD_NORM_MAX_PARTS));
    const Pending<T> pending{(const T*)delta, parts, n_parts, stride};
    // a thread for every 4-element group where 1,024 reach (measured on an MI355X, 64 rows with 4 partial sums: width
    // 3,584 6.5 us with 256 threads, 4.9 with 512, 4.5 with 1,024; width 5,120 5.7 with 512, 5.1 with 1,024; width 896
    // 3.4 us with any); from the width alone: the sum of squares has one order per model
    const int threads = hidden <= 1024 ? 256 : hidden <= 2048 ? 512 : 1024;
    if (vec && threads == 256)
        add_rmsnorm_vec_kernel<T, WT, 256><<<R, 256, 0, stream>>>(resid, pending, rows, (const WT*)weight, (T*)out, hidden, eps);
    else if (vec && threads == 512)
        add_rmsnorm_vec_kernel<T, WT, 512><<<R, 512, 0, stream>>>(resid, pending, rows, (const WT*)weight, (T*)out, hidden, eps);
    else if (vec)
        add_rmsnorm_vec_kernel<T, WT, 1024><<<R, 1024, 0, stream>>>(resid, pending, rows, (const WT*)weight, (T*)out, hidden, eps);
    else
        add_rmsnorm_kernel<T, WT><<<R, 256, 0, stream>>>(resid, pending, rows, (const WT*)weight, (T*)out, hidden, eps);
}

static int add_rmsnorm_any(float* resid, const void* delta, const float* parts, int n_parts, size_t stride, const int* rows,
                           const void* weight, int w_dtype, void* out, int dtype, int R, int hidden, float eps,
                           hipStream_t stream) {
    if (R <= 0) return TM_OK;
    if (hidden <= 0 || !(eps > 0.f)) return TM_ERR_ARG;
    if (dtype == TM_F32 && w_dtype == TM_F32)
        launch_add_rmsnorm<float, float>(resid, delta, parts, n_parts, stride, rows, weight, out, R, hidden, eps, stream);
    else if (dtype == TM_BF16 && w_dtype == TM_BF16)
        launch_add_rmsnorm<bf16_t, bf16_t>(resid, delta, parts, n_parts, stride, rows, weight, out, R, hidden, eps, stream);
    else if (dtype == TM_BF16 && w_dtype == TM_F32)
        launch_add_rmsnorm<bf16_t, float>(resid, delta, parts, n_parts, stride, rows, weight, out, R, hidden, eps, stream);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

extern "C" int tm_add_rmsnorm(float* resid, const void* delta, const int* rows, const void* weight,
                              int w_dtype, void* out, int dtype, int R, int hidden, float eps,
                              hipStream_t stream) {
    return add_rmsnorm_any(resid, delta, nullptr, 0, 0, rows, weight, w_dtype, out, dtype, R, hidden, eps, stream);
}

// The same, with what is to be added given as the 32-bit partial sums of a product whose K was split over blocks:
// parts[p * stride + i], p < n_parts, added in the order of p and rounded to `dtype` before they meet the residual.
extern "C" int tm_add_rmsnorm_parts(float* resid, const float* parts, int n_parts, size_t stride, const int* rows,
                                    const void* weight, int w_dtype, void* out, int dtype, int R, int hidden, float eps,
                                    hipStream_t stream) {
    if (!parts || n_parts < 1 || n_parts > 16) return TM_ERR_ARG;
    return add_rmsnorm_any(resid, nullptr, parts, n_parts, stride, rows, weight, w_dtype, out, dtype, R, hidden, eps, stream);
}

// out[i] = round(sum over p of parts[p * stride + i]) in `dtype`: the partial sums as the tensor the product would
// have stored.
template <typename T>
__global__ void sum_parts_kernel(const float* __restrict__ parts, int n_parts, size_t stride, T* __restrict__ out, size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    float s = parts[i];
    for (int p = 1; p < n_parts; ++p) s += parts[p * stride + i];
    Elem<T>::store(out + i, s);
}

extern "C" int tm_sum_parts(const float* parts, int n_parts, size_t stride, void* out, int dtype, size_t n,
                            hipStream_t stream) {
    if (n == 0) return TM_OK;
    if (!parts || n_parts < 1 || !out) return TM_ERR_ARG;
    const unsigned blocks = (unsigned)((n + 255) / 256);
    if (dtype == TM_BF16) sum_parts_kernel<bf16_t><<<blocks, 256, 0, stream>>>(parts, n_parts, stride, (bf16_t*)out, n);
    else if (dtype == TM_F32) sum_parts_kernel<float><<<blocks, 256, 0, stream>>>(parts, n_parts, stride, (float*)out, n);
    else return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// Rotary position encoding of q and k in place, then k and v of every token to its cache slot.
//   qkv row = [H heads of q | KVH heads of k | KVH heads of v], each D wide.
//   pairs (j, j + rot/2) for j < rot/2; elements >= rot pass through
//                                                    (reference src/infer/model/layers.py:55-64;
//                                                     cache write: src/infer/kv/paged_cache.py:40-43)
//   cos/sin: [max_pos, rot/2] 32-bit; cos == nullptr means no rotation (cache write only).
//   slot = page * page_size + place in the page; slot < 0: k and v are not stored (padding rows).
//   K pool [pages, page_size, KVH, D]; V pool [pages, KVH, D, page_size]: the values of one page
//   lie key-contiguous for each (head, d), which is how the MFMA attention kernels read them.
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ void rope_kv_write_kernel(T* __restrict__ qkv, int H, int KVH, int D, int rot,
                                     const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                     const int* __restrict__ positions, const int* __restrict__ slots,
                                     T* __restrict__ k_pool, T* __restrict__ v_pool, int page, int write_kv) {
    // one block per token; its threads walk (head, pair) for q and k and (head, d) for v
    const int t = blockIdx.x;
    const int width = (H + 2 * KVH) * D;
    T* row = qkv + (size_t)t * width;
    const int slot = slots ? slots[t] : -1;
    const bool store = write_kv && slot >= 0;
    const int half = rot / 2;
    const float* c = cos_t ? cos_t + (size_t)positions[t] * half : nullptr;
    const float* s = cos_t ? sin_t + (size_t)positions[t] * half : nullptr;
    if (cos_t) {
        for (int idx = threadIdx.x; idx < (H + KVH) * half; idx += blockDim.x) {
            const int hh = idx / half, j = idx - hh * half;
            T* x = row + (size_t)hh * D;
            const float x1 = Elem<T>::load(x + j), x2 = Elem<T>::load(x + j + half);
            float y1, y2;
            rotate_pair(x1, x2, c[j], s[j], y1, y2);
            Elem<T>::store(x + j, y1);
            Elem<T>::store(x + j + half, y2);
            if (store && hh >= H) {
                T* dst = k_pool + ((size_t)slot * KVH + (hh - H)) * D;
                Elem<T>::store(dst + j, y1);
                Elem<T>::store(dst + j + half, y2);
            }
        }
    }
    if (!store) return;
    // the part of k that is not rotated (all of it without a table) and v
    const int tail = D - rot * (cos_t ? 1 : 0);
    const int k_from = cos_t ? rot : 0;
    for (int idx = threadIdx.x; idx < KVH * tail; idx += blockDim.x) {
        const int kvh = idx / tail, j = k_from + idx - kvh * tail;
        k_pool[((size_t)slot * KVH + kvh) * D + j] = row[(size_t)(H + kvh) * D + j];
    }
    const int pg = slot / page, in_page = slot % page;
    for (int idx = threadIdx.x; idx < KVH * D; idx += blockDim.x) {
        const int kvh = idx / D, j = idx - kvh * D;
        v_pool[(((size_t)pg * KVH + kvh) * D + j) * page + in_page] = row[(size_t)(H + KVH + kvh) * D + j];
    }
}

extern "C" int tm_rope_kv_write(void* qkv, int dtype, int T, int H, int KVH, int D, int rot,
                                const float* cos_t, const float* sin_t, const int* positions,
                                const int* slots, void* k_pool, void* v_pool, int page, int write_kv,
                                hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (H <= 0 || KVH <= 0 || D <= 0 || rot < 0 || rot > D || (rot & 1)) return TM_ERR_ARG;
    if (cos_t && (!sin_t || !positions)) return TM_ERR_ARG;
    if (write_kv && (!slots || !k_pool || !v_pool || page <= 0)) return TM_ERR_ARG;
    const int grid = T;
    if (dtype == TM_F32)
        rope_kv_write_kernel<float><<<grid, 256, 0, stream>>>((float*)qkv, H, KVH, D, rot, cos_t, sin_t, positions,
                                                            slots, (float*)k_pool, (float*)v_pool, page, write_kv);
    else if (dtype == TM_BF16)
        rope_kv_write_kernel<bf16_t><<<grid, 256, 0, stream>>>((bf16_t*)qkv, H, KVH, D, rot, cos_t, sin_t,
                                                             positions, slots, (bf16_t*)k_pool, (bf16_t*)v_pool,
                                                             page, write_kv);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// out[t, i] = silu(gu[t, i]) * gu[t, I + i]           (reference src/infer/model/layers.py:164)
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ void silu_mul_kernel(const T* __restrict__ gu, T* __restrict__ out, int I, size_t total) {
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (size_t)gridDim.x * blockDim.x) {
        const size_t t = idx / I;
        const int i = (int)(idx - t * I);
        const float g = Elem<T>::load(gu + t * 2 * I + i);
        const float u = Elem<T>::load(gu + t * 2 * I + I + i);
        Elem<T>::store(out + idx, g / (1.f + expf(-g)) * u);
    }
}

// bfloat16 rows whose width is a multiple of 8: eight elements (16 bytes) per thread and step
__global__ void silu_mul_bf16x8_kernel(const bf16_t* __restrict__ gu, bf16_t* __restrict__ out, int I, size_t groups) {
    const int per_row = I / 8;
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < groups;
         idx += (size_t)gridDim.x * blockDim.x) {
        const size_t t = idx / per_row;
        const int i = (int)(idx - t * per_row) * 8;
        const uint4 gv = *(const uint4*)(gu + t * 2 * I + i);
        const uint4 uv = *(const uint4*)(gu + t * 2 * I + I + i);
        const uint32_t gw[4] = {gv.x, gv.y, gv.z, gv.w}, uw[4] = {uv.x, uv.y, uv.z, uv.w};
        uint32_t ow[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const float g0 = __uint_as_float(gw[k] << 16), g1 = __uint_as_float(gw[k] & 0xffff0000u);
            const float u0 = __uint_as_float(uw[k] << 16), u1 = __uint_as_float(uw[k] & 0xffff0000u);
            const float r0 = g0 / (1.f + expf(-g0)) * u0, r1 = g1 / (1.f + expf(-g1)) * u1;
            ow[k] = (uint32_t)f32_to_bf16(r0) | ((uint32_t)f32_to_bf16(r1) << 16);
        }
        *(uint4*)(out + t * I + i) = uint4{ow[0], ow[1], ow[2], ow[3]};
    }
}

extern "C" int tm_silu_mul(const void* gu, void* out, int dtype, int T, int I, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (I <= 0) return TM_ERR_ARG;
    const size_t total = (size_t)T * I;
    if (dtype == TM_BF16 && I % 8 == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0) {
        const size_t groups = total / 8;
        size_t want = (groups + 255) / 256;
        silu_mul_bf16x8_kernel<<<(int)(want < 65536 ? want : 65536), 256, 0, stream>>>((const bf16_t*)gu, (bf16_t*)out,
                                                                                  I, groups);
        TM_CHECK_LAUNCH();
        return TM_OK;
    }
    size_t want = (total + 255) / 256;
    const int blocks = (int)(want < 16384 ? want : 16384);
    if (dtype == TM_F32)
        silu_mul_kernel<float><<<blocks, 256, 0, stream>>>((const float*)gu, (float*)out, I, total);
    else if (dtype == TM_BF16)
        silu_mul_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)gu, (bf16_t*)out, I, total);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// out[i] = gelu_tanh(in[i]) = 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), computed in 32-bit (in place allowed)
// ------------------------------------------------------------------------------------------
__device__ __forceinline__ float gelu_tanh_f32(float z) {
    const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return 0.5f * z * (1.f + tanhf(u));
}

// the square of relu, also in 32-bit
__device__ __forceinline__ float relu2_f32(float z) {
    const float r = fmaxf(z, 0.f);
    return r * r;
}

enum { ACT_GELU_TANH = 0, ACT_RELU2 = 1 };

template <int ACT>
__device__ __forceinline__ float act_f32(float z) { return ACT == ACT_RELU2 ? relu2_f32(z) : gelu_tanh_f32(z); }

template <typename T, int ACT>
__global__ void activation_kernel(const T* __restrict__ in, T* __restrict__ out, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x)
        Elem<T>::store(out + i, act_f32<ACT>(Elem<T>::load(in + i)));
}

// bfloat16, eight elements (16 bytes) per thread and step
template <int ACT>
__global__ void activation_bf16x8_kernel(const bf16_t* __restrict__ in, bf16_t* __restrict__ out, size_t groups) {
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < groups; idx += (size_t)gridDim.x * blockDim.x) {
        const uint4 v = *(const uint4*)(in + 8 * idx);
        const uint32_t w[4] = {v.x, v.y, v.z, v.w};
        uint32_t o[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const float a = act_f32<ACT>(__uint_as_float(w[k] << 16)), b = act_f32<ACT>(__uint_as_float(w[k] & 0xffff0000u));
            o[k] = (uint32_t)f32_to_bf16(a) | ((uint32_t)f32_to_bf16(b) << 16);
        }
        *(uint4*)(out + 8 * idx) = uint4{o[0], o[1], o[2], o[3]};
    }
}

template <int ACT>
static int launch_activation(const void* in, void* out, int dtype, long long n, hipStream_t stream) {
    if (n <= 0) return TM_OK;
    if (!in || !out) return TM_ERR_ARG;
    if (dtype == TM_BF16 && n % 8 == 0 && ((uintptr_t)in % 16) == 0 && ((uintptr_t)out % 16) == 0) {
        const size_t groups = (size_t)n / 8, want = (groups + 255) / 256;
        activation_bf16x8_kernel<ACT><<<(int)(want < 65536 ? want : 65536), 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, groups);
        TM_CHECK_LAUNCH();
        return TM_OK;
    }
    const size_t want = ((size_t)n + 255) / 256;
    const int blocks = (int)(want < 16384 ? want : 16384);
    if (dtype == TM_F32)
        activation_kernel<float, ACT><<<blocks, 256, 0, stream>>>((const float*)in, (float*)out, (size_t)n);
    else if (dtype == TM_BF16)
        activation_kernel<bf16_t, ACT><<<blocks, 256, 0, stream>>>((const bf16_t*)in, (bf16_t*)out, (size_t)n);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// out[t, i] = gelu_tanh(gu[t, i]) * gu[t, I + i]: the gated feed-forward's activation with the tanh form of GELU on the gate,
// computed in 32-bit and rounded once; gu [T, 2I] (gate columns, then up columns).
template <typename T>
__global__ void gelu_mul_kernel(const T* __restrict__ gu, T* __restrict__ out, int I, size_t total) {
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total; idx += (size_t)gridDim.x * blockDim.x) {
        const size_t t = idx / I;
        const int i = (int)(idx - t * I);
        const float g = Elem<T>::load(gu + t * 2 * I + i);
        const float u = Elem<T>::load(gu + t * 2 * I + I + i);
        Elem<T>::store(out + idx, gelu_tanh_f32(g) * u);
    }
}

extern "C" int tm_gelu_mul(const void* gu, void* out, int dtype, int T, int I, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (I <= 0 || !gu || !out) return TM_ERR_ARG;
    const size_t total = (size_t)T * I;
    const size_t want = (total + 255) / 256;
    const int blocks = (int)(want < 16384 ? want : 16384);
    if (dtype == TM_F32)
        gelu_mul_kernel<float><<<blocks, 256, 0, stream>>>((const float*)gu, (float*)out, I, total);
    else if (dtype == TM_BF16)
        gelu_mul_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)gu, (bf16_t*)out, I, total);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// out[t, i] = g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = up held to +-limit: the clamped gated activation, computed in
// 32-bit and rounded once; gu [T, 2I] (gate columns, then up columns). Eight elements a thread where the rows come in whole
// pieces of eight.
template <typename T, int N>
__global__ __launch_bounds__(256) void clamped_glu_kernel(const T* __restrict__ gu, T* __restrict__ out, int I, float alpha,
                                                          float limit) {
    const size_t t = blockIdx.y;
    const int i = (blockIdx.x * 256 + threadIdx.x) * N;
    if (i >= I) return;
    const T* gr = gu + t * 2 * I + i;
    T* o = out + t * I + i;
    if constexpr (N == 1) {
        Elem<T>::store(o, clamped_glu_f32(Elem<T>::load(gr), Elem<T>::load(gr + I), alpha, limit));
    } else {
        __align__(16) T g[N], u[N], r[N];
#pragma unroll
        for (int p = 0; p < (int)(N * sizeof(T) / 16); ++p) {
            ((uint4*)g)[p] = ((const uint4*)gr)[p];
            ((uint4*)u)[p] = ((const uint4*)(gr + I))[p];
        }
#pragma unroll
        for (int j = 0; j < N; ++j) Elem<T>::store(r + j, clamped_glu_f32(Elem<T>::load(g + j), Elem<T>::load(u + j), alpha, limit));
#pragma unroll
        for (int p = 0; p < (int)(N * sizeof(T) / 16); ++p) ((uint4*)o)[p] = ((const uint4*)r)[p];
    }
}

template <typename T>
static void launch_clamped_glu(const void* gu, void* out, int T_rows, int I, float alpha, float limit, hipStream_t stream) {
    const bool pieces = I % 8 == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0;
    for (int t0 = 0; t0 < T_rows; t0 += 65535) {
        const int rows = T_rows - t0 < 65535 ? T_rows - t0 : 65535;
        const T* src = (const T*)gu + (size_t)t0 * 2 * I;
        T* dst = (T*)out + (size_t)t0 * I;
        if (pieces) clamped_glu_kernel<T, 8><<<dim3((I / 8 + 255) / 256, rows), 256, 0, stream>>>(src, dst, I, alpha, limit);
        else clamped_glu_kernel<T, 1><<<dim3((I + 255) / 256, rows), 256, 0, stream>>>(src, dst, I, alpha, limit);
    }
}

extern "C" int tm_clamped_glu(const void* gu, void* out, int dtype, int T, int I, float alpha, float limit, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (I <= 0 || !gu || !out || !(limit > 0.f)) return TM_ERR_ARG;
    if (dtype == TM_F32) launch_clamped_glu<float>(gu, out, T, I, alpha, limit, stream);
    else if (dtype == TM_BF16) launch_clamped_glu<bf16_t>(gu, out, T, I, alpha, limit, stream);
    else return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

extern "C" int tm_gelu_tanh(const void* in, void* out, int dtype, long long n, hipStream_t stream) {
    return launch_activation<ACT_GELU_TANH>(in, out, dtype, n, stream);
}

// out[i] = relu(in[i])^2 (in place allowed)
extern "C" int tm_relu2(const void* in, void* out, int dtype, long long n, hipStream_t stream) {
    return launch_activation<ACT_RELU2>(in, out, dtype, n, stream);
}

// ------------------------------------------------------------------------------------------
// type conversion of a flat array
// ------------------------------------------------------------------------------------------
template <typename TI, typename TO>
__global__ void convert_kernel(const TI* __restrict__ in, TO* __restrict__ out, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x)
        Elem<TO>::store(out + i, Elem<TI>::load(in + i));
}

extern "C" int tm_convert(const void* in, int in_dtype, void* out, int out_dtype, long long n,
                          hipStream_t stream) {
    if (n <= 0) return TM_OK;
    size_t want = ((size_t)n + 255) / 256;
    const int blocks = (int)(want < 16384 ? want : 16384);
    if (in_dtype == TM_BF16 && out_dtype == TM_F32)
        convert_kernel<bf16_t, float><<<blocks, 256, 0, stream>>>((const bf16_t*)in, (float*)out, (size_t)n);
    else if (in_dtype == TM_F32 && out_dtype == TM_BF16)
        convert_kernel<float, bf16_t><<<blocks, 256, 0, stream>>>((const float*)in, (bf16_t*)out, (size_t)n);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// x <- x * scale, then with cap > 0: cap * tanh(x / cap), in place, 32-bit (an output head's scaled and capped logits)
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void scale_cap_kernel(float* __restrict__ x, size_t n, float scale, float cap) {
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
        const float v = x[i] * scale;
        x[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
    }
}

extern "C" int tm_scale_cap(float* x, long long n, float scale, float cap, hipStream_t stream) {
    if (n <= 0) return TM_OK;
    if (!x || !(cap >= 0.f)) return TM_ERR_ARG;
    const long long want = (n + 255) / 256;
    scale_cap_kernel<<<(int)(want < 16384 ? want : 16384), 256, 0, stream>>>(x, (size_t)n, scale, cap);
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------
// out[t] = table[ids[t]] * scale + waves, waves[2 i] = sin(p f[i]), waves[2 i + 1] = cos(p f[i]) with p the token's position;
// angles, sines and the sum in 32-bit. f holds ceil(hidden / 2) frequencies. A thread has two pairs where the rows come in pieces of
// four (WIDE), else one.
// ------------------------------------------------------------------------------------------
template <typename T, bool WIDE>
__global__ __launch_bounds__(256) void embed_waves_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                                         const int* __restrict__ positions, const float* __restrict__ f,
                                                         float* __restrict__ out, int hidden, int vocab, float scale) {
    const int t = blockIdx.x;
    int id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);       // the host rejects such ids; never read outside
    const float p = (float)positions[t];
    const T* row = table + (size_t)id * hidden;
    float* o = out + (size_t)t * hidden;
    if constexpr (WIDE) {
        const int c = 4 * (blockIdx.y * 256 + threadIdx.x);
        if (c >= hidden) return;
        const float2 fr = *(const float2*)(f + c / 2);
        T x[4];
        if constexpr (sizeof(T) == 4) *(uint4*)x = *(const uint4*)(row + c);
        else *(uint2*)x = *(const uint2*)(row + c);
        float s0, c0, s1, c1;
        sincosf(p * fr.x, &s0, &c0);
        sincosf(p * fr.y, &s1, &c1);
        *(float4*)(o + c) = float4{Elem<T>::load(x) * scale + s0, Elem<T>::load(x + 1) * scale + c0, Elem<T>::load(x + 2) * scale + s1,
                                   Elem<T>::load(x + 3) * scale + c1};
    } else {
        const int i = blockIdx.y * 256 + threadIdx.x;
        if (2 * i >= hidden) return;
        float s, c;
        sincosf(p * f[i], &s, &c);
        o[2 * i] = Elem<T>::load(row + 2 * i) * scale + s;
        if (2 * i + 1 < hidden) o[2 * i + 1] = Elem<T>::load(row + 2 * i + 1) * scale + c;
    }
}

template <typename T>
static void launch_embed_waves(const T* table, const int* ids, const int* positions, const float* f, float* out, int n, int hidden,
                               int vocab, float scale, hipStream_t stream) {
    const bool wide = hidden % 4 == 0 && (uintptr_t)table % (4 * sizeof(T)) == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)f % 8 == 0;
    const int per = wide ? 1024 : 512;
    const dim3 grid(n, (hidden + per - 1) / per);
    if (wide) embed_waves_kernel<T, true><<<grid, 256, 0, stream>>>(table, ids, positions, f, out, hidden, vocab, scale);
    else embed_waves_kernel<T, false><<<grid, 256, 0, stream>>>(table, ids, positions, f, out, hidden, vocab, scale);
}

extern "C" int tm_embed_waves(const void* table, int dtype, const int* ids, const int* positions, const float* f, float* out, int T,
                              int hidden, int vocab, float scale, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (!table || !ids || !positions || !f || !out || hidden <= 0 || hidden > 65535 * 512 || vocab <= 0) return TM_ERR_ARG;
    if (dtype == TM_F32)
        launch_embed_waves<float>((const float*)table, ids, positions, f, out, T, hidden, vocab, scale, stream);
    else if (dtype == TM_BF16)
        launch_embed_waves<bf16_t>((const bf16_t*)table, ids, positions, f, out, T, hidden, vocab, scale, stream);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}
