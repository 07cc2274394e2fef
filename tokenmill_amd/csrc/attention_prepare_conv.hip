// What stands between the projection of q, k and v and an attention over the paged cache, for mixers with a short causal
// convolution over time on every projected channel:
//
//   proj row (model's type) = [H heads of q, D wide | G heads of k, D wide | G heads of v, Dv wide | ...]
//   u = sum_j w[c, j] * row(t - taps + 1 + j)[c]      rows before the step's own come from the request's state [taps - 1, channels]
//   q and k of u normed over the whole projection (or head by head, `per_head`), the first `rot` channels of every head turned by
//   the token's position, q to q_out, k and v to the token's cache slot: the operands and layouts of attention_prepare.hip
//
// Everything between the loads and the stores is 32-bit. A block a token, of more threads in a step of few tokens (a token's sums are
// then ordered otherwise). The rows from first_single on are the step's single tokens, one a request (request n_portions + row - first_single): a
// single token's block is the only one that touches its request's state, and moves it on itself. The state of the requests with
// longer portions is moved on by tm_delta_conv_state afterwards (other blocks still read it here).
#include "common.h"
#include "api.h"

#define CP_THREADS 256
#define CP_WIDE 1024                    // threads of a token's block in a step of few tokens
#define CP_MAX_TAPS 16
#define CP_MAX_FLOATS (36 * 1024)       // q and k of a token in LDS, and a norm per head of theirs

// VEC consecutive elements
template <typename T, int VEC> struct Vec { T v[VEC]; };
template <typename T, int VEC>
__device__ __forceinline__ Vec<T, VEC> vec_load(const T* p) {
    if constexpr (VEC == 1) return Vec<T, 1>{{*p}};
    else {
        union { Vec<T, VEC> v; uint4 q; uint2 d; } u;
        if constexpr (sizeof(T) * VEC == 16) u.q = *(const uint4*)p;
        else u.d = *(const uint2*)p;
        return u.v;
    }
}
template <typename T, int VEC>
__device__ __forceinline__ void vec_store(T* p, const Vec<T, VEC>& x) {
    if constexpr (VEC == 1) *p = x.v[0];
    else {
        union { Vec<T, VEC> v; uint4 q; uint2 d; } u;
        u.v = x;
        if constexpr (sizeof(T) * VEC == 16) *(uint4*)p = u.q;
        else *(uint2*)p = u.d;
    }
}

// VEC channels from c on of the token behind the convolution. TAPS 0: any number. For a single token (`move`) the state moves on.
template <typename T, int VEC, int TAPS>
__device__ __forceinline__ void cp_conv(const T* __restrict__ proj, int ld, const T* __restrict__ conv_w, T* __restrict__ st, int C,
                                        int taps_, int first, int i, int c, bool move, float (&out)[VEC]) {
    const int taps = TAPS > 0 ? TAPS : taps_;
    Vec<T, VEC> w[TAPS > 0 ? TAPS : 1];             // VEC rows of `taps` weights lie behind each other
    if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j] = vec_load<T, VEC>(conv_w + (size_t)c * TAPS + VEC * j);
    }
    auto weight = [&](int e, int j) {
        if constexpr (TAPS > 0) return Elem<T>::load(&w[(e * TAPS + j) / VEC].v[(e * TAPS + j) % VEC]);
        else return Elem<T>::load(conv_w + (size_t)(c + e) * taps + j);
    };
#pragma unroll
    for (int e = 0; e < VEC; ++e) out[e] = 0.f;
    Vec<T, VEC> x[TAPS > 0 ? TAPS : CP_MAX_TAPS];
#pragma unroll
    for (int j = 0; j < (TAPS > 0 ? TAPS : CP_MAX_TAPS); ++j) {
        if (j >= taps) break;
        const int at = i - (taps - 1) + j;          // < 0: before this step's rows, in the state
        x[j] = at >= 0 ? vec_load<T, VEC>(proj + (size_t)(first + at) * ld + c) : vec_load<T, VEC>(st + (size_t)(taps - 1 + at) * C + c);
    }
#pragma unroll
    for (int j = 0; j < (TAPS > 0 ? TAPS : CP_MAX_TAPS); ++j) {
        if (j >= taps) break;
#pragma unroll
        for (int e = 0; e < VEC; ++e) out[e] += weight(e, j) * Elem<T>::load(&x[j].v[e]);
    }
    if (move) {
#pragma unroll
        for (int j = 0; j + 1 < (TAPS > 0 ? TAPS : CP_MAX_TAPS); ++j) {
            if (j + 1 >= taps) break;
            vec_store<T, VEC>(st + (size_t)j * C + c, x[j + 1]);
        }
    }
}

template <typename T, int VEC, int TAPS, int NT>
__global__ __launch_bounds__(NT) void conv_norm_rope_store_kernel(
    const T* __restrict__ proj, int ld, const T* __restrict__ conv_w, T* __restrict__ conv_state, int taps, const int* __restrict__ cu,
    const int* __restrict__ state_slots, const int* __restrict__ seq_of_token, int first_single, int n_portions, T* __restrict__ q_out, int H,
    int G, int D, int Dv, int rot, int interleaved, const float* __restrict__ q_w, const float* __restrict__ k_w, float eps, int per_head,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, const int* __restrict__ positions, const int* __restrict__ slots,
    T* __restrict__ k_pool, T* __restrict__ v_pool, int page) {
    extern __shared__ __align__(16) float lds[];
    __shared__ float red[NT / TM_WAVE];
    const int t = blockIdx.x, tid = threadIdx.x;
    const int Q = H * D, K = G * D, QK = Q + K, V = G * Dv, C = QK + V;
    float* xs = lds;                                // q and k behind the convolution
    float* inv_head = lds + QK;                     // [H + G] with per_head
    const bool single = t >= first_single;
    const int s = single ? n_portions + t - first_single : seq_of_token[t];
    const int first = single ? t : cu[s], i = t - first;
    T* st = conv_state + (size_t)state_slots[s] * (taps - 1) * C;
    const int slot = slots[t];
    float sq = 0.f, sk = 0.f;
    for (int c = tid * VEC; c < QK; c += NT * VEC) {        // (Q is a multiple of VEC: a piece is all of q or all of k)
        float u[VEC];
        cp_conv<T, VEC, TAPS>(proj, ld, conv_w, st, C, taps, first, i, c, single, u);
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            xs[c + e] = u[e];
            ss += u[e] * u[e];
        }
        if (c < Q) sq += ss;
        else sk += ss;
    }
    if (slot >= 0 || single) {
        const size_t vbase = slot >= 0 ? (size_t)(slot / page) * V * page + slot % page : 0;
        for (int c = tid * VEC; c < V; c += NT * VEC) {
            float u[VEC];
            cp_conv<T, VEC, TAPS>(proj, ld, conv_w, st, C, taps, first, i, QK + c, single, u);
            if (slot >= 0)
#pragma unroll
                for (int e = 0; e < VEC; ++e) Elem<T>::store(v_pool + vbase + (size_t)(c + e) * page, u[e]);
        }
    }
    float rq = 1.f, rk = 1.f;
    const bool normed = q_w != nullptr;
    if (normed && per_head) {                       // a wavefront a head
        __syncthreads();
        const int wave = tid / TM_WAVE, lane = tid % TM_WAVE;
        for (int hh = wave; hh < H + G; hh += NT / TM_WAVE) {
            float ss = 0.f;
            for (int d = lane; d < D; d += TM_WAVE) ss += xs[hh * D + d] * xs[hh * D + d];
            ss = wave_sum(ss);
            if (lane == 0) inv_head[hh] = 1.0f / sqrtf(ss / (float)D + eps);
        }
    } else if (normed) {
        rq = 1.0f / sqrtf(block_sum<NT>(sq, red) / (float)Q + eps);
        rk = 1.0f / sqrtf(block_sum<NT>(sk, red) / (float)K + eps);
    }
    __syncthreads();
    const int half = cos_t ? rot / 2 : 0;
    const float* cs = half ? cos_t + (size_t)positions[t] * half : nullptr;
    const float* sn = half ? sin_t + (size_t)positions[t] * half : nullptr;
    T* qo = q_out + (size_t)t * Q;
    T* ko = slot >= 0 ? k_pool + (size_t)slot * K : nullptr;
    // channel c of q | k, normed
    auto value = [&](int c) {
        float x = xs[c];
        if (!normed) return x;
        const int hh = c / D;
        const float r = per_head ? inv_head[hh] : c < Q ? rq : rk;
        const int wi = per_head ? c - hh * D : c < Q ? c : c - Q;
        return (c < Q ? q_w : k_w)[wi] * (x * r);
    };
    auto put = [&](int c, float y) {
        if (c < Q) Elem<T>::store(qo + c, y);
        else if (ko) Elem<T>::store(ko + (c - Q), y);
    };
    if (half) {
        for (int idx = tid; idx < (H + G) * half; idx += NT) {
            const int hh = idx / half, j = idx % half;
            const int a = hh * D + (interleaved ? 2 * j : j), b = hh * D + (interleaved ? 2 * j + 1 : j + half);
            float y1, y2;
            rotate_pair(value(a), value(b), cs[j], sn[j], y1, y2);
            put(a, y1);
            put(b, y2);
        }
        const int rest = D - 2 * half;
        for (int idx = tid; idx < (H + G) * rest; idx += NT) {
            const int c = idx / rest * D + 2 * half + idx % rest;
            put(c, value(c));
        }
        return;
    }
    for (int c = tid * VEC; c < QK; c += NT * VEC) {
        if (c >= Q && !ko) continue;
        Vec<T, VEC> y;
#pragma unroll
        for (int e = 0; e < VEC; ++e) Elem<T>::store(&y.v[e], value(c + e));
        vec_store<T, VEC>(c < Q ? qo + c : ko + (c - Q), y);
    }
}

extern "C" int tm_conv_norm_rope_store(const void* proj, int ld, int dtype, const void* conv_w, void* conv_state, int taps,
                                       const int* cu_q_lens, const int* state_slots, const int* seq_of_token, int T, int first_single,
                                       int n_portions, void* q_out, int H, int G, int D, int Dv, int rot, int interleaved, const float* q_w,
                                       const float* k_w, float eps, int per_head, const float* cos_t, const float* sin_t,
                                       const int* positions, const int* slots, void* k_pool, void* v_pool, int page, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (!proj || !conv_w || taps < 1 || taps > CP_MAX_TAPS || (taps > 1 && !conv_state) || !cu_q_lens || !state_slots || !seq_of_token ||
        first_single < 0 || first_single > T || n_portions < 0 || !q_out || H <= 0 || G <= 0 || D <= 0 || Dv <= 0 || rot < 0 || rot > D ||
        (rot & 1) || (q_w == nullptr) != (k_w == nullptr) || (q_w && !(eps > 0.f)) || (cos_t && rot && (!sin_t || !positions)) || !slots ||
        !k_pool || !v_pool || page <= 0 || (dtype != TM_F32 && dtype != TM_BF16))
        return TM_ERR_ARG;
    const long long floats = (long long)(H + G) * D + H + G, channels = (long long)(H + G) * D + (long long)G * Dv;
    if (floats > CP_MAX_FLOATS || ld < channels) return TM_ERR_ARG;
    const int e = dtype == TM_F32 ? 4 : 2, b = 4 * e;
    auto al = [&](const void* p) { return ((uintptr_t)p % b) == 0; };
    const bool vec = D % 4 == 0 && (G * Dv) % 4 == 0 && ld % 4 == 0 && al(proj) && al(conv_w) && al(conv_state) && al(q_out) && al(k_pool);
    const size_t bytes = (size_t)floats * sizeof(float);
#define CP_RUN(T_, V_, TAPS_, NT_)                                                                                                            \
    do {                                                                                                                                  \
        auto fn = conv_norm_rope_store_kernel<T_, V_, TAPS_, NT_>;                                                                         \
        if (bytes > 48 * 1024 && hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, CP_MAX_FLOATS * 4) != hipSuccess) \
            return TM_ERR_LAUNCH;                                                                                                         \
        fn<<<T, NT_, bytes, stream>>>((const T_*)proj, ld, (const T_*)conv_w, (T_*)conv_state, taps, cu_q_lens, state_slots,       \
                                             seq_of_token, first_single, n_portions, (T_*)q_out, H, G, D, Dv, rot, interleaved, q_w, k_w, \
                                             eps, per_head, cos_t, sin_t, positions, slots, (T_*)k_pool, (T_*)v_pool, page);              \
    } while (0)
#define CP_GO(T_, V_, TAPS_)                     \
    do {                                         \
        if (T < 256) CP_RUN(T_, V_, TAPS_, CP_WIDE); \
        else CP_RUN(T_, V_, TAPS_, CP_THREADS);  \
    } while (0)
#define CP_TAPS(T_)                                     \
    if (!vec) CP_GO(T_, 1, 0);                          \
    else switch (taps) {                                \
        case 1: CP_GO(T_, 4, 1); break;                 \
        case 2: CP_GO(T_, 4, 2); break;                 \
        case 3: CP_GO(T_, 4, 3); break;                 \
        case 4: CP_GO(T_, 4, 4); break;                 \
        default: CP_GO(T_, 4, 0);                       \
    }
    if (dtype == TM_F32) { CP_TAPS(float) } else { CP_TAPS(bf16_t) }
#undef CP_TAPS
#undef CP_GO
#undef CP_RUN
    TM_CHECK_LAUNCH();
    return TM_OK;
}
