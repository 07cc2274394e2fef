// Single tokens through a recurrent mixer in one launch: everything between the input projections and the output projection.
//
//   tm_retention_step   rotation, S <- decay S + k v^T, o = S^T q, o / rms(o) * silu(g); with `silu` q, k and v are silu of the
//                       projection; with o_out the heads' o go there in 32-bit as they are (a norm over all heads follows)
//   tm_delta_step       short convolutions and their state, silu, unit norms, step sizes and decays,
//                       S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q,   rms norm with a weight, gate
//
// A block is a request and a head of the retention, or a request and a q/k head of the delta rule with all value heads that
// read it (so that nobody else touches the convolution state of its channels); its sixteen wavefronts share the state: a wavefront has
// 64 columns and a share of their rows, a lane a column, so that a row is read and written in runs of 256 bytes. A column's partial
// sums are added in the order of the wavefronts. All of it is 32-bit but the operands of the model's type; the result is rounded
// once. The same mathematics as retention.hip and delta_rule.hip, sums in another order.
#include "common.h"
#include "api.h"

#define RS_WAVES 16
#define RS_THREADS (RS_WAVES * TM_WAVE)
#define RS_MAX_D 256
#define RS_MAX_TAPS 16

__device__ __forceinline__ float rs_silu(float z) { return z / (1.0f + expf(-z)); }

// ------------------------------------------------------------------------------------------------ retention

// grid (H, requests). Column groups of 64: nc = ceil(Dv / 64) <= 16; wavefront w takes group w % nc and the rows of share w / nc of
// RG = 16 / nc shares.
template <typename T>
__global__ __launch_bounds__(RS_THREADS) void retention_step_kernel(const T* __restrict__ proj, int ld, const float* __restrict__ cos_t,
                                                                   const float* __restrict__ sin_t, int rot, const int* __restrict__ positions,
                                                                   const float* __restrict__ decay, float* __restrict__ state,
                                                                   const int* __restrict__ slots, T* __restrict__ y, int H, int D, int Dv,
                                                                   float k_scale, float eps, int silu, float* __restrict__ o_out) {
    auto in = [&](const T* p) {
        const float z = Elem<T>::load(p);
        return silu ? rs_silu(z) : z;
    };
    __shared__ float q_s[RS_MAX_D], k_s[RS_MAX_D], part[RS_THREADS], red[RS_WAVES];
    const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, wave = tid / TM_WAVE, lane = tid % TM_WAVE;
    const T* row = proj + (size_t)t * ld;
    const T* q = row + h * D;
    const T* k = row + H * D + h * D;
    const int half = rot / 2;
    for (int j = tid; j < half; j += RS_THREADS) {
        const float c = cos_t[(size_t)positions[t] * half + j], s = sin_t[(size_t)positions[t] * half + j];
        float a, b;
        rotate_pair(in(q + j), in(q + j + half), c, s, a, b);
        q_s[j] = a;
        q_s[j + half] = b;
        rotate_pair(in(k + j), in(k + j + half), c, s, a, b);
        k_s[j] = a * k_scale;
        k_s[j + half] = b * k_scale;
    }
    for (int d = rot + tid; d < D; d += RS_THREADS) {
        q_s[d] = in(q + d);
        k_s[d] = in(k + d) * k_scale;
    }
    const int nc = (Dv + TM_WAVE - 1) / TM_WAVE, RG = RS_WAVES / nc;
    const int cg = wave % nc, rg = wave / nc;
    const int e = cg * TM_WAVE + lane;
    const bool mine = rg < RG && e < Dv;
    const float v = mine ? in(row + 2 * H * D + h * Dv + e) : 0.f;
    const float a = decay[h * D];
    float* st = state + (((size_t)slots[t] * H + h) * D) * Dv + (mine ? e : 0);
    __syncthreads();
    const int R = (D + RG - 1) / RG, d0 = rg * R, d1 = min(D, d0 + R);
    float acc = 0.f;
    if (mine) {
        int d = d0;
        for (; d + 8 <= d1; d += 8) {                   // eight rows on their way at a time
            float S[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) S[i] = st[(size_t)(d + i) * Dv];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                S[i] = a * S[i] + k_s[d + i] * v;
                acc += S[i] * q_s[d + i];
                st[(size_t)(d + i) * Dv] = S[i];
            }
        }
        for (; d < d1; ++d) {
            const float S = a * st[(size_t)d * Dv] + k_s[d] * v;
            acc += S * q_s[d];
            st[(size_t)d * Dv] = S;
        }
    }
    part[tid] = acc;
    __syncthreads();
    // threads 0 .. 64 nc - 1: the columns' results, and the head's norm
    float o = 0.f;
    const bool out = tid < Dv;
    if (out)
        for (int i = 0; i < RG; ++i) o += part[i * nc * TM_WAVE + tid];
    if (o_out) {
        if (out) o_out[((size_t)t * H + h) * Dv + tid] = o;
        return;
    }
    const float ss = block_sum<RS_THREADS>(o * o, red);
    if (out) {
        const float g = Elem<T>::load(row + 2 * H * D + H * Dv + h * Dv + tid);
        Elem<T>::store(y + ((size_t)t * H + h) * Dv + tid, o * (1.0f / sqrtf(ss / (float)Dv + eps)) * rs_silu(g));
    }
}

extern "C" int tm_retention_step(const void* proj, int ld, int dtype, const float* cos_t, const float* sin_t, int rot, const int* positions,
                                 const float* decay, float* state, const int* state_slots, void* y, int n, int H, int D, int Dv,
                                 float k_scale, float eps, int silu, float* o_out, hipStream_t stream) {
    if (n <= 0) return TM_OK;
    if (!proj || !decay || !state || !state_slots || (!y && !o_out) || H <= 0 || D <= 0 || D > RS_MAX_D || Dv <= 0 || Dv > RS_THREADS || rot < 0 || rot > D ||
        (rot & 1) || (rot && (!cos_t || !sin_t || !positions)) || ld < (o_out ? H * (2 * D + Dv) : 2 * H * (D + Dv)) || n > 65535 || !(eps > 0.f))
        return TM_ERR_ARG;
    const dim3 grid(H, n);
    if (dtype == TM_F32)
        retention_step_kernel<float><<<grid, RS_THREADS, 0, stream>>>((const float*)proj, ld, cos_t, sin_t, rot, positions, decay, state,
                                                                      state_slots, (float*)y, H, D, Dv, k_scale, eps, silu, o_out);
    else if (dtype == TM_BF16)
        retention_step_kernel<bf16_t><<<grid, RS_THREADS, 0, stream>>>((const bf16_t*)proj, ld, cos_t, sin_t, rot, positions, decay, state,
                                                                       state_slots, (bf16_t*)y, H, D, Dv, k_scale, eps, silu, o_out);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------------ delta rule

// A channel of the token behind the convolution and silu; the request's convolution state moves on by the token. TAPS 0: any number,
// one after the other.
template <typename T, int TAPS>
__device__ __forceinline__ float rs_conv_taps(const T* __restrict__ x, const T* __restrict__ conv_w, T* __restrict__ st, int C, int taps,
                                              int c) {
    const T now = x[c];
    const T* w = conv_w + (size_t)c * taps;
    float acc = 0.f;
    if constexpr (TAPS > 0) {
        T held[TAPS > 1 ? TAPS - 1 : 1];
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) held[j] = st[(size_t)j * C + c];
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) acc += Elem<T>::load(w + j) * Elem<T>::load(held + j);
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) st[(size_t)j * C + c] = j + 1 < TAPS - 1 ? held[j + 1] : now;
    } else {
        for (int j = 0; j < taps - 1; ++j) {
            const T held = st[(size_t)j * C + c];
            acc += Elem<T>::load(w + j) * Elem<T>::load(&held);
            if (j > 0) st[(size_t)(j - 1) * C + c] = held;
        }
        st[(size_t)(taps - 2) * C + c] = now;
    }
    acc += Elem<T>::load(w + taps - 1) * Elem<T>::load(&now);
    return rs_silu(acc);
}

template <typename T>
__device__ __forceinline__ float rs_conv(const T* __restrict__ x, const T* __restrict__ conv_w, T* __restrict__ st, int C, int taps, int c) {
    switch (taps) {
        case 1: return rs_conv_taps<T, 1>(x, conv_w, st, C, taps, c);
        case 2: return rs_conv_taps<T, 2>(x, conv_w, st, C, taps, c);
        case 3: return rs_conv_taps<T, 3>(x, conv_w, st, C, taps, c);
        case 4: return rs_conv_taps<T, 4>(x, conv_w, st, C, taps, c);
        default: return rs_conv_taps<T, 0>(x, conv_w, st, C, taps, c);
    }
}

// grid (G, requests). The columns of the group's rep = H / G value heads stand side by side, every head's filled up to a multiple of
// 64: nc = rep ceil(Dv / 64) <= 16 groups; wavefront w takes group w % nc and the rows of share w / nc of RG = 16 / nc shares, at most
// RMAX of them. LDS: q, k [D]; v [rep Dv]; decays [rep D]; two partial sums a thread; o [rep Dv].
template <typename T, int RMAX>
__global__ __launch_bounds__(RS_THREADS) void delta_step_kernel(const T* __restrict__ proj, int ld, const T* __restrict__ conv_w,
                                                               T* __restrict__ conv_state, const float* __restrict__ ba, int ldba,
                                                               const float* __restrict__ z, int ldz, const float* __restrict__ a_log,
                                                               const float* __restrict__ dt_bias, const T* __restrict__ gate, int ldg,
                                                               int sigmoid, const float* __restrict__ norm_w, float* __restrict__ state,
                                                               const int* __restrict__ slots, T* __restrict__ y, int H, int G, int D, int Dv,
                                                               int taps, float unit_eps, float eps) {
    extern __shared__ float lds[];
    __shared__ float sums[4], inv[RS_WAVES];
    const int g = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, wave = tid / TM_WAVE, lane = tid % TM_WAVE;
    const int rep = H / G, C = 2 * G * D + H * Dv;
    float* q_s = lds;
    float* k_s = q_s + D;
    float* v_s = k_s + D;
    float* g_s = v_s + rep * Dv;
    float* part = g_s + rep * D;                        // [2][RS_THREADS]
    float* o_s = part + 2 * RS_THREADS;
    const T* row = proj + (size_t)t * ld;
    T* cst = conv_state + (size_t)slots[t] * (taps - 1) * C;
    // the state's rows of this thread: on their way while the operands are made
    const int per_head = (Dv + TM_WAVE - 1) / TM_WAVE, nc = rep * per_head, RG = RS_WAVES / nc;
    const int cg = wave % nc, rg = wave / nc, hh = cg / per_head, e = (cg % per_head) * TM_WAVE + lane;
    const int h = g * rep + hh;
    const bool mine = rg < RG && e < Dv;
    const int R = (D + RG - 1) / RG, d0 = rg * R;
    float* st = state + (((size_t)slots[t] * H + h) * D) * Dv + (mine ? e : 0);
    float S[RMAX];
#pragma unroll
    for (int i = 0; i < RMAX; ++i) S[i] = (mine && i < R && d0 + i < D) ? st[(size_t)(d0 + i) * Dv] : 0.f;
    for (int c = tid; c < 2 * D + rep * Dv; c += RS_THREADS) {
        const int at = c < D ? g * D + c : c < 2 * D ? G * D + g * D + (c - D) : 2 * G * D + g * rep * Dv + (c - 2 * D);
        lds[c] = rs_conv<T>(row, conv_w, cst, C, taps, at);      // q_s, k_s and v_s lie behind each other
    }
    for (int n = tid; n < rep * D; n += RS_THREADS) {
        const int head = g * rep + n / D;
        const float a = z ? z[(size_t)t * ldz + (size_t)g * rep * D + n] + dt_bias[(size_t)g * rep * D + n]
                          : ba[(size_t)t * ldba + H + head] + dt_bias[head];
        const float sp = fmaxf(a, 0.f) + log1pf(expf(-fabsf(a)));            // softplus
        g_s[n] = expf(-expf(a_log[head]) * sp);
    }
    __syncthreads();
    if (wave < 3) {                                     // sum q^2, sum k^2, q . k
        float s = 0.f;
        for (int d = lane; d < D; d += TM_WAVE) s += (wave == 1 ? k_s[d] : q_s[d]) * (wave == 0 ? q_s[d] : k_s[d]);
        s = wave_sum(s);
        if (lane == 0) sums[wave] = s;
    }
    __syncthreads();
    const float iq = (1.0f / sqrtf((float)D)) / sqrtf(sums[0] + unit_eps), ik = 1.0f / sqrtf(sums[1] + unit_eps), kq = sums[2] * iq * ik;
    float dk = 0.f, dq = 0.f;
#pragma unroll
    for (int i = 0; i < RMAX; ++i)
        if (i < R && d0 + i < D) {
            S[i] *= g_s[hh * D + d0 + i];
            dk += S[i] * (k_s[d0 + i] * ik);
            dq += S[i] * (q_s[d0 + i] * iq);
        }
    part[tid] = dk;
    part[RS_THREADS + tid] = dq;
    __syncthreads();
    if (mine) {
        dk = dq = 0.f;
        for (int i = 0; i < RG; ++i) {
            dk += part[i * nc * TM_WAVE + cg * TM_WAVE + lane];
            dq += part[RS_THREADS + i * nc * TM_WAVE + cg * TM_WAVE + lane];
        }
        const float beta = 1.0f / (1.0f + expf(-ba[(size_t)t * ldba + h]));
        const float u = beta * (v_s[hh * Dv + e] - dk);
#pragma unroll
        for (int i = 0; i < RMAX; ++i)
            if (i < R && d0 + i < D) st[(size_t)(d0 + i) * Dv] = S[i] + (k_s[d0 + i] * ik) * u;
        if (rg == 0) o_s[hh * Dv + e] = dq + u * kq;
    }
    __syncthreads();
    if (wave < rep) {                                   // a wavefront a head's norm
        float s = 0.f;
        for (int c = lane; c < Dv; c += TM_WAVE) s += o_s[wave * Dv + c] * o_s[wave * Dv + c];
        s = wave_sum(s);
        if (lane == 0) inv[wave] = 1.0f / sqrtf(s / (float)Dv + eps);
    }
    __syncthreads();
    for (int c = tid; c < rep * Dv; c += RS_THREADS) {
        const float x = Elem<T>::load(gate + (size_t)t * ldg + (size_t)g * rep * Dv + c);
        Elem<T>::store(y + (size_t)t * H * Dv + (size_t)g * rep * Dv + c,
                       norm_w[c % Dv] * (o_s[c] * inv[c / Dv]) * ((sigmoid ? 1.f : x) / (1.f + expf(-x))));
    }
}

// rows of a thread for these sizes, or 0: not taken
static int delta_step_rows(int H, int G, int D, int Dv) {
    if (H <= 0 || G <= 0 || H % G || D <= 0 || D > RS_MAX_D || Dv <= 0) return 0;
    const long long nc = (long long)(H / G) * ((Dv + TM_WAVE - 1) / TM_WAVE);
    if (nc > RS_WAVES) return 0;
    const int RG = RS_WAVES / (int)nc, R = (D + RG - 1) / RG;
    return R <= 32 ? R : 0;
}

extern "C" int tm_delta_step_takes(int H, int G, int D, int Dv) { return delta_step_rows(H, G, D, Dv) > 0 ? 1 : 0; }

// Operands as tm_delta_prepare's, of n single tokens: row t of proj, ba, z, gate and y is request t, whose state row is state_slots[t].
extern "C" int tm_delta_step(const void* proj, int ld, const void* conv_w, void* conv_state, const float* ba, int ldba, const float* z, int ldz,
                             const float* a_log, const float* dt_bias, const void* gate, int ldg, int sigmoid, const float* norm_w,
                             float* state, const int* state_slots, void* y, int n, int H, int G, int D, int Dv, int taps, float unit_eps,
                             float eps, int dtype, hipStream_t stream) {
    if (n <= 0) return TM_OK;
    const int R = delta_step_rows(H, G, D, Dv);
    if (!R || !proj || !conv_w || !ba || !a_log || !dt_bias || !gate || !norm_w || !state || !state_slots || !y || taps < 1 || taps > RS_MAX_TAPS ||
        (taps > 1 && !conv_state) || ld < 2 * G * D + H * Dv || ldba < (z ? H : 2 * H) || (z && ldz < H * D) || ldg < H * Dv || n > 65535 ||
        !(unit_eps > 0.f) || !(eps > 0.f) || (dtype != TM_F32 && dtype != TM_BF16))
        return TM_ERR_ARG;
    const int rep = H / G;
    const size_t lds = ((size_t)2 * D + rep * Dv + rep * D + 2 * RS_THREADS + rep * Dv) * sizeof(float);     // 23 KB at most
    const dim3 grid(G, n);
#define RS_GO(T_, R_)                                                                                                                \
    delta_step_kernel<T_, R_><<<grid, RS_THREADS, lds, stream>>>((const T_*)proj, ld, (const T_*)conv_w, (T_*)conv_state, ba, ldba, z, ldz, a_log, \
                                                                 dt_bias, (const T_*)gate, ldg, sigmoid, norm_w, state, state_slots, (T_*)y, H, \
                                                                 G, D, Dv, taps, unit_eps, eps)
    if (dtype == TM_F32) {
        if (R <= 16) RS_GO(float, 16); else RS_GO(float, 32);
    } else {
        if (R <= 16) RS_GO(bf16_t, 16); else RS_GO(bf16_t, 32);
    }
#undef RS_GO
    TM_CHECK_LAUNCH();
    return TM_OK;
}
