// What a retention's recurrence reads, from the stacked projection of a step: 32-bit rows [q (H D) | k (H D) | v (H Dv)]
//
//   (with `silu` q, k and v are silu of the projection)   q and k with the first `rot` channels of every head turned by the token's position (pairs (j, j + rot/2)), k times k_scale,
//   v as projected
//
// so that nothing is rounded between the projection and the recurrence (gla.hip, with decays that do not change from token
// to token). A wavefront a token and head.
#include "common.h"
#include "api.h"

template <typename T>
__global__ __launch_bounds__(TM_WAVE) void retention_prepare_kernel(const T* __restrict__ proj, int ld, const float* __restrict__ cos_t,
                                                                   const float* __restrict__ sin_t, int rot,
                                                                   const int* __restrict__ positions, float* __restrict__ rows, int ldr,
                                                                   int H, int D, int Dv, float k_scale, int silu) {
    auto in = [&](const T* p) {
        const float z = Elem<T>::load(p);
        return silu ? z / (1.0f + expf(-z)) : z;
    };
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const T* q = proj + (size_t)t * ld + h * D;
    const T* k = q + H * D;
    const T* v = proj + (size_t)t * ld + 2 * H * D + h * Dv;
    float* qo = rows + (size_t)t * ldr + h * D;
    float* ko = qo + H * D;
    float* vo = rows + (size_t)t * ldr + 2 * H * D + h * Dv;
    const int half = rot / 2;
    const float* cs = half ? cos_t + (size_t)positions[t] * half : nullptr;
    const float* sn = half ? sin_t + (size_t)positions[t] * half : nullptr;
    for (int j = lane; j < half; j += TM_WAVE) {
        const float c = cs[j], s = sn[j];
        float a, b;
        rotate_pair(in(q + j), in(q + j + half), c, s, a, b);
        qo[j] = a;
        qo[j + half] = b;
        rotate_pair(in(k + j), in(k + j + half), c, s, a, b);
        ko[j] = a * k_scale;
        ko[j + half] = b * k_scale;
    }
    for (int d = rot + lane; d < D; d += TM_WAVE) {
        qo[d] = in(q + d);
        ko[d] = in(k + d) * k_scale;
    }
    for (int e = lane; e < Dv; e += TM_WAVE) vo[e] = in(v + e);
}

extern "C" int tm_retention_prepare(const void* proj, int ld, int dtype, const float* cos_t, const float* sin_t, int rot,
                                    const int* positions, float* rows, int ldr, int T, int H, int D, int Dv, float k_scale, int silu,
                                    hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (!proj || !rows || H <= 0 || H > 65535 || D <= 0 || Dv <= 0 || rot < 0 || rot > D || (rot & 1) ||
        (rot && (!cos_t || !sin_t || !positions)) || ld < H * (2 * D + Dv) || ldr < H * (2 * D + Dv))
        return TM_ERR_ARG;
    const dim3 grid(T, H);
    if (dtype == TM_F32)
        retention_prepare_kernel<float><<<grid, TM_WAVE, 0, stream>>>((const float*)proj, ld, cos_t, sin_t, rot, positions, rows, ldr, H, D,
                                                                      Dv, k_scale, silu);
    else if (dtype == TM_BF16)
        retention_prepare_kernel<bf16_t><<<grid, TM_WAVE, 0, stream>>>((const bf16_t*)proj, ld, cos_t, sin_t, rot, positions, rows, ldr, H,
                                                                       D, Dv, k_scale, silu);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}
