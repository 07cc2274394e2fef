// Recurrences with a matrix of state per request and head, over the portions of prompts, in chunks of 64 tokens on the 32-bit
// matrix unit. Inside a chunk the recurrence is written out as products of small matrices; only the state crosses from one
// chunk to the next.
//
// Delta rule (delta_rule.hip), S_t = g_t S_(t-1) + k_t u_t^T with u_t = beta_t (v_t - (g_t S_(t-1))^T k_t), o_t = S_t^T q_t, g_t a
// decay per key channel (or per head: the same for all channels). With G_t = g_1 ... g_t, channel by channel, from the state S at
// the chunk's start:
//
//   (I + A) U = B (V - (G K) S),   A_ts = beta_t sum_d k_td k_sd G_td / G_sd  (s < t),   B = diag(beta)
//   U = U0 + W S,                  U0 = (I + A)^-1 B V,   W = -(I + A)^-1 B (G K)
//   O = (G Q) S + P U,             P_ts = sum_d q_td k_sd G_td / G_sd         (s <= t)
//   S' = G_n S + (G_n / G K)^T U
//
// Retention (retention.hip), S_t = decay S_(t-1) + k_t v_t^T: the same with U = V and G_t = decay^t.
//
//   tm_delta_chunks      per chunk and head: W, U0, P, G Q, (G_n / G K)^T and G_n, from the rows of tm_delta_prepare
//   tm_retention_chunks  likewise P, G Q, (G_n / G K)^T and G_n, from the rows of tm_retention_prepare
//   tm_chunk_chain       the chain over a request's chunks: writes o and the request's new state
//
// No ratio of decays is ever above one or taken of two underflowed numbers: logarithms are summed inside sub-blocks of 16 tokens,
// a pair of tokens of one sub-block takes the exponential of their difference, and across sub-blocks each side brings a factor of
// at most one (from its own token to a sub-block border between the two). All of it is 32-bit; a token's result depends on its
// own request's rows and state only, and on the cutting of the prompt by the order of 32-bit sums.
#include "common.h"
#include "api.h"

#define CS_C 64                              // tokens of a chunk
#define CS_SUB 16                            // tokens of a sub-block
#define CS_A_STRIDE 68                       // floats between rows of A in LDS (16-byte aligned)
#define CS_PREP 512
#define CS_CHAIN 256

typedef float cs_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ cs_f32x4 cs_mfma(float a, float b, cs_f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// ------------------------------------------------------------------------------------------------ the delta rule's chunks

// grid (H, chunks). DP: the key size rounded up (64 or 128); channels from D on are zeros everywhere.
template <int DP>
__global__ __launch_bounds__(CS_PREP) void delta_chunks_kernel(const float* __restrict__ rows, int ld, const int* __restrict__ cu_chunk,
                                                              float* __restrict__ Wm, float* __restrict__ Qm, float* __restrict__ Km,
                                                              float* __restrict__ Pm, float* __restrict__ gam, float* __restrict__ u0,
                                                              int H, int G, int D, int Dv, int per_channel) {
    constexpr int LD = DP + 4;
    extern __shared__ __align__(16) float lds[];
    // what is read at addresses without a lane in them stands first, inside the reach of an instruction's own offset
    float* As = lds;                                    // [64][CS_A_STRIDE]
    float* beta = As + CS_C * CS_A_STRIDE;              // [64]
    float* tot = beta + CS_C;                           // [4][DP]: a sub-block's sum
    float* Ks = tot + 4 * DP;                           // [64][LD]
    float* Ls = Ks + CS_C * LD;                         // log2 of the decays, summed inside a sub-block
    float* Qs = Ls + CS_C * LD;
    const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x;
    const int g_head = h / (H / G);
    const int row0 = cu_chunk[c], n = cu_chunk[c + 1] - row0;
    const int C = 2 * G * D + H * Dv;
    const size_t at = (size_t)c * H + h;
    for (int idx = tid; idx < CS_C * DP; idx += CS_PREP) {
        const int t = idx / DP, d = idx % DP;
        float k = 0.f, q = 0.f, lg = 0.f;
        if (t < n && d < D) {
            const float* row = rows + (size_t)(row0 + t) * ld;
            q = row[g_head * D + d];
            k = row[G * D + g_head * D + d];
            // a decay below 2^-150 is zero to everything it multiplies
            lg = fmaxf(log2f(per_channel ? row[C + 2 * H + G + h * D + d] : row[C + H + h]), -150.f);
        }
        Ks[t * LD + d] = k;
        Qs[t * LD + d] = q;
        Ls[t * LD + d] = lg;
    }
    if (tid < CS_C) beta[tid] = tid < n ? rows[(size_t)(row0 + tid) * ld + C + h] : 0.f;
    __syncthreads();
    for (int idx = tid; idx < 4 * DP; idx += CS_PREP) {
        const int I = idx / DP, d = idx % DP;
        float sum = 0.f;
#pragma unroll
        for (int t = 0; t < CS_SUB; ++t) {
            sum += Ls[(CS_SUB * I + t) * LD + d];
            Ls[(CS_SUB * I + t) * LD + d] = sum;
        }
        tot[I * DP + d] = sum;
    }
    __syncthreads();
    float* Pg = Pm + at * CS_C * CS_C;
    // pairs of one sub-block: a thread a pair
    for (int p = tid; p < 4 * CS_SUB * CS_SUB; p += CS_PREP) {
        const int I = p >> 8, t = CS_SUB * I + ((p >> 4) & 15), s = CS_SUB * I + (p & 15);
        float a = 0.f, b = 0.f;
        if (s <= t) {
            for (int d = 0; d < DP; d += 4) {
                const cs_f32x4 kt = *(const cs_f32x4*)(Ks + t * LD + d), qt = *(const cs_f32x4*)(Qs + t * LD + d);
                const cs_f32x4 ks = *(const cs_f32x4*)(Ks + s * LD + d);
                const cs_f32x4 lt = *(const cs_f32x4*)(Ls + t * LD + d), lsv = *(const cs_f32x4*)(Ls + s * LD + d);
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float e = ks[i] * __builtin_amdgcn_exp2f(lt[i] - lsv[i]);
                    a += kt[i] * e;
                    b += qt[i] * e;
                }
            }
        }
        As[t * CS_A_STRIDE + s] = s < t ? beta[t] * a : 0.f;
        Pg[t * CS_C + s] = b;
    }
    // pairs of two sub-blocks I > J: a wavefront two of them, on the matrix unit
    {
        const int wave = __builtin_amdgcn_readfirstlane(tid / TM_WAVE), lane = tid % TM_WAVE, r = lane % 16, g = lane / 16;
        if (wave < 6) {
            const int I = wave < 1 ? 1 : wave < 3 ? 2 : 3, J = wave < 1 ? 0 : wave < 3 ? wave - 1 : wave - 3;
            const int tr = CS_SUB * I + r, sr = CS_SUB * J + r;
            cs_f32x4 accA = {0.f, 0.f, 0.f, 0.f}, accP = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
            for (int dt = 0; dt < DP / 16; ++dt) {
                const int d = 16 * dt + 4 * g;
                const cs_f32x4 kt = *(const cs_f32x4*)(Ks + tr * LD + d), qt = *(const cs_f32x4*)(Qs + tr * LD + d);
                const cs_f32x4 lt = *(const cs_f32x4*)(Ls + tr * LD + d);
                const cs_f32x4 ks = *(const cs_f32x4*)(Ks + sr * LD + d), lsv = *(const cs_f32x4*)(Ls + sr * LD + d);
                cs_f32x4 between = *(const cs_f32x4*)(tot + J * DP + d) - lsv;              // from token s to the end of its sub-block,
                for (int M = J + 1; M < I; ++M) between += *(const cs_f32x4*)(tot + M * DP + d);     // and on to the start of t's
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float ft = __builtin_amdgcn_exp2f(lt[i]), ks_i = ks[i] * __builtin_amdgcn_exp2f(between[i]);
                    accA = cs_mfma(kt[i] * ft, ks_i, accA);
                    accP = cs_mfma(qt[i] * ft, ks_i, accP);
                }
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = CS_SUB * I + 4 * g + i, s = CS_SUB * J + r;
                As[t * CS_A_STRIDE + s] = beta[t] * accA[i];
                Pg[t * CS_C + s] = accP[i];
            }
        }
    }
    // what the chain reads of the tokens themselves
    float* Qg = Qm + at * CS_C * DP;
    float* Kg = Km + at * CS_C * DP;
    for (int idx = tid; idx < CS_C * DP; idx += CS_PREP) {
        const int t = idx / DP, d = idx % DP;
        float before = Ls[t * LD + d];
        for (int M = 0; M < t / CS_SUB; ++M) before += tot[M * DP + d];
        Qg[idx] = Qs[t * LD + d] * __builtin_amdgcn_exp2f(before);
    }
    for (int idx = tid; idx < CS_C * DP; idx += CS_PREP) {
        const int d = idx / CS_C, t = idx % CS_C, I = t / CS_SUB;
        float after = tot[I * DP + d] - Ls[t * LD + d];
        for (int M = I + 1; M < 4; ++M) after += tot[M * DP + d];
        Kg[idx] = Ks[t * LD + d] * __builtin_amdgcn_exp2f(after);
    }
    for (int d = tid; d < DP; d += CS_PREP)
        gam[at * DP + d] = __builtin_amdgcn_exp2f(tot[d] + tot[DP + d] + tot[2 * DP + d] + tot[3 * DP + d]);
    __syncthreads();
    // (I + A) X = B (G K) and = B V, a thread a column, from the first token on; the columns of the first DP threads are W's
    float* Wg = Wm + at * CS_C * DP;
    for (int col = tid; col < DP + Dv; col += CS_PREP) {
        const bool is_w = __builtin_amdgcn_readfirstlane(col) < DP;      // the same for a wavefront's lanes (DP is a multiple of 64)
        float x[CS_C];
        if (is_w) {
            float before = 0.f;
#pragma unroll
            for (int t = 0; t < CS_C; ++t) {
                x[t] = beta[t] * (Ks[t * LD + col] * __builtin_amdgcn_exp2f(before + Ls[t * LD + col]));
                if (t % CS_SUB == CS_SUB - 1) before += tot[t / CS_SUB * DP + col];
            }
        } else {
            // rows beyond the chunk's last: the last one again, with a beta of zero
            const float* v = rows + (size_t)row0 * ld + 2 * G * D + h * Dv + (col - DP);
            int off = 0;
#pragma unroll
            for (int t = 0; t < CS_C; ++t) {
                x[t] = beta[t] * v[off];
                off += t + 1 < n ? ld : 0;
                asm volatile("" : "+v"(off));            // (else 64 offsets are made ahead and held)
            }
        }
#pragma unroll
        for (int t = 1; t < CS_C; ++t) {
            float p0 = 0.f, p1 = 0.f;
#pragma unroll
            for (int s = 0; s < t; s += 4) {             // A is zero from its diagonal on
                const cs_f32x4 a = *(const cs_f32x4*)(As + t * CS_A_STRIDE + s);
                p0 += a[0] * x[s];
                p1 += a[1] * x[s + 1];
                p0 += a[2] * x[s + 2];
                p1 += a[3] * x[s + 3];
            }
            x[t] -= p0 + p1;
        }
        if (is_w) {
#pragma unroll
            for (int t = 0; t < CS_C; ++t) Wg[t * DP + col] = -x[t];
        } else {
            float* u = u0 + (size_t)c * CS_C * H * Dv + (size_t)h * Dv + (col - DP);
            int off = 0;
#pragma unroll
            for (int t = 0; t < CS_C; ++t) {
                u[off] = x[t];
                off += H * Dv;
                asm volatile("" : "+v"(off));
            }
        }
    }
}

static size_t delta_chunks_lds(int DP) { return ((size_t)3 * CS_C * (DP + 4) + CS_C * CS_A_STRIDE + 4 * DP + CS_C) * sizeof(float); }

// rows as tm_delta_prepare writes them; chunk c holds the rows cu_chunk[c] .. cu_chunk[c + 1] - 1 (1 to 64 of one request). Km, Qm,
// Wm float [n, H, 64 * DP] (Km as [DP][64]), Pm [n, H, 64, 64], gam [n, H, DP] with DP = 64 or 128 >= D, u0 [64 n, H Dv]
// (a chunk's 64 rows each, zeros behind its tokens).
extern "C" int tm_delta_chunks(const float* rows, int ld, const int* cu_chunk, int n_chunks, float* Wm, float* Qm, float* Km, float* Pm,
                               float* gam, float* u0, int H, int G, int D, int DP, int Dv, int per_channel, hipStream_t stream) {
    if (n_chunks <= 0) return TM_OK;
    if (!rows || !cu_chunk || !Wm || !Qm || !Km || !Pm || !gam || !u0 || H <= 0 || G <= 0 || H % G || D <= 0 || D > DP || Dv <= 0 ||
        n_chunks > 65535 ||
        (long long)ld < 2LL * G * D + (long long)H * Dv + 2 * H + G + (per_channel ? (long long)H * D : 0))
        return TM_ERR_ARG;
    const dim3 grid(H, n_chunks);
    const size_t lds = delta_chunks_lds(DP);
#define CS_GO(DP_)                                                                                                                   \
    do {                                                                                                                             \
        if (hipFuncSetAttribute((const void*)delta_chunks_kernel<DP_>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return TM_ERR_LAUNCH;                                                                                                    \
        delta_chunks_kernel<DP_><<<grid, CS_PREP, lds, stream>>>(rows, ld, cu_chunk, Wm, Qm, Km, Pm, gam, u0, H, G, D, Dv, per_channel); \
    } while (0)
    if (DP == 64) CS_GO(64);
    else if (DP == 128) CS_GO(128);
    else return TM_ERR_ARG;
#undef CS_GO
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------------ a retention's chunks

// grid (H, chunks)
template <int DP>
__global__ __launch_bounds__(CS_CHAIN) void retention_chunks_kernel(const float* __restrict__ rows, int ld, const int* __restrict__ cu_chunk,
                                                                   const float* __restrict__ decay, float* __restrict__ Qm,
                                                                   float* __restrict__ Km, float* __restrict__ Pm, float* __restrict__ gam,
                                                                   int H, int D) {
    constexpr int LD = DP + 4;
    extern __shared__ __align__(16) float lds[];
    float* Ks = lds;                                    // [64][LD]
    float* Qs = Ks + CS_C * LD;
    float* pw = Qs + CS_C * LD;                         // [65]: the decay's powers
    const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x;
    const int row0 = cu_chunk[c], n = cu_chunk[c + 1] - row0;
    const size_t at = (size_t)c * H + h;
    for (int idx = tid; idx < CS_C * DP; idx += CS_CHAIN) {
        const int t = idx / DP, d = idx % DP;
        const float* row = rows + (size_t)(row0 + t) * ld + h * D;
        const bool in = t < n && d < D;
        Qs[t * LD + d] = in ? row[d] : 0.f;
        Ks[t * LD + d] = in ? row[H * D + d] : 0.f;
    }
    if (tid <= CS_C) {                                  // each power by itself in 64-bit, rounded once
        const double x = (double)decay[h * D];
        double v = 1.0;
        for (int i = 0; i < tid; ++i) v *= x;
        pw[tid] = (float)v;
    }
    __syncthreads();
    float* Pg = Pm + at * CS_C * CS_C;
    const int wave = __builtin_amdgcn_readfirstlane(tid / TM_WAVE), lane = tid % TM_WAVE, r = lane % 16, g = lane / 16;
    for (int p = wave; p < 10; p += CS_CHAIN / TM_WAVE) {           // tiles on and below the diagonal
        const int I = p < 1 ? 0 : p < 3 ? 1 : p < 6 ? 2 : 3, J = p - I * (I + 1) / 2;
        cs_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int dt = 0; dt < DP / 16; ++dt) {
            const cs_f32x4 q4 = *(const cs_f32x4*)(Qs + (16 * I + r) * LD + 16 * dt + 4 * g);
            const cs_f32x4 k4 = *(const cs_f32x4*)(Ks + (16 * J + r) * LD + 16 * dt + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = cs_mfma(q4[i], k4[i], acc);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * I + 4 * g + i, s = 16 * J + r;
            Pg[t * CS_C + s] = s <= t ? acc[i] * pw[t - s] : 0.f;
        }
    }
    float* Qg = Qm + at * CS_C * DP;
    float* Kg = Km + at * CS_C * DP;
    for (int idx = tid; idx < CS_C * DP; idx += CS_CHAIN) {
        const int t = idx / DP, d = idx % DP;
        Qg[idx] = Qs[t * LD + d] * pw[t + 1];
    }
    for (int idx = tid; idx < CS_C * DP; idx += CS_CHAIN) {
        const int d = idx / CS_C, t = idx % CS_C;
        Kg[idx] = t < n ? Ks[t * LD + d] * pw[n - 1 - t] : 0.f;
    }
    for (int d = tid; d < DP; d += CS_CHAIN) gam[at * DP + d] = pw[n];
}

// rows as tm_retention_prepare writes them, decay float [H * D] (a head's D equal), the rest as tm_delta_chunks.
extern "C" int tm_retention_chunks(const float* rows, int ld, const int* cu_chunk, int n_chunks, const float* decay, float* Qm, float* Km,
                                   float* Pm, float* gam, int H, int D, int DP, hipStream_t stream) {
    if (n_chunks <= 0) return TM_OK;
    if (!rows || !cu_chunk || !decay || !Qm || !Km || !Pm || !gam || H <= 0 || D <= 0 || D > DP || n_chunks > 65535 || ld < 2 * H * D)
        return TM_ERR_ARG;
    const dim3 grid(H, n_chunks);
    const size_t lds = ((size_t)2 * CS_C * (DP + 4) + CS_C + 4) * sizeof(float);
#define CS_GO(DP_)                                                                                                                   \
    do {                                                                                                                             \
        if (lds > 64 * 1024 &&                                                                                                       \
            hipFuncSetAttribute((const void*)retention_chunks_kernel<DP_>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return TM_ERR_LAUNCH;                                                                                                    \
        retention_chunks_kernel<DP_><<<grid, CS_CHAIN, lds, stream>>>(rows, ld, cu_chunk, decay, Qm, Km, Pm, gam, H, D);             \
    } while (0)
    if (DP == 64) CS_GO(64);
    else if (DP == 128) CS_GO(128);
    else return TM_ERR_ARG;
#undef CS_GO
    TM_CHECK_LAUNCH();
    return TM_OK;
}

// ------------------------------------------------------------------------------------------------ the chain

// What a wavefront reads of a chunk, in the operands' places: rows r of its 16 tokens (or of its tiles of key channels), sixteen
// bytes at channel (or token) 4 g of every tile of 16.
template <int NDT, bool HAS_W>
struct ChunkRegs {
    static constexpr int NJ = NDT / 4;                  // tiles of 16 key channels of a wavefront's share of the state
    cs_f32x4 w[HAS_W ? NDT : 1], q[NDT], p[4], k[NJ][4], gam[NJ];
    float u[4];
};

template <int NDT, bool HAS_W>
__device__ __forceinline__ void load_chunk(ChunkRegs<NDT, HAS_W>& x, const float* __restrict__ Wm, const float* __restrict__ Qm,
                                           const float* __restrict__ Km, const float* __restrict__ Pm, const float* __restrict__ gam,
                                           const float* __restrict__ u0, int ldu, size_t at, int row0, int n, int wave, int r, int g,
                                           bool col) {
    constexpr int DP = 16 * NDT, NJ = ChunkRegs<NDT, HAS_W>::NJ;
    const size_t mine = (at * CS_C + 16 * wave + r) * DP + 4 * g;
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
        if (HAS_W) x.w[dt] = *(const cs_f32x4*)(Wm + mine + 16 * dt);
        x.q[dt] = *(const cs_f32x4*)(Qm + mine + 16 * dt);
    }
#pragma unroll
    for (int tt = 0; tt < 4; ++tt)
        if (tt <= wave) x.p[tt] = *(const cs_f32x4*)(Pm + (at * CS_C + 16 * wave + r) * CS_C + 16 * tt + 4 * g);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int dt = wave * NJ + j;
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) x.k[j][tt] = *(const cs_f32x4*)(Km + (at * DP + 16 * dt + r) * CS_C + 16 * tt + 4 * g);
        x.gam[j] = *(const cs_f32x4*)(gam + at * DP + 16 * dt + 4 * g);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * g + i;
        x.u[i] = (col && t < n) ? u0[(size_t)(row0 + t) * ldu] : 0.f;
    }
}

// grid (H, ceil(Dv / 16), requests); a block is four wavefronts and 16 columns of a request's and head's state. A wavefront owns 16
// of a chunk's tokens (rows of U and O) and a quarter of the state's rows. The matrix unit leaves a 16x16 result with four
// consecutive rows in a lane, and takes its second operand one row a lane: with the rows of every product's inner sum dealt the
// same way (row 16 tile + 4 g + i to lane group g, instruction i) a result is the next product's operand as it lies. U and S go
// through LDS (column by column, so that a lane's four rows are one piece) because every wavefront needs all their rows. The next
// chunk's operands are asked for before the current chunk is worked on.
// Neighbouring blocks are heads, so that (heads in multiples of eight) the blocks that read one head's chunks share an L2.
template <int NDT, bool HAS_W>
__global__ __launch_bounds__(CS_CHAIN) void chunk_chain_kernel(const float* __restrict__ Wm, const float* __restrict__ Qm,
                                                              const float* __restrict__ Km, const float* __restrict__ Pm,
                                                              const float* __restrict__ gam, const float* __restrict__ u0, int ldu,
                                                              float* __restrict__ o, float* __restrict__ state,
                                                              const int* __restrict__ cu_chunk, const int* __restrict__ first_chunk,
                                                              const int* __restrict__ state_slots, int H, int D, int Dv) {
    constexpr int DP = 16 * NDT, NJ = ChunkRegs<NDT, HAS_W>::NJ, SLD = DP + 4, ULD = CS_C + 4;
    __shared__ __align__(16) float Ss[16 * SLD], Us[16 * ULD];      // [column][row]
    const int h = blockIdx.x, s = blockIdx.z;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TM_WAVE), lane = threadIdx.x % TM_WAVE, r = lane % 16, g = lane / 16;
    const int e = blockIdx.y * 16 + r;
    const bool col = e < Dv;
    const int c0 = first_chunk[s], c1 = first_chunk[s + 1];
    if (c1 <= c0) return;                                           // the whole block
    float* st = state + (((size_t)state_slots[s] * H + h) * D) * Dv + (col ? e : 0);
    const float* u_col = u0 + (size_t)h * Dv + (col ? e : 0);
    cs_f32x4 S[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int d0 = 16 * (wave * NJ + j) + 4 * g;
#pragma unroll
        for (int i = 0; i < 4; ++i) S[j][i] = (col && d0 + i < D) ? st[(size_t)(d0 + i) * Dv] : 0.f;
        *(cs_f32x4*)(Ss + r * SLD + d0) = S[j];
    }
    ChunkRegs<NDT, HAS_W> now, next;
    int row0 = cu_chunk[c0], row1 = cu_chunk[c0 + 1];
    load_chunk<NDT, HAS_W>(now, Wm, Qm, Km, Pm, gam, u_col, ldu, (size_t)c0 * H + h, HAS_W ? c0 * CS_C : row0, row1 - row0, wave, r, g, col);
    __syncthreads();
    for (int c = c0; c < c1; ++c) {
        const int n = row1 - row0;
        const int cn = c + 1 < c1 ? c + 1 : c;                      // the last chunk asks for itself again
        const int nrow0 = cu_chunk[cn], nrow1 = cu_chunk[cn + 1];
        load_chunk<NDT, HAS_W>(next, Wm, Qm, Km, Pm, gam, u_col, ldu, (size_t)cn * H + h, HAS_W ? cn * CS_C : nrow0,
                                 nrow1 - nrow0, wave, r, g, col);
        // U = U0 + W S, O = (G Q) S
        cs_f32x4 U = {now.u[0], now.u[1], now.u[2], now.u[3]}, O = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            const cs_f32x4 s4 = *(const cs_f32x4*)(Ss + r * SLD + 16 * dt + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (HAS_W) U = cs_mfma(now.w[dt][i], s4[i], U);
                O = cs_mfma(now.q[dt][i], s4[i], O);
            }
        }
        *(cs_f32x4*)(Us + r * ULD + 16 * wave + 4 * g) = U;
        __syncthreads();                                            // U is whole, and every wavefront has read S
        // S <- G_n S + (G_n / G K)^T U, O += P U
#pragma unroll
        for (int j = 0; j < NJ; ++j) S[j] = now.gam[j] * S[j];
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
            const cs_f32x4 u4 = *(const cs_f32x4*)(Us + r * ULD + 16 * tt + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (tt <= wave) O = cs_mfma(now.p[tt][i], u4[i], O);
#pragma unroll
                for (int j = 0; j < NJ; ++j) S[j] = cs_mfma(now.k[j][tt][i], u4[i], S[j]);
            }
        }
#pragma unroll
        for (int j = 0; j < NJ; ++j) *(cs_f32x4*)(Ss + r * SLD + 16 * (wave * NJ + j) + 4 * g) = S[j];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * g + i;
            if (col && t < n) o[((size_t)(row0 + t) * H + h) * Dv + e] = O[i];
        }
        __syncthreads();                                            // S is whole, and every wavefront has read U
        now = next;
        row0 = nrow0;
        row1 = nrow1;
    }
#pragma unroll
    for (int j = 0; j < NJ; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NJ + j) + 4 * g + i;
            if (col && d < D) st[(size_t)d * Dv] = S[j][i];
        }
}

// The chunks first_chunk[s] .. first_chunk[s + 1] - 1 of every request s, in order, from and to the request's row of state
// [slots, H, D, Dv]. Wm null: U is U0 itself (a retention: u0 are the values, a row a token of
// the step); else u0 holds 64 rows a chunk. u0: column h Dv + e of rows ldu apart; o [T, H Dv].
extern "C" int tm_chunk_chain(const float* Wm, const float* Qm, const float* Km, const float* Pm, const float* gam, const float* u0,
                              int ldu, float* o, float* state, const int* cu_chunk, const int* first_chunk, const int* state_slots,
                              int S, int H, int D, int DP, int Dv, hipStream_t stream) {
    if (S <= 0) return TM_OK;
    if (!Qm || !Km || !Pm || !gam || !u0 || !o || !state || !cu_chunk || !first_chunk || !state_slots || H <= 0 || D <= 0 || D > DP ||
        Dv <= 0 || S > 65535 || (Dv + 15) / 16 > 65535 || ldu < H * Dv)
        return TM_ERR_ARG;
    const dim3 grid(H, (Dv + 15) / 16, S);
#define CS_GO(NDT_, W_)                                                                                                              \
    chunk_chain_kernel<NDT_, W_><<<grid, CS_CHAIN, 0, stream>>>(Wm, Qm, Km, Pm, gam, u0, ldu, o, state, cu_chunk, first_chunk,       \
                                                                state_slots, H, D, Dv)
    if (DP == 64) { if (Wm) CS_GO(4, true); else CS_GO(4, false); }
    else if (DP == 128) { if (Wm) CS_GO(8, true); else CS_GO(8, false); }
    else return TM_ERR_ARG;
#undef CS_GO
    TM_CHECK_LAUNCH();
    return TM_OK;
}
