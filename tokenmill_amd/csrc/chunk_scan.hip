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
// The chain's operands are stored in the order its lanes take them: a matrix [rows, inner] as tiles of 16 x 16, tile after tile along
// the inner dimension, and in a tile the four consecutive inner elements of lane (row + 16 * quarter) behind each other, so that a
// wavefront's load of a tile is one run of 1,024 bytes (`cs_at`). U0 likewise as it lies in the results' lanes.
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
#define CS_I_STRIDE 20                       // and of the inverses of its diagonal blocks
#define CS_PREP 512
#define CS_CHAIN 256

typedef float cs_f32x4 __attribute__((ext_vector_type(4)));

// Where element (row, inner) of a matrix with `tiles` tiles along its inner dimension is stored
__device__ __forceinline__ int cs_at(int row, int inner, int tiles) {
    return (((row >> 4) * tiles + (inner >> 4)) * 64 + ((inner >> 2) & 3) * 16 + (row & 15)) * 4 + (inner & 3);
}

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
    const int wave = __builtin_amdgcn_readfirstlane(tid / TM_WAVE), lane = tid % TM_WAVE, r = lane % 16, g = lane / 16;
    if (wave < 5) {
        // pairs of one sub-block: four lanes (a quarter of the channels each) take two tokens t and four tokens s; a sub-block
        // has 20 such blocks on and below its diagonal: quads of s per pair of t: 1 1 2 2 3 3 4 4
        const int task = tid / 4, part = tid % 4, I = task / 20, k = task % 20;
        const int tp = k < 2 ? k : k < 6 ? 2 + (k - 2) / 2 : k < 12 ? 4 + (k - 6) / 3 : 6 + (k - 12) / 4;
        const int sq = k < 2 ? 0 : k < 6 ? (k - 2) % 2 : k < 12 ? (k - 6) % 3 : (k - 12) % 4;
        const int t0 = CS_SUB * I + 2 * tp, s0 = CS_SUB * I + 4 * sq;
        float pa[2][4], pb[2][4];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) pa[i][j] = pb[i][j] = 0.f;
#pragma unroll 1
        for (int d = 4 * part; d < DP; d += 16) {
            cs_f32x4 kt[2], qt[2], lt[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                kt[i] = *(const cs_f32x4*)(Ks + (t0 + i) * LD + d);
                qt[i] = *(const cs_f32x4*)(Qs + (t0 + i) * LD + d);
                lt[i] = *(const cs_f32x4*)(Ls + (t0 + i) * LD + d);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const cs_f32x4 ks = *(const cs_f32x4*)(Ks + (s0 + j) * LD + d), lsv = *(const cs_f32x4*)(Ls + (s0 + j) * LD + d);
#pragma unroll
                for (int i = 0; i < 2; ++i)
#pragma unroll
                    for (int m = 0; m < 4; ++m) {
                        // (a pair with s after t is dropped below; its exponent is held to zero so that it stays finite)
                        const float e = ks[m] * __builtin_amdgcn_exp2f(fminf(lt[i][m] - lsv[m], 0.f));
                        pa[i][j] += kt[i][m] * e;
                        pb[i][j] += qt[i][m] * e;
                    }
            }
        }
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                pa[i][j] += __shfl_xor(pa[i][j], 1, TM_WAVE);
                pa[i][j] += __shfl_xor(pa[i][j], 2, TM_WAVE);
                pb[i][j] += __shfl_xor(pb[i][j], 1, TM_WAVE);
                pb[i][j] += __shfl_xor(pb[i][j], 2, TM_WAVE);
            }
        if (part < 2) {                                 // lane 0 writes A's two rows, lane 1 P's
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                const int t = t0 + i;
                cs_f32x4 v;
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    v[j] = part == 0 ? (s0 + j < t ? beta[t] * pa[i][j] : 0.f) : (s0 + j <= t ? pb[i][j] : 0.f);
                if (part == 0) *(cs_f32x4*)(As + t * CS_A_STRIDE + s0) = v;
                else *(cs_f32x4*)(Pg + cs_at(t, s0, 4)) = v;
            }
        } else if (sq == tp / 2) {                      // and the quads behind the diagonal's are zeros
            for (int z = s0 + 4; z < CS_SUB * (I + 1); z += 4)
#pragma unroll
                for (int i = 0; i < 2; ++i) {
                    if (part == 2) *(cs_f32x4*)(As + (t0 + i) * CS_A_STRIDE + z) = cs_f32x4{0.f, 0.f, 0.f, 0.f};
                    else *(cs_f32x4*)(Pg + cs_at(t0 + i, z, 4)) = cs_f32x4{0.f, 0.f, 0.f, 0.f};
                }
        }
    } else {
        // pairs of two sub-blocks I > J on the matrix unit: three wavefronts, two of the six products each
#pragma unroll 1
        for (int p = 2 * (wave - 5); p < 2 * (wave - 5) + 2; ++p) {
            const int I = p < 1 ? 1 : p < 3 ? 2 : 3, J = p < 1 ? 0 : p < 3 ? p - 1 : p - 3;
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
                Pg[cs_at(t, s, 4)] = accP[i];
            }
        }
    }
    // what the chain reads of the tokens themselves
    float* Qg = Qm + at * CS_C * DP;
    float* Kg = Km + at * CS_C * DP;
    // (a wavefront writes tile after tile: idx / 64 is the tile, the lane its place in it)
    for (int tile = wave; tile < 4 * (DP / 16); tile += CS_PREP / TM_WAVE) {
        const int I = tile / (DP / 16), t = CS_SUB * I + r, d = 16 * (tile % (DP / 16)) + 4 * g;
        cs_f32x4 v = *(const cs_f32x4*)(Ls + t * LD + d);
        for (int M = 0; M < I; ++M) v += *(const cs_f32x4*)(tot + M * DP + d);
        const cs_f32x4 q4 = *(const cs_f32x4*)(Qs + t * LD + d);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = q4[i] * __builtin_amdgcn_exp2f(v[i]);
        *(cs_f32x4*)(Qg + (tile * 64 + lane) * 4) = v;
    }
    for (int tile = wave; tile < 4 * (DP / 16); tile += CS_PREP / TM_WAVE) {
        const int I = tile % 4, d = 16 * (tile / 4) + r;
        float rest = tot[I * DP + d];
        for (int M = I + 1; M < 4; ++M) rest += tot[M * DP + d];
        cs_f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = CS_SUB * I + 4 * g + i;
            v[i] = Ks[t * LD + d] * __builtin_amdgcn_exp2f(rest - Ls[t * LD + d]);
        }
        *(cs_f32x4*)(Kg + (tile * 64 + lane) * 4) = v;
    }
    for (int d = tid; d < DP; d += CS_PREP)
        gam[at * DP + d] = __builtin_amdgcn_exp2f(tot[d] + tot[DP + d] + tot[2 * DP + d] + tot[3 * DP + d]);
    __syncthreads();
    // the inverses of I + A's four 16x16 blocks on the diagonal: a wavefront a block, a lane a column, from the first row on
    float* inv = Qs;                                    // [4][16][CS_I_STRIDE]: the queries are no longer needed
    if (wave < 4 && lane < 16) {
        const float* a = As + CS_SUB * wave * CS_A_STRIDE + CS_SUB * wave;
        float x[CS_SUB];
#pragma unroll
        for (int t = 0; t < CS_SUB; ++t) {
            float v = t == lane ? 1.f : 0.f;
#pragma unroll
            for (int s = 0; s < t; ++s) v -= a[t * CS_A_STRIDE + s] * x[s];
            x[t] = v;
        }
#pragma unroll
        for (int t = 0; t < CS_SUB; ++t) inv[(CS_SUB * wave + t) * CS_I_STRIDE + lane] = x[t];
    }
    __syncthreads();
    // (I + A) X = B (G K) and = B V in blocks of 16 rows, a wavefront 16 columns at a time: X_I = inv_I (B_I - sum over J < I of
    // A_IJ X_J). A block of X lies in the lanes as the next product takes it. The first DP columns are W's.
    float* Wg = Wm + at * CS_C * DP;
    const int v_tiles = (Dv + 15) / 16;
    float* ug = u0 + at * v_tiles * CS_C * 16;
    for (int tile = wave; tile < DP / 16 + v_tiles; tile += CS_PREP / TM_WAVE) {
        const bool is_w = tile < DP / 16;
        const int e = (is_w ? tile : tile - DP / 16) * 16 + r;
        const int ev = e < Dv ? e : Dv - 1;             // a column beyond the last repeats it; nobody stores what comes of it
        cs_f32x4 X[4];
        float before = 0.f;
#pragma unroll
        for (int I = 0; I < 4; ++I) {
            cs_f32x4 acc;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = CS_SUB * I + 4 * g + i;
                if (is_w) {
                    acc[i] = beta[t] * (Ks[t * LD + e] * __builtin_amdgcn_exp2f(before + Ls[t * LD + e]));
                } else {                                // rows beyond the chunk's last: the last one again, with a beta of zero
                    const int tc = t < n ? t : n - 1;
                    acc[i] = beta[t] * rows[(size_t)(row0 + tc) * ld + 2 * G * D + h * Dv + ev];
                }
            }
            if (is_w) before += tot[I * DP + e];
#pragma unroll
            for (int J = 0; J < I; ++J) {
                const cs_f32x4 a4 = *(const cs_f32x4*)(As + (CS_SUB * I + r) * CS_A_STRIDE + CS_SUB * J + 4 * g);
#pragma unroll
                for (int i = 0; i < 4; ++i) acc = cs_mfma(-a4[i], X[J][i], acc);
            }
            const cs_f32x4 t4 = *(const cs_f32x4*)(inv + (CS_SUB * I + r) * CS_I_STRIDE + 4 * g);
            X[I] = cs_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < 4; ++i) X[I] = cs_mfma(t4[i], acc[i], X[I]);
            if (is_w) {
#pragma unroll
                for (int i = 0; i < 4; ++i) Wg[cs_at(CS_SUB * I + 4 * g + i, e, DP / 16)] = -X[I][i];
            } else {
                *(cs_f32x4*)(ug + (((tile - DP / 16) * 4 + I) * 64 + lane) * 4) = X[I];
            }
        }
    }
}

static size_t delta_chunks_lds(int DP) { return ((size_t)3 * CS_C * (DP + 4) + CS_C * CS_A_STRIDE + 4 * DP + CS_C) * sizeof(float); }

// rows as tm_delta_prepare writes them; chunk c holds the rows cu_chunk[c] .. cu_chunk[c + 1] - 1 (1 to 64 of one request). Km, Qm,
// Wm float [n, H, 64 * DP], Pm [n, H, 64 * 64], gam [n, H, DP] with DP = 64 or 128 >= D, u0
// [n, H, ceil(Dv / 16), 64 * 16]; matrices in the chain's order.
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
            Pg[cs_at(t, s, 4)] = s <= t ? acc[i] * pw[t - s] : 0.f;
        }
    }
    float* Qg = Qm + at * CS_C * DP;
    float* Kg = Km + at * CS_C * DP;
    for (int tile = wave; tile < 4 * (DP / 16); tile += CS_CHAIN / TM_WAVE) {
        const int t = 16 * (tile / (DP / 16)) + r, d = 16 * (tile % (DP / 16)) + 4 * g;
        *(cs_f32x4*)(Qg + (tile * 64 + lane) * 4) = *(const cs_f32x4*)(Qs + t * LD + d) * pw[t + 1];
    }
    for (int tile = wave; tile < 4 * (DP / 16); tile += CS_CHAIN / TM_WAVE) {
        const int d = 16 * (tile / 4) + r;
        cs_f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * (tile % 4) + 4 * g + i;
            v[i] = t < n ? Ks[t * LD + d] * pw[n - 1 - t] : 0.f;
        }
        *(cs_f32x4*)(Kg + (tile * 64 + lane) * 4) = v;
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

// What a wavefront reads of a chunk, in the operands' places.
template <int NDT, bool HAS_W>
struct ChunkRegs {
    static constexpr int NJ = NDT / 4;                  // tiles of 16 key channels of a wavefront's share of the state
    cs_f32x4 w[HAS_W ? NDT : 1], q[NDT], p[4], k[NJ][4], gam[NJ], u;
};

// Where a wavefront's operands of one (chunk, head) start.
template <int NDT, bool HAS_W>
struct ChunkPlaces {
    const float *w, *q, *p, *k, *gam, *u;
    int u_row[4];                                       // without W: offsets of the lane's four rows of values

    __device__ __forceinline__ ChunkPlaces(const float* Wm, const float* Qm, const float* Km, const float* Pm, const float* gm, const float* u0,
                                           int ldu, size_t at, int row0, int n, int wave, int r, int g) {
        const int lane = 16 * g + r;
        const size_t mine = (at * 4 + wave) * NDT * 256 + 4 * lane;
        w = Wm + mine;
        q = Qm + mine;
        p = Pm + (at * 4 + wave) * 4 * 256 + 4 * lane;
        k = Km + (at * NDT + wave * (NDT / 4)) * 4 * 256 + 4 * lane;
        gam = gm + (at * NDT + wave * (NDT / 4)) * 16 + 4 * g;
        u = HAS_W ? u0 + at * ldu + (wave * 64 + lane) * 4 : u0 + (size_t)row0 * ldu;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * g + i;        // a row behind the chunk's tokens meets zeros everywhere: any will do
            u_row[i] = (t < n ? t : n - 1) * ldu;
        }
    }
    __device__ __forceinline__ cs_f32x4 load_u() const {
        return HAS_W ? *(const cs_f32x4*)u : cs_f32x4{u[u_row[0]], u[u_row[1]], u[u_row[2]], u[u_row[3]]};
    }
};

// grid (H, ceil(Dv / 16), requests); a block is four wavefronts and 16 columns of a request's and head's state. A wavefront owns 16
// of a chunk's tokens (rows of U and O) and a quarter of the state's rows. The matrix unit leaves a 16x16 result with four
// consecutive rows in a lane, and takes its second operand one row a lane: with the rows of every product's inner sum dealt the
// same way (row 16 tile + 4 g + i to lane group g, instruction i) a result is the next product's operand as it lies. U and S go
// through LDS (column by column, so that a lane's four rows are one piece) because every wavefront needs all their rows. An
// operand's registers are filled with the next chunk's as soon as its products are issued (the last chunk asks for itself again), a
// few loads at a time between the products: asked for in one go they hold up the products behind them. Every load is unconditional:
// behind a test the compiler waits for what is on its way.
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
    const float* u_mine = HAS_W ? u0 + (size_t)blockIdx.y * CS_C * 16 : u0 + (size_t)h * Dv + (col ? e : 0);
    if (HAS_W) ldu = gridDim.y * CS_C * 16;                         // from one (chunk, head) to the next
    cs_f32x4 S[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int d0 = 16 * (wave * NJ + j) + 4 * g;
#pragma unroll
        for (int i = 0; i < 4; ++i) S[j][i] = (col && d0 + i < D) ? st[(size_t)(d0 + i) * Dv] : 0.f;
        *(cs_f32x4*)(Ss + r * SLD + d0) = S[j];
    }
    ChunkRegs<NDT, HAS_W> x;
    int row0 = cu_chunk[c0], n = cu_chunk[c0 + 1] - row0;
    {
        const ChunkPlaces<NDT, HAS_W> at(Wm, Qm, Km, Pm, gam, u_mine, ldu, (size_t)c0 * H + h, row0, n, wave, r, g);
        x.u = at.load_u();                                          // in the order in which the loop uses and asks for them again
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            if (HAS_W) x.w[dt] = *(const cs_f32x4*)(at.w + 256 * dt);
            x.q[dt] = *(const cs_f32x4*)(at.q + 256 * dt);
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
            x.p[tt] = *(const cs_f32x4*)(at.p + 256 * tt);          // (beyond the diagonal: not looked at)
#pragma unroll
            for (int j = 0; j < NJ; ++j) x.k[j][tt] = *(const cs_f32x4*)(at.k + (4 * j + tt) * 256);
        }
#pragma unroll
        for (int j = 0; j < NJ; ++j) x.gam[j] = *(const cs_f32x4*)(at.gam + 16 * j);
    }
    __syncthreads();
    for (int c = c0; c < c1; ++c) {
        const int cn = c + 1 < c1 ? c + 1 : c;
        const int nrow0 = cu_chunk[cn], nn = cu_chunk[cn + 1] - nrow0;
        const ChunkPlaces<NDT, HAS_W> next(Wm, Qm, Km, Pm, gam, u_mine, ldu, (size_t)cn * H + h, nrow0, nn, wave, r, g);
        // U = U0 + W S, O = (G Q) S
        cs_f32x4 U = x.u, O = {0.f, 0.f, 0.f, 0.f};
        x.u = next.load_u();
        cs_f32x4 s4 = *(const cs_f32x4*)(Ss + r * SLD + 4 * g);
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            const cs_f32x4 ahead = *(const cs_f32x4*)(Ss + r * SLD + 16 * (dt + 1 < NDT ? dt + 1 : dt) + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (HAS_W) U = cs_mfma(x.w[dt][i], s4[i], U);
                O = cs_mfma(x.q[dt][i], s4[i], O);
            }
            if (HAS_W) x.w[dt] = *(const cs_f32x4*)(next.w + 256 * dt);
            x.q[dt] = *(const cs_f32x4*)(next.q + 256 * dt);
            s4 = ahead;
            __builtin_amdgcn_sched_barrier(0);
        }
        *(cs_f32x4*)(Us + r * ULD + 16 * wave + 4 * g) = U;
        __syncthreads();                                            // U is whole, and every wavefront has read S
        // S <- G_n S + (G_n / G K)^T U, O += P U
        cs_f32x4 u4 = *(const cs_f32x4*)(Us + r * ULD + 4 * g);
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            S[j] = x.gam[j] * S[j];
            x.gam[j] = *(const cs_f32x4*)(next.gam + 16 * j);
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
            const cs_f32x4 ahead = *(const cs_f32x4*)(Us + r * ULD + 16 * (tt < 3 ? tt + 1 : tt) + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < NJ; ++j) S[j] = cs_mfma(x.k[j][tt][i], u4[i], S[j]);
            if (tt <= wave) {
#pragma unroll
                for (int i = 0; i < 4; ++i) O = cs_mfma(x.p[tt][i], u4[i], O);
            }
            x.p[tt] = *(const cs_f32x4*)(next.p + 256 * tt);
#pragma unroll
            for (int j = 0; j < NJ; ++j) x.k[j][tt] = *(const cs_f32x4*)(next.k + (4 * j + tt) * 256);
            u4 = ahead;
            __builtin_amdgcn_sched_barrier(0);
        }
#pragma unroll
        for (int j = 0; j < NJ; ++j) *(cs_f32x4*)(Ss + r * SLD + 16 * (wave * NJ + j) + 4 * g) = S[j];
        float* out = o + ((size_t)row0 * H + h) * Dv + e;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * g + i;
            if (col && t < n) out[(size_t)t * H * Dv] = O[i];
        }
        __syncthreads();                                            // S is whole, and every wavefront has read U
        row0 = nrow0;
        n = nn;
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
// [slots, H, D, Dv]. Wm null: U is U0 itself (a retention: u0 are the values, column
// h Dv + e of rows ldu apart, a row a token of the step); else u0 is tm_delta_chunks' own. o [T, H Dv].
extern "C" int tm_chunk_chain(const float* Wm, const float* Qm, const float* Km, const float* Pm, const float* gam, const float* u0,
                              int ldu, float* o, float* state, const int* cu_chunk, const int* first_chunk, const int* state_slots,
                              int S, int H, int D, int DP, int Dv, hipStream_t stream) {
    if (S <= 0) return TM_OK;
    if (!Qm || !Km || !Pm || !gam || !u0 || !o || !state || !cu_chunk || !first_chunk || !state_slots || H <= 0 || D <= 0 || D > DP ||
        Dv <= 0 || S > 65535 || (Dv + 15) / 16 > 65535 || (!Wm && ldu < H * Dv))
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
