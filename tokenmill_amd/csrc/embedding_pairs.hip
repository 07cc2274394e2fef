// Embedding rows to which a second table adds a row per pair of neighbouring tokens:
//
//   out[t] = table[id_t] * scale + pairs[b_t]
//   b_t = (id_(t-1) * mul_prev + id_t * mul_cur) mod buckets;  buckets (the table's last row) for a request's first token
//
// The token before a step's first row of a request lives in the request's state slot, which the same launch moves on to
// the step's last token of the request. The pair's number is 64-bit arithmetic; the row is summed in 32-bit.
#include "common.h"
#include "api.h"

#define EP_THREADS 256

// A block a token. The block of a request's first row of the step is the only one that touches the request's state: it
// reads the token before, then writes the step's last one, so no other block's order matters.
template <typename T>
__global__ __launch_bounds__(EP_THREADS) void embed_pairs_kernel(const T* __restrict__ table, const T* __restrict__ pairs,
                                                                 const int* __restrict__ ids, const int* __restrict__ positions,
                                                                 const int* __restrict__ cu, const int* __restrict__ slots,
                                                                 const int* __restrict__ seq_of_token, int* __restrict__ prev_state,
                                                                 float* __restrict__ out, int hidden, int vocab, float scale, int buckets,
                                                                 long long mul_prev, long long mul_cur) {
    __shared__ int row_s;
    const int t = blockIdx.x;
    int id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);       // the host rejects such ids; never read outside
    if (threadIdx.x == 0) {
        const int s = seq_of_token[t], first = cu[s];
        int prev = t > first ? ids[t - 1] : 0;
        if (t == first) {
            int* mine = prev_state + slots[s];
            prev = *mine;
            *mine = ids[cu[s + 1] - 1];
        }
        const long long mixed = ((long long)prev * mul_prev + (long long)id * mul_cur) % buckets;
        row_s = positions[t] == 0 ? buckets : (int)(mixed < 0 ? mixed + buckets : mixed);
    }
    __syncthreads();
    const T* a = table + (size_t)id * hidden;
    const T* b = pairs + (size_t)row_s * hidden;
    float* o = out + (size_t)t * hidden;
    for (int c = threadIdx.x; c < hidden; c += EP_THREADS) o[c] = Elem<T>::load(a + c) * scale + Elem<T>::load(b + c);
}

extern "C" int tm_embed_pairs(const void* table, const void* pairs, int dtype, const int* ids, const int* positions, const int* cu_q_lens,
                              const int* state_slots, const int* seq_of_token, int* prev_state, float* out, int T, int hidden, int vocab,
                              float scale, int buckets, long long mul_prev, long long mul_cur, hipStream_t stream) {
    if (T <= 0) return TM_OK;
    if (!table || !pairs || !ids || !positions || !cu_q_lens || !state_slots || !seq_of_token || !prev_state || !out || hidden <= 0 ||
        vocab <= 0 || buckets <= 0)
        return TM_ERR_ARG;
    if (dtype == TM_F32)
        embed_pairs_kernel<float><<<T, EP_THREADS, 0, stream>>>((const float*)table, (const float*)pairs, ids, positions, cu_q_lens, state_slots,
                                                                seq_of_token, prev_state, out, hidden, vocab, scale, buckets, mul_prev, mul_cur);
    else if (dtype == TM_BF16)
        embed_pairs_kernel<bf16_t><<<T, EP_THREADS, 0, stream>>>((const bf16_t*)table, (const bf16_t*)pairs, ids, positions, cu_q_lens,
                                                                 state_slots, seq_of_token, prev_state, out, hidden, vocab, scale, buckets,
                                                                 mul_prev, mul_cur);
    else
        return TM_ERR_ARG;
    TM_CHECK_LAUNCH();
    return TM_OK;
}
