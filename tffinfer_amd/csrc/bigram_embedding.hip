// An embedding with a second table of rows for pairs of neighbouring tokens:
//   x_t = E[token_t] + B[(token_(t-1) * mul_prev + token_t * mul_cur) mod buckets],   for a sequence's first token
//   x_0 = E[token_0] + B[buckets].
// The token before a portion's first one is part of the request's state: one int32 per state slot.  The block of
// a portion's first token alone reads it, and then leaves the portion's last token there for the next step.
// E is row-major or in the fragment order of the matrix-core products (a table that also serves as output head), B
// is row-major of the same element type.  x is float32; `copy`, if given, gets the same rows.
#include "common.h"
#include "tffinfer_kernels.h"

struct BigramEmbedArgs {
    const int32_t *ids, *positions, *token_req, *cu_tokens, *slots;
    int32_t* last;               // [slots][last_row]
    size_t last_row;
    long long mul_prev, mul_cur, buckets;
    float *out, *copy;
    int W, V, KB;                // KB: k-blocks of 32 of a packed E, 0: row-major
};

// eight neighbouring elements 8 c .. 8 c + 7 of row id of E
template <typename T>
__device__ __forceinline__ const T* bigram_chunk(const T* table, int id, int c, const BigramEmbedArgs& a) {
    if (a.KB) return table + (size_t)(id / 16) * a.KB * 512 + (id % 16) * 8 + (size_t)(c / 4) * 512 + (c % 4) * 128;
    return table + (size_t)id * a.W + (size_t)c * 8;
}

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void bigram_embed_kernel(const T* __restrict__ table, const T* __restrict__ pairs,
                                                           const BigramEmbedArgs a) {
    const int t = blockIdx.x, r = a.token_req[t], t0 = a.cu_tokens[r];
    const int tok = a.ids[t];
    const bool bad = tok < 0 || tok >= a.V;
    const int id = bad ? 0 : tok;
    const bool head = t == t0;
    int32_t* const kept = a.last + (size_t)a.slots[r] * a.last_row;
    const int prev = head ? *kept : a.ids[t - 1];
    if (head) {
        __syncthreads();         // every thread has read what one of them replaces
        if (threadIdx.x == 0) *kept = a.ids[a.cu_tokens[r + 1] - 1];
    }
    long long row = a.buckets;
    if (a.positions[t] > 0) {
        row = ((long long)prev * a.mul_prev + (long long)tok * a.mul_cur) % a.buckets;
        if (row < 0) row += a.buckets;
    }
    const T* p = pairs + (size_t)row * a.W;
    float* o = a.out + (size_t)t * a.W;
    float* o2 = a.copy ? a.copy + (size_t)t * a.W : nullptr;
    if constexpr (VEC) {         // W a multiple of 8, everything 16-byte aligned
        for (int c = threadIdx.x; c < a.W / 8; c += 256) {
            const T* e = bigram_chunk(table, id, c, a);
            float v[8];
            if constexpr (sizeof(T) == 2) {
                union { uint4 u; T h[8]; } x, y;
                x.u = *reinterpret_cast<const uint4*>(e);
                y.u = *reinterpret_cast<const uint4*>(p + (size_t)c * 8);
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] = to_f32(x.h[i]) + to_f32(y.h[i]);
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] = to_f32(e[i]) + to_f32(p[(size_t)c * 8 + i]);
            }
            if (bad) {
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] = __builtin_nanf("");
            }
            const float4 lo = make_float4(v[0], v[1], v[2], v[3]), hi = make_float4(v[4], v[5], v[6], v[7]);
            *reinterpret_cast<float4*>(o + (size_t)c * 8) = lo;
            *reinterpret_cast<float4*>(o + (size_t)c * 8 + 4) = hi;
            if (o2) {
                *reinterpret_cast<float4*>(o2 + (size_t)c * 8) = lo;
                *reinterpret_cast<float4*>(o2 + (size_t)c * 8 + 4) = hi;
            }
        }
    } else {
        for (int i = threadIdx.x; i < a.W; i += 256) {
            const float v = bad ? __builtin_nanf("") : to_f32(bigram_chunk(table, id, i / 8, a)[i % 8]) + to_f32(p[i]);
            o[i] = v;
            if (o2) o2[i] = v;
        }
    }
}

// row_width: elements of a row of a packed E (W rounded up to 8); packed 0: E is [V, W].
TFF_API int tff_bigram_embed(const void* table, int packed, int row_width, const void* pairs, const int32_t* ids,
                             const int32_t* positions, const int32_t* token_req, const int32_t* cu_tokens,
                             const int32_t* state_slots, int32_t* last, size_t last_row, int64_t mul_prev, int64_t mul_cur,
                             int64_t buckets, float* out, float* copy, int T, int W, int V, int dtype, tff_stream_t stream) {
    TFF_REQUIRE(table && pairs && ids && positions && token_req && cu_tokens && state_slots && last && out, "bigram_embed: null pointer");
    TFF_REQUIRE(T >= 0 && W > 0 && V > 0 && buckets > 0 && last_row >= 1 && (!packed || (row_width >= W && row_width % 8 == 0)),
                "bigram_embed: bad sizes T=%d W=%d V=%d", T, W, V);
    TFF_REQUIRE(!packed || dtype == TFF_BF16, "bigram_embed: only a bfloat16 table is packed");
    if (T == 0) return 0;
    const BigramEmbedArgs a{ids, positions, token_req, cu_tokens, state_slots, last, last_row, mul_prev, mul_cur, buckets, out, copy,
                            W, V, packed ? (row_width + 31) / 32 : 0};
    hipStream_t s = (hipStream_t)stream;
    const bool vec = W % 8 == 0 && ((uintptr_t)table % 16) == 0 && ((uintptr_t)pairs % 16) == 0 && ((uintptr_t)out % 16) == 0 &&
                     ((uintptr_t)copy % 16) == 0;
#define BE_GO(TT, VEC) bigram_embed_kernel<TT, VEC><<<T, 256, 0, s>>>((const TT*)table, (const TT*)pairs, a)
    if (dtype == TFF_F32) { if (vec) BE_GO(float, true); else BE_GO(float, false); }
    else if (dtype == TFF_BF16) { if (vec) BE_GO(bf16_t, true); else BE_GO(bf16_t, false); }
    else return tff_fail("bigram_embed: unknown dtype %d", dtype);
#undef BE_GO
    return tff_check_launch("bigram_embed");
}
