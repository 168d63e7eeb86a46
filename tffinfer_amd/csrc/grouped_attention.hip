// What stands around the paged attention kernels in a grouped attention whose queries carry a temperature that grows
// with the position and whose window has the mean keys of whole blocks of tokens before it.
//
// tff_grouped_qkv_store:  from the joint projection (float32): biases, an RMS norm over all of a token's q (and of its k)
//                         at once, rotation of q and k, the temperature on q, q laid out with the cache's head size, the
//                         token's key and value into its slot.
// tff_pool_keys:          for every token of the step that ends a block of P tokens: the means of the block's P keys and
//                         values, as the pages hold them, into the block's slot.
// tff_gate_heads:         a head's output times one gate per head and a scale, heads brought together.
#include "common.h"
#include "tffinfer_kernels.h"

struct GroupedRot {
    const float* cs;     // the position's [pair][cos, sin], or null
    int dims;            // rotated elements of a head (even)
    int pairing;         // 0: (i, i + dims/2), 1: (2i, 2i+1)
};

// Elements of a head come two by two: place p < dims / 2 is the p-th pair that turns, the others two neighbours behind
// the turned part.  f(element, its value): elements from D to P - 1 are zeros.
template <typename V, typename F>
__device__ __forceinline__ void grouped_pair(int p, int D, const GroupedRot r, V value, F f) {
    const int half = r.cs ? r.dims >> 1 : 0;
    if (p < half) {
        const int i = r.pairing == 0 ? p : 2 * p, j = r.pairing == 0 ? p + half : 2 * p + 1;
        const float u = value(i), w = value(j), c = r.cs[2 * p], s = r.cs[2 * p + 1];
        // the pair (u, w) becomes (u c - w s, w c + u s)
        f(i, fmaf(u, c, -(w * s)));
        f(j, fmaf(w, c, u * s));
    } else {
        const int i = 2 * p;
        f(i, i < D ? value(i) : 0.f);
        f(i + 1, i + 1 < D ? value(i + 1) : 0.f);
    }
}

// What happens to the projections before rotation.
struct GroupedPre {
    const float* bias;                 // [H D + G D + G E] in the projection's column order, or null
    const float *q_norm, *k_norm;      // [H D], [G D]: RMS norms over the whole of q and of k, or null
    float eps;
};

// Blocks (token, y): y < q_blocks works through `per_q` query heads; the others through `per_kv` kv heads each: their key
// and value rows into the token's slot.  Elements past a head's own size are zeros.  With a norm every block forms the
// sum of squares it needs by itself, always in the same order (its threads are as many whatever the step).
#define GQ_THREADS 128
#define GQ_WIDE 512      // threads with a norm, and where few tokens wait for one another's loads
#define GQ_HEADS 8

// 1 / sqrt(mean over x[0 .. n) of (x + bias)^2 + eps), the result in every thread of the block
template <int NT>
__device__ __forceinline__ float grouped_rms(const float* __restrict__ x, const float* __restrict__ bias, int n, float eps, bool vec,
                                             float* red) {
    float ss = 0.f;
    if (vec) {
#pragma unroll 8
        for (int c = threadIdx.x * 4; c < n; c += NT * 4) {
            float4 v = *reinterpret_cast<const float4*>(x + c);
            if (bias) {
                const float4 b = *reinterpret_cast<const float4*>(bias + c);
                v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
            }
            ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
        }
    } else {
        for (int c = threadIdx.x; c < n; c += NT) {
            const float v = x[c] + (bias ? bias[c] : 0.f);
            ss = fmaf(v, v, ss);
        }
    }
    ss = rows_sum(row16_sum(ss));
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NT / 64; ++i) ss += red[i];
    return 1.0f / sqrtf(ss / (float)n + eps);
}

template <typename TC, int NT>
__global__ __launch_bounds__(NT) void grouped_qkv_store_kernel(
    const float* __restrict__ proj, size_t row, const float* __restrict__ cos_sin, int rot_dims, int pairing, int max_pos,
    float temp_coef, int temp_every, const GroupedPre pre, const int32_t* __restrict__ positions, const int32_t* __restrict__ slots,
    TC* __restrict__ q_out, TC* __restrict__ k_cache, TC* __restrict__ v_cache, int page_size, int H, int G, int D, int E, int P,
    int q_blocks, int per_q, int per_kv, int vec) {
    __shared__ float red[NT / 64];
    const int t = blockIdx.x, y = blockIdx.y, tid = threadIdx.x;
    const float* x = proj + (size_t)t * row;
    const int pos = max(positions[t], 0), tpos = min(pos, max(max_pos - 1, 0));
    const GroupedRot rot{(cos_sin && rot_dims) ? cos_sin + (size_t)tpos * rot_dims : nullptr, rot_dims, pairing};
    const int half = P >> 1;                 // places of a head
    if (y < q_blocks) {
        const float temp = temp_coef != 0.f ? 1.0f + temp_coef * logf((float)((pos + 1) / temp_every + 1)) : 1.0f;
        const float rr = pre.q_norm ? grouped_rms<NT>(x, pre.bias, H * D, pre.eps, vec, red) : 1.0f;
        TC* qo = q_out + (size_t)t * H * P;
        const int h0 = y * per_q, count = (min(H, h0 + per_q) - h0) * half;
        for (int idx = tid; idx < count; idx += NT) {
            const int h = h0 + idx / half, p = idx % half, c0 = h * D;
            TC* const qh = qo + (size_t)h * P;
            grouped_pair(p, D, rot,
                [&](int e) {
                    float v = x[c0 + e];
                    if (pre.bias) v += pre.bias[c0 + e];
                    return pre.q_norm ? v * rr * pre.q_norm[c0 + e] : v;
                },
                [&](int e, float v) { qh[e] = from_f32<TC>(v * temp); });
        }
        return;
    }
    const int slot = slots[t];
    if (slot < 0) return;      // (the whole block: a token that writes no key)
    const int page = slot / page_size, off = slot - page * page_size;
    const size_t ck = (size_t)H * D;
    const float* xk = x + ck;
    const float* bk = pre.bias ? pre.bias + ck : nullptr;
    const float rr = pre.k_norm ? grouped_rms<NT>(xk, bk, G * D, pre.eps, vec, red) : 1.0f;
    const int g0 = (y - q_blocks) * per_kv, groups = min(G, g0 + per_kv) - g0;
    for (int idx = tid; idx < groups * half; idx += NT) {
        const int g = g0 + idx / half, p = idx % half, c0 = g * D;
        TC* const kd = k_cache + (((size_t)page * G + g) * page_size + off) * P;
        grouped_pair(p, D, rot,
            [&](int e) {
                float v = xk[c0 + e];
                if (bk) v += bk[c0 + e];
                return pre.k_norm ? v * rr * pre.k_norm[c0 + e] : v;
            },
            [&](int e, float v) { kd[e] = from_f32<TC>(v); });
    }
    for (int idx = tid; idx < groups * P; idx += NT) {
        const int g = g0 + idx / P, e = idx % P;
        const size_t cv = ck + (size_t)G * D + (size_t)g * E + e;
        TC* const vd = v_cache + ((size_t)page * G + g) * P * page_size + off;
        vd[(size_t)e * page_size] = from_f32<TC>(e < E ? x[cv] + (pre.bias ? pre.bias[cv] : 0.f) : 0.f);
    }
}

TFF_API int tff_grouped_qkv_store(const float* proj, size_t row, const float* cos_sin, int rot_dims, int pairing, int max_pos,
                                  float temp_coef, int temp_every, const float* bias, const float* q_norm, const float* k_norm,
                                  float norm_eps, const int32_t* positions, const int32_t* slots, void* q_out, void* k_cache,
                                  void* v_cache, int page_size, int num_pages, int T, int H, int G, int D, int E, int P, int store,
                                  int dtype, tff_stream_t stream) {
    TFF_REQUIRE(proj && positions && q_out && (!store || (slots && k_cache && v_cache)), "grouped_qkv_store: null pointer");
    TFF_REQUIRE(T >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && E > 0 && P >= D && P >= E && temp_every > 0,
                "grouped_qkv_store: bad sizes H=%d G=%d D=%d E=%d P=%d", H, G, D, E, P);
    TFF_REQUIRE(P % 2 == 0, "grouped_qkv_store: a cache head of %d elements must be even", P);
    TFF_REQUIRE(row >= (size_t)H * D + (store ? (size_t)G * (D + E) : 0), "grouped_qkv_store: rows of %zu are too short", row);
    TFF_REQUIRE(rot_dims >= 0 && rot_dims <= D && rot_dims % 2 == 0 && (rot_dims == 0 || (cos_sin && max_pos > 0)) &&
                (pairing == 0 || pairing == 1), "grouped_qkv_store: %d rotated elements of a head of %d need an even count and a table", rot_dims, D);
    TFF_REQUIRE(page_size > 0 && num_pages > 0, "grouped_qkv_store: bad cache geometry");
    if (T == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    // (with a norm over all heads, many tokens fill the GPU with a block each for q and for k: nothing is summed twice)
    const bool whole = (q_norm || k_norm) && T >= 128;
    const int per_q = whole ? H : GQ_HEADS, per_kv = whole ? G : 1;
    const int q_blocks = (H + per_q - 1) / per_q, kv_blocks = store ? (G + per_kv - 1) / per_kv : 0;
    const int vec = D % 4 == 0 && row % 4 == 0 && ((uintptr_t)proj % 16) == 0 && ((uintptr_t)bias % 16) == 0;
    TFF_REQUIRE(q_blocks + kv_blocks <= 65535, "grouped_qkv_store: too many heads");
    const dim3 grid(T, q_blocks + kv_blocks);
    const bool wide = q_norm || k_norm || T < 128;
#define GQ_LAUNCH(TC, NT)                                                                                                      \
    grouped_qkv_store_kernel<TC, NT><<<grid, NT, 0, s>>>(proj, row, cos_sin, rot_dims, pairing, max_pos, temp_coef, temp_every, \
                                                         GroupedPre{bias, q_norm, k_norm, norm_eps}, positions, slots, (TC*)q_out, \
                                                         (TC*)k_cache, (TC*)v_cache, page_size, H, G, D, E, P, q_blocks, per_q, per_kv, vec)
    if (dtype == TFF_F32 && wide) GQ_LAUNCH(float, GQ_WIDE);
    else if (dtype == TFF_F32) GQ_LAUNCH(float, GQ_THREADS);
    else if (dtype == TFF_BF16 && wide) GQ_LAUNCH(bf16_t, GQ_WIDE);
    else if (dtype == TFF_BF16) GQ_LAUNCH(bf16_t, GQ_THREADS);
    else return tff_fail("grouped_qkv_store: unknown dtype %d", dtype);
#undef GQ_LAUNCH
    return tff_check_launch("grouped_qkv_store");
}

// Blocks (token, kv head); the tokens are those that `tokens` lists, or all of the step's, of which those that end no
// block leave at once.  The sum runs over the block's tokens in their order; a thread takes elements tid, tid + 128, ...
// Where the tokens' keys and values lie is worked out by the threads side by side, PK_RUN tokens at a time.
#define PK_THREADS 128
#define PK_RUN 64

template <typename TC>
__global__ __launch_bounds__(PK_THREADS) void pool_keys_kernel(TC* __restrict__ k_cache, TC* __restrict__ v_cache,
                                                               const int32_t* __restrict__ block_tables, int bt_stride,
                                                               const int32_t* __restrict__ pool_tables, int pt_stride,
                                                               const int32_t* __restrict__ token_req,
                                                               const int32_t* __restrict__ positions,
                                                               const int32_t* __restrict__ slots,
                                                               const int32_t* __restrict__ tokens, int page_size, int pool, int G,
                                                               int d) {
    __shared__ size_t koff[PK_RUN], voff[PK_RUN];
    const int t = tokens ? tokens[blockIdx.x] : (int)blockIdx.x, g = blockIdx.y, tid = threadIdx.x;
    const int pos = positions[t];
    if (slots[t] < 0 || (pos + 1) % pool) return;      // (the whole block)
    const int r = token_req[t], blk = pos / pool, first = pos + 1 - pool;
    const int32_t* bt = block_tables + (size_t)r * bt_stride;
    const int dpage = pool_tables[(size_t)r * pt_stride + blk / page_size], dslot = blk % page_size;
    const float f = 1.0f / (float)pool;
    const size_t dhead = ((size_t)dpage * G + g) * page_size * d;
    for (int e0 = 0; e0 < d; e0 += PK_THREADS) {
        const int e = min(e0 + tid, d - 1);
        float ks = 0.f, vs = 0.f;
        for (int i0 = 0; i0 < pool; i0 += PK_RUN) {
            const int cnt = min(PK_RUN, pool - i0);
            if (i0 || e0) __syncthreads();             // the run before is read
            if (tid < cnt) {
                const int j = first + i0 + tid, slot = j % page_size;
                const size_t head = ((size_t)bt[j / page_size] * G + g) * page_size * d;
                koff[tid] = head + (size_t)slot * d;
                voff[tid] = head + slot;
            }
            __syncthreads();
#pragma unroll 8
            for (int i = 0; i < cnt; ++i) {
                ks += to_f32(k_cache[koff[i] + e]);
                vs += to_f32(v_cache[voff[i] + (size_t)e * page_size]);
            }
        }
        if (e0 + tid < d) {
            k_cache[dhead + (size_t)dslot * d + e] = from_f32<TC>(ks * f);
            v_cache[dhead + (size_t)e * page_size + dslot] = from_f32<TC>(vs * f);
        }
    }
}

TFF_API int tff_pool_keys(void* k_cache, void* v_cache, const int32_t* block_tables, int bt_stride, const int32_t* pool_tables,
                          int pt_stride, const int32_t* token_req, const int32_t* positions, const int32_t* slots,
                          const int32_t* tokens, int page_size, int num_pages, int pool, int T, int G, int d, int dtype, tff_stream_t stream) {
    TFF_REQUIRE(k_cache && v_cache && block_tables && pool_tables && token_req && positions && slots, "pool_keys: null pointer");
    TFF_REQUIRE(T >= 0 && G > 0 && G <= 65535 && d > 0 && pool > 0 && page_size > 0 && num_pages > 0 && bt_stride > 0 && pt_stride > 0,
                "pool_keys: bad sizes");
    if (T == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(T, G);
    if (dtype == TFF_F32)
        pool_keys_kernel<float><<<grid, PK_THREADS, 0, s>>>((float*)k_cache, (float*)v_cache, block_tables, bt_stride, pool_tables, pt_stride,
                                                            token_req, positions, slots, tokens, page_size, pool, G, d);
    else if (dtype == TFF_BF16)
        pool_keys_kernel<bf16_t><<<grid, PK_THREADS, 0, s>>>((bf16_t*)k_cache, (bf16_t*)v_cache, block_tables, bt_stride, pool_tables,
                                                             pt_stride, token_req, positions, slots, tokens, page_size, pool, G, d);
    else
        return tff_fail("pool_keys: unknown dtype %d", dtype);
    return tff_check_launch("pool_keys");
}

// out[t, h E + e] = o[t, h P + e] * sigmoid(g[t, h]) * scale      (g null: no gate); rows of out out_row apart
template <typename T>
__global__ __launch_bounds__(256) void gate_heads_kernel(const T* __restrict__ o, size_t o_row, int P, const float* __restrict__ g,
                                                         size_t g_row, float scale, T* __restrict__ out, size_t out_row, int HE, int E,
                                                         size_t count) {
    const size_t id = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (id >= count) return;
    const size_t t = id / HE;
    const int c = (int)(id - t * HE), h = c / E, e = c - h * E;
    const float f = g ? scale / (1.0f + expf(-g[t * g_row + h])) : scale;
    out[t * out_row + c] = from_f32<T>(to_f32(o[t * o_row + (size_t)h * P + e]) * f);
}

// The same, eight neighbouring elements a thread (E, P and the rows' strides multiples of 8).
__global__ __launch_bounds__(256) void gate_heads8_kernel(const bf16_t* __restrict__ o, size_t o_row, int P, const float* __restrict__ g,
                                                          size_t g_row, float scale, bf16_t* __restrict__ out, size_t out_row, int HE8,
                                                          int E8, size_t count) {
    const size_t id = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (id >= count) return;
    const size_t t = id / HE8;
    const int c = (int)(id - t * HE8), h = c / E8, e = c - h * E8;
    const float f = g ? scale / (1.0f + expf(-g[t * g_row + h])) : scale;
    union { uint4 u; bf16_t b[8]; } x;
    x.u = *reinterpret_cast<const uint4*>(o + t * o_row + (size_t)h * P + e * 8);
#pragma unroll
    for (int i = 0; i < 8; ++i) x.b[i] = (bf16_t)((float)x.b[i] * f);
    *reinterpret_cast<uint4*>(out + t * out_row + (size_t)c * 8) = x.u;
}

TFF_API int tff_gate_heads(const void* o, size_t o_row, int P, const float* g, size_t g_row, float scale, void* out, size_t out_row,
                           int T, int H, int E, int dtype, tff_stream_t stream) {
    TFF_REQUIRE(o && out, "gate_heads: null pointer");
    TFF_REQUIRE(T >= 0 && H > 0 && E > 0 && P >= E && o_row >= (size_t)H * P && out_row >= (size_t)H * E && (!g || g_row >= (size_t)H),
                "gate_heads: bad sizes");
    if (T == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const size_t count = (size_t)T * H * E;
    const unsigned blocks = (unsigned)((count + 255) / 256);
    if (dtype == TFF_BF16 && E % 8 == 0 && P % 8 == 0 && o_row % 8 == 0 && out_row % 8 == 0 && ((uintptr_t)o % 16) == 0 &&
        ((uintptr_t)out % 16) == 0) {
        gate_heads8_kernel<<<(unsigned)((count / 8 + 255) / 256), 256, 0, s>>>((const bf16_t*)o, o_row, P, g, g_row, scale, (bf16_t*)out,
                                                                               out_row, H * E / 8, E / 8, count / 8);
        return tff_check_launch("gate_heads");
    }
    if (dtype == TFF_F32)
        gate_heads_kernel<float><<<blocks, 256, 0, s>>>((const float*)o, o_row, P, g, g_row, scale, (float*)out, out_row, H * E, E, count);
    else if (dtype == TFF_BF16)
        gate_heads_kernel<bf16_t><<<blocks, 256, 0, s>>>((const bf16_t*)o, o_row, P, g, g_row, scale, (bf16_t*)out, out_row, H * E, E, count);
    else
        return tff_fail("gate_heads: unknown dtype %d", dtype);
    return tff_check_launch("gate_heads");
}
