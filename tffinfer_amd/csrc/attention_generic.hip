// Attention over the paged cache for any head size, group size, page size and
// window, in float32 arithmetic: the path of the 32-bit model, and the yardstick
// the matrix-core kernels are checked against.
//
// One wave per (token, q head).  Keys are taken 64 at a time, one per lane:
//   s_j = (q . k_j) * scale                   (scale after the product; with a cap c > 0, s_j <- c tanh(s_j / c);
//                                              reference paged_flash_attention.cu:723)
//   visible iff  lo <= j <= pos               (causal: mask_op.cu:37-43; lo from the window)
// With pools, keys of whole blocks of `pool` tokens (found through tables of their own) come before the
// window's: block b is visible iff its last token is (b + 1) pool - 1 <= pos - window.
//   running max m and sum l over chunks       (paged_flash_attention.cu:746-790)
//   o = sum_j exp(s_j - m) v_j / l            (l also holds e^(sink - m) of the head, if sinks are given)
// q head h reads kv head h / (nq / nkv)       (paged_flash_attention.cu:891-892).
// Keys lie [page, kv head, slot, element], values [page, kv head, element, slot].
// Keys are found by block id arithmetic, not by a table of addresses as in the
// reference (src/kernel/cuda/get_row.cu:73-109).
#include "common.h"
#include "tffinfer_kernels.h"

#define AG_MAX_D 1024     // (a kernel for head sizes up to 512, one for those beyond: the accumulators are registers)

template <typename T, typename TC, int MAXD>
__global__ __launch_bounds__(64) void attention_generic_kernel(
    const T* __restrict__ q, int q_stride, T* __restrict__ out, const TC* __restrict__ k_cache,
    const TC* __restrict__ v_cache, const int32_t* __restrict__ block_tables, int bt_stride,
    const int32_t* __restrict__ token_req, const int32_t* __restrict__ positions, int nq, int nkv,
    int d, int page_size, int window, float scale, const float* __restrict__ sinks, float softcap,
    const int32_t* __restrict__ pool_tables, int pt_stride, int pool) {
    __shared__ float qs[MAXD];
    __shared__ long long voff[64];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int G = nq / nkv;
    const int g = h / G;
    const int r = token_req[t];
    const int pos = positions[t];
    const int blocks_seen = pool > 0 ? max(0, pos - window + 1) / pool : 0;

    const T* qp = q + (size_t)t * q_stride + (size_t)h * d;
    for (int e = lane; e < d; e += 64) qs[e] = to_f32(qp[e]);
    __syncthreads();

    float m = -INFINITY, l = 0.f;
    float acc[MAXD / 64];
#pragma unroll
    for (int i = 0; i < MAXD / 64; ++i) acc[i] = 0.f;

    // first the keys of the blocks before the window, if there are any, then the tokens' own
    for (int part = blocks_seen > 0 ? 0 : 1; part < 2; ++part) {
    const int lo = (part == 1 && window > 0) ? max(0, pos - window + 1) : 0;
    const int hi = part == 1 ? pos : blocks_seen - 1;
    const int32_t* bt = part == 1 ? block_tables + (size_t)r * bt_stride : pool_tables + (size_t)r * pt_stride;
    for (int base = lo; base <= hi; base += 64) {
        const int j = base + lane;
        const bool valid = j <= hi;
        float s = -INFINITY;
        long long off = 0;
        if (valid) {
            const int page = bt[j / page_size];
            const long long head_base = ((long long)page * nkv + g) * page_size * d;
            off = head_base + (j % page_size);   // values: [element][slot]
            const TC* kp = k_cache + head_base + (long long)(j % page_size) * d;
            float dot = 0.f;
            for (int e = 0; e < d; ++e) dot = fmaf(qs[e], to_f32(kp[e]), dot);
            s = dot * scale;
            if (softcap > 0.f) s = softcap * tanhf(s / softcap);      // a cap on the scores, before the mask
        }
        __syncthreads();  // earlier readers of voff are done
        voff[lane] = off;
        const float cmax = wave_max(s);
        const float m_new = fmaxf(m, cmax);
        const float p = valid ? expf(s - m_new) : 0.f;
        const float corr = expf(m - m_new);  // 0 on the first chunk (m = -inf)
        l = l * corr + wave_sum(p);
        m = m_new;
        __syncthreads();
        const int nvalid = min(64, hi - base + 1);
#pragma unroll
        for (int i = 0; i < MAXD / 64; ++i) acc[i] *= corr;
        for (int jj = 0; jj < nvalid; ++jj) {
            const float pj = __shfl(p, jj, 64);
            const TC* vp = v_cache + voff[jj];
#pragma unroll
            for (int i = 0; i < MAXD / 64; ++i) {
                const int e = lane + 64 * i;
                if (e < d) acc[i] = fmaf(pj, to_f32(vp[(long long)e * page_size]), acc[i]);
            }
        }
    }
    }
    T* op = out + (size_t)t * nq * d + (size_t)h * d;
    // a sink: one more term e^sink in the denominator, with no key and no value, not scaled
    if (sinks) l += expf(sinks[h] - m);
    const float inv = 1.0f / l;
#pragma unroll
    for (int i = 0; i < MAXD / 64; ++i) {
        const int e = lane + 64 * i;
        if (e < d) op[e] = from_f32<T>(acc[i] * inv);
    }
}

TFF_API int tff_attention_generic(const void* q, int q_stride, void* out, const void* k_cache,
                                  const void* v_cache, const int32_t* block_tables, int bt_stride,
                                  const int32_t* token_req, const int32_t* positions, int T, int nq,
                                  int nkv, int d, int page_size, int num_pages, int window,
                                  float scale, const float* sinks, float softcap, const int32_t* pool_tables,
                                  int pt_stride, int pool, int dtype, int cache_dtype, tff_stream_t stream) {
    TFF_REQUIRE(q && out && k_cache && v_cache && block_tables && token_req && positions,
                "attention: null pointer");
    TFF_REQUIRE(T >= 0 && nq > 0 && nkv > 0 && nq % nkv == 0,
                "attention: %d query heads are not a multiple of %d key heads", nq, nkv);
    TFF_REQUIRE(d > 0 && d <= AG_MAX_D, "attention: head size %d not supported (1..%d)", d, AG_MAX_D);
    TFF_REQUIRE(page_size > 0 && num_pages > 0 && bt_stride > 0 && window >= 0,
                "attention: bad cache geometry page_size=%d pages=%d table stride=%d window=%d",
                page_size, num_pages, bt_stride, window);
    TFF_REQUIRE(q_stride >= nq * d, "attention: query row stride %d below %d", q_stride, nq * d);
    TFF_REQUIRE(dtype == cache_dtype, "attention: cache type %d differs from activation type %d",
                cache_dtype, dtype);
    TFF_REQUIRE(nq <= 65535, "attention: too many heads");
    TFF_REQUIRE(pool >= 0 && (pool == 0 || (window > 0 && pool_tables && pt_stride > 0)),
                "attention: keys of blocks of %d tokens stand before a window and need their tables", pool);
    if (T == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    dim3 grid(T, nq);
#define TFF_AG(TT, MAXD)                                                                                            \
    attention_generic_kernel<TT, TT, MAXD><<<grid, 64, 0, s>>>((const TT*)q, q_stride, (TT*)out, (const TT*)k_cache, \
                                                              (const TT*)v_cache, block_tables, bt_stride, token_req, \
                                                              positions, nq, nkv, d, page_size, window, scale, sinks, softcap, \
                                                              pool_tables, pt_stride, pool)
    if (dtype == TFF_F32) {
        if (d <= 512) TFF_AG(float, 512); else TFF_AG(float, AG_MAX_D);
    } else if (dtype == TFF_BF16) {
        if (d <= 512) TFF_AG(bf16_t, 512); else TFF_AG(bf16_t, AG_MAX_D);
    } else {
        return tff_fail("attention: unknown dtype %d", dtype);
    }
#undef TFF_AG
    return tff_check_launch("attention_generic");
}
