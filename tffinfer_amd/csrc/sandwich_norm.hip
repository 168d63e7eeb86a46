// The norms of a layer that norms before and after each sublayer, and the convolution over time of what the
// sublayers read.
//
// tff_add_layernorm, per row:
//   d = (planes of a, in order) + bias                                       one sublayer's result, or
//   d = (planes of a) + bias + b_scale[row] * (planes of b)                  two results, one with a factor per row, or
//   d = (rms(a) * wa + rms(b) * wb) / 2                                      two normed results side by side
//   y = layernorm(d; nw, nb) * scale                                         (nw null: y = d; scale null: 1)
//   resid <- resid + y + extra;   h = layernorm(resid; w, b)                 -> out
//   (extra: a row for every row of the step, or one row for all; a layer norm's bias may be null)
//   with a convolution (steps of one token a request):  h <- h + sum_j cw[j] h_(t - taps + 1 + j), the earlier
//   h from the request's state row, which moves on by one
// Every part is optional: without a term the stream is only normed; with `rows` the norm of those rows leaves
// and resid stays as it is; without resid out is y itself.
// A layer norm takes two passes over its row's registers: the mean first, then the squares of what is left after
// subtracting it (no difference of moments).  Everything is float32; one block a row, the row in registers, a
// reduction costs one barrier.
//
// tff_input_conv: the same convolution for portions of any length: out = h + conv(h) over each request's tokens of
// the step, inputs before the portion from the state, the last taps - 1 inputs left there.
#include "common.h"
#include "tffinfer_kernels.h"

#define SN_MAX_W 16384
#define SN_MAX_TAPS 32

struct SandwichTerm {
    const float* a;            // null: no term
    const float* b;            // the second of two results, or null
    const float* b_scale;      // a factor per row on b (null: 1), where the two are not normed
    const float *wa, *wb;      // their RMS norms' weights, or null
    const float* bias;         // added to a
    const float *nw, *nb;      // the layer norm of the term, or null
    const float* scale;
    size_t plane_a, plane_b;
    int planes_a, planes_b;
    float pair_eps, n_eps;
    const float* extra;        // added to the stream beside the term, rows extra_row apart (0: one row for all), or null
    size_t extra_row;
};

struct SandwichConv {
    const float* w;            // [taps][W], or null
    float* state;              // [slots][state_row], the inputs [taps - 1][W] at off, oldest first
    const int32_t* slots;
    size_t state_row, off;
    int taps;
};

// Sum over the block; red: NT / 64 floats that no earlier call used since the last barrier after its reads.
template <int NT>
__device__ __forceinline__ float sn_total(float v, float* red) {
    v = rows_sum(row16_sum(v));
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NT / 64; ++i) s += red[i];
    return s;
}

template <int VEC>
__device__ __forceinline__ void sn_load(float (&v)[VEC], const float* p) {
    if constexpr (VEC == 4) {
        const float4 x = *reinterpret_cast<const float4*>(p);
        v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
    } else {
        v[0] = *p;
    }
}
template <int VEC, typename TO>
__device__ __forceinline__ void sn_store(TO* p, const float (&v)[VEC]) {
    if constexpr (VEC == 4) {
        if constexpr (sizeof(TO) == 4) {
            *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
            union { bf16_t h[4]; uint2 u; } pk;
#pragma unroll
            for (int e = 0; e < 4; ++e) pk.h[e] = (bf16_t)v[e];
            *reinterpret_cast<uint2*>(p) = pk.u;
        }
    } else {
        *p = from_f32<TO>(v[0]);
    }
}

// What a thread needs of the vectors as long as a row (weights, biases, the convolution's taps and state).  With few
// elements a thread (EARLY) everything is asked for at the start, so that a step of few rows, which nothing else
// hides, waits for memory once; with many it is fetched where it is used.
#define SN_EARLY_TAPS 4

template <int IT, int VEC, bool EARLY>
struct SandwichVector {
    float v[EARLY ? IT : 1][VEC];
    const float* p;
    __device__ __forceinline__ void ask(const float* src, int W, int tid, int nt) {
        p = src;
        if constexpr (EARLY) {
#pragma unroll
            for (int it = 0; it < IT; ++it) {
#pragma unroll
                for (int u = 0; u < VEC; ++u) v[it][u] = 0.f;
                const int e = (it * nt + tid) * VEC;
                if (src && e < W) sn_load<VEC>(v[it], src + e);
            }
        }
    }
    __device__ __forceinline__ void take(float (&out)[VEC], int it, int e) const {
        if constexpr (EARLY) {
#pragma unroll
            for (int u = 0; u < VEC; ++u) out[u] = v[it][u];
        } else if (p) {
            sn_load<VEC>(out, p + e);
        } else {
#pragma unroll
            for (int u = 0; u < VEC; ++u) out[u] = 0.f;
        }
    }
};

template <typename TO, int NT, int VPT, int VEC>
__global__ __launch_bounds__(NT) void add_layernorm_kernel(float* __restrict__ resid, const SandwichTerm tm,
                                                           const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                           TO* __restrict__ out, const int32_t* __restrict__ rows, int W,
                                                           const SandwichConv cv) {
    constexpr int IT = VPT / VEC;
    constexpr bool EARLY = VPT <= 4;
    __shared__ float red[6][NT / 64];
    const int i = blockIdx.x, tid = threadIdx.x;
    const size_t row = rows ? (size_t)rows[i] : (size_t)i;
    const float inv_w = 1.0f / (float)W;
    const size_t at = row * W;
    float* const xr = resid ? resid + at : nullptr;
    const float* const ar = tm.a ? tm.a + at : nullptr;
    const float* const br = tm.b ? tm.b + at : nullptr;
    const float bs = br && tm.b_scale ? tm.b_scale[row] : 1.0f;
    const int slot = cv.w ? cv.slots[i] : 0;
    float x[IT][VEC], d[IT][VEC], p2[IT][VEC];
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int e = (it * NT + tid) * VEC;
#pragma unroll
        for (int u = 0; u < VEC; ++u) x[it][u] = d[it][u] = p2[it][u] = 0.f;
        if (e < W) {
            if (xr) sn_load<VEC>(x[it], xr + e);
            if (ar) sn_load<VEC>(d[it], ar + e);
            if (br) sn_load<VEC>(p2[it], br + e);
            if (tm.extra) {
                float t[VEC];
                sn_load<VEC>(t, tm.extra + row * tm.extra_row + e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) x[it][u] += t[u];
            }
        }
    }
    SandwichVector<IT, VEC, EARLY> vbias, vwa, vwb, vnw, vnb, vsc, vw, vb;
    vbias.ask(tm.bias, W, tid, NT);
    vwa.ask(tm.wa, W, tid, NT);
    vwb.ask(tm.wb, W, tid, NT);
    vnw.ask(tm.nw, W, tid, NT);
    vnb.ask(tm.nb, W, tid, NT);
    vsc.ask(tm.scale, W, tid, NT);
    vw.ask(w, W, tid, NT);
    vb.ask(b, W, tid, NT);
    float* const st = cv.w && cv.taps > 1 ? cv.state + (size_t)slot * cv.state_row + cv.off : nullptr;
    float cw[EARLY ? SN_EARLY_TAPS : 1][EARLY ? IT : 1][VEC], cs[EARLY ? SN_EARLY_TAPS : 1][EARLY ? IT : 1][VEC];
    const bool early_conv = EARLY && cv.w && cv.taps <= SN_EARLY_TAPS;
    if constexpr (EARLY) {
        if (early_conv) {
#pragma unroll
            for (int j = 0; j < SN_EARLY_TAPS; ++j)
#pragma unroll
                for (int it = 0; it < IT; ++it) {
                    const int e = (it * NT + tid) * VEC;
#pragma unroll
                    for (int u = 0; u < VEC; ++u) cw[j][it][u] = cs[j][it][u] = 0.f;
                    if (j < cv.taps && e < W) {
                        sn_load<VEC>(cw[j][it], cv.w + (size_t)j * W + e);
                        if (j < cv.taps - 1) {
#pragma unroll
                            for (int u = 0; u < VEC; ++u) cs[j][it][u] = st[(size_t)j * W + e + u];
                        }
                    }
                }
        }
    }
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int e = (it * NT + tid) * VEC;
        if (e < W) {
            float t[VEC];
            for (int p = 1; p < tm.planes_a; ++p) {
                sn_load<VEC>(t, ar + p * tm.plane_a + e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) d[it][u] += t[u];
            }
            for (int p = 1; p < tm.planes_b; ++p) {
                sn_load<VEC>(t, br + p * tm.plane_b + e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) p2[it][u] += t[u];
            }
            if (br && !tm.wa) {
#pragma unroll
                for (int u = 0; u < VEC; ++u) d[it][u] = fmaf(p2[it][u], bs, d[it][u]);
            }
            if (tm.bias) {
                vbias.take(t, it, e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) d[it][u] += t[u];
            }
        }
    }
    // v <- (v - mean) / sqrt(variance + eps) * lw + lb, elements past the row left at what they are
    auto layernorm = [&](float (&v)[IT][VEC], const auto& lw, const auto& lb, float le, float* r0, float* r1) {
        float s = 0.f;
#pragma unroll
        for (int it = 0; it < IT; ++it)
#pragma unroll
            for (int u = 0; u < VEC; ++u) s += v[it][u];        // (zeros past the row)
        const float mean = sn_total<NT>(s, r0) * inv_w;
        s = 0.f;
#pragma unroll
        for (int it = 0; it < IT; ++it)
#pragma unroll
            for (int u = 0; u < VEC; ++u) {
                const float c = (it * NT + tid) * VEC < W ? v[it][u] - mean : 0.f;
                v[it][u] = c;
                s = fmaf(c, c, s);
            }
        const float rr = 1.0f / sqrtf(sn_total<NT>(s, r1) * inv_w + le);
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int e = (it * NT + tid) * VEC;
            if (e < W) {
                float a[VEC], c[VEC];
                lw.take(a, it, e);
                lb.take(c, it, e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) v[it][u] = fmaf(v[it][u] * rr, a[u], c[u]);
            }
        }
    };
    if (br && tm.wa) {
        float s0 = 0.f, s1 = 0.f;
#pragma unroll
        for (int it = 0; it < IT; ++it)
#pragma unroll
            for (int u = 0; u < VEC; ++u) {
                s0 = fmaf(d[it][u], d[it][u], s0);
                s1 = fmaf(p2[it][u], p2[it][u], s1);
            }
        s0 = rows_sum(row16_sum(s0));
        s1 = rows_sum(row16_sum(s1));
        if ((tid & 63) == 0) { red[4][tid >> 6] = s0; red[5][tid >> 6] = s1; }
        __syncthreads();
        s0 = s1 = 0.f;
#pragma unroll
        for (int q = 0; q < NT / 64; ++q) { s0 += red[4][q]; s1 += red[5][q]; }
        const float fa = 0.5f / sqrtf(s0 * inv_w + tm.pair_eps), fb = 0.5f / sqrtf(s1 * inv_w + tm.pair_eps);
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int e = (it * NT + tid) * VEC;
            if (e < W) {
                float a[VEC], c[VEC];
                vwa.take(a, it, e);
                vwb.take(c, it, e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) d[it][u] = d[it][u] * fa * a[u] + p2[it][u] * fb * c[u];
            }
        }
    }
    if (ar) {
        if (tm.nw) layernorm(d, vnw, vnb, tm.n_eps, red[0], red[1]);
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int e = (it * NT + tid) * VEC;
            if (e < W) {
                if (tm.scale) {
                    float c[VEC];
                    vsc.take(c, it, e);
#pragma unroll
                    for (int u = 0; u < VEC; ++u) d[it][u] *= c[u];
                }
#pragma unroll
                for (int u = 0; u < VEC; ++u) x[it][u] += d[it][u];
            }
        }
    }
    if ((ar || tm.extra) && xr && !rows) {
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int e = (it * NT + tid) * VEC;
            if (e < W) sn_store<VEC, float>(xr + e, x[it]);
        }
    }
    if (w) layernorm(x, vw, vb, eps, red[2], red[3]);
    if (cv.w) {
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int e = (it * NT + tid) * VEC;
            if (e < W) {
                float y[VEC];
#pragma unroll
                for (int u = 0; u < VEC; ++u) y[u] = 0.f;
                bool done = false;
                if constexpr (EARLY) {
                    if (early_conv) {
                        done = true;
#pragma unroll
                        for (int j = 0; j < SN_EARLY_TAPS; ++j) {
                            const bool last = j == cv.taps - 1;
                            if (j < cv.taps) {
#pragma unroll
                                for (int u = 0; u < VEC; ++u) {
                                    y[u] = fmaf(cw[j][it][u], last ? x[it][u] : cs[j][it][u], y[u]);
                                    if (j > 0) st[(size_t)(j - 1) * W + e + u] = last ? x[it][u] : cs[j][it][u];
                                }
                            }
                        }
                    }
                }
                if (!done) {
                    for (int j = 0; j < cv.taps; ++j) {
                        float c[VEC];
                        sn_load<VEC>(c, cv.w + (size_t)j * W + e);
                        const bool last = j == cv.taps - 1;
#pragma unroll
                        for (int u = 0; u < VEC; ++u) {
                            const float h = last ? x[it][u] : st[(size_t)j * W + e + u];
                            y[u] = fmaf(c[u], h, y[u]);
                            if (j > 0) st[(size_t)(j - 1) * W + e + u] = h;
                        }
                    }
                }
#pragma unroll
                for (int u = 0; u < VEC; ++u) x[it][u] += y[u];
            }
        }
    }
    TO* const orow = out + (size_t)i * W;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int e = (it * NT + tid) * VEC;
        if (e < W) sn_store<VEC, TO>(orow + e, x[it]);
    }
}

TFF_API int tff_add_layernorm(float* resid, const float* a, int planes_a, size_t plane_a, const float* b, int planes_b,
                              size_t plane_b, const float* b_scale, const float* wa, const float* wb, float pair_eps, const float* bias,
                              const float* nw, const float* nb, float n_eps, const float* scale, const float* w,
                              const float* beta, float eps, void* out, const int32_t* rows, int n, int W, const float* conv_w,
                              int taps, float* state, size_t state_row, size_t state_off, const int32_t* state_slots,
                              const float* extra, size_t extra_row, int out_dtype, tff_stream_t stream) {
    TFF_REQUIRE((resid || a) && out, "add_layernorm: null pointer");
    TFF_REQUIRE(n >= 0 && W > 0 && W <= SN_MAX_W, "add_layernorm: rows of %d (up to %d)", W, SN_MAX_W);
    TFF_REQUIRE(!a || planes_a >= 1, "add_layernorm: a term without planes");
    TFF_REQUIRE(!b || (a && (!wa) == (!wb) && planes_b >= 1), "add_layernorm: the second of two results needs the first, and both weights or none");
    TFF_REQUIRE((nw || !nb) && (w || !beta) && (!nw || a), "add_layernorm: a norm takes a weight, and a bias or none");
    TFF_REQUIRE(!extra || (resid && (extra_row == 0 || extra_row >= (size_t)W)), "add_layernorm: rows of %zu to add to a stream of %d", extra_row, W);
    TFF_REQUIRE(!rows || resid, "add_layernorm: chosen rows of no stream");
    TFF_REQUIRE(!conv_w || (taps >= 1 && taps <= SN_MAX_TAPS && !rows && (taps == 1 || (state && state_slots &&
                state_off + (size_t)(taps - 1) * W <= state_row))), "add_layernorm: a convolution of %d taps (up to %d) needs its state", taps, SN_MAX_TAPS);
    if (n == 0) return 0;
    const SandwichTerm tm{a, b, b_scale, wa, wb, bias, nw, nb, scale, plane_a, plane_b, planes_a, planes_b, pair_eps, n_eps, extra, extra_row};
    const SandwichConv cv{conv_w, state, state_slots, state_row, state_off, taps};
    hipStream_t s = (hipStream_t)stream;
    auto ok16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool vec = W % 4 == 0 && plane_a % 4 == 0 && plane_b % 4 == 0 && ok16(resid) && ok16(a) && ok16(b) && ok16(wa) && ok16(wb) &&
                     ok16(bias) && ok16(nw) && ok16(nb) && ok16(scale) && ok16(w) && ok16(beta) && ok16(out) && ok16(conv_w) && ok16(extra) && extra_row % 4 == 0;
    TFF_REQUIRE(vec || W <= 8192, "add_layernorm: rows of %d (more than 8192) must be a multiple of 4 wide and 16-byte aligned", W);
#define SN_LAUNCH(TO, NT, VPT, VEC) add_layernorm_kernel<TO, NT, VPT, VEC><<<n, NT, 0, s>>>(resid, tm, w, beta, eps, (TO*)out, rows, W, cv)
#define SN_SIZES(TO)                                                                         \
    do {                                                                                     \
        if (!vec) {                                                                          \
            if (W <= 1024) SN_LAUNCH(TO, 256, 4, 1);                                         \
            else if (W <= 4096) SN_LAUNCH(TO, 1024, 4, 1);                                   \
            else SN_LAUNCH(TO, 1024, 8, 1);                                                  \
        } else if (W <= 1024) SN_LAUNCH(TO, 256, 4, 4);                                      \
        else if (W <= 4096 && n <= 256) SN_LAUNCH(TO, 1024, 4, 4);                           \
        else if (W <= 2048) SN_LAUNCH(TO, 256, 8, 4);                                        \
        else if (W <= 4096) SN_LAUNCH(TO, 256, 16, 4);                                       \
        else SN_LAUNCH(TO, 1024, 16, 4);                                                     \
    } while (0)
    if (out_dtype == TFF_F32) SN_SIZES(float);
    else if (out_dtype == TFF_BF16) SN_SIZES(bf16_t);
    else return tff_fail("add_layernorm: unknown dtype %d", out_dtype);
#undef SN_SIZES
#undef SN_LAUNCH
    return tff_check_launch("add_layernorm");
}

// Items (row of the step's tables, first place in the request's portion) of up to `chunk` tokens; a thread takes
// VEC neighbouring channels through an item's tokens, the taps' inputs in registers.  The first item of a portion
// alone reads the state (chunk >= taps - 1) and alone leaves the new one there, each thread its own channels.

template <typename TO, int TAPS, int VEC>
__global__ __launch_bounds__(256) void input_conv_kernel(const float* __restrict__ h, const float* __restrict__ w, int taps_any,
                                                         float* __restrict__ state, size_t state_row, size_t off,
                                                         const int32_t* __restrict__ items, int chunk, const int32_t* __restrict__ cu_tokens,
                                                         const int32_t* __restrict__ slots, TO* __restrict__ out, int W) {
    const int e = (blockIdx.y * 256 + threadIdx.x) * VEC;
    if (e >= W) return;
    const int r = items[2 * blockIdx.x], i0 = items[2 * blockIdx.x + 1];
    const int t0 = cu_tokens[r], n = cu_tokens[r + 1] - t0;
    const int i1 = min(n, i0 + chunk);
    const int taps = TAPS ? TAPS : taps_any;
    float* st = state ? state + (size_t)slots[r] * state_row + off : nullptr;
    const float* base = h + (size_t)t0 * W + e;
    // input at place i of the portion (before it: the state's)
    auto input = [&](float (&v)[VEC], int i) {
        if (i >= 0) {
            sn_load<VEC>(v, base + (size_t)i * W);
        } else {
#pragma unroll
            for (int u = 0; u < VEC; ++u) v[u] = st[(size_t)(i + taps - 1) * W + e + u];
        }
    };
    if constexpr (TAPS > 0) {
        float wr[TAPS][VEC], x[TAPS][VEC];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) sn_load<VEC>(wr[j], w + (size_t)j * W + e);
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) input(x[j + 1], i0 - (TAPS - 1) + j);
        for (int i = i0; i < i1; ++i) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
                for (int u = 0; u < VEC; ++u) x[j][u] = x[j + 1][u];
            sn_load<VEC>(x[TAPS - 1], base + (size_t)i * W);
            float y[VEC];
#pragma unroll
            for (int u = 0; u < VEC; ++u) {
                float a = 0.f;
#pragma unroll
                for (int j = 0; j < TAPS; ++j) a = fmaf(wr[j][u], x[j][u], a);
                y[u] = x[TAPS - 1][u] + a;
            }
            sn_store<VEC, TO>(out + (size_t)(t0 + i) * W + e, y);
        }
    } else {
        for (int i = i0; i < i1; ++i) {
            float y[VEC], v[VEC], c[VEC];
#pragma unroll
            for (int u = 0; u < VEC; ++u) y[u] = v[u] = 0.f;
            for (int j = 0; j < taps; ++j) {
                input(v, i - (taps - 1) + j);
                sn_load<VEC>(c, w + (size_t)j * W + e);
#pragma unroll
                for (int u = 0; u < VEC; ++u) y[u] = fmaf(c[u], v[u], y[u]);
            }
#pragma unroll
            for (int u = 0; u < VEC; ++u) y[u] += v[u];
            sn_store<VEC, TO>(out + (size_t)(t0 + i) * W + e, y);
        }
    }
    if (i0 == 0) {
        for (int j = 0; j < taps - 1; ++j) {        // ascending: what is read lies behind what was written
            float v[VEC];
            input(v, n - (taps - 1) + j);
#pragma unroll
            for (int u = 0; u < VEC; ++u) st[(size_t)j * W + e + u] = v[u];
        }
    }
}

TFF_API int tff_input_conv(const float* h, const float* w, int taps, float* state, size_t state_row, size_t state_off,
                           const int32_t* items, int num_items, int chunk, const int32_t* cu_tokens, const int32_t* state_slots,
                           void* out, int W, int out_dtype, tff_stream_t stream) {
    TFF_REQUIRE(h && w && items && cu_tokens && out, "input_conv: null pointer");
    TFF_REQUIRE(num_items >= 0 && W > 0 && taps >= 1 && taps <= SN_MAX_TAPS && chunk >= 1 && chunk >= taps - 1,
                "input_conv: rows of %d, %d taps (up to %d), items of %d tokens", W, taps, SN_MAX_TAPS, chunk);
    TFF_REQUIRE(taps == 1 || (state && state_slots && state_off + (size_t)(taps - 1) * W <= state_row),
                "input_conv: state rows of %zu do not hold %d rows of %d", state_row, taps - 1, W);
    if (num_items == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const bool vec = W % 4 == 0 && ((uintptr_t)h % 16) == 0 && ((uintptr_t)w % 16) == 0 && ((uintptr_t)out % 16) == 0;
    const int per = vec ? 1024 : 256;
    const dim3 grid(num_items, (W + per - 1) / per);
    if (taps == 1) state = nullptr;
#define SC_GO(TO, TAPS, VEC) input_conv_kernel<TO, TAPS, VEC><<<grid, 256, 0, s>>>(h, w, taps, state, state_row, state_off, items, chunk, \
                                                                                  cu_tokens, state_slots, (TO*)out, W)
#define SC_TAPS(TO)                                                                               \
    do {                                                                                          \
        if (!vec) SC_GO(TO, 0, 1);                                                                \
        else if (taps == 2) SC_GO(TO, 2, 4);                                                      \
        else if (taps == 3) SC_GO(TO, 3, 4);                                                      \
        else if (taps == 4) SC_GO(TO, 4, 4);                                                      \
        else SC_GO(TO, 0, 4);                                                                     \
    } while (0)
    if (out_dtype == TFF_F32) SC_TAPS(float);
    else if (out_dtype == TFF_BF16) SC_TAPS(bf16_t);
    else return tff_fail("input_conv: unknown dtype %d", out_dtype);
#undef SC_TAPS
#undef SC_GO
    return tff_check_launch("input_conv");
}
