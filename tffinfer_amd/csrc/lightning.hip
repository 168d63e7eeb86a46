// A linear recurrence with a fixed decay per head: per request and head a matrix S [key channel, value channel],
//   S <- decay S + k_t v_t^T,   o_t = S^T q_t,      q, k, v = silu of their projections, all float32.
// A request's state row: [heads][value channel][key channel] (S transposed: the key channels of one value channel
// lie side by side, as the lanes that share the channel read them).
//
// tff_lightning:         the recurrence over each request's tokens of the step, token by token.
// tff_lightning_chunks:  the same for portions of many tokens, in chunks of 64.  With S the state before a chunk of n
//                        tokens and g the decay,
//                          o_i = g^(i+1) S^T q_i + sum over j <= i of g^(i-j) (q_i . k_j) v_j,
//                          S  <- g^n S + sum over j of g^(n-1-j) k_j v_j^T:
//                        what a chunk adds to the state depends on its own tokens only, so all chunks form it at once
//                        (1), a pass over the chunks' sums leaves in each one's place the state before it (2), and all
//                        chunks form their outputs at once (3).  The products run on the matrix cores in float32.
// tff_row_norm_gate:  out = o / sqrt(mean over the row of o^2 + eps) * w * sigmoid(gate).
#include "common.h"
#include "tffinfer_kernels.h"

// (the hardware's exponential and reciprocal: a few units in the last place of float32)
__device__ __forceinline__ float lt_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// Block: sixteen value channels of one head of one request; a row of sixteen lanes shares a value channel, lane s
// holding the key channels s, s + 16, ...  No LDS and no barrier: for steps of a few tokens a request.
template <int KPL>
__global__ __launch_bounds__(256) void lightning_few_kernel(const float* __restrict__ proj, size_t ldp,
                                                            const float* __restrict__ decay, float* __restrict__ state,
                                                            size_t state_row, const int32_t* __restrict__ cu_tokens,
                                                            const int32_t* __restrict__ state_slots, float* __restrict__ o, int H,
                                                            int D, int E) {
    const int h = blockIdx.y, r = blockIdx.z, tid = threadIdx.x, s = tid & 15;
    const int j = blockIdx.x * 16 + (tid >> 4), jc = min(j, E - 1);
    const int t0 = cu_tokens[r], n = cu_tokens[r + 1] - t0;
    const bool live = j < E;
    const float g = decay[h];
    float* sp = state + (size_t)state_slots[r] * state_row + ((size_t)h * E + jc) * D + s;
    if (n <= 0) return;
    // a token's projections are asked for while the token before is worked on, the first one's with the state
    float S[KPL], qn[KPL], kn[KPL], vn;
    const float* p = proj + (size_t)t0 * ldp;
    const size_t oq = (size_t)h * D + s, ok = oq + (size_t)H * D, ov = 2 * (size_t)H * D + (size_t)h * E + jc;
    auto ask = [&](const float* row) {
#pragma unroll
        for (int m = 0; m < KPL; ++m) {
            const bool in = s + 16 * m < D;
            qn[m] = in ? row[oq + 16 * m] : 0.f;
            kn[m] = in ? row[ok + 16 * m] : 0.f;
        }
        vn = row[ov];
    };
    ask(p);
#pragma unroll
    for (int m = 0; m < KPL; ++m) S[m] = (live && s + 16 * m < D) ? sp[16 * m] : 0.f;
    for (int t = 0; t < n; ++t) {
        float kk[KPL], qq[KPL];
#pragma unroll
        for (int m = 0; m < KPL; ++m) {
            qq[m] = lt_silu(qn[m]);         // (silu(0) = 0)
            kk[m] = lt_silu(kn[m]);
        }
        const float v = lt_silu(vn);
        p += ldp;
        if (t + 1 < n) ask(p);
        float a = 0.f;
#pragma unroll
        for (int m = 0; m < KPL; ++m) {
            S[m] = fmaf(kk[m], v, g * S[m]);
            a = fmaf(S[m], qq[m], a);
        }
        a = row16_sum(a);
        if (s == 0 && live) o[(size_t)(t0 + t) * H * E + (size_t)h * E + j] = a;
    }
    if (live) {
#pragma unroll
        for (int m = 0; m < KPL; ++m)
            if (s + 16 * m < D) sp[16 * m] = S[m];
    }
}

TFF_API int tff_lightning(const float* proj, size_t ldp, const float* decay, float* state, size_t state_row,
                          const int32_t* cu_tokens, const int32_t* state_slots, float* o, int R, int H, int D, int E,
                          tff_stream_t stream) {
    TFF_REQUIRE(proj && decay && state && cu_tokens && state_slots && o, "lightning: null pointer");
    TFF_REQUIRE(R >= 0 && H > 0 && D > 0 && D <= 256 && E > 0, "lightning: bad sizes heads=%d dim=%d vdim=%d (dim up to 256)", H, D, E);
    TFF_REQUIRE(ldp >= 2 * (size_t)H * D + (size_t)H * E && (size_t)H * E * D <= state_row,
                "lightning: rows of %zu or state rows of %zu are too short", ldp, state_row);
    TFF_REQUIRE(H <= 65535 && R <= 65535, "lightning: too many heads or requests");
    if (R == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((E + 15) / 16, H, R);
#define LT_LAUNCH(KPL) lightning_few_kernel<KPL><<<grid, 256, 0, s>>>(proj, ldp, decay, state, state_row, cu_tokens, state_slots, o, H, D, E)
    if (D <= 16) LT_LAUNCH(1);
    else if (D <= 32) LT_LAUNCH(2);
    else if (D <= 64) LT_LAUNCH(4);
    else if (D <= 128) LT_LAUNCH(8);
    else LT_LAUNCH(16);
#undef LT_LAUNCH
    return tff_check_launch("lightning");
}

// ------------------------------------------------------------------- chunks ---
// Items (row of the step's tables, first place in the request's portion) of up to LC tokens.  A 16 x 16 x 4 product of
// the matrix cores takes, from lane (r = lane & 15, g = lane >> 4), element [r][k = g] of either operand; which index of
// the inner dimension k stands for is free as long as both operands agree, so step s of four takes k = 4 g + s of
// sixteen inner indices: a lane reads its four steps' elements as one run of 16 bytes.  Its result: lane (r, g) holds rows
// 4 g .. 4 g + 3 (of the first operand) of column r (of the second).  Rows in LDS are LS floats apart.
#define LC 64
#define LS 68

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float lt_floatx4;

// acc += a[16 rows][64] . b[16 rows][64]^T, a and b pointing at the rows' first elements in LDS
__device__ __forceinline__ void lt_mma64(lt_floatx4& acc, const float* a, const float* b, int r, int g) {
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
        const float4 x = *reinterpret_cast<const float4*>(a + r * LS + kb * 16 + g * 4);
        const float4 y = *reinterpret_cast<const float4*>(b + r * LS + kb * 16 + g * 4);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc, 0, 0, 0);
    }
}

// g^n for g >= 0 (0^0 = 1)
__device__ __forceinline__ float lt_power(float log2_g, int n) { return n == 0 ? 1.0f : exp2f((float)n * log2_g); }

// Columns c0 .. c0 + 63 of 64 rows of a projection into LDS, silu applied; rows past n and columns past `cols` are zeros.
// TRANSPOSED: dst[column][row], else dst[row][column].
template <bool TRANSPOSED, bool VEC>
__device__ __forceinline__ void lt_load(float* dst, const float* __restrict__ src, size_t ld, int n, int c0, int cols) {
    if constexpr (VEC) {
        // (a multiple of four columns, 16-byte aligned rows)
        for (int x = threadIdx.x; x < LC * 16; x += 256) {
            int t, c;
            if constexpr (TRANSPOSED) { t = x & 63; c = (x >> 6) * 4; }       // (neighbouring lanes write neighbouring words)
            else { t = x >> 4; c = (x & 15) * 4; }
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (t < n && c0 + c < cols) v = *reinterpret_cast<const float4*>(src + (size_t)t * ld + c0 + c);
            v.x = lt_silu(v.x); v.y = lt_silu(v.y); v.z = lt_silu(v.z); v.w = lt_silu(v.w);       // (silu(0) = 0)
            if constexpr (TRANSPOSED) {
                dst[(c + 0) * LS + t] = v.x;
                dst[(c + 1) * LS + t] = v.y;
                dst[(c + 2) * LS + t] = v.z;
                dst[(c + 3) * LS + t] = v.w;
            } else {
                *reinterpret_cast<float4*>(dst + t * LS + c) = v;
            }
        }
    } else {
        for (int x = threadIdx.x; x < LC * 64; x += 256) {
            const int t = x >> 6, c = x & 63;
            const float v = (t < n && c0 + c < cols) ? lt_silu(src[(size_t)t * ld + c0 + c]) : 0.f;
            dst[TRANSPOSED ? c * LS + t : t * LS + c] = v;
        }
    }
}

// (1) sums[item][h][e][d] = sum over the chunk's tokens of g^(n-1-j) v_j[e] k_j[d]: blocks of 64 value channels x 64 key
// channels, a wave sixteen value channels.
template <bool VEC>
__global__ __launch_bounds__(256) void lightning_sums_kernel(const float* __restrict__ proj, size_t ldp, const float* __restrict__ decay,
                                                             const int32_t* __restrict__ items, const int32_t* __restrict__ cu_tokens,
                                                             float* __restrict__ sums, int H, int D, int E, int d_blocks) {
    __shared__ __attribute__((aligned(16))) float kt[64 * LS], vt[64 * LS];
    const int item = blockIdx.x, h = blockIdx.y, eb = blockIdx.z / d_blocks, db = blockIdx.z - eb * d_blocks;
    const int r = items[2 * item], i0 = items[2 * item + 1];
    const int t0 = cu_tokens[r] + i0, n = min(LC, cu_tokens[r + 1] - t0);
    const float* p = proj + (size_t)t0 * ldp;
    lt_load<true, VEC>(kt, p + (size_t)(H + h) * D, ldp, n, db * 64, D);
    lt_load<true, VEC>(vt, p + 2 * (size_t)H * D + (size_t)h * E, ldp, n, eb * 64, E);
    __syncthreads();
    const float lg = log2f(decay[h]);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, lr = lane & 15, g = lane >> 4;
    // (each wave weighs the rows of its own value channels: no other wave reads them)
    for (int x = lane; x < 16 * LC; x += 64) {
        const int e = x >> 6, t = x & 63;
        if (t < n) vt[(w * 16 + e) * LS + t] *= lt_power(lg, n - 1 - t);
    }
    __syncthreads();
    float* out = sums + (((size_t)item * H + h) * E + eb * 64 + w * 16) * D + db * 64;
#pragma unroll
    for (int dt = 0; dt < 4; ++dt) {
        lt_floatx4 acc = {0.f, 0.f, 0.f, 0.f};
        lt_mma64(acc, vt + w * 16 * LS, kt + dt * 16 * LS, lr, g);
        const int d = dt * 16 + lr;
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (eb * 64 + w * 16 + g * 4 + u < E && db * 64 + d < D) out[(size_t)(g * 4 + u) * D + d] = acc[u];
    }
}

// (2) per request, head and element: the state goes through the request's chunks; each chunk's sum is replaced by the
// state before the chunk, the last state goes back.  The sums of LP chunks are asked for at once.
#define LP 8
__global__ __launch_bounds__(256) void lightning_scan_kernel(float* __restrict__ sums, const float* __restrict__ decay,
                                                             float* __restrict__ state, size_t state_row,
                                                             const int32_t* __restrict__ item_start, const int32_t* __restrict__ cu_tokens,
                                                             const int32_t* __restrict__ slots, int H, int ED) {
    const int r = blockIdx.z, h = blockIdx.y, x = blockIdx.x * 256 + threadIdx.x;
    if (x >= ED) return;
    const int first = item_start[r], last = item_start[r + 1], n = cu_tokens[r + 1] - cu_tokens[r];
    const float lg = log2f(decay[h]);
    const float full = lt_power(lg, LC);
    float* sp = state + (size_t)slots[r] * state_row + (size_t)h * ED + x;
    const size_t step = (size_t)H * ED;
    float* q = sums + (size_t)first * step + (size_t)h * ED + x;
    float S = *sp;
    for (int c = first; c < last; c += LP) {
        float v[LP];
#pragma unroll
        for (int u = 0; u < LP; ++u) v[u] = c + u < last ? q[u * step] : 0.f;
#pragma unroll
        for (int u = 0; u < LP; ++u) {
            if (c + u < last) {
                q[u * step] = S;
                const int m = min(LC, n - (c + u - first) * LC);
                S = fmaf(m == LC ? full : lt_power(lg, m), S, v[u]);
            }
        }
        q += LP * step;
    }
    *sp = S;
}

// (3) o[64 tokens][64 value channels] of a chunk; a wave sixteen tokens.
template <bool VEC>
__global__ __launch_bounds__(256) void lightning_outputs_kernel(const float* __restrict__ proj, size_t ldp, const float* __restrict__ decay,
                                                                const int32_t* __restrict__ items, const int32_t* __restrict__ cu_tokens,
                                                                const float* __restrict__ sums, float* __restrict__ o, int H, int D, int E) {
    __shared__ __attribute__((aligned(16))) float qs[LC * LS], ks[LC * LS], ss[LC * LS];
    const int item = blockIdx.x, h = blockIdx.y, eb = blockIdx.z;
    const int r = items[2 * item], i0 = items[2 * item + 1];
    const int t0 = cu_tokens[r] + i0, n = min(LC, cu_tokens[r + 1] - t0);
    const float* p = proj + (size_t)t0 * ldp;
    const float* before = sums + (((size_t)item * H + h) * E + eb * 64) * D;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, lr = lane & 15, g = lane >> 4;
    lt_floatx4 pa[4], oa[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) pa[u] = oa[u] = lt_floatx4{0.f, 0.f, 0.f, 0.f};
    for (int d0 = 0; d0 < D; d0 += 64) {
        if (d0) __syncthreads();
        lt_load<false, VEC>(qs, p + (size_t)h * D, ldp, n, d0, D);
        lt_load<false, VEC>(ks, p + (size_t)(H + h) * D, ldp, n, d0, D);
        for (int x = threadIdx.x; x < 64 * 64; x += 256) {
            const int e = x >> 6, d = x & 63;
            ss[e * LS + d] = (eb * 64 + e < E && d0 + d < D) ? before[(size_t)e * D + d0 + d] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            if (u <= w) lt_mma64(pa[u], qs + w * 16 * LS, ks + u * 16 * LS, lr, g);      // (tokens of later tiles are not seen)
            lt_mma64(oa[u], qs + w * 16 * LS, ss + u * 16 * LS, lr, g);
        }
    }
    __syncthreads();            // the tiles are read: qs takes the weighed scores, ks the values
    lt_load<true, VEC>(ks, p + 2 * (size_t)H * D + (size_t)h * E, ldp, n, eb * 64, E);
    const float lg = log2f(decay[h]);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int i = w * 16 + g * 4 + u;               // this lane's token of result row u
        const float f = lt_power(lg, i + 1);
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            oa[t][u] *= f;
            const int j = t * 16 + lr;
            qs[i * LS + j] = j <= i ? pa[t][u] * lt_power(lg, i - j) : 0.f;
        }
    }
    __syncthreads();
    float* out = o + (size_t)t0 * H * E + (size_t)h * E + eb * 64;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        lt_mma64(oa[t], qs + w * 16 * LS, ks + t * 16 * LS, lr, g);
        const int e = t * 16 + lr;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int i = w * 16 + g * 4 + u;
            if (i < n && eb * 64 + e < E) out[(size_t)i * H * E + e] = oa[t][u];
        }
    }
}

TFF_API int tff_lightning_chunk(void) { return LC; }

TFF_API int tff_lightning_chunks(const float* proj, size_t ldp, const float* decay, float* state, size_t state_row,
                                 const int32_t* items, const int32_t* item_start, int num_items, const int32_t* cu_tokens,
                                 const int32_t* state_slots, float* sums, float* o, int R, int H, int D, int E, tff_stream_t stream) {
    TFF_REQUIRE(proj && decay && state && items && item_start && cu_tokens && state_slots && sums && o, "lightning_chunks: null pointer");
    TFF_REQUIRE(R >= 0 && num_items >= 0 && H > 0 && D > 0 && E > 0, "lightning_chunks: bad sizes heads=%d dim=%d vdim=%d", H, D, E);
    TFF_REQUIRE(ldp >= 2 * (size_t)H * D + (size_t)H * E && (size_t)H * E * D <= state_row,
                "lightning_chunks: rows of %zu or state rows of %zu are too short", ldp, state_row);
    const int d_blocks = (D + 63) / 64, e_blocks = (E + 63) / 64;
    TFF_REQUIRE(H <= 65535 && R <= 65535 && (long)d_blocks * e_blocks <= 65535, "lightning_chunks: too many heads, requests or channels");
    if (R == 0 || num_items == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const bool vec = D % 4 == 0 && E % 4 == 0 && ldp % 4 == 0 && ((uintptr_t)proj % 16) == 0;
    const dim3 g1(num_items, H, d_blocks * e_blocks), g2((E * D + 255) / 256, H, R), g3(num_items, H, e_blocks);
    if (vec) lightning_sums_kernel<true><<<g1, 256, 0, s>>>(proj, ldp, decay, items, cu_tokens, sums, H, D, E, d_blocks);
    else lightning_sums_kernel<false><<<g1, 256, 0, s>>>(proj, ldp, decay, items, cu_tokens, sums, H, D, E, d_blocks);
    if (int rc = tff_check_launch("lightning_sums")) return rc;
    lightning_scan_kernel<<<g2, 256, 0, s>>>(sums, decay, state, state_row, item_start, cu_tokens, state_slots, H, E * D);
    if (int rc = tff_check_launch("lightning_scan")) return rc;
    if (vec) lightning_outputs_kernel<true><<<g3, 256, 0, s>>>(proj, ldp, decay, items, cu_tokens, sums, o, H, D, E);
    else lightning_outputs_kernel<false><<<g3, 256, 0, s>>>(proj, ldp, decay, items, cu_tokens, sums, o, H, D, E);
    return tff_check_launch("lightning_outputs");
}

// One block a row.
template <typename TO, int NT>
__global__ __launch_bounds__(NT) void row_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ g, size_t g_row,
                                                           const float* __restrict__ w, float eps, TO* __restrict__ out, int N) {
    __shared__ float red[NT / 64];
    const size_t t = blockIdx.x;
    const float* orow = o + t * N;
    const float* grow = g + t * g_row;
    float ss = 0.f;
    for (int e = threadIdx.x; e < N; e += NT) ss = fmaf(orow[e], orow[e], ss);
    ss = rows_sum(row16_sum(ss));
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NT / 64; ++i) ss += red[i];
    const float rr = 1.0f / sqrtf(ss / (float)N + eps);
    for (int e = threadIdx.x; e < N; e += NT)
        out[t * N + e] = from_f32<TO>(orow[e] * rr * w[e] * (1.0f / (1.0f + expf(-grow[e]))));
}

TFF_API int tff_row_norm_gate(const float* o, const float* g, size_t g_row, const float* w, float eps, void* out, int T, int N,
                              int out_dtype, tff_stream_t stream) {
    TFF_REQUIRE(o && g && w && out, "row_norm_gate: null pointer");
    TFF_REQUIRE(T >= 0 && N > 0 && g_row >= (size_t)N, "row_norm_gate: bad sizes");
    if (T == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const bool few = T <= 256 && N > 1024;
#define RG_LAUNCH(TO)                                                                                         \
    do {                                                                                                      \
        if (few) row_norm_gate_kernel<TO, 1024><<<T, 1024, 0, s>>>(o, g, g_row, w, eps, (TO*)out, N);         \
        else row_norm_gate_kernel<TO, 256><<<T, 256, 0, s>>>(o, g, g_row, w, eps, (TO*)out, N);               \
    } while (0)
    if (out_dtype == TFF_F32) RG_LAUNCH(float);
    else if (out_dtype == TFF_BF16) RG_LAUNCH(bf16_t);
    else return tff_fail("row_norm_gate: unknown dtype %d", out_dtype);
#undef RG_LAUNCH
    return tff_check_launch("row_norm_gate");
}
