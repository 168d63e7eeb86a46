// A linear recurrence with a fixed decay per head: per request and head a matrix S [key channel, value channel],
//   S <- decay S + k_t v_t^T,   o_t = S^T q_t,      q, k, v = silu of their projections, all float32.
// A request's state row: [heads][value channel][key channel] (S transposed: the key channels of one value channel
// lie side by side, as the lanes that share the channel read them).
//
// tff_lightning:      the recurrence over each request's tokens of the step.
// tff_row_norm_gate:  out = o / sqrt(mean over the row of o^2 + eps) * w * sigmoid(gate).
#include "common.h"
#include "tffinfer_kernels.h"

__device__ __forceinline__ float lt_silu(float z) { return z / (1.0f + expf(-z)); }

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
    float S[KPL];
#pragma unroll
    for (int m = 0; m < KPL; ++m) S[m] = (live && s + 16 * m < D) ? sp[16 * m] : 0.f;
    for (int t = 0; t < n; ++t) {
        const float* p = proj + (size_t)(t0 + t) * ldp;
        const float* pq = p + (size_t)h * D + s;
        const float* pk = pq + (size_t)H * D;
        float kk[KPL], qq[KPL];
#pragma unroll
        for (int m = 0; m < KPL; ++m) {
            const bool in = s + 16 * m < D;
            qq[m] = in ? lt_silu(pq[16 * m]) : 0.f;
            kk[m] = in ? lt_silu(pk[16 * m]) : 0.f;
        }
        const float v = lt_silu(p[2 * (size_t)H * D + (size_t)h * E + jc]);
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
                          int max_tokens, tff_stream_t stream) {
    TFF_REQUIRE(proj && decay && state && cu_tokens && state_slots && o, "lightning: null pointer");
    TFF_REQUIRE(R >= 0 && H > 0 && D > 0 && D <= 256 && E > 0, "lightning: bad sizes heads=%d dim=%d vdim=%d (dim up to 256)", H, D, E);
    TFF_REQUIRE(ldp >= 2 * (size_t)H * D + (size_t)H * E && (size_t)H * E * D <= state_row,
                "lightning: rows of %zu or state rows of %zu are too short", ldp, state_row);
    TFF_REQUIRE(H <= 65535 && R <= 65535, "lightning: too many heads or requests");
    (void)max_tokens;
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
