// Two linear recurrences over a matrix S [key channel, value channel] per request and head, all float32:
//
//   TFF_LR_DECAY  (a decay per key channel):   S <- diag(alpha_t) S + k_t v_t^T,   o_t = S^T q_t
//                 alpha = sigmoid(z)^(1/tau),  z = A2 (A1 x) + bias
//   TFF_LR_EXP    (exponential gates per head): with log gates i and f, a running maximum m (zero at the start)
//                 m_t = max(f + m_(t-1), i),  S <- exp(f + m_(t-1) - m_t) S + exp(i - m_t) k_t v_t^T,  n likewise with k_t,
//                 o_t = S^T q_t / (max(|n . q_t|, exp(-m_t)) + den_eps)
//                 i = cap tanh((zi + bi) / cap),  f = logsigmoid(cap tanh((zf + bf) / cap))
//
// then per head  y = o / sqrt(mean o^2 + eps) * w * gate(g),  gate = silu or sigmoid.
//
// A request's state row: [heads][value channel][key channel] (S transposed: the key channels of one value channel lie
// side by side); with exponential gates n is one more value channel (whose v is 1), behind a head's others, and
// the heads' m follow all matrices.
//
// tff_recurrence_few:    for steps of a few tokens a request: one block per request and head does everything from the
//                        projections to y.
// tff_recurrence_chunks: for longer portions, in chunks of 64 tokens.  With S the state before a chunk and c_i the sum of the
//                        log decays up to token i of it,
//                          o_i = S^T (q_i e^(c_i)) + sum over j <= i of (sum over d of q_id k_jd e^(c_id - c_jd)) v_j,
//                          S  <- e^(c_n) S + sum over j of (k_j e^(c_n - c_j)) v_j^T
//                        (exponential gates: c is one number per head, and the terms carry e^(i_j - m)).  No factor is larger than
//                        1: differences are taken before exponentials, for a channel-wise decay relative to the start of
//                        the row's sixteen tokens, within the sixteen pair by pair.  Every chunk's own sum (1), a scan over a request's chunks
//                        that leaves the state before each one in its place (2), all outputs (3).  Products on the
//                        matrix cores in float32.
#include "common.h"
#include "tffinfer_kernels.h"

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float lr_floatx4;

__device__ __forceinline__ float lr_logsigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float lr_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float lr_gate(float z, int sigmoid) {
    const float s = 1.0f / (1.0f + expf(-z));
    return sigmoid ? s : z * s;
}
#define LR_LOG2E 1.44269504088896340736f

// -------------------------------------------------------------- a few tokens ---
// Block: one head of one request, its threads in rows of sixteen lanes; a row shares a value channel, lane s holding
// the key channels 64 m + 4 s .. + 3.  Up to `tm` tokens pass at a time: their q, k, v, gates and decays go to LDS,
// every row takes its value channels through all of them with S in registers, then a wave per token norms and gates.
template <int KIND, int M, int IT, bool VEC, typename TO>
__global__ __launch_bounds__(1024) void lr_few_kernel(const TffRecurrence a, int tm) {
    extern __shared__ __attribute__((aligned(16))) float lr_lds[];
    constexpr bool EXPG = KIND == TFF_LR_EXP;
    constexpr int DP = 64 * M, KPL = 4 * M, NS = EXPG ? IT + 1 : IT;      // (the last place of the first row is for n)
    const int D = a.D, E = a.E, E1 = EXPG ? E + 1 : E;
    float* const lq = lr_lds;
    float* const lk = lq + tm * DP;
    float* const la = lk + tm * DP;                        // decays (channel-wise), or nothing
    float* const lv = la + (EXPG ? 0 : tm * DP);
    float* const lg = lv + tm * E;                         // the norm's weight times the gate
    float* const lo = lg + tm * E;
    float* const lc = lo + tm * E1;                        // exponential gates: keep, put, exp(-m) of a token
    const int h = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, nt = blockDim.x;
    const int row = tid >> 4, s = tid & 15, rows = nt >> 4, lane = tid & 63, wave = tid >> 6;
    const int t0 = a.cu_tokens[r], n = a.cu_tokens[r + 1] - t0;
    if (n <= 0) return;                                    // (the whole block)
    float* const srow = a.state + (size_t)a.state_slots[r] * a.state_row;
    float* const S0 = srow + (size_t)h * E1 * D;
    float* const mp = srow + (size_t)a.H * E1 * D + h;     // (exponential gates)
    float m_run = (EXPG && wave == 0) ? *mp : 0.f;
    float S[NS][KPL];
    // the value channel of place u of a row; E1: none
    auto channel = [&](int e0, int u) {
        if (u == IT) return e0 == 0 ? E : E1;
        const int e = e0 + u * rows;
        return e < E ? e : E1;
    };
    auto load = [&](int e0) {
#pragma unroll
        for (int u = 0; u < NS; ++u) {
            const int e = channel(e0, u);
            const float* p = S0 + (size_t)e * D;
#pragma unroll
            for (int m = 0; m < M; ++m) {
                const int d = 64 * m + 4 * s;
                if constexpr (VEC) {
                    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (e < E1 && d < D) x = *reinterpret_cast<const float4*>(p + d);
                    S[u][4 * m] = x.x; S[u][4 * m + 1] = x.y; S[u][4 * m + 2] = x.z; S[u][4 * m + 3] = x.w;
                } else {
#pragma unroll
                    for (int c = 0; c < 4; ++c) S[u][4 * m + c] = (e < E1 && d + c < D) ? p[d + c] : 0.f;
                }
            }
        }
    };
    auto store = [&](int e0) {
#pragma unroll
        for (int u = 0; u < NS; ++u) {
            const int e = channel(e0, u);
            float* p = S0 + (size_t)e * D;
#pragma unroll
            for (int m = 0; m < M; ++m) {
                const int d = 64 * m + 4 * s;
                if constexpr (VEC) {
                    if (e < E1 && d < D) *reinterpret_cast<float4*>(p + d) = make_float4(S[u][4 * m], S[u][4 * m + 1], S[u][4 * m + 2], S[u][4 * m + 3]);
                } else {
#pragma unroll
                    for (int c = 0; c < 4; ++c)
                        if (e < E1 && d + c < D) p[d + c] = S[u][4 * m + c];
                }
            }
        }
    };
    auto take = [&](float (&x)[KPL], const float* p) {
#pragma unroll
        for (int m = 0; m < M; ++m) {
            const float4 y = *reinterpret_cast<const float4*>(p + 64 * m + 4 * s);
            x[4 * m] = y.x; x[4 * m + 1] = y.y; x[4 * m + 2] = y.z; x[4 * m + 3] = y.w;
        }
    };
    for (int p0 = 0; p0 < n; p0 += tm) {
        const int cnt = min(tm, n - p0);
        const size_t tp = (size_t)(t0 + p0);
        load(row);                                         // (asked for before anything waits)
        if (p0) __syncthreads();                           // the tokens before are read
        for (int x = tid; x < cnt * DP; x += nt) {
            const int tk = x / DP, d = x - tk * DP;
            const size_t c = (size_t)h * D + d, at = (tp + tk) * a.ld + c;
            const bool in = d < D;
            lq[x] = in ? a.q[at] * a.q_scale : 0.f;
            lk[x] = in ? a.k[at] : 0.f;
            if constexpr (!EXPG) {
                float al = 0.f;
                if (in) {
                    float z = a.a_bias[c];
                    const float* a1 = a.a1 + (tp + tk) * a.ld;
                    const float* a2 = a.a2 + c;
                    const size_t step = (size_t)a.H * D;
                    int i = 0;
                    for (; i + 16 <= a.rank; i += 16) {      // (sixteen loads in flight)
                        float x[16], y[16];
#pragma unroll
                        for (int j = 0; j < 16; ++j) { x[j] = a2[(i + j) * step]; y[j] = a1[i + j]; }
#pragma unroll
                        for (int j = 0; j < 16; ++j) z = fmaf(x[j], y[j], z);
                    }
                    for (; i < a.rank; ++i) z = fmaf(a2[i * step], a1[i], z);
                    al = expf(lr_logsigmoid(z) * a.inv_tau);
                }
                la[x] = al;
            }
        }
        for (int x = tid; x < cnt * E; x += nt) {
            const int tk = x / E, e = x - tk * E;
            const size_t at = (tp + tk) * a.ld + (size_t)h * E + e;
            lv[x] = a.v[at];
            lg[x] = lr_gate(a.gate[at], a.sigmoid_gate) * a.w[(a.w_per_head ? (size_t)h * E : 0) + e];
        }
        if constexpr (EXPG) {
            if (wave == 0) {
                float li = 0.f, lf = 0.f, keep = 0.f, put = 0.f, fl = 0.f;
                if (lane < cnt) {
                    const size_t at = (tp + lane) * a.ld + h;
                    li = a.cap * tanhf((a.ig[at] + a.i_bias[h]) / a.cap);
                    lf = lr_logsigmoid(a.cap * tanhf((a.fg[at] + a.f_bias[h]) / a.cap));
                }
                for (int j = 0; j < cnt; ++j) {
                    const float fj = __shfl(lf, j, 64), ij = __shfl(li, j, 64);
                    const float mn = fmaxf(fj + m_run, ij);
                    if (lane == j) { keep = expf(fj + m_run - mn); put = expf(ij - mn); fl = expf(-mn); }
                    m_run = mn;
                }
                if (lane < cnt) { lc[3 * lane] = keep; lc[3 * lane + 1] = put; lc[3 * lane + 2] = fl; }
            }
        }
        __syncthreads();
        for (int e0 = row, base = 0; base < E; base += rows * IT, e0 += rows * IT) {
            if (base) load(e0);
            for (int tk = 0; tk < cnt; ++tk) {
                float kk[KPL], qq[KPL], al[EXPG ? 1 : KPL];
                take(kk, lk + tk * DP);
                take(qq, lq + tk * DP);
                if constexpr (!EXPG) take(al, la + tk * DP);
                const float keep = EXPG ? lc[3 * tk] : 0.f, put = EXPG ? lc[3 * tk + 1] : 1.f;
#pragma unroll
                for (int u = 0; u < NS; ++u) {
                    if (u == IT && e0 != 0) break;
                    const int e = channel(e0, u);
                    const float v = e < E ? lv[tk * E + e] * put : put;
                    float acc = 0.f;
#pragma unroll
                    for (int m = 0; m < KPL; ++m) {
                        S[u][m] = fmaf(kk[m], v, (EXPG ? keep : al[EXPG ? 0 : m]) * S[u][m]);
                        acc = fmaf(S[u][m], qq[m], acc);
                    }
                    acc = row16_sum(acc);
                    if (s == 0 && e < E1) lo[tk * E1 + e] = acc;
                }
            }
            store(e0);
        }
        __syncthreads();
        for (int tk = wave; tk < cnt; tk += nt >> 6) {
            const float* x = lo + tk * E1;
            const float den = EXPG ? fmaxf(fabsf(x[EXPG ? E : 0]), lc[3 * tk + 2]) + a.den_eps : 1.0f;
            float ss = 0.f;
            for (int e = lane; e < E; e += 64) {
                const float o = EXPG ? x[e] / den : x[e];
                ss = fmaf(o, o, ss);
            }
            ss = rows_sum(row16_sum(ss));
            const float rr = a.out_scale / sqrtf(ss / (float)E + a.eps);
            TO* out = reinterpret_cast<TO*>(a.out) + (tp + tk) * a.out_row + (size_t)h * E;
            for (int e = lane; e < E; e += 64) {
                const float o = EXPG ? x[e] / den : x[e];
                out[e] = from_f32<TO>(o * rr * lg[tk * E + e]);
            }
        }
    }
    if (EXPG && tid == 0) *mp = m_run;
}

static int lr_check(const TffRecurrence* a, const char* what) {
    TFF_REQUIRE(a && a->q && a->k && a->v && a->gate && a->w && a->state && a->cu_tokens && a->state_slots && a->out, "%s: null pointer", what);
    TFF_REQUIRE(a->kind == TFF_LR_DECAY || a->kind == TFF_LR_EXP, "%s: unknown recurrence %d", what, a->kind);
    TFF_REQUIRE(a->R >= 0 && a->H > 0 && a->D > 0 && a->D <= 256 && a->E > 0, "%s: bad sizes heads=%d dim=%d vdim=%d (dim up to 256)", what,
                a->H, a->D, a->E);
    const bool ex = a->kind == TFF_LR_EXP;
    const size_t need = (size_t)a->H * (a->E + (ex ? 1 : 0)) * a->D + (ex ? a->H : 0);
    TFF_REQUIRE(a->state_row >= need && a->out_row >= (size_t)a->H * a->E && a->ld >= (size_t)a->H * a->E && a->ld >= (size_t)a->H * a->D,
                "%s: rows of %zu, state rows of %zu or result rows of %zu are too short", what, a->ld, a->state_row, a->out_row);
    TFF_REQUIRE(a->H <= 65535 && a->R <= 65535, "%s: too many heads or requests", what);
    if (ex) TFF_REQUIRE(a->ig && a->fg && a->i_bias && a->f_bias && a->cap > 0.f, "%s: the gates need their columns, biases and cap", what);
    else TFF_REQUIRE(a->a1 && a->a2 && a->a_bias && a->rank > 0, "%s: the decay needs its two matrices and bias", what);
    TFF_REQUIRE(a->out_dtype == TFF_F32 || a->out_dtype == TFF_BF16, "%s: unknown dtype %d", what, a->out_dtype);
    return 0;
}

#define LR_FEW_LDS (60 * 1024)

TFF_API int tff_recurrence_few(const TffRecurrence* p, int max_tokens, tff_stream_t stream) {
    if (int rc = lr_check(p, "recurrence_few")) return rc;
    const TffRecurrence a = *p;
    if (a.R == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const bool ex = a.kind == TFF_LR_EXP;
    const int M = a.D <= 64 ? 1 : a.D <= 128 ? 2 : 4, DP = 64 * M;
    const size_t per = ((ex ? 2 : 3) * (size_t)DP + 3 * (size_t)a.E + 4) * sizeof(float);
    int tm = (int)(LR_FEW_LDS / per);
    TFF_REQUIRE(tm >= 1, "recurrence_few: heads of %d and %d channels do not fit LDS", a.D, a.E);
    if (max_tokens > 0 && tm > max_tokens) tm = max_tokens;
    if (tm > 16) tm = 16;
    const size_t lds = (per * tm + 15) & ~(size_t)15;
    const int nt = a.E <= 16 ? 256 : a.E <= 32 ? 512 : 1024;
    const bool vec = a.D % 4 == 0 && a.state_row % 4 == 0 && ((uintptr_t)a.state % 16) == 0;
    const dim3 grid(a.H, a.R);
#define LR_GO(K, MM, V, TO) lr_few_kernel<K, MM, 2, V, TO><<<grid, nt, lds, s>>>(a, tm)
#define LR_M(K, V, TO) do { if (M == 1) LR_GO(K, 1, V, TO); else if (M == 2) LR_GO(K, 2, V, TO); else LR_GO(K, 4, V, TO); } while (0)
#define LR_V(K, TO) do { if (vec) LR_M(K, true, TO); else LR_M(K, false, TO); } while (0)
    if (ex && a.out_dtype == TFF_BF16) LR_V(TFF_LR_EXP, bf16_t);
    else if (ex) LR_V(TFF_LR_EXP, float);
    else if (a.out_dtype == TFF_BF16) LR_V(TFF_LR_DECAY, bf16_t);
    else LR_V(TFF_LR_DECAY, float);
#undef LR_V
#undef LR_M
#undef LR_GO
    return tff_check_launch("recurrence_few");
}

// ------------------------------------------------------------------- chunks ---
// Items (row of the step's tables, first place in the request's portion) of up to LRC tokens.  A 16 x 16 x 4 product of
// the matrix cores takes element [r][k = g] of either operand from lane (r = lane & 15, g = lane >> 4); its result: lane
// (r, g) holds rows 4 g .. 4 g + 3 (of the first operand) of column r (of the second).
#define LRC 64
#define LRS 68       // floats between rows whose lanes read four neighbours (the inner index runs along the row)
#define LRV 80       // floats between rows whose lanes read one column each (the inner index runs down the rows)
#define LR_FUSED_E 256   // value channels up to which the outputs' kernel also norms and gates
#define LRR 32       // inner size of the decay's second product that is worked through at a time

// -log1p(e^(-|z|)) + min(z, 0) with the hardware's exponential and logarithm: log u for u = 1 + e is off by the rounding of
// the sum, which the factor e / (u - 1) takes out again (D. Goldberg, "What Every Computer Scientist Should Know About
// Floating-Point Arithmetic", theorem 4).
__device__ __forceinline__ float lr_logsigmoid_fast(float z) {
    const float e = __expf(-fabsf(z)), u = 1.0f + e, d = u - 1.0f;
    return fminf(z, 0.f) - (d == 0.f ? e : __logf(u) * (e * __builtin_amdgcn_rcpf(d)));
}

// (0a) channel-wise decay: cum[t][h D + d] = the sum of log2 alpha from the chunk's first token to t.  A wave takes sixteen
// of the chunk's tokens, its lanes 64 channels; the waves' sums meet in LDS.
__global__ __launch_bounds__(256) void lr_decay_kernel(const TffRecurrence a, const int32_t* __restrict__ items, float* __restrict__ cum) {
    __shared__ __attribute__((aligned(16))) float a1s[LRR * LRS];
    __shared__ float tot[4][64];
    const int r = items[2 * blockIdx.x], i0 = items[2 * blockIdx.x + 1];
    const int t0 = a.cu_tokens[r] + i0, n = min(LRC, a.cu_tokens[r + 1] - t0);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int HD = a.H * a.D, c = blockIdx.y * 64 + lane, cc = min(c, HD - 1);
    float z[16];
    const float b = a.a_bias[cc];
#pragma unroll
    for (int t = 0; t < 16; ++t) z[t] = b;
    for (int r0 = 0; r0 < a.rank; r0 += LRR) {
        if (r0) __syncthreads();
        const int nr = min(LRR, a.rank - r0);
        for (int x = threadIdx.x; x < LRR * LRC; x += 256) {
            const int t = x / LRR, i = x % LRR;
            a1s[i * LRS + t] = (t < n && i < nr) ? a.a1[(size_t)(t0 + t) * a.ld + r0 + i] : 0.f;
        }
        __syncthreads();
#pragma unroll 4
        for (int i = 0; i < nr; ++i) {
            const float q = a.a2[(size_t)(r0 + i) * HD + cc];
#pragma unroll
            for (int t = 0; t < 16; t += 4) {
                const float4 x = *reinterpret_cast<const float4*>(a1s + i * LRS + w * 16 + t);
                z[t] = fmaf(q, x.x, z[t]);
                z[t + 1] = fmaf(q, x.y, z[t + 1]);
                z[t + 2] = fmaf(q, x.z, z[t + 2]);
                z[t + 3] = fmaf(q, x.w, z[t + 3]);
            }
        }
    }
    const float f = a.inv_tau * LR_LOG2E;
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        sum = fmaf(lr_logsigmoid_fast(z[t]), f, sum);
        z[t] = sum;
    }
    tot[w][lane] = sum;
    __syncthreads();
    sum = 0.f;
    for (int j = 0; j < w; ++j) sum += tot[j][lane];
    float* out = cum + (size_t)(t0 + w * 16) * HD + c;
#pragma unroll
    for (int t = 0; t < 16; ++t)
        if (w * 16 + t < n && c < HD) out[(size_t)t * HD] = sum + z[t];
}

// (0b) exponential gates, per request and head, sixteen chunks at a time (a wave each).  With b the sums of f within a
// chunk, w_j = i_j - b_j, m' the maximum before the chunk and x_i = max(m', w_0 .. w_i):  m_i = b_i + x_i, a chunk's
// state decays by e^(m' - x_i) up to token i and token j's term counts e^(w_j - x_i).
//   w, x, fl: [T][H] (fl = e^(-m_i));  before, last: [items][H] = m', x of the chunk's last token.
__global__ __launch_bounds__(1024) void lr_gates_kernel(const TffRecurrence a, const int32_t* __restrict__ item_start, float* __restrict__ w,
                                                        float* __restrict__ x, float* __restrict__ fl, float* __restrict__ before,
                                                        float* __restrict__ last) {
    __shared__ float tot[16][2];
    const int h = blockIdx.x, r = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int first = item_start[r], count = item_start[r + 1] - first;
    const int t0 = a.cu_tokens[r], n = a.cu_tokens[r + 1] - t0;
    if (n <= 0) return;                      // (the whole block)
    float* const mp = a.state + (size_t)a.state_slots[r] * a.state_row + (size_t)a.H * (a.E + 1) * a.D + h;
    float m = *mp;
    const float ib = a.i_bias[h], fb = a.f_bias[h];
    for (int c0 = 0; c0 < count; c0 += 16) {
        const int c = c0 + wave, t = c * LRC + lane;
        float li = -INFINITY, lf = 0.f;
        if (t < n) {
            const size_t at = (size_t)(t0 + t) * a.ld + h;
            li = a.cap * tanhf((a.ig[at] + ib) / a.cap);
            lf = lr_logsigmoid(a.cap * tanhf((a.fg[at] + fb) / a.cap));
        }
        float b = lf;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float y = __shfl_up(b, o, 64);
            if (lane >= o) b += y;
        }
        const float wj = li - b;
        float px = wj;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float y = __shfl_up(px, o, 64);
            if (lane >= o) px = fmaxf(px, y);
        }
        if (c0) __syncthreads();
        if (lane == 63) { tot[wave][0] = b; tot[wave][1] = px; }
        __syncthreads();
        float mine = m;
        for (int j = 0; j < 16; ++j) {
            if (j == wave) mine = m;
            if (c0 + j < count) m = tot[j][0] + fmaxf(m, tot[j][1]);
        }
        if (t < n) {
            const size_t at = (size_t)(t0 + t) * a.H + h;
            const float xi = fmaxf(mine, px);
            w[at] = wj;
            x[at] = xi;
            fl[at] = expf(-(b + xi));
            if (lane == 0) before[(size_t)(first + c) * a.H + h] = mine;
            if (lane == LRC - 1 || t == n - 1) last[(size_t)(first + c) * a.H + h] = xi;
        }
    }
    if (threadIdx.x == 0) *mp = m;
}

// Columns c0 .. c0 + 63 of 64 rows (ld apart) into LDS rows of LS floats, each element through f(value, row, column from
// c0); rows past n repeat the last one where `repeat`, else they and columns past `cols` are zeros.
template <bool VEC, int LS, typename F>
__device__ __forceinline__ void lr_load(float* dst, const float* __restrict__ src, size_t ld, int n, int c0, int cols, bool repeat, F f) {
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int x = i * 256 + threadIdx.x, t = x >> 4, c = (x & 15) * 4;
            const int ts = repeat ? min(t, n - 1) : t;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (ts < n && c0 + c < cols) {
                v = *reinterpret_cast<const float4*>(src + (size_t)ts * ld + c0 + c);
                v = f(v, t, c);
            }
            *reinterpret_cast<float4*>(dst + t * LS + c) = v;
        }
    } else {
        for (int x = threadIdx.x; x < LRC * 16; x += 256) {
            const int t = x >> 4, c = (x & 15) * 4;
            const int ts = repeat ? min(t, n - 1) : t;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (ts < n) {
                const float* p = src + (size_t)ts * ld + c0 + c;
                if (c0 + c < cols) v.x = p[0];
                if (c0 + c + 1 < cols) v.y = p[1];
                if (c0 + c + 2 < cols) v.z = p[2];
                if (c0 + c + 3 < cols) v.w = p[3];
                v = f(v, t, c);
            }
            *reinterpret_cast<float4*>(dst + t * LS + c) = v;
        }
    }
}

// acc += A[16 rows][64] . B[16 rows][64]^T, both along the rows in LDS; a in registers (four runs of four), b by address
__device__ __forceinline__ void lr_mma64(lr_floatx4& acc, const float4 (&x)[4], const float4 (&y)[4]) {
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[kb].x, y[kb].x, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[kb].y, y[kb].y, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[kb].z, y[kb].z, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[kb].w, y[kb].w, acc, 0, 0, 0);
    }
}
__device__ __forceinline__ void lr_rows(float4 (&x)[4], const float* p, int r, int g) {
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) x[kb] = *reinterpret_cast<const float4*>(p + r * LRS + kb * 16 + g * 4);
}
__device__ __forceinline__ float4 lr_mul(const float4& a, const float4& b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }
__device__ __forceinline__ float4 lr_exp2_diff(const float4& a, const float4& b) {
    return make_float4(lr_exp2(a.x - b.x), lr_exp2(a.y - b.y), lr_exp2(a.z - b.z), lr_exp2(a.w - b.w));
}

struct LrWork {
    const int32_t *items, *item_start;
    const float* cum;                            // channel-wise decay
    const float *w, *x, *fl, *before, *last;     // exponential gates
    float* sums;                                 // [items][H][E1][D]
    float* o;                                    // [T][H E], where the outputs' norm is left to another kernel
};

// (1) sums[item][h][e][d] = sum over the chunk's tokens of (k_j[d] times its decay to the chunk's end) v_j[e]: blocks of 64 value
// channels x 64 key channels, a wave sixteen value channels.
template <int KIND, bool VEC>
__global__ __launch_bounds__(256) void lr_sums_kernel(const TffRecurrence a, const LrWork k, int d_blocks) {
    constexpr bool EXPG = KIND == TFF_LR_EXP;
    __shared__ __attribute__((aligned(16))) float ks[LRC * LRV], vs[LRC * LRV];
    __shared__ float wt[LRC];
    const int item = blockIdx.x, h = blockIdx.y, eb = blockIdx.z / d_blocks, db = blockIdx.z - eb * d_blocks;
    const int r = k.items[2 * item], i0 = k.items[2 * item + 1];
    const int t0 = a.cu_tokens[r] + i0, n = min(LRC, a.cu_tokens[r + 1] - t0);
    const int D = a.D, E = a.E, E1 = EXPG ? E + 1 : E;
    if constexpr (EXPG) {
        if (threadIdx.x < LRC) {
            const int t = threadIdx.x;
            wt[t] = t < n ? __expf(k.w[(size_t)(t0 + t) * a.H + h] - k.last[(size_t)item * a.H + h]) : 0.f;
        }
        __syncthreads();
    }
    auto same = [](const float4& v, int, int) { return v; };
    const float* kp = a.k + (size_t)t0 * a.ld + (size_t)h * D;
    const float* vp = a.v + (size_t)t0 * a.ld + (size_t)h * E;
    if constexpr (EXPG) {
        lr_load<VEC, LRV>(ks, kp, a.ld, n, db * 64, D, false, same);
        lr_load<VEC, LRV>(vs, vp, a.ld, n, eb * 64, E, false, [&](const float4& v, int t, int) {
            const float f = wt[t];
            return make_float4(v.x * f, v.y * f, v.z * f, v.w * f);
        });
    } else {
        const size_t HD = (size_t)a.H * D;
        const float* cp = k.cum + (size_t)t0 * HD + (size_t)h * D + db * 64;
        const float* cl = cp + (size_t)(n - 1) * HD;
        const int left = D - db * 64;
        lr_load<VEC, LRV>(ks, kp, a.ld, n, db * 64, D, false, [&](const float4& v, int t, int c) {
            const float* p = cp + (size_t)t * HD;
            float4 x, y;
            if constexpr (VEC) {
                x = *reinterpret_cast<const float4*>(cl + c);
                y = *reinterpret_cast<const float4*>(p + c);
            } else {
                const int c1 = min(c + 1, left - 1), c2 = min(c + 2, left - 1), c3 = min(c + 3, left - 1);
                c = min(c, left - 1);
                x = make_float4(cl[c], cl[c1], cl[c2], cl[c3]);
                y = make_float4(p[c], p[c1], p[c2], p[c3]);
            }
            return lr_mul(v, lr_exp2_diff(x, y));
        });
        lr_load<VEC, LRV>(vs, vp, a.ld, n, eb * 64, E, false, same);
    }
    __syncthreads();
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, lr = lane & 15, g = lane >> 4;
    float av[16];
#pragma unroll
    for (int q = 0; q < 16; ++q) av[q] = vs[(4 * q + g) * LRV + w * 16 + lr];
    float* out = k.sums + (((size_t)item * a.H + h) * E1 + eb * 64 + w * 16) * D + db * 64;
#pragma unroll
    for (int dt = 0; dt < 4; ++dt) {
        lr_floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int q = 0; q < 16; ++q) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(av[q], ks[(4 * q + g) * LRV + dt * 16 + lr], acc, 0, 0, 0);
        const int d = dt * 16 + lr;
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (eb * 64 + w * 16 + g * 4 + u < E && db * 64 + d < D) out[(size_t)(g * 4 + u) * D + d] = acc[u];
    }
    if constexpr (EXPG) {
        if (eb == 0 && threadIdx.x < 64 && db * 64 + (int)threadIdx.x < D) {       // n: the value channel whose v is 1
            float acc = 0.f;
            for (int t = 0; t < n; ++t) acc = fmaf(wt[t], ks[t * LRV + threadIdx.x], acc);
            k.sums[(((size_t)item * a.H + h) * E1 + E) * D + db * 64 + threadIdx.x] = acc;
        }
    }
}

// (2) per request, head and element: the state goes through the request's chunks; each chunk's sum is replaced by the
// state before the chunk, the last state goes back.  The sums of LRP chunks are asked for at once.
#define LRP 8
template <int KIND>
__global__ __launch_bounds__(256) void lr_scan_kernel(const TffRecurrence a, const LrWork k) {
    constexpr bool EXPG = KIND == TFF_LR_EXP;
    const int ED = (EXPG ? a.E + 1 : a.E) * a.D;
    const int r = blockIdx.z, h = blockIdx.y, x = blockIdx.x * 256 + threadIdx.x;
    if (x >= ED) return;
    const int first = k.item_start[r], last = k.item_start[r + 1], t0 = a.cu_tokens[r], n = a.cu_tokens[r + 1] - t0;
    float* sp = a.state + (size_t)a.state_slots[r] * a.state_row + (size_t)h * ED + x;
    const size_t step = (size_t)a.H * ED;
    float* q = k.sums + (size_t)first * step + (size_t)h * ED + x;
    const size_t HD = (size_t)a.H * a.D;
    const float* cum = EXPG ? nullptr : k.cum + (size_t)h * a.D + x % a.D;
    float S = *sp;
    for (int c = first; c < last; c += LRP) {
        float v[LRP], f[LRP];
#pragma unroll
        for (int u = 0; u < LRP; ++u) {
            v[u] = f[u] = 0.f;
            if (c + u < last) {
                v[u] = q[u * step];
                if constexpr (EXPG) f[u] = k.before[(size_t)(c + u) * a.H + h] - k.last[(size_t)(c + u) * a.H + h];
                else f[u] = cum[(size_t)(t0 + min(n, (c + u - first + 1) * LRC) - 1) * HD];
            }
        }
#pragma unroll
        for (int u = 0; u < LRP; ++u) {
            if (c + u < last) {
                q[u * step] = S;
                S = fmaf(EXPG ? __expf(f[u]) : lr_exp2(f[u]), S, v[u]);
            }
        }
        q += LRP * step;
    }
    *sp = S;
}

// (3) the outputs of a chunk's 64 tokens, EB blocks of 64 value channels; a wave sixteen tokens.  FUSED: all of the head's
// value channels are in the block, and norm, weight and gate are applied here; else o goes out as it is.
template <int KIND, int EB, bool VEC, typename TO, bool FUSED>
__global__ __launch_bounds__(256) void lr_outputs_kernel(const TffRecurrence a, const LrWork k) {
    constexpr bool EXPG = KIND == TFF_LR_EXP;
    constexpr int TILE = LRC * LRS;
    __shared__ __attribute__((aligned(16))) float lds[(EXPG ? 3 : 4) * TILE];
    __shared__ float ws[LRC], xs[LRC], dn[LRC];
    float* const qs = lds;                       // then the weighed scores
    float* const ss = lds + TILE;
    float* const ks = lds + 2 * TILE;
    float* const cs = lds + 3 * TILE;            // (channel-wise decay)
    float* const vs = lds + TILE;                // then the values, rows LRV apart, over ss and ks
    static_assert(LRC * LRV <= 2 * TILE, "the values fit where the state and the keys were");
    const int item = blockIdx.x, h = blockIdx.y, e_first = blockIdx.z * EB * 64;
    const int r = k.items[2 * item], i0 = k.items[2 * item + 1];
    const int t0 = a.cu_tokens[r] + i0, n = min(LRC, a.cu_tokens[r + 1] - t0);
    const int D = a.D, E = a.E, E1 = EXPG ? E + 1 : E;
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, g = lane >> 4;
    const size_t HD = (size_t)a.H * D;
    const float* qp = a.q + (size_t)t0 * a.ld + (size_t)h * D;
    const float* kp = a.k + (size_t)t0 * a.ld + (size_t)h * D;
    const float* vp = a.v + (size_t)t0 * a.ld + (size_t)h * E;
    const float* sb = k.sums + ((size_t)item * a.H + h) * E1 * D;
    const bool busy = w * 16 < n;                // (waves without tokens only help with the loads)
    const float qsc = a.q_scale;
    auto same = [](const float4& v, int, int) { return v; };
    auto scaled = [&](const float4& v, int, int) { return make_float4(v.x * qsc, v.y * qsc, v.z * qsc, v.w * qsc); };
    if constexpr (EXPG) {
        if (tid < LRC) {
            const size_t at = (size_t)(t0 + min(tid, n - 1)) * a.H + h;
            ws[tid] = k.w[at];
            xs[tid] = k.x[at];
            dn[tid] = k.fl[at];
        }
    }
    const float mb = EXPG ? k.before[(size_t)item * a.H + h] : 0.f;
    lr_floatx4 pa[4], oa[EB][4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        pa[u] = lr_floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int b = 0; b < EB; ++b) oa[b][u] = lr_floatx4{0.f, 0.f, 0.f, 0.f};
    }
    float qn = 0.f;                              // a quarter of q . n of token tid / 4
    for (int d0 = 0; d0 < D; d0 += 64) {
        if (d0) __syncthreads();
        lr_load<VEC, LRS>(qs, qp, a.ld, n, d0, D, false, scaled);
        lr_load<VEC, LRS>(ks, kp, a.ld, n, d0, D, false, same);
        if constexpr (!EXPG) lr_load<VEC, LRS>(cs, k.cum + (size_t)t0 * HD + (size_t)h * D, HD, n, d0, D, true, same);
        lr_load<VEC, LRS>(ss, sb + (size_t)e_first * D, D, min(64, E - e_first), d0, D, false, same);
        __syncthreads();
        float4 qx[4];                            // this wave's rows of q, decayed to where the state is (the chunk's start)
        if (busy) {
            lr_rows(qx, qs + w * 16 * LRS, lr, g);
            if constexpr (EXPG) {
#pragma unroll
                for (int u = 0; u < 4; ++u)
                    if (u <= w) {
                        float4 y[4];
                        lr_rows(y, ks + u * 16 * LRS, lr, g);
                        lr_mma64(pa[u], qx, y);
                    }
            } else {
                // within the sixteen tokens of the wave pair by pair (lane: token lr as key, tokens 4 g .. 4 g + 3 as queries)
                float dg[4] = {0.f, 0.f, 0.f, 0.f};
                const float* kj = ks + (w * 16 + lr) * LRS;
                const float* cj = cs + (w * 16 + lr) * LRS;
                for (int c = 0; c < min(64, D - d0); c += 4) {
                    const float4 y = *reinterpret_cast<const float4*>(kj + c), cy = *reinterpret_cast<const float4*>(cj + c);
#pragma unroll
                    for (int u = 0; u < 4; ++u) {
                        const int at = (w * 16 + g * 4 + u) * LRS + c;
                        const float4 q4 = *reinterpret_cast<const float4*>(qs + at);
                        const float4 f = lr_exp2_diff(*reinterpret_cast<const float4*>(cs + at), cy);
                        dg[u] = fmaf(q4.x * y.x, f.x, dg[u]);
                        dg[u] = fmaf(q4.y * y.y, f.y, dg[u]);
                        dg[u] = fmaf(q4.z * y.z, f.z, dg[u]);
                        dg[u] = fmaf(q4.w * y.w, f.w, dg[u]);
                    }
                }
                float4 ci[4], rf[4], qd[4];      // the sums up to the wave's tokens and to the token before its first
                lr_rows(ci, cs + w * 16 * LRS, lr, g);
#pragma unroll
                for (int kb = 0; kb < 4; ++kb) {
                    rf[kb] = w ? *reinterpret_cast<const float4*>(cs + (w * 16 - 1) * LRS + kb * 16 + g * 4) : make_float4(0.f, 0.f, 0.f, 0.f);
                    qd[kb] = lr_mul(qx[kb], lr_exp2_diff(ci[kb], rf[kb]));
                    qx[kb] = lr_mul(qx[kb], lr_exp2_diff(ci[kb], make_float4(0.f, 0.f, 0.f, 0.f)));
                }
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    if (u < w) {
                        float4 y[4], cy[4];
                        lr_rows(y, ks + u * 16 * LRS, lr, g);
                        lr_rows(cy, cs + u * 16 * LRS, lr, g);
#pragma unroll
                        for (int kb = 0; kb < 4; ++kb) y[kb] = lr_mul(y[kb], lr_exp2_diff(rf[kb], cy[kb]));
                        lr_mma64(pa[u], qd, y);
                    } else if (u == w) {
#pragma unroll
                        for (int i = 0; i < 4; ++i) pa[u][i] += (lr <= g * 4 + i) ? dg[i] : 0.f;      // (later keys are not seen)
                    }
                }
            }
        }
        if constexpr (EXPG) {
            const float* np = sb + (size_t)E * D + d0;
            const float* q4 = qs + (tid >> 2) * LRS + (tid & 3) * 16;
            for (int c = 0; c < 16; ++c) {
                const int d = (tid & 3) * 16 + c;
                if (d0 + d < D) qn = fmaf(q4[c], np[d], qn);
            }
        }
#pragma unroll
        for (int b = 0; b < EB; ++b) {
            if (b) {
                __syncthreads();
                if (e_first + b * 64 < E)
                    lr_load<VEC, LRS>(ss, sb + (size_t)(e_first + b * 64) * D, D, min(64, E - e_first - b * 64), d0, D, false, same);
                __syncthreads();
            }
            if (busy && e_first + b * 64 < E) {
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    float4 y[4];
                    lr_rows(y, ss + u * 16 * LRS, lr, g);
                    lr_mma64(oa[b][u], qx, y);
                }
            }
        }
    }
    __syncthreads();            // the tiles are read: qs takes the weighed scores, vs the values
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int i = w * 16 + g * 4 + u;               // this lane's token of result row u
        const float xi = EXPG ? xs[i] : 0.f, f = EXPG ? __expf(mb - xi) : 1.0f;
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if constexpr (EXPG) {
#pragma unroll
                for (int b = 0; b < EB; ++b) oa[b][t][u] *= f;
            }
            const int j = t * 16 + lr;
            qs[i * LRS + j] = j <= i ? (EXPG ? pa[t][u] * __expf(ws[j] - xi) : pa[t][u]) : 0.f;
        }
    }
    lr_load<VEC, LRV>(vs, vp, a.ld, n, e_first, E, false, same);
    __syncthreads();
    if constexpr (EXPG) {
        const int i = tid >> 2;
        float nq = qn * __expf(mb - xs[i]);
        const float* p = qs + i * LRS + (tid & 3) * 16;
#pragma unroll
        for (int c = 0; c < 16; ++c) nq += p[c];
        nq += __shfl_xor(nq, 1, 64);
        nq += __shfl_xor(nq, 2, 64);
        const float den = fmaxf(fabsf(nq), dn[i]) + a.den_eps;
        if ((tid & 3) == 0) dn[i] = den;         // (the four lanes of a token read it before one of them writes)
    }
    float ap[16];
    if (busy) {
#pragma unroll
        for (int q = 0; q < 16; ++q) ap[q] = q < 4 * (w + 1) ? qs[(w * 16 + lr) * LRS + 4 * q + g] : 0.f;
    }
#pragma unroll
    for (int b = 0; b < EB; ++b) {
        if (b) {
            __syncthreads();
            if (e_first + b * 64 < E) lr_load<VEC, LRV>(vs, vp, a.ld, n, e_first + b * 64, E, false, same);
            __syncthreads();
        }
        if (busy && e_first + b * 64 < E) {
#pragma unroll
            for (int t = 0; t < 4; ++t) {
#pragma unroll
                for (int q = 0; q < 16; ++q)
                    if (q < 4 * (w + 1)) oa[b][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ap[q], vs[(4 * q + g) * LRV + t * 16 + lr], oa[b][t], 0, 0, 0);
            }
        }
    }
    if constexpr (EXPG) __syncthreads();         // dn
    if (!busy) return;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int i = w * 16 + g * 4 + u;
        if constexpr (EXPG) {
            const float inv = dn[i];
#pragma unroll
            for (int b = 0; b < EB; ++b)
#pragma unroll
                for (int t = 0; t < 4; ++t) oa[b][t][u] /= inv;
        }
        if constexpr (FUSED) {
            float sq = 0.f;
#pragma unroll
            for (int b = 0; b < EB; ++b)
#pragma unroll
                for (int t = 0; t < 4; ++t) sq = fmaf(oa[b][t][u], oa[b][t][u], sq);
            sq = row16_sum(sq);
            const float rr = a.out_scale / sqrtf(sq / (float)E + a.eps);
            if (i < n) {
                const float* gp = a.gate + (size_t)(t0 + i) * a.ld + (size_t)h * E;
                const float* wp = a.w + (a.w_per_head ? (size_t)h * E : 0);
                TO* out = reinterpret_cast<TO*>(a.out) + (size_t)(t0 + i) * a.out_row + (size_t)h * E;
#pragma unroll
                for (int b = 0; b < EB; ++b)
#pragma unroll
                    for (int t = 0; t < 4; ++t) {
                        const int e = b * 64 + t * 16 + lr;
                        if (e < E) out[e] = from_f32<TO>(oa[b][t][u] * rr * wp[e] * lr_gate(gp[e], a.sigmoid_gate));
                    }
            }
        } else if (i < n) {
            float* out = k.o + ((size_t)(t0 + i) * a.H + h) * E;
#pragma unroll
            for (int b = 0; b < EB; ++b)
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const int e = e_first + b * 64 + t * 16 + lr;
                    if (e < E) out[e] = oa[b][t][u];
                }
        }
    }
}

// One wave per (token, head): y = o / sqrt(mean over the head of o^2 + eps) * w * gate(g).
template <typename TO>
__global__ __launch_bounds__(256) void lr_norm_gate_kernel(const TffRecurrence a, const float* __restrict__ o, int pairs) {
    const int id = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (id >= pairs) return;
    const int t = id / a.H, h = id % a.H, E = a.E;
    const float* x = o + ((size_t)t * a.H + h) * E;
    float ss = 0.f;
    for (int e = lane; e < E; e += 64) ss = fmaf(x[e], x[e], ss);
    ss = rows_sum(row16_sum(ss));
    const float rr = a.out_scale / sqrtf(ss / (float)E + a.eps);
    const float* gp = a.gate + (size_t)t * a.ld + (size_t)h * E;
    const float* w = a.w + (a.w_per_head ? (size_t)h * E : 0);
    TO* out = reinterpret_cast<TO*>(a.out) + (size_t)t * a.out_row + (size_t)h * E;
    for (int e = lane; e < E; e += 64) out[e] = from_f32<TO>(x[e] * rr * w[e] * lr_gate(gp[e], a.sigmoid_gate));
}

TFF_API int tff_recurrence_chunk(void) { return LRC; }

// Room for the chunks' form: sums, then the decays' sums or the gates' tables, then the outputs where their norm is apart.
TFF_API size_t tff_recurrence_workspace_bytes(int kind, int T, int items, int H, int D, int E) {
    if (T <= 0 || items <= 0 || H <= 0 || D <= 0 || E <= 0) return 0;
    const bool ex = kind == TFF_LR_EXP;
    size_t n = (size_t)items * H * (E + (ex ? 1 : 0)) * D;
    n = (n + 3) & ~(size_t)3;
    n += ex ? 3 * (size_t)T * H + 2 * (size_t)items * H : (size_t)T * H * D;
    n = (n + 3) & ~(size_t)3;
    if (E > LR_FUSED_E) n += (size_t)T * H * E;
    return n * sizeof(float);
}

TFF_API int tff_recurrence_chunks(const TffRecurrence* p, int T, const int32_t* items, const int32_t* item_start, int num_items,
                                  float* workspace, size_t workspace_bytes, tff_stream_t stream) {
    if (int rc = lr_check(p, "recurrence_chunks")) return rc;
    const TffRecurrence a = *p;
    TFF_REQUIRE(items && item_start && workspace && num_items >= 0 && T >= 0 && ((uintptr_t)workspace % 16) == 0, "recurrence_chunks: null pointer");
    if (a.R == 0 || num_items == 0 || T == 0) return 0;
    TFF_REQUIRE(workspace_bytes >= tff_recurrence_workspace_bytes(a.kind, T, num_items, a.H, a.D, a.E), "recurrence_chunks: a workspace of %zu bytes is too small", workspace_bytes);
    const bool ex = a.kind == TFF_LR_EXP;
    const int E1 = a.E + (ex ? 1 : 0), d_blocks = (a.D + 63) / 64, e_blocks = (a.E + 63) / 64;
    TFF_REQUIRE((long)d_blocks * e_blocks <= 65535 && ((long)a.H * a.D + 63) / 64 <= 65535, "recurrence_chunks: too many channels");
    hipStream_t s = (hipStream_t)stream;
    LrWork k{items, item_start, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, workspace, nullptr};
    float* q = workspace + ((((size_t)num_items * a.H * E1 * a.D) + 3) & ~(size_t)3);
    if (ex) {
        float *w = q, *x = w + (size_t)T * a.H, *fl = x + (size_t)T * a.H, *before = fl + (size_t)T * a.H, *last = before + (size_t)num_items * a.H;
        k.w = w; k.x = x; k.fl = fl; k.before = before; k.last = last;
        q = last + (size_t)num_items * a.H;
        lr_gates_kernel<<<dim3(a.H, a.R), 1024, 0, s>>>(a, item_start, w, x, fl, before, last);
        if (int rc = tff_check_launch("recurrence_gates")) return rc;
    } else {
        k.cum = q;
        lr_decay_kernel<<<dim3(num_items, (a.H * a.D + 63) / 64), 256, 0, s>>>(a, items, q);
        q += (size_t)T * a.H * a.D;
        if (int rc = tff_check_launch("recurrence_decay")) return rc;
    }
    k.o = workspace + (((size_t)(q - workspace) + 3) & ~(size_t)3);
    auto ok16 = [](const void* x) { return ((uintptr_t)x % 16) == 0; };
    const bool vec = a.D % 4 == 0 && a.E % 4 == 0 && a.ld % 4 == 0 && ok16(a.q) && ok16(a.k) && ok16(a.v);
    const dim3 g1(num_items, a.H, d_blocks * e_blocks), g2((E1 * a.D + 255) / 256, a.H, a.R);
#define LR_SUMS(K) do { if (vec) lr_sums_kernel<K, true><<<g1, 256, 0, s>>>(a, k, d_blocks); else lr_sums_kernel<K, false><<<g1, 256, 0, s>>>(a, k, d_blocks); } while (0)
    if (ex) LR_SUMS(TFF_LR_EXP); else LR_SUMS(TFF_LR_DECAY);
#undef LR_SUMS
    if (int rc = tff_check_launch("recurrence_sums")) return rc;
    if (ex) lr_scan_kernel<TFF_LR_EXP><<<g2, 256, 0, s>>>(a, k);
    else lr_scan_kernel<TFF_LR_DECAY><<<g2, 256, 0, s>>>(a, k);
    if (int rc = tff_check_launch("recurrence_scan")) return rc;
    const bool bf = a.out_dtype == TFF_BF16;
    const int eb = a.E <= 64 ? 1 : a.E <= 128 ? 2 : 4;
    const dim3 g3(num_items, a.H, (e_blocks + eb - 1) / eb);
#define LR_OUT(K, EB, V, TO, FU) lr_outputs_kernel<K, EB, V, TO, FU><<<g3, 256, 0, s>>>(a, k)
#define LR_OUT_V(K, EB, TO, FU) do { if (vec) LR_OUT(K, EB, true, TO, FU); else LR_OUT(K, EB, false, TO, FU); } while (0)
#define LR_OUT_K(K)                                          \
    do {                                                     \
        if (a.E > LR_FUSED_E) LR_OUT_V(K, 4, float, false);  \
        else if (eb == 1 && bf) LR_OUT_V(K, 1, bf16_t, true); \
        else if (eb == 1) LR_OUT_V(K, 1, float, true);       \
        else if (eb == 2 && bf) LR_OUT_V(K, 2, bf16_t, true); \
        else if (eb == 2) LR_OUT_V(K, 2, float, true);       \
        else if (bf) LR_OUT_V(K, 4, bf16_t, true);           \
        else LR_OUT_V(K, 4, float, true);                    \
    } while (0)
    if (ex) LR_OUT_K(TFF_LR_EXP); else LR_OUT_K(TFF_LR_DECAY);
#undef LR_OUT_K
#undef LR_OUT_V
#undef LR_OUT
    if (int rc = tff_check_launch("recurrence_outputs")) return rc;
    if (a.E > LR_FUSED_E) {
        const int pairs = T * a.H;
        if (bf) lr_norm_gate_kernel<bf16_t><<<(pairs + 3) / 4, 256, 0, s>>>(a, k.o, pairs);
        else lr_norm_gate_kernel<float><<<(pairs + 3) / 4, 256, 0, s>>>(a, k.o, pairs);
        return tff_check_launch("recurrence_norm_gate");
    }
    return 0;
}
