// Gated linear attention over a packed batch, with per-slot state: a recurrence whose state is a matrix a head and
// whose decay is a number a head and key channel,
//     S <- diag(a_t) S + k_t v_t^T;   o_t = S^T (q_scale q_t)            S: [dk, dv], zero at the start
//     a_t = sigmoid(z_t)^(1/tau),  z_t = W_up low_t + b,  low_t the rank-R first half of a low-rank product
// q, k, v and low are column blocks of one projection's rows (q and k heads x dk, v heads x dv, low R wide), in the
// engine's element type; the decays, the state and everything behind the projection are float.  ln a = -softplus(-z) /
// tau, so a decay near zero or one keeps its precision.
//
//  * channel_decay_kernel: the decays of a step's tokens, float [n, heads*dk].
//  * gla_scan_kernel: steps of many tokens.  A workgroup owns one (sequence, head, C * 256 / L columns of dv) and walks
//    tokens in order; a column's dk state values are spread over L neighbouring lanes in pieces of 4 (state index
//    (j L + l) 4 + e: neighbouring lanes read neighbouring 16 bytes of LDS), and a lane holds C columns, which share
//    the q, k and decays it reads.  Tokens pass through LDS in tiles, the next tile is asked for while the current one
//    is walked.
//    A sequence may be cut into segments of `seg_len` tokens that run at the same time: the first one starts from the
//    slot's state, the others from zero.  A segment then also leaves its state and the product of its decays, and every
//    token's q times the product of the decays since the segment's start.
//  * gla_carry_kernel: the states at the segments' starts, one segment after the other, and the slot's new state.
//  * gla_fix_kernel: o_t += S_start^T (q_t * product of decays) for the segments behind the first, a product on the
//    matrix cores in float (v_mfma_f32_16x16x4_f32).  Only decays multiply the carried state, so nothing is divided by
//    a small number.
//  * gla_step_kernel: steps of one token a sequence, a workgroup a (sequence, head): the decays, one pass over the
//    state, each head's RMS norm (a weight of dv numbers shared by the heads) and the gate's nonlinearity, written as
//    the output projection reads it.
#include "common.h"

typedef float gfloatx4_t __attribute__((ext_vector_type(4)));

// sigmoid(z)^(1/tau)
__device__ inline float decay_of(float z, float inv_tau) {
    return expf(-(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * inv_tau);
}

#define DECAY_TOKENS 8
// grid (ceil(n / DECAY_TOKENS), ceil(C / 256)), 256 threads: a thread owns a channel for DECAY_TOKENS tokens
template <typename T>
__global__ __launch_bounds__(256) void channel_decay_kernel(const T* __restrict__ low, long ld, int R,
                                                            const float* __restrict__ up, const float* __restrict__ bias,
                                                            float inv_tau, float* __restrict__ out, int n, int C) {
    constexpr int RC = 64;
    __shared__ float ls[RC][DECAY_TOKENS];
    const int c = blockIdx.y * 256 + threadIdx.x, t0 = blockIdx.x * DECAY_TOKENS;
    float z[DECAY_TOKENS];
    const float b = c < C ? bias[c] : 0.f;
#pragma unroll
    for (int t = 0; t < DECAY_TOKENS; ++t) z[t] = b;
    for (int r0 = 0; r0 < R; r0 += RC) {
        const int rn = min(RC, R - r0);
        __syncthreads();
        for (int i = threadIdx.x; i < rn * DECAY_TOKENS; i += 256) {
            const int r = i % rn, t = i / rn;
            ls[r][t] = to_f32(low[(long)min(t0 + t, n - 1) * ld + r0 + r]);
        }
        __syncthreads();
        if (c < C)
            for (int r = 0; r < rn; ++r) {
                const float w = up[(long)(r0 + r) * C + c];       // up is stored [R][C]: neighbouring threads, neighbouring words
#pragma unroll
                for (int t = 0; t < DECAY_TOKENS; ++t) z[t] += w * ls[r][t];
            }
    }
    if (c >= C) return;
#pragma unroll
    for (int t = 0; t < DECAY_TOKENS; ++t)
        if (t0 + t < n) out[(long)(t0 + t) * C + c] = decay_of(z[t], inv_tau);
}

extern "C" const char* cpmcu_channel_decay(const void* low, int dtype, long ld, int R, const float* up, const float* bias,
                                           float inv_tau, float* out, int n, int C, hipStream_t stream) {
    CPMCU_REQUIRE(n > 0 && C > 0 && R > 0 && ld >= R, "channel_decay: empty shape n=%d channels=%d rank=%d", n, C, R);
    CPMCU_REQUIRE(low && up && bias && out, "channel_decay: null pointer");
    dim3 grid((n + DECAY_TOKENS - 1) / DECAY_TOKENS, (C + 255) / 256);
    CPMCU_REQUIRE(grid.y <= 65535, "channel_decay: %d channels exceed the launch grid", C);
    if (dtype == CPMCU_F32)
        channel_decay_kernel<float><<<grid, 256, 0, stream>>>((const float*)low, ld, R, up, bias, inv_tau, out, n, C);
    else if (dtype == CPMCU_BF16)
        channel_decay_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)low, ld, R, up, bias, inv_tau, out, n, C);
    else
        CPMCU_FAIL("channel_decay: unknown dtype %d", dtype);
    CPMCU_LAUNCH_CHECK("channel_decay");
    return nullptr;
}

// rows: T [n, ld] with q heads at column q_off, k at k_off, v at v_off; decay float [n, heads*dk];
// state float [slots][heads][dv][dk]; y float [n, heads*dv].
// n_seg > 1: seg_state float [B * n_seg][heads][dv][dk], seg_decay float [B * n_seg][heads][dk], qa float [n, heads*dk]
template <int NR, int TT, int L, int C, typename T>
__global__ __launch_bounds__(256) void gla_scan_kernel(const T* __restrict__ rows, long ld, long q_off, long k_off,
                                                       long v_off, const float* __restrict__ decay,
                                                       float* __restrict__ state, float* __restrict__ y,
                                                       const int* __restrict__ cu_q, const int* __restrict__ seq_slot,
                                                       int heads, int dk, int dv, float q_scale, int n_seg, int seg_len,
                                                       float* __restrict__ seg_state, float* __restrict__ seg_decay,
                                                       float* __restrict__ qa) {
    constexpr int PB = 256 / L;                     // lane groups a workgroup
    constexpr int NS = NR * L;                      // state values a column, padded
    constexpr int QK = TT * NS / 256;               // q (k, decay) values a thread brings a tile
    constexpr int VV = (TT * PB * C + 255) / 256;
    static_assert(NR % 4 == 0 && TT * NS % 256 == 0, "tile shape");
    __shared__ __attribute__((aligned(16))) float qs[TT][NS], ks[TT][NS], as[TT][NS];
    __shared__ float vs[TT][PB * C];
    const int b = blockIdx.x / n_seg, seg = blockIdx.x % n_seg, h = blockIdx.y, p0 = blockIdx.z * PB * C;
    const int first = cu_q[b] + seg * seg_len;
    const int n_q = n_seg > 1 ? min(seg_len, cu_q[b + 1] - first) : cu_q[b + 1] - first;
    if (n_q <= 0) return;                           // (the whole workgroup)
    const int slot = seq_slot[b];
    const int g = threadIdx.x / L, l = threadIdx.x % L;
    float S[C][NR];
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int p = p0 + g * C + c;
        const float* sp = state + (((long)slot * heads + h) * dv + min(p, dv - 1)) * dk;
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const int n = ((i >> 2) * L + l) * 4 + (i & 3);
            S[c][i] = (seg == 0 && p < dv && n < dk) ? sp[n] : 0.f;
        }
    }
    const bool writes_qa = n_seg > 1 && blockIdx.z == 0;
    float run = 1.f;                                // the channel's product of decays since the segment's start
    float rq[QK], rk[QK], ra[QK], rv[VV];
    auto fetch = [&](int t0) {
        const int tn = min(TT, n_q - t0);
#pragma unroll
        for (int i = 0; i < QK; ++i) {
            const int e = threadIdx.x + i * 256, tt = e / NS, n = e % NS;
            const bool ok = tt < tn && n < dk;
            const long t = first + t0 + min(tt, tn - 1);
            const long col = (long)h * dk + min(n, dk - 1);
            const float q = to_f32(rows[t * ld + q_off + col]), k = to_f32(rows[t * ld + k_off + col]), a = decay[t * heads * dk + col];
            rq[i] = ok ? q * q_scale : 0.f;
            rk[i] = ok ? k : 0.f;
            ra[i] = ok ? a : 0.f;
        }
#pragma unroll
        for (int i = 0; i < VV; ++i) {
            const int e = threadIdx.x + i * 256, tt = e / (PB * C), p = p0 + e % (PB * C);
            const float v = to_f32(rows[(long)(first + t0 + min(tt, tn - 1)) * ld + v_off + (long)h * dv + min(p, dv - 1)]);
            rv[i] = (tt < tn && p < dv) ? v : 0.f;
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < n_q; t0 += TT) {
        const int tn = min(TT, n_q - t0);
        __syncthreads();
#pragma unroll
        for (int i = 0; i < QK; ++i) {
            const int e = threadIdx.x + i * 256;
            qs[e / NS][e % NS] = rq[i];
            ks[e / NS][e % NS] = rk[i];
            as[e / NS][e % NS] = ra[i];
        }
#pragma unroll
        for (int i = 0; i < VV; ++i) {
            const int e = threadIdx.x + i * 256;
            if (e < TT * PB * C) vs[e / (PB * C)][e % (PB * C)] = rv[i];
        }
        __syncthreads();
        if (t0 + TT < n_q) fetch(t0 + TT);
        for (int tt = 0; tt < tn; ++tt) {
            float o[C], v[C];
#pragma unroll
            for (int c = 0; c < C; ++c) {
                o[c] = 0.f;
                v[c] = vs[tt][g * C + c];
            }
#pragma unroll
            for (int j = 0; j < NR / 4; ++j) {
                const float4 q4 = *(const float4*)&qs[tt][(j * L + l) * 4];
                const float4 k4 = *(const float4*)&ks[tt][(j * L + l) * 4];
                const float4 a4 = *(const float4*)&as[tt][(j * L + l) * 4];
                const float q[4] = {q4.x, q4.y, q4.z, q4.w}, k[4] = {k4.x, k4.y, k4.z, k4.w}, a[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int c = 0; c < C; ++c) {
                        const float s = fmaf(a[e], S[c][4 * j + e], k[e] * v[c]);
                        S[c][4 * j + e] = s;
                        o[c] = fmaf(s, q[e], o[c]);
                    }
            }
#pragma unroll
            for (int c = 0; c < C; ++c) {
                o[c] = lanes_sum<L>(o[c]);
                const int p = p0 + g * C + c;
                if (l == 0 && p < dv) y[(long)(first + t0 + tt) * heads * dv + (long)h * dv + p] = o[c];
            }
        }
        if (writes_qa && (int)threadIdx.x < dk) {
            for (int tt = 0; tt < tn; ++tt) {
                run *= as[tt][threadIdx.x];
                qa[(long)(first + t0 + tt) * heads * dk + (long)h * dk + threadIdx.x] = qs[tt][threadIdx.x] * run;
            }
        }
    }
    float* base = n_seg > 1 ? seg_state + ((long)blockIdx.x * heads + h) * dv * dk : state + ((long)slot * heads + h) * (long)dv * dk;
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int p = p0 + g * C + c;
        if (p < dv)
#pragma unroll
            for (int i = 0; i < NR; ++i) {
                const int n = ((i >> 2) * L + l) * 4 + (i & 3);
                if (n < dk) base[(long)p * dk + n] = S[c][i];
            }
    }
    if (writes_qa && (int)threadIdx.x < dk) seg_decay[((long)blockIdx.x * heads + h) * dk + threadIdx.x] = run;
}

// grid (B, heads, ceil(dv * dk / 256)): seg_state[b][s] becomes the state at the START of segment s, the slot gets the last
__global__ __launch_bounds__(256) void gla_carry_kernel(float* __restrict__ state, const int* __restrict__ cu_q,
                                                        const int* __restrict__ seq_slot, int heads, int dk, int dv,
                                                        int n_seg, int seg_len, float* __restrict__ seg_state,
                                                        const float* __restrict__ seg_decay) {
    const int b = blockIdx.x, h = blockIdx.y;
    const long i = (long)blockIdx.z * 256 + threadIdx.x;
    if (i >= (long)dv * dk) return;
    const int segs = (cu_q[b + 1] - cu_q[b] + seg_len - 1) / seg_len;
    if (segs <= 0) return;
    const int n = (int)(i % dk);
    float carried = 0.f;                             // segment 0 started from the slot's state
    for (int s = 0; s < segs; ++s) {
        const long at = ((long)(b * n_seg + s) * heads + h) * dv * dk + i;
        const float end = seg_state[at] + (s ? seg_decay[((long)(b * n_seg + s) * heads + h) * dk + n] * carried : 0.f);
        seg_state[at] = carried;
        carried = end;
    }
    state[((long)seq_slot[b] * heads + h) * dv * dk + i] = carried;
}

// grid (B * n_seg, heads, ceil(dv / 64)), 256 threads: a wavefront takes 16 columns of dv and the segment's tokens 16 at a
// time: y[t, p] += sum_n qa[t, n] S_start[p][n]
__global__ __launch_bounds__(256) void gla_fix_kernel(const float* __restrict__ qa, const float* __restrict__ seg_state,
                                                      float* __restrict__ y, const int* __restrict__ cu_q, int heads,
                                                      int dk, int dv, int n_seg, int seg_len) {
    const int b = blockIdx.x / n_seg, seg = blockIdx.x % n_seg, h = blockIdx.y;
    const int first = cu_q[b] + seg * seg_len, n_q = min(seg_len, cu_q[b + 1] - first);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
    const int p0 = blockIdx.z * 64 + wave * 16;
    if (seg == 0 || n_q <= 0 || p0 >= dv) return;    // (no barrier in this kernel)
    const float* sp = seg_state + (((long)blockIdx.x * heads + h) * dv + min(p0 + r, dv - 1)) * dk;
    constexpr int TB = 4;                            // tiles of 16 tokens that share the state's operand
    for (int t0 = 0; t0 < n_q; t0 += 16 * TB) {
        gfloatx4_t acc[TB];
        const float* qp[TB];
#pragma unroll
        for (int u = 0; u < TB; ++u) {
            acc[u] = gfloatx4_t{0.f, 0.f, 0.f, 0.f};
            qp[u] = qa + (long)(first + min(t0 + u * 16 + r, n_q - 1)) * heads * dk + (long)h * dk;
        }
        int n0 = 0;
        if (dk % 4 == 0)                             // 16 features at a time: a lane brings 4 neighbouring ones of its rows
            for (; n0 + 16 <= dk; n0 += 16) {
                const float4 s = *(const float4*)(sp + n0 + 4 * g);
                float4 q[TB];
#pragma unroll
                for (int u = 0; u < TB; ++u) q[u] = *(const float4*)(qp[u] + n0 + 4 * g);
#pragma unroll
                for (int u = 0; u < TB; ++u) {
                    acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[u].x, s.x, acc[u], 0, 0, 0);
                    acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[u].y, s.y, acc[u], 0, 0, 0);
                    acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[u].z, s.z, acc[u], 0, 0, 0);
                    acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[u].w, s.w, acc[u], 0, 0, 0);
                }
            }
        for (; n0 < dk; n0 += 4) {
            const int n = min(n0 + g, dk - 1);
            const float s = n0 + g < dk ? sp[n] : 0.f;
#pragma unroll
            for (int u = 0; u < TB; ++u) acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(qp[u][n], s, acc[u], 0, 0, 0);
        }
        // lane (column r, g): acc[u][i] belongs to token t0 + 16 u + 4 g + i
        if (p0 + r < dv)
#pragma unroll
            for (int u = 0; u < TB; ++u)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = t0 + u * 16 + 4 * g + i;
                    if (t < n_q) y[(long)(first + t) * heads * dv + (long)h * dv + p0 + r] += acc[u][i];
                }
    }
}

extern "C" const char* cpmcu_gla_scan(const void* rows, int dtype, long ld, long q_off, long k_off, long v_off,
                                      const float* decay, float* state, float* y, const int* cu_q, const int* seq_slot,
                                      int n_seqs, int heads, int dk, int dv, float q_scale, int n_seg, int seg_len,
                                      float* seg_state, float* seg_decay, float* qa, hipStream_t stream) {
    CPMCU_REQUIRE(n_seqs > 0 && heads > 0 && dk > 0 && dv > 0, "gla_scan: empty shape");
    CPMCU_REQUIRE(dk <= 256, "gla_scan: a key size of %d is not supported (at most 256)", dk);
    CPMCU_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && ld >= q_off + (long)heads * dk && ld >= k_off + (long)heads * dk &&
                  ld >= v_off + (long)heads * dv, "gla_scan: rows of %ld too short", ld);
    CPMCU_REQUIRE(rows && decay && state && y && cu_q && seq_slot, "gla_scan: null pointer");
    CPMCU_REQUIRE(n_seg >= 1 && (n_seg == 1 || (seg_len > 0 && seg_state && seg_decay && qa)), "gla_scan: %d segments of %d tokens without scratch", n_seg, seg_len);
    // 16 lanes a column where a column is long enough for them, 8 otherwise; two columns a lane where enough workgroups remain
    const int lanes = dk > 32 ? 16 : 8;
    const int groups = 256 / lanes;
    const long wgs2 = (long)n_seqs * n_seg * heads * ((dv + 2 * groups - 1) / (2 * groups));
    const int cols = (dv > groups && wgs2 >= 256) ? 2 : 1;
    const dim3 grid((unsigned)(n_seqs * n_seg), heads, (dv + groups * cols - 1) / (groups * cols));
    CPMCU_REQUIRE(heads <= 65535 && grid.z <= 65535, "gla_scan: shape exceeds the launch grid");
#define LAUNCH(NRv, TTv, Lv, Cv, Tv)                                                                                  \
    gla_scan_kernel<NRv, TTv, Lv, Cv, Tv><<<grid, 256, 0, stream>>>((const Tv*)rows, ld, q_off, k_off, v_off, decay,   \
                                                                    state, y, cu_q, seq_slot, heads, dk, dv, q_scale, \
                                                                    n_seg, seg_len, seg_state, seg_decay, qa)
#define BY_COLS(NRv, TTv, Lv, Tv)                        \
    do {                                                 \
        if (cols == 2) LAUNCH(NRv, TTv, Lv, 2, Tv);      \
        else LAUNCH(NRv, TTv, Lv, 1, Tv);                \
    } while (0)
#define BY_SIZE(Tv)                                      \
    do {                                                 \
        if (lanes == 8) BY_COLS(4, 32, 8, Tv);           \
        else if (dk <= 64) BY_COLS(4, 32, 16, Tv);       \
        else if (dk <= 128) BY_COLS(8, 16, 16, Tv);      \
        else BY_COLS(16, 8, 16, Tv);                     \
    } while (0)
    if (dtype == CPMCU_F32) BY_SIZE(float);
    else if (dtype == CPMCU_BF16) BY_SIZE(bf16_t);
    else CPMCU_FAIL("gla_scan: unknown dtype %d", dtype);
#undef BY_SIZE
#undef BY_COLS
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("gla_scan");
    if (n_seg > 1) {
        const long per = ((long)dv * dk + 255) / 256;
        CPMCU_REQUIRE(per <= 65535, "gla_scan: a state of %d x %d exceeds the launch grid", dk, dv);
        gla_carry_kernel<<<dim3(n_seqs, heads, (unsigned)per), 256, 0, stream>>>(state, cu_q, seq_slot, heads, dk, dv, n_seg,
                                                                                seg_len, seg_state, seg_decay);
        CPMCU_LAUNCH_CHECK("gla_carry");
        gla_fix_kernel<<<dim3(n_seqs * n_seg, heads, (dv + 63) / 64), 256, 0, stream>>>(qa, seg_state, y, cu_q, heads, dk, dv,
                                                                                        n_seg, seg_len);
        CPMCU_LAUNCH_CHECK("gla_fix");
    }
    return nullptr;
}

// grid (B, heads), NT threads: 16 lanes a column of the state.  rows: T [n, ld]; sequence b's one token is row cu_q[b];
// up float [R][heads*dk]; out T [n, heads*dv].
// out = rms(o) * norm_w (per head) * silu(gate), or * sigmoid(gate) with gate_sigmoid
template <typename T>
__global__ __launch_bounds__(1024) void gla_step_kernel(const T* __restrict__ rows, long ld, long q_off, long k_off,
                                                        long v_off, long g_off, long low_off, int R,
                                                        const float* __restrict__ up, const float* __restrict__ bias,
                                                        float inv_tau, const float* __restrict__ norm_w, float eps,
                                                        int gate_sigmoid, float* __restrict__ state, T* __restrict__ out,
                                                        const int* __restrict__ cu_q, const int* __restrict__ seq_slot,
                                                        int heads, int dk, int dv, float q_scale) {
    extern __shared__ float sm[];                    // q, k, a: [dkp] each; then o: [dv]
    __shared__ float red[17];
    const int b = blockIdx.x, h = blockIdx.y, NT = blockDim.x;
    const int dkp = (dk + 63) & ~63;
    float *qs = sm, *ks = sm + dkp, *as = sm + 2 * dkp, *os = sm + 3 * dkp;
    const long t = cu_q[b];
    const T* row = rows + t * ld;
    float* sp = state + ((long)seq_slot[b] * heads + h) * (long)dv * dk;
    const int g = threadIdx.x >> 4, l = threadIdx.x & 15, G = NT >> 4;
    // a column's share of a lane: pieces of 4 values, the first column asked for before the decays are formed
    float S[16];
    auto load = [&](int p) {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int n = ((i >> 2) * 16 + l) * 4 + (i & 3);
            S[i] = (p < dv && n < dk) ? sp[(long)p * dk + n] : 0.f;
        }
    };
    auto load4s = [&](int p) {                       // dk a multiple of 4
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = (j * 16 + l) * 4;
            const float4 v = (p < dv && n < dk) ? *(const float4*)(sp + (long)p * dk + n) : make_float4(0.f, 0.f, 0.f, 0.f);
            S[4 * j] = v.x; S[4 * j + 1] = v.y; S[4 * j + 2] = v.z; S[4 * j + 3] = v.w;
        }
    };
    const bool vec = dk % 4 == 0;
    if (vec) load4s(g);
    else load(g);
    // decays: 4 neighbouring lanes a channel
    for (int c0 = 0; c0 < dkp; c0 += NT / 4) {
        const int c = c0 + (threadIdx.x >> 2), part = threadIdx.x & 3;
        float z = 0.f;
        if (c < dk)
            for (int r = part; r < R; r += 4) z += up[(long)r * heads * dk + (long)h * dk + c] * to_f32(row[low_off + r]);
        z = lanes_sum<4>(z);
        if (part == 0 && c < dkp) as[c] = c < dk ? decay_of(z + bias[(long)h * dk + c], inv_tau) : 0.f;
    }
    for (int c = threadIdx.x; c < dkp; c += NT) {
        qs[c] = c < dk ? to_f32(row[q_off + (long)h * dk + c]) * q_scale : 0.f;
        ks[c] = c < dk ? to_f32(row[k_off + (long)h * dk + c]) : 0.f;
    }
    __syncthreads();
    float ss = 0.f;
    for (int p = g; p < dv; p += G) {
        const float v = to_f32(row[v_off + (long)h * dv + p]);
        float o = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = (j * 16 + l) * 4;
            if (n >= dkp) break;
            const float4 q4 = *(const float4*)(qs + n), k4 = *(const float4*)(ks + n), a4 = *(const float4*)(as + n);
            S[4 * j] = fmaf(a4.x, S[4 * j], k4.x * v);
            S[4 * j + 1] = fmaf(a4.y, S[4 * j + 1], k4.y * v);
            S[4 * j + 2] = fmaf(a4.z, S[4 * j + 2], k4.z * v);
            S[4 * j + 3] = fmaf(a4.w, S[4 * j + 3], k4.w * v);
            o += (S[4 * j] * q4.x + S[4 * j + 1] * q4.y) + (S[4 * j + 2] * q4.z + S[4 * j + 3] * q4.w);
            if (vec) {
                if (n < dk) *(float4*)(sp + (long)p * dk + n) = make_float4(S[4 * j], S[4 * j + 1], S[4 * j + 2], S[4 * j + 3]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < dk) sp[(long)p * dk + n + e] = S[4 * j + e];
            }
        }
        if (vec) load4s(p + G);
        else load(p + G);
        o = row16_sum(o);
        if (l == 0) {
            os[p] = o;
            ss += o * o;
        }
    }
    const float r = 1.0f / sqrtf(block_sum(ss, red) / (float)dv + eps);     // (its barriers make os visible)
    for (int p = threadIdx.x; p < dv; p += NT) {
        const float gt = to_f32(row[g_off + (long)h * dv + p]);
        const float s = 1.0f / (1.0f + expf(-gt));
        out[(t * heads + h) * dv + p] = from_f32<T>(os[p] * r * norm_w[p] * (gate_sigmoid ? s : gt * s));
    }
}

extern "C" const char* cpmcu_gla_step(const void* rows, int dtype, long ld, long q_off, long k_off, long v_off, long g_off,
                                      long low_off, int R, const float* up, const float* bias, float inv_tau,
                                      const float* norm_w, float eps, int gate_sigmoid, float* state, void* out,
                                      const int* cu_q, const int* seq_slot, int n_seqs, int heads, int dk, int dv,
                                      float q_scale, hipStream_t stream) {
    CPMCU_REQUIRE(n_seqs > 0 && heads > 0 && dk > 0 && dv > 0 && R > 0, "gla_step: empty shape");
    CPMCU_REQUIRE(dk <= 256, "gla_step: a key size of %d is not supported (at most 256)", dk);
    CPMCU_REQUIRE(dv <= 8192, "gla_step: a value size of %d does not fit the kernel's LDS", dv);
    CPMCU_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && g_off >= 0 && low_off >= 0 && ld >= q_off + (long)heads * dk &&
                  ld >= k_off + (long)heads * dk && ld >= v_off + (long)heads * dv && ld >= g_off + (long)heads * dv &&
                  ld >= low_off + R, "gla_step: rows of %ld too short", ld);
    CPMCU_REQUIRE(rows && up && bias && norm_w && state && out && cu_q && seq_slot, "gla_step: null pointer");
    CPMCU_REQUIRE(heads <= 65535, "gla_step: %d heads exceed the launch grid", heads);
    int nt = 1024;
    while (nt > 256 && nt / 16 > dv) nt /= 2;
    const size_t lds = (3 * ((dk + 63) & ~63) + dv) * sizeof(float);
    const dim3 grid(n_seqs, heads);
#define LAUNCH(Tv)                                                                                                      \
    gla_step_kernel<Tv><<<grid, nt, lds, stream>>>((const Tv*)rows, ld, q_off, k_off, v_off, g_off, low_off, R, up, bias, \
                                                   inv_tau, norm_w, eps, gate_sigmoid, state, (Tv*)out, cu_q, seq_slot, \
                                                   heads, dk, dv, q_scale)
    if (dtype == CPMCU_F32) LAUNCH(float);
    else if (dtype == CPMCU_BF16) LAUNCH(bf16_t);
    else CPMCU_FAIL("gla_step: unknown dtype %d", dtype);
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("gla_step");
    return nullptr;
}
