// Row kernels of layers whose norm is followed by a short convolution, whose residual takes a normed input of the
// token itself, or whose residual is replaced at the start of a pass:
//
//  * norm_rows_kernel: one pass over a token's row,
//        y = y_scale * (sum of the branch's partial sums) + y_bias           (if a branch is pending)
//        y <- y / sqrt(mean(y^2) + y_eps) * y_norm_w                         (if the branch has a norm of its own)
//        x <- x + y, or x <- y (`replace`); written back unless `rows` selects rows
//        h = x as it is, its layer norm (x - mean) / sqrt(mean((x - mean)^2) + eps) * w, or its RMS norm
//    and h goes out in either element type (rows may be `ld_out` apart).  With convolutions, for steps in which
//    every row is a sequence of its own (decoding): out_k = h + sum_j c_k[j] h_(t - taps + 1 + j), k = 1, 2, the
//    earlier h from the sequence's slot, which then moves on by one.  Float statistics; the row stays in registers.
//  * conv_rows_kernel: the same convolution for steps that bring several tokens a sequence, reading h from memory;
//    conv_rows_remember_kernel then moves the slots on to the step's last inputs.
//  * add_rows_kernel: x += A + F (partial sums and biases), and x again in the activations' element type: what a
//    product that reads the residual itself takes.
//  * gated_lookup_kernel: g[t, j] = act(z[t, j]) * table[id_t, off + j]; lookup_strip_kernel does the product z = x W^T
//    as well, for decode steps of at most 16 tokens in bf16.
#include "common.h"
#include "vec4.h"

enum { ROWS_NORM_NONE = 0, ROWS_NORM_LAYER = 1, ROWS_NORM_RMS = 2 };

// V neighbouring columns
template <int V> struct Cols { float v[V]; };
template <typename T>
__device__ inline Cols<4> load_cols(const T* p, Cols<4>*) {
    const float4 f = load4(p);
    return Cols<4>{{f.x, f.y, f.z, f.w}};
}
template <typename T>
__device__ inline Cols<1> load_cols(const T* p, Cols<1>*) { return Cols<1>{{to_f32(*p)}}; }
template <int V, typename T>
__device__ inline Cols<V> load_cols(const T* p) { return load_cols(p, (Cols<V>*)nullptr); }
template <typename T>
__device__ inline void store_cols(T* p, const Cols<4>& c) { store4(p, c.v[0], c.v[1], c.v[2], c.v[3]); }
template <typename T>
__device__ inline void store_cols(T* p, const Cols<1>& c) { *p = from_f32<T>(c.v[0]); }
template <typename T>
__device__ inline Cols<4> sum_cols(const T* p, int parts, long stride, Cols<4>*) {
    const float4 f = sum_parts4(p, parts, stride);
    return Cols<4>{{f.x, f.y, f.z, f.w}};
}
template <typename T>
__device__ inline Cols<1> sum_cols(const T* p, int parts, long stride, Cols<1>*) {
    float s = 0.f;
    for (int i = 0; i < parts; ++i) s += to_f32(p[i * stride]);
    return Cols<1>{{s}};
}
template <int V, typename T>
__device__ inline Cols<V> sum_cols(const T* p, int parts, long stride) { return sum_cols(p, parts, stride, (Cols<V>*)nullptr); }

// A row a workgroup; thread i holds columns V * (i + k * blockDim) .. + V, k < K.
template <typename YT, typename OT, int V, int K>
__global__ __launch_bounds__(1024) void norm_rows_kernel(
    float* __restrict__ X, const YT* __restrict__ Y, int nparts, long part_stride, float y_scale,
    const float* __restrict__ y_bias, const float* __restrict__ y_norm_w, float y_eps, int replace, int norm,
    const float* __restrict__ w, float eps, OT* __restrict__ out, long ld_out, const int* __restrict__ rows, int H,
    const float* __restrict__ conv1, const float* __restrict__ conv2, int taps, float* __restrict__ conv_state,
    const int* __restrict__ slots, OT* __restrict__ out2) {
    __shared__ float red[17];
    const long r = rows ? rows[blockIdx.x] : blockIdx.x;
    Cols<V> u[K];
    float ss = 0.f, sum = 0.f;
#pragma unroll
    for (int k = 0; k < K; ++k) {
        const int c = V * (threadIdx.x + k * blockDim.x);
#pragma unroll
        for (int e = 0; e < V; ++e) u[k].v[e] = 0.f;
        if (c >= H || !Y) continue;
        u[k] = sum_cols<V>(Y + r * H + c, nparts, part_stride);
#pragma unroll
        for (int e = 0; e < V; ++e) {
            u[k].v[e] = u[k].v[e] * y_scale + (y_bias ? y_bias[c + e] : 0.f);
            ss += u[k].v[e] * u[k].v[e];
        }
    }
    float yr = 1.f;
    if (y_norm_w) yr = 1.0f / sqrtf(block_sum(ss, red) / (float)H + y_eps);
#pragma unroll
    for (int k = 0; k < K; ++k) {
        const int c = V * (threadIdx.x + k * blockDim.x);
        if (c >= H) continue;
        if (y_norm_w) {
            const Cols<V> g = load_cols<V>(y_norm_w + c);
#pragma unroll
            for (int e = 0; e < V; ++e) u[k].v[e] = u[k].v[e] * yr * g.v[e];
        }
        if (!replace) {
            const Cols<V> x = load_cols<V>(X + r * H + c);
#pragma unroll
            for (int e = 0; e < V; ++e) u[k].v[e] += x.v[e];
        }
        if (!rows && Y) store_cols(X + r * H + c, u[k]);
#pragma unroll
        for (int e = 0; e < V; ++e) sum += u[k].v[e];
    }
    if (norm != ROWS_NORM_NONE) {
        const float mean = norm == ROWS_NORM_LAYER ? block_sum(sum, red) / (float)H : 0.f;
        float sq = 0.f;
#pragma unroll
        for (int k = 0; k < K; ++k) {
            if (V * (int)(threadIdx.x + k * blockDim.x) >= H) continue;
#pragma unroll
            for (int e = 0; e < V; ++e) {
                u[k].v[e] -= mean;
                sq += u[k].v[e] * u[k].v[e];
            }
        }
        const float inv = 1.0f / sqrtf(block_sum(sq, red) / (float)H + eps);
#pragma unroll
        for (int k = 0; k < K; ++k) {
            const int c = V * (threadIdx.x + k * blockDim.x);
            if (c >= H) continue;
            const Cols<V> g = load_cols<V>(w + c);
#pragma unroll
            for (int e = 0; e < V; ++e) u[k].v[e] = u[k].v[e] * inv * g.v[e];
        }
    }
    if (!out) return;
    OT* o = out + (long)blockIdx.x * ld_out;
    if (!conv1) {
#pragma unroll
        for (int k = 0; k < K; ++k) {
            const int c = V * (threadIdx.x + k * blockDim.x);
            if (c < H) store_cols(o + c, u[k]);
        }
        return;
    }
    float* st = taps > 1 ? conv_state + (long)slots[r] * (taps - 1) * H : nullptr;
    OT* o2 = conv2 ? out2 + (long)blockIdx.x * ld_out : nullptr;
#pragma unroll
    for (int k = 0; k < K; ++k) {
        const int c = V * (threadIdx.x + k * blockDim.x);
        if (c >= H) continue;
        Cols<V> a1 = u[k], a2 = u[k];
        for (int j = 0; j < taps; ++j) {
            Cols<V> s = u[k];
            if (j < taps - 1) {
                s = load_cols<V>(st + (long)j * H + c);
                if (j > 0) store_cols(st + (long)(j - 1) * H + c, s);
            }
            const Cols<V> w1 = load_cols<V>(conv1 + (long)j * H + c);
#pragma unroll
            for (int e = 0; e < V; ++e) a1.v[e] += w1.v[e] * s.v[e];
            if (conv2) {
                const Cols<V> w2 = load_cols<V>(conv2 + (long)j * H + c);
#pragma unroll
                for (int e = 0; e < V; ++e) a2.v[e] += w2.v[e] * s.v[e];
            }
        }
        if (taps > 1) store_cols(st + (long)(taps - 2) * H + c, u[k]);
        store_cols(o + c, a1);
        if (conv2) store_cols(o2 + c, a2);
    }
}

static bool aligned16r(const void* p) { return ((uintptr_t)p % 16) == 0; }

extern "C" const char* cpmcu_norm_rows(float* X, const void* Y, int y_dtype, int nparts, long part_stride, float y_scale,
                                       const float* y_bias, const float* y_norm_w, float y_eps, int replace, int norm,
                                       const float* w, float eps, void* out, int out_dtype, long ld_out, const int* rows,
                                       int n_out, int H, const float* conv1, const float* conv2, int taps,
                                       float* conv_state, const int* slots, void* out2, hipStream_t stream) {
    CPMCU_REQUIRE(n_out > 0 && H > 0 && X, "norm_rows: empty shape rows=%d width=%d", n_out, H);
    CPMCU_REQUIRE(norm >= ROWS_NORM_NONE && norm <= ROWS_NORM_RMS && (norm == ROWS_NORM_NONE || w), "norm_rows: norm kind %d", norm);
    CPMCU_REQUIRE(Y || (!replace && !y_norm_w && !y_bias), "norm_rows: a branch is missing");
    CPMCU_REQUIRE(!Y || nparts >= 1, "norm_rows: nparts=%d", nparts);
    CPMCU_REQUIRE(out || (!conv1 && Y), "norm_rows: nothing to write");
    CPMCU_REQUIRE(!out || ld_out >= H, "norm_rows: output rows of %ld for %d columns", ld_out, H);
    CPMCU_REQUIRE(!conv2 || (conv1 && out2), "norm_rows: the second convolution comes with the first and an output");
    CPMCU_REQUIRE(!conv1 || (taps >= 1 && !rows && (taps == 1 || (conv_state && slots))), "norm_rows: %d convolution taps", taps);
    CPMCU_REQUIRE(y_dtype == CPMCU_F32 || y_dtype == CPMCU_BF16, "norm_rows: unknown branch dtype %d", y_dtype);
    CPMCU_REQUIRE(out_dtype == CPMCU_F32 || out_dtype == CPMCU_BF16, "norm_rows: unknown output dtype %d", out_dtype);
    const bool vec = H % 4 == 0 && ld_out % 4 == 0 && aligned16r(X) && (!Y || (aligned16r(Y) && part_stride % 4 == 0)) &&
                     (!y_norm_w || aligned16r(y_norm_w)) && (!w || aligned16r(w)) && (!out || aligned16r(out)) &&
                     (!out2 || aligned16r(out2)) && (!conv1 || aligned16r(conv1)) && (!conv2 || aligned16r(conv2)) &&
                     (!conv_state || aligned16r(conv_state));
    const int cols = vec ? H / 4 : H, kmax = vec ? 4 : 8, cap = n_out >= 512 ? 256 : 1024;
    int block = 64;
    while (block < cap && block < cols) block *= 2;
    while (block < 1024 && block * kmax < cols) block *= 2;
    CPMCU_REQUIRE(block * kmax >= cols, "norm_rows: a width of %d is not supported", H);
    const bool one = block >= cols;
#define LAUNCH(YT, OT, Vv, Kv)                                                                                        \
    norm_rows_kernel<YT, OT, Vv, Kv><<<n_out, block, 0, stream>>>(X, (const YT*)Y, nparts, part_stride, y_scale, y_bias, \
                                                                  y_norm_w, y_eps, replace, norm, w, eps, (OT*)out,    \
                                                                  ld_out, rows, H, conv1, conv2, taps, conv_state,    \
                                                                  slots, (OT*)out2)
#define BY_SHAPE(YT, OT)                        \
    do {                                        \
        if (vec && one) LAUNCH(YT, OT, 4, 1);   \
        else if (vec) LAUNCH(YT, OT, 4, 4);     \
        else if (one) LAUNCH(YT, OT, 1, 1);     \
        else LAUNCH(YT, OT, 1, 8);              \
    } while (0)
    if (y_dtype == CPMCU_F32 && out_dtype == CPMCU_F32) BY_SHAPE(float, float);
    else if (y_dtype == CPMCU_F32) BY_SHAPE(float, bf16_t);
    else if (out_dtype == CPMCU_F32) BY_SHAPE(bf16_t, float);
    else BY_SHAPE(bf16_t, bf16_t);
#undef BY_SHAPE
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("norm_rows");
    return nullptr;
}

// grid (ceil(H / (256 V)), chunks of CONV_TOKENS tokens, sequences).  TAPS > 0: known at compile time, the last inputs
// slide through registers; 0: any number, every tap read from memory (the CU's cache holds the neighbours).
#define CONV_TOKENS 8
template <typename IT, typename OT, int V, int TAPS>
__global__ __launch_bounds__(256) void conv_rows_kernel(const IT* __restrict__ h, const float* __restrict__ conv1,
                                                        const float* __restrict__ conv2, int taps_rt,
                                                        const float* __restrict__ state, OT* __restrict__ out1,
                                                        OT* __restrict__ out2, const int* __restrict__ cu_q,
                                                        const int* __restrict__ seq_slot, int H) {
    const int taps = TAPS > 0 ? TAPS : taps_rt;
    const int c = V * (blockIdx.x * 256 + threadIdx.x), b = blockIdx.z;
    const long q0 = cu_q[b];
    const int len = cu_q[b + 1] - (int)q0, i0 = blockIdx.y * CONV_TOKENS;
    if (c >= H || i0 >= len) return;
    const int i1 = min(i0 + CONV_TOKENS, len);
    const float* st = taps > 1 ? state + (long)seq_slot[b] * (taps - 1) * H : nullptr;
    auto input = [&](int i) {          // the sequence's input i of this step; before its start, from the slot
        return i >= 0 ? load_cols<V>(h + (q0 + i) * H + c) : load_cols<V>(st + (long)(taps - 1 + i) * H + c);
    };
    constexpr int HN = TAPS > 1 ? TAPS - 1 : 1;
    Cols<V> hist[HN], w1[TAPS > 0 ? TAPS : 1], w2[TAPS > 0 ? TAPS : 1];
    if (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
            w1[j] = load_cols<V>(conv1 + (long)j * H + c);
            if (conv2) w2[j] = load_cols<V>(conv2 + (long)j * H + c);
            if (j < TAPS - 1) hist[j] = input(i0 - (TAPS - 1) + j);
        }
    }
    for (int i = i0; i < i1; ++i) {
        const Cols<V> cur = input(i);
        Cols<V> a1 = cur, a2 = cur;
        if (TAPS > 0) {
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
                const Cols<V> s = j < TAPS - 1 ? hist[j < HN ? j : 0] : cur;
#pragma unroll
                for (int e = 0; e < V; ++e) {
                    a1.v[e] += w1[j].v[e] * s.v[e];
                    if (conv2) a2.v[e] += w2[j].v[e] * s.v[e];
                }
            }
#pragma unroll
            for (int j = 0; j + 1 < HN; ++j) hist[j] = hist[j + 1];
            hist[HN - 1] = cur;
        } else {
            for (int j = 0; j < taps; ++j) {
                const Cols<V> s = j < taps - 1 ? input(i - (taps - 1) + j) : cur;
                const Cols<V> x1 = load_cols<V>(conv1 + (long)j * H + c);
#pragma unroll
                for (int e = 0; e < V; ++e) a1.v[e] += x1.v[e] * s.v[e];
                if (conv2) {
                    const Cols<V> x2 = load_cols<V>(conv2 + (long)j * H + c);
#pragma unroll
                    for (int e = 0; e < V; ++e) a2.v[e] += x2.v[e] * s.v[e];
                }
            }
        }
        store_cols(out1 + (q0 + i) * H + c, a1);
        if (conv2) store_cols(out2 + (q0 + i) * H + c, a2);
    }
}

// grid (ceil(H / 256), sequences): slot row j becomes the sequence's input len - (taps - 1) + j.  Rows are written in
// rising order and only read further on, so a step shorter than the slot's memory shifts it in place.
template <typename IT>
__global__ __launch_bounds__(256) void conv_rows_remember_kernel(const IT* __restrict__ h, int taps, float* __restrict__ state,
                                                                 const int* __restrict__ cu_q,
                                                                 const int* __restrict__ seq_slot, int H) {
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
    const long q0 = cu_q[b];
    const int len = cu_q[b + 1] - (int)q0;
    if (c >= H || len <= 0) return;
    float* st = state + (long)seq_slot[b] * (taps - 1) * H + c;
    for (int j = 0; j < taps - 1; ++j) {
        const int i = len - (taps - 1) + j;
        st[(long)j * H] = i >= 0 ? to_f32(h[(q0 + i) * H + c]) : st[(long)(j + len) * H];
    }
}

extern "C" const char* cpmcu_conv_rows(const void* h, int h_dtype, const float* conv1, const float* conv2, int taps,
                                       float* state, void* out1, void* out2, int out_dtype, const int* cu_q,
                                       const int* seq_slot, int n_seqs, int max_q, int H, int update_state,
                                       hipStream_t stream) {
    CPMCU_REQUIRE(n_seqs > 0 && max_q > 0 && H > 0 && taps >= 1 && h && conv1 && out1, "conv_rows: empty shape");
    CPMCU_REQUIRE(taps == 1 || state, "conv_rows: the slots' last inputs are missing");
    CPMCU_REQUIRE(!conv2 || out2, "conv_rows: the second convolution needs an output");
    const bool vec = H % 4 == 0 && aligned16r(h) && aligned16r(conv1) && (!conv2 || (aligned16r(conv2) && aligned16r(out2))) &&
                     aligned16r(out1) && (!state || aligned16r(state));
    const int chunks = (max_q + CONV_TOKENS - 1) / CONV_TOKENS;
    CPMCU_REQUIRE(chunks <= 65535 && n_seqs <= 65535, "conv_rows: %d tokens of a sequence or %d sequences exceed the launch grid", max_q, n_seqs);
    const int V = vec ? 4 : 1;
    dim3 grid((H + 256 * V - 1) / (256 * V), chunks, n_seqs);
#define LAUNCH(IT, OT, Vv, Tv)                                                                                       \
    conv_rows_kernel<IT, OT, Vv, Tv><<<grid, 256, 0, stream>>>((const IT*)h, conv1, conv2, taps, state, (OT*)out1,   \
                                                               (OT*)out2, cu_q, seq_slot, H)
#define BY_SHAPE(IT, OT)                             \
    do {                                             \
        if (vec && taps == 4) LAUNCH(IT, OT, 4, 4);  \
        else if (vec) LAUNCH(IT, OT, 4, 0);          \
        else LAUNCH(IT, OT, 1, 0);                   \
    } while (0)
    if (h_dtype == CPMCU_F32 && out_dtype == CPMCU_F32) BY_SHAPE(float, float);
    else if (h_dtype == CPMCU_F32 && out_dtype == CPMCU_BF16) BY_SHAPE(float, bf16_t);
    else if (h_dtype == CPMCU_BF16 && out_dtype == CPMCU_BF16) BY_SHAPE(bf16_t, bf16_t);
    else CPMCU_FAIL("conv_rows: unsupported dtypes in=%d out=%d", h_dtype, out_dtype);
#undef BY_SHAPE
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("conv_rows");
    if (update_state && taps > 1) {
        dim3 rgrid((H + 255) / 256, n_seqs);
        if (h_dtype == CPMCU_F32)
            conv_rows_remember_kernel<float><<<rgrid, 256, 0, stream>>>((const float*)h, taps, state, cu_q, seq_slot, H);
        else
            conv_rows_remember_kernel<bf16_t><<<rgrid, 256, 0, stream>>>((const bf16_t*)h, taps, state, cu_q, seq_slot, H);
        CPMCU_LAUNCH_CHECK("conv_rows_remember");
    }
    return nullptr;
}

template <typename AT, typename FT, typename OT, int V>
__global__ __launch_bounds__(256) void add_rows_kernel(float* __restrict__ X, const AT* __restrict__ a, int a_parts,
                                                       long a_stride, const float* __restrict__ a_bias,
                                                       const FT* __restrict__ f, int f_parts, long f_stride,
                                                       const float* __restrict__ f_bias, OT* __restrict__ out, long ld_out,
                                                       long total, int H) {
    for (long i = V * ((long)blockIdx.x * 256 + threadIdx.x); i < total; i += V * (long)gridDim.x * 256) {
        const long t = i / H;
        const int c = (int)(i - t * H);
        Cols<V> x = load_cols<V>(X + i);
        if (a) {
            const Cols<V> v = sum_cols<V>(a + i, a_parts, a_stride);
#pragma unroll
            for (int e = 0; e < V; ++e) x.v[e] += v.v[e] + (a_bias ? a_bias[c + e] : 0.f);
        }
        if (f) {
            const Cols<V> v = sum_cols<V>(f + i, f_parts, f_stride);
#pragma unroll
            for (int e = 0; e < V; ++e) x.v[e] += v.v[e] + (f_bias ? f_bias[c + e] : 0.f);
        }
        if (a || f) store_cols(X + i, x);
        if (out) store_cols(out + t * ld_out + c, x);
    }
}

extern "C" const char* cpmcu_add_rows(float* X, const void* a, int a_dtype, int a_parts, long a_stride, const float* a_bias,
                                      const void* f, int f_dtype, int f_parts, long f_stride, const float* f_bias, void* out,
                                      int out_dtype, long ld_out, int n, int H, hipStream_t stream) {
    CPMCU_REQUIRE(n > 0 && H > 0 && X && (a || f || out), "add_rows: empty shape");
    CPMCU_REQUIRE((!a || a_parts >= 1) && (!f || f_parts >= 1) && (!out || ld_out >= H), "add_rows: bad branch or output rows");
    const int ad = a ? a_dtype : CPMCU_F32, fd = f ? f_dtype : CPMCU_F32, od = out ? out_dtype : CPMCU_F32;
    const bool vec = H % 4 == 0 && aligned16r(X) && (!a || (aligned16r(a) && a_stride % 4 == 0)) &&
                     (!f || (aligned16r(f) && f_stride % 4 == 0)) && (!out || (aligned16r(out) && ld_out % 4 == 0));
    const long total = (long)n * H, work = vec ? total / 4 : total;
    const int blocks = (int)((work + 255) / 256 < 8192 ? (work + 255) / 256 : 8192);
#define LAUNCH(AT, FT, OT)                                                                                              \
    do {                                                                                                                \
        if (vec) add_rows_kernel<AT, FT, OT, 4><<<blocks, 256, 0, stream>>>(X, (const AT*)a, a_parts, a_stride, a_bias,   \
                                                                            (const FT*)f, f_parts, f_stride, f_bias,     \
                                                                            (OT*)out, ld_out, total, H);                 \
        else add_rows_kernel<AT, FT, OT, 1><<<blocks, 256, 0, stream>>>(X, (const AT*)a, a_parts, a_stride, a_bias,      \
                                                                        (const FT*)f, f_parts, f_stride, f_bias,         \
                                                                        (OT*)out, ld_out, total, H);                     \
    } while (0)
#define BY_OUT(AT, FT)                                  \
    do {                                                \
        if (od == CPMCU_F32) LAUNCH(AT, FT, float);     \
        else LAUNCH(AT, FT, bf16_t);                    \
    } while (0)
    CPMCU_REQUIRE((od == CPMCU_F32 || od == CPMCU_BF16) && ad >= 0 && ad <= 1 && fd >= 0 && fd <= 1, "add_rows: unknown dtypes");
    if (ad == CPMCU_F32 && fd == CPMCU_F32) BY_OUT(float, float);
    else if (ad == CPMCU_F32) BY_OUT(float, bf16_t);
    else if (fd == CPMCU_F32) BY_OUT(bf16_t, float);
    else BY_OUT(bf16_t, bf16_t);
#undef BY_OUT
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("add_rows");
    return nullptr;
}

template <typename ZT, typename T>
__global__ __launch_bounds__(256) void gated_lookup_kernel(const ZT* __restrict__ z, int parts, long stride,
                                                           const T* __restrict__ table, long ld_table, long off,
                                                           const int* __restrict__ ids, T* __restrict__ out, long total,
                                                           int D, int act) {
    for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < total; i += (long)gridDim.x * 256) {
        const long t = i / D;
        const int j = (int)(i - t * D);
        float v = 0.f;
        for (int p = 0; p < parts; ++p) v += to_f32(z[(long)p * stride + i]);
        out[i] = from_f32<T>(gate_act(v, act) * to_f32(table[(long)ids[t] * ld_table + off + j]));
    }
}

extern "C" const char* cpmcu_gated_lookup(const void* z, int z_dtype, int parts, long stride, const void* table, int dtype,
                                          long ld_table, long off, const int* ids, void* out, int n, int D, int act,
                                          hipStream_t stream) {
    CPMCU_REQUIRE(n > 0 && D > 0 && parts >= 1 && off >= 0 && off + D <= ld_table, "gated_lookup: %d columns from %ld of rows of %ld", D, off, ld_table);
    CPMCU_REQUIRE(act == CPMCU_ACT_SILU || act == CPMCU_ACT_GELU_TANH, "gated_lookup: unknown nonlinearity %d", act);
    const long total = (long)n * D;
    const int blocks = (int)((total + 255) / 256 < 8192 ? (total + 255) / 256 : 8192);
#define LAUNCH(ZT, T)                                                                                                \
    gated_lookup_kernel<ZT, T><<<blocks, 256, 0, stream>>>((const ZT*)z, parts, stride, (const T*)table, ld_table, off, \
                                                           ids, (T*)out, total, D, act)
    if (z_dtype == CPMCU_F32 && dtype == CPMCU_F32) LAUNCH(float, float);
    else if (z_dtype == CPMCU_F32 && dtype == CPMCU_BF16) LAUNCH(float, bf16_t);
    else if (z_dtype == CPMCU_BF16 && dtype == CPMCU_BF16) LAUNCH(bf16_t, bf16_t);
    else CPMCU_FAIL("gated_lookup: unsupported dtypes z=%d table=%d", z_dtype, dtype);
#undef LAUNCH
    CPMCU_LAUNCH_CHECK("gated_lookup");
    return nullptr;
}

// The product and the lookup of a decode step in one launch: a workgroup owns a strip of 16 columns over all of K, its NW
// wavefronts take a contiguous share of the 128-column blocks each (weight tiled as for the other strip kernels: [strip
// of 16 rows][128-column block][i][lane][8], zero padded), add up through LDS, and the first one finishes.
typedef __bf16 rbf16x8_t __attribute__((ext_vector_type(8)));
typedef float rfloatx4_t __attribute__((ext_vector_type(4)));

template <int PF, int NW>
__global__ __launch_bounds__(NW * 64) void lookup_strip_kernel(const bf16_t* __restrict__ A, const bf16_t* __restrict__ W, int M,
                                                               int D, int K, const bf16_t* __restrict__ table, long ld_table,
                                                               long off, const int* __restrict__ ids,
                                                               bf16_t* __restrict__ out, int act) {
    __shared__ float red[NW - 1][4][64];
    const int strip = blockIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
    const int lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
    const int nkb = (K + 127) / 128, per_wave = (nkb + NW - 1) / NW;
    const int kb0 = wave * per_wave, kb1 = min(kb0 + per_wave, nkb);
    const bf16_t* wp = W + (long)strip * nkb * 2048 + lane * 8;
    const bf16_t* ap = A + (long)min(r, M - 1) * K;             // rows beyond the step repeat its last token
    const int col = strip * 16 + 4 * g;
    // what the end needs is asked for first: the table's numbers of this lane's token and columns
    float e[4];
    const bf16_t* tp = table + (long)ids[min(r, M - 1)] * ld_table + off;
#pragma unroll
    for (int i = 0; i < 4; ++i) e[i] = to_f32(tp[min(col + i, D - 1)]);
    rfloatx4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int kb = kb0; kb < kb1; kb += PF) {
        // a block beyond the wavefront's last repeats the matrix's last and is not multiplied; columns beyond K repeat
        // the row's last 8 and meet the weight's zero padding
        rbf16x8_t wv[PF][4], av[PF][4];
#pragma unroll
        for (int j = 0; j < PF; ++j) {
            const int kbc = min(kb + j, nkb - 1);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                wv[j][i] = *(const rbf16x8_t*)(wp + ((long)kbc * 4 + i) * 512);
                av[j][i] = *(const rbf16x8_t*)(ap + min(kbc * 128 + i * 32 + g * 8, K - 8));
            }
        }
#pragma unroll
        for (int j = 0; j < PF; ++j)
            if (kb + j < kb1) {
#pragma unroll
                for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[j][i], av[j][i], acc, 0, 0, 0);
            }
    }
    if (wave > 0) {
#pragma unroll
        for (int i = 0; i < 4; ++i) red[wave - 1][i][lane] = acc[i];
    }
    __syncthreads();
    if (wave > 0 || r >= M) return;
    // lane (token r, g): acc[i] is column 16 * strip + 4g + i
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        float z = acc[i];
#pragma unroll
        for (int w = 0; w < NW - 1; ++w) z += red[w][i][lane];
        if (col + i < D) out[(long)r * D + col + i] = f32_to_bf16(gate_act(z, act) * e[i]);
    }
}

extern "C" const char* cpmcu_lookup_strip(const void* A, const void* W, int M, int D, int K, const void* table, long ld_table,
                                          long off, const int* ids, void* out, int act, hipStream_t stream) {
    CPMCU_REQUIRE(M > 0 && M <= 16, "lookup_strip: %d tokens (1..16 are taken)", M);
    CPMCU_REQUIRE(D > 0 && K > 0 && K % 8 == 0 && off >= 0 && off + D <= ld_table, "lookup_strip: %d columns, K=%d (a multiple of 8)", D, K);
    CPMCU_REQUIRE(A && W && table && ids && out && (uintptr_t)A % 16 == 0 && (uintptr_t)W % 16 == 0, "lookup_strip: operands must be 16-byte aligned");
    CPMCU_REQUIRE(act == CPMCU_ACT_SILU || act == CPMCU_ACT_GELU_TANH, "lookup_strip: unknown nonlinearity %d", act);
    lookup_strip_kernel<4, 8><<<(D + 15) / 16, 512, 0, stream>>>((const bf16_t*)A, (const bf16_t*)W, M, D, K, (const bf16_t*)table,
                                                               ld_table, off, ids, (bf16_t*)out, act);
    CPMCU_LAUNCH_CHECK("lookup_strip");
    return nullptr;
}
