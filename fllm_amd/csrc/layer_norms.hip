// Layer norms (the mean taken off first, no bias) and the small passes of designs that use them.  All arithmetic is float32; the
// element type only says how operands are stored.  A row's result depends on that row alone: sums run in a fixed order.
//
//   layernorm         out = (x - mean) * rsqrt(mean (x - mean)^2 + eps) * w, of every row or of the rows named; with a second
//                     weight vector (and eps) both norms of a row in one pass.
//   layernorm_conv    the same for steps of one row a segment, the first norm through a short convolution over time on its way.
//   normed_pair_sum   out (+)= a x / rms(x) wx + b y / rms(y) wy.
//   cast_rows, softcap, gelu_side: a stream's rows in the compute type; cap * tanh(x / cap); gelu(z) times a part of the rows'
//                     tokens' rows in a table.
//   side_gate         gelu_side of z = W x in one kernel, for steps of few rows.
#include "api.h"
#include "common.h"

namespace {

constexpr int kBlock = 256;
constexpr int kWaves = kBlock / kWave;
constexpr int kMaxKeep = 15;

// N > 0: the row (at most N * kBlock values) stays in registers between the mean, the deviations and the output; 0: any width
template <typename T, int N>
__global__ void __launch_bounds__(kBlock)
layernorm_kernel(const float *__restrict__ x, const int32_t *__restrict__ rows, const float *__restrict__ w1, float eps1, T *__restrict__ out1,
                 const float *__restrict__ w2, float eps2, T *__restrict__ out2, int width) {
    __shared__ float scratch[kWaves];
    const size_t i = blockIdx.x;
    const float *src = x + (rows ? (size_t)rows[i] : i) * width;
    T *d1 = out1 + i * width, *d2 = out2 == nullptr ? nullptr : out2 + i * width;
    if constexpr (N > 0) {
        float v[N];
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < N; j++) {
            const int c = threadIdx.x + j * kBlock;
            v[j] = c < width ? src[c] : 0.f;
            sum += v[j];
        }
        const float mean = block_sum<kWaves>(sum, scratch) / (float)width;
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < N; j++) {
            v[j] -= mean;
            if (threadIdx.x + j * kBlock < width) ss = fmaf(v[j], v[j], ss);
        }
        const float var = block_sum<kWaves>(ss, scratch) / (float)width;
        const float inv1 = 1.0f / sqrtf(var + eps1), inv2 = 1.0f / sqrtf(var + eps2);
#pragma unroll
        for (int j = 0; j < N; j++) {
            const int c = threadIdx.x + j * kBlock;
            if (c >= width) break;
            d1[c] = from_f32<T>(v[j] * (inv1 * w1[c]));
            if (d2 != nullptr) d2[c] = from_f32<T>(v[j] * (inv2 * w2[c]));
        }
    } else {
        float sum = 0.f;
        for (int c = threadIdx.x; c < width; c += kBlock) sum += src[c];
        const float mean = block_sum<kWaves>(sum, scratch) / (float)width;
        float ss = 0.f;
        for (int c = threadIdx.x; c < width; c += kBlock) {
            const float d = src[c] - mean;
            ss = fmaf(d, d, ss);
        }
        const float var = block_sum<kWaves>(ss, scratch) / (float)width;
        const float inv1 = 1.0f / sqrtf(var + eps1), inv2 = 1.0f / sqrtf(var + eps2);
        for (int c = threadIdx.x; c < width; c += kBlock) {
            const float d = src[c] - mean;
            d1[c] = from_f32<T>(d * (inv1 * w1[c]));
            if (d2 != nullptr) d2[c] = from_f32<T>(d * (inv2 * w2[c]));
        }
    }
}

// grid (rows, blocks of kBlock channels): every workgroup of a row sums the row itself, in layernorm_kernel's order, so that no
// thread loops over channels behind the sums and all it reads is on its way at once.  The first norm's value is rounded to T before
// the convolution, as layernorm_kernel's output is.  A thread owns a channel of the state: it reads the old entries before it
// writes any.
template <typename T, int N>
__global__ void __launch_bounds__(kBlock)
layernorm_conv_kernel(const float *__restrict__ x, const float *__restrict__ w1, float eps1, const float *__restrict__ conv, int taps,
                      T *__restrict__ state, const int32_t *__restrict__ row_seg, const int32_t *__restrict__ slots, T *__restrict__ out1,
                      const float *__restrict__ w2, float eps2, T *__restrict__ out2, int width) {
    __shared__ float scratch[kWaves];
    const int r = blockIdx.x, c = blockIdx.y * kBlock + threadIdx.x;
    const bool mine = c < width;
    T *d1 = out1 + (size_t)r * width, *d2 = out2 == nullptr ? nullptr : out2 + (size_t)r * width;
    const int seg = row_seg[r];
    if (seg < 0) {      // padding row
        if (mine) d1[c] = from_f32<T>(0.f);
        if (mine && d2 != nullptr) d2[c] = from_f32<T>(0.f);
        return;
    }
    const int keep = taps - 1;
    T *old = state + (size_t)slots[seg] * keep * width;
    const float *wc = conv + (size_t)c * taps;
    T held[kMaxKeep];
#pragma unroll
    for (int i = 0; i < kMaxKeep; i++)
        if (i < keep && mine) held[i] = old[(size_t)i * width + c];
    const float *src = x + (size_t)r * width;
    const float own = mine ? src[c] : 0.f, a1 = mine ? w1[c] : 0.f, a2 = mine && d2 != nullptr ? w2[c] : 0.f;
    float v[N];
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < N; j++) {
        const int at = threadIdx.x + j * kBlock;
        v[j] = at < width ? src[at] : 0.f;
        sum += v[j];
    }
    const float mean = block_sum<kWaves>(sum, scratch) / (float)width;
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < N; j++) {
        v[j] -= mean;
        if (threadIdx.x + j * kBlock < width) ss = fmaf(v[j], v[j], ss);
    }
    const float var = block_sum<kWaves>(ss, scratch) / (float)width;
    if (!mine) return;
    const float inv1 = 1.0f / sqrtf(var + eps1), inv2 = 1.0f / sqrtf(var + eps2);
    const T h = from_f32<T>((own - mean) * (inv1 * a1));
    const float now = to_f32<T>(h);
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < kMaxKeep; i++) {      // oldest input first; entry i moves to i - 1
        if (i >= keep) break;
        acc = fmaf(wc[i], to_f32<T>(held[i]), acc);
        if (i > 0) old[(size_t)(i - 1) * width + c] = held[i];
    }
    if (keep > 0) old[(size_t)(keep - 1) * width + c] = h;
    acc = fmaf(wc[keep], now, acc);
    d1[c] = from_f32<T>(now + acc);
    if (d2 != nullptr) d2[c] = from_f32<T>((own - mean) * (inv2 * a2));
}

__global__ void __launch_bounds__(kBlock)
normed_pair_sum_kernel(float *__restrict__ out, const float *__restrict__ x, const float *__restrict__ wx, float a, const float *__restrict__ y,
                       const float *__restrict__ wy, float b, float eps, int width, int accumulate) {
    __shared__ float scratch[kWaves];
    const size_t r = blockIdx.x;
    const float *xr = x + r * width, *yr = y + r * width;
    float *dst = out + r * width;
    float sx = 0.f, sy = 0.f;
#pragma unroll 4
    for (int c = threadIdx.x; c < width; c += kBlock) {
        const float u = xr[c], v = yr[c];
        sx = fmaf(u, u, sx);
        sy = fmaf(v, v, sy);
    }
    sx = block_sum<kWaves>(sx, scratch);
    sy = block_sum<kWaves>(sy, scratch);
    const float fx = a / sqrtf(sx / (float)width + eps), fy = b / sqrtf(sy / (float)width + eps);
#pragma unroll 4
    for (int c = threadIdx.x; c < width; c += kBlock) {
        const float v = xr[c] * fx * wx[c] + yr[c] * fy * wy[c];
        dst[c] = accumulate ? dst[c] + v : v;
    }
}

template <typename T>
__global__ void __launch_bounds__(kBlock) cast_rows_kernel(const float *__restrict__ x, T *__restrict__ out, size_t total) {
    for (size_t i = blockIdx.x * (size_t)kBlock + threadIdx.x; i < total; i += (size_t)gridDim.x * kBlock) out[i] = from_f32<T>(x[i]);
}

__global__ void __launch_bounds__(kBlock) softcap_kernel(float *__restrict__ x, size_t total, float cap) {
    for (size_t i = blockIdx.x * (size_t)kBlock + threadIdx.x; i < total; i += (size_t)gridDim.x * kBlock) x[i] = cap * tanhf(x[i] / cap);
}

__device__ __forceinline__ float gelu_tanh(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

__device__ __forceinline__ void load8(const float *p, float (&v)[8]) {
    *(f32x4_t *)v = *(const f32x4_t *)p;
    *(f32x4_t *)(v + 4) = *(const f32x4_t *)(p + 4);
}

__device__ __forceinline__ void load8(const bf16_t *p, float (&v)[8]) {
    const bf16x8_t a = *(const bf16x8_t *)p;
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] = (float)a[e];
}

template <typename T>
__global__ void __launch_bounds__(kBlock)
gelu_side_kernel(const T *__restrict__ z, const int32_t *__restrict__ ids, const T *__restrict__ table, int vocab, int table_width, int offset,
                 T *__restrict__ out, int rows, int dim) {
    for (size_t i = blockIdx.x * (size_t)kBlock + threadIdx.x; i < (size_t)rows * dim; i += (size_t)gridDim.x * kBlock) {
        const size_t r = i / dim;
        const int c = (int)(i - r * dim);
        int id = ids[r];
        id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);      // ids are validated on the host; never read outside the table
        out[i] = from_f32<T>(gelu_tanh(to_f32<T>(z[i])) * to_f32<T>(table[(size_t)id * table_width + offset + c]));
    }
}

// One workgroup an output lane d: z = W[d] . x for the R rows of the step (x rounded to T first, as cast_rows gives it), then
// gelu_side of it.  dims that are multiples of 8 lie side by side in 16-byte loads.
template <typename T, int R>
__global__ void __launch_bounds__(kBlock)
side_gate_kernel(const float *__restrict__ x, const T *__restrict__ w, const int32_t *__restrict__ ids, const T *__restrict__ table, int vocab,
                 int table_width, int offset, T *__restrict__ out, int rows, int width, int dim) {
    __shared__ float part[kWaves][R];
    const int d = blockIdx.x, lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const T *wr = w + (size_t)d * width;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.f;
    for (int c0 = threadIdx.x * 8; c0 < width; c0 += kBlock * 8) {
        float wv[8];
        load8(wr + c0, wv);
#pragma unroll
        for (int r = 0; r < R; r++) {
            const float *xr = x + (size_t)(r < rows ? r : 0) * width + c0;
            const f32x4_t a = *(const f32x4_t *)xr, b = *(const f32x4_t *)(xr + 4);
#pragma unroll
            for (int e = 0; e < 4; e++) acc[r] = fmaf(wv[e], to_f32<T>(from_f32<T>(a[e])), acc[r]);
#pragma unroll
            for (int e = 0; e < 4; e++) acc[r] = fmaf(wv[4 + e], to_f32<T>(from_f32<T>(b[e])), acc[r]);
        }
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
        acc[r] = wave_sum(acc[r]);
        if (lane == 0) part[wave][r] = acc[r];
    }
    const int r = threadIdx.x;
    float e = 0.f;
    if (r < rows) {
        int id = ids[r];
        id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);      // ids are validated on the host; never read outside the table
        e = to_f32<T>(table[(size_t)id * table_width + offset + d]);
    }
    __syncthreads();
    if (r >= rows) return;
    float z = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; w++) z += part[w][r];
    out[(size_t)r * dim + d] = from_f32<T>(gelu_tanh(z) * e);
}

int small_grid(size_t total) {
    const size_t blocks = (total + kBlock - 1) / kBlock;
    return (int)(blocks < 4096 ? (blocks ? blocks : 1) : 4096);
}

template <typename T>
void launch_layernorm(const float *x, const int32_t *rows, const float *w1, float eps1, T *out1, const float *w2, float eps2, T *out2, int count,
                      int width, hipStream_t stream) {
#define FLLM_LN(N) hipLaunchKernelGGL((layernorm_kernel<T, N>), dim3(count), dim3(kBlock), 0, stream, x, rows, w1, eps1, out1, w2, eps2, out2, width)
    if (width <= 4 * kBlock) FLLM_LN(4);
    else if (width <= 8 * kBlock) FLLM_LN(8);
    else if (width <= 32 * kBlock) FLLM_LN(32);
    else FLLM_LN(0);
#undef FLLM_LN
}

}  // namespace

extern "C" int fllm_layernorm(const float *x, const int32_t *rows, const float *w1, float eps1, void *out1, const float *w2, float eps2, void *out2,
                              int count, int width, int out_dtype, hipStream_t stream) {
    FLLM_REQUIRE(count >= 0 && width > 0, "layernorm: bad sizes count=%d width=%d", count, width);
    FLLM_REQUIRE(x && w1 && out1 && ((w2 == nullptr) == (out2 == nullptr)) && eps1 > 0.f && (w2 == nullptr || eps2 > 0.f), "layernorm: operands missing");
    if (count == 0) return 0;
    if (out_dtype == FLLM_F32) launch_layernorm<float>(x, rows, w1, eps1, (float *)out1, w2, eps2, (float *)out2, count, width, stream);
    else if (out_dtype == FLLM_BF16) launch_layernorm<bf16_t>(x, rows, w1, eps1, (bf16_t *)out1, w2, eps2, (bf16_t *)out2, count, width, stream);
    else FLLM_REQUIRE(false, "layernorm: unknown dtype %d", out_dtype);
    return fllm_check_launch("layernorm");
}

extern "C" int fllm_layernorm_conv(const float *x, const float *w1, float eps1, const float *conv, int taps, void *state, const int32_t *row_seg,
                                   const int32_t *slots, void *out1, const float *w2, float eps2, void *out2, int rows, int width, int out_dtype,
                                   hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && width > 0 && width <= 32 * kBlock && taps >= 1 && taps - 1 <= kMaxKeep, "layernorm_conv: bad sizes");
    FLLM_REQUIRE(x && w1 && conv && (state || taps == 1) && row_seg && slots && out1 && ((w2 == nullptr) == (out2 == nullptr)) && eps1 > 0.f &&
                     (w2 == nullptr || eps2 > 0.f), "layernorm_conv: operands missing");
    if (rows == 0) return 0;
    const dim3 grid(rows, (width + kBlock - 1) / kBlock);
#define FLLM_LNC(T, N)                                                                                                                       \
    hipLaunchKernelGGL((layernorm_conv_kernel<T, N>), grid, dim3(kBlock), 0, stream, x, w1, eps1, conv, taps, (T *)state, row_seg, slots,      \
                       (T *)out1, w2, eps2, (T *)out2, width)
#define FLLM_LNC_N(T)                                       \
    do {                                                    \
        if (width <= 4 * kBlock) FLLM_LNC(T, 4);            \
        else if (width <= 8 * kBlock) FLLM_LNC(T, 8);       \
        else FLLM_LNC(T, 32);                               \
    } while (0)
    if (out_dtype == FLLM_F32) FLLM_LNC_N(float);
    else if (out_dtype == FLLM_BF16) FLLM_LNC_N(bf16_t);
    else FLLM_REQUIRE(false, "layernorm_conv: unknown dtype %d", out_dtype);
#undef FLLM_LNC_N
#undef FLLM_LNC
    return fllm_check_launch("layernorm_conv");
}

// 0: launched; negative: error; 1: declined (more than 8 rows, a width that is no multiple of 8)
extern "C" int fllm_side_gate(const float *x, const void *w, const int32_t *ids, const void *table, int vocab, int table_width, int offset, void *out,
                              int rows, int width, int dim, int dtype, hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && width > 0 && dim > 0 && vocab > 0 && offset >= 0 && offset + dim <= table_width, "side_gate: bad sizes");
    FLLM_REQUIRE(x && w && ids && table && out, "side_gate: operands missing");
    if (rows == 0) return 0;
    if (rows > 8 || width % 8 != 0 || (((uintptr_t)x | (uintptr_t)w) & 15) != 0) return 1;
#define FLLM_SIDE(T, R)                                                                                                                      \
    hipLaunchKernelGGL((side_gate_kernel<T, R>), dim3(dim), dim3(kBlock), 0, stream, x, (const T *)w, ids, (const T *)table, vocab, table_width, \
                       offset, (T *)out, rows, width, dim)
#define FLLM_SIDE_R(T)                            \
    do {                                          \
        if (rows == 1) FLLM_SIDE(T, 1);           \
        else if (rows == 2) FLLM_SIDE(T, 2);      \
        else if (rows <= 4) FLLM_SIDE(T, 4);      \
        else FLLM_SIDE(T, 8);                     \
    } while (0)
    if (dtype == FLLM_F32) FLLM_SIDE_R(float);
    else if (dtype == FLLM_BF16) FLLM_SIDE_R(bf16_t);
    else FLLM_REQUIRE(false, "side_gate: unknown dtype %d", dtype);
#undef FLLM_SIDE_R
#undef FLLM_SIDE
    return fllm_check_launch("side_gate");
}

extern "C" int fllm_normed_pair_sum(float *out, const float *x, const float *wx, float a, const float *y, const float *wy, float b, float eps,
                                    int rows, int width, int accumulate, hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && width > 0 && eps > 0.f, "normed_pair_sum: bad sizes");
    FLLM_REQUIRE(out && x && wx && y && wy, "normed_pair_sum: operands missing");
    if (rows == 0) return 0;
    hipLaunchKernelGGL(normed_pair_sum_kernel, dim3(rows), dim3(kBlock), 0, stream, out, x, wx, a, y, wy, b, eps, width, accumulate);
    return fllm_check_launch("normed_pair_sum");
}

extern "C" int fllm_cast_rows(const float *x, void *out, size_t total, int dtype, hipStream_t stream) {
    FLLM_REQUIRE(x && out, "cast_rows: operands missing");
    if (total == 0) return 0;
    if (dtype == FLLM_F32) hipLaunchKernelGGL(cast_rows_kernel<float>, dim3(small_grid(total)), dim3(kBlock), 0, stream, x, (float *)out, total);
    else if (dtype == FLLM_BF16) hipLaunchKernelGGL(cast_rows_kernel<bf16_t>, dim3(small_grid(total)), dim3(kBlock), 0, stream, x, (bf16_t *)out, total);
    else FLLM_REQUIRE(false, "cast_rows: unknown dtype %d", dtype);
    return fllm_check_launch("cast_rows");
}

extern "C" int fllm_softcap(float *x, size_t total, float cap, hipStream_t stream) {
    FLLM_REQUIRE(x && cap > 0.f, "softcap: bad operands");
    if (total == 0) return 0;
    hipLaunchKernelGGL(softcap_kernel, dim3(small_grid(total)), dim3(kBlock), 0, stream, x, total, cap);
    return fllm_check_launch("softcap");
}

extern "C" int fllm_gelu_side(const void *z, const int32_t *ids, const void *table, int vocab, int table_width, int offset, void *out, int rows,
                              int dim, int dtype, hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && dim > 0 && vocab > 0 && offset >= 0 && offset + dim <= table_width, "gelu_side: bad sizes");
    FLLM_REQUIRE(z && ids && table && out, "gelu_side: operands missing");
    if (rows == 0) return 0;
    const int grid = small_grid((size_t)rows * dim);
    if (dtype == FLLM_F32)
        hipLaunchKernelGGL(gelu_side_kernel<float>, dim3(grid), dim3(kBlock), 0, stream, (const float *)z, ids, (const float *)table, vocab,
                           table_width, offset, (float *)out, rows, dim);
    else if (dtype == FLLM_BF16)
        hipLaunchKernelGGL(gelu_side_kernel<bf16_t>, dim3(grid), dim3(kBlock), 0, stream, (const bf16_t *)z, ids, (const bf16_t *)table, vocab,
                           table_width, offset, (bf16_t *)out, rows, dim);
    else
        FLLM_REQUIRE(false, "gelu_side: unknown dtype %d", dtype);
    return fllm_check_launch("gelu_side");
}
