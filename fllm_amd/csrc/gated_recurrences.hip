// Recurrences whose gates the token itself chooses, plain forms: float32 arithmetic, both element types, any sizes.
//
//   gated_linear_attention  S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t per head, alpha = sigmoid(z + b)^(1 / tau) one
//                           number a key channel; S float32 [dim][vdim] in the sequence's state slot.  Token after token, the
//                           state in registers (values in groups of four lanes) or in LDS (any sizes).
//   min_recurrence          S_t = (1 - z) S_(t-1) + z c lane by lane, z = sigmoid(a + b_z), c = u + 1/2 where u = x + b_x >= 0 and
//                           sigmoid(u) below; out = S silu(g).  Segments in parts of 64 tokens side by side.
//
// A row's result depends on its own sequence alone, never on the rest of the batch.
#include "api.h"
#include "common.h"
#include "segment_parts.h"

int fllm_gated_linear_chunked(const void *q, const void *k, const void *v, int ld, const float *z, const float *bias, float inv_tau,
                              float query_scale, float *state, const int32_t *row_seg, const int32_t *seg_start, const int32_t *slots,
                              int num_segs, float *out, int rows, int heads, int dim, int vdim, int dtype, float *carried,
                              hipStream_t stream);   // gated_linear_mfma.hip; 1: sizes declined

namespace {

constexpr int kBlock = 256;
constexpr int kWaves = kBlock / kWave;

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
// sigmoid(z)^(1 / tau) through its logarithm: -softplus(-z) / tau, which neither overflows nor loses small decays
__device__ __forceinline__ float decay_of(float z, float inv_tau) {
    return expf(-(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * inv_tau);
}

// ---- gated linear attention ------------------------------------------------------------------------------------------------
// One workgroup a (segment, head, slice of VB value lanes), the slice of the state in LDS: thread (g, j) owns rows g, g + G, ..
// of column j.
template <typename T>
__global__ void __launch_bounds__(kBlock)
gated_linear_kernel(const T *__restrict__ q, const T *__restrict__ k, const T *__restrict__ v, int ld, const float *__restrict__ z,
                    const float *__restrict__ bias, float inv_tau, float query_scale, float *__restrict__ state,
                    const int32_t *__restrict__ row_seg, const int32_t *__restrict__ seg_start, const int32_t *__restrict__ slots,
                    float *__restrict__ out, int heads, int dim, int vdim, int VB) {
    extern __shared__ float smem[];
    const int G = kBlock / VB;
    float *S = smem;                    // dim * VB
    float *qs = S + (size_t)dim * VB;   // dim
    float *ks = qs + dim;               // dim
    float *as = ks + dim;               // dim
    float *part = as + dim;             // G * VB
    const int seg = blockIdx.x, h = blockIdx.y, j0 = blockIdx.z * VB;
    const int r0 = seg_start[seg], n = seg_start[seg + 1] - r0;
    if (n <= 0) return;
    const int j = threadIdx.x % VB, g = threadIdx.x / VB;
    const bool live = j0 + j < vdim;
    if (row_seg[r0] < 0) {   // padding rows: no state is touched
        if (g == 0 && live)
            for (int t = 0; t < n; t++) out[((size_t)(r0 + t) * heads + h) * vdim + j0 + j] = 0.f;
        return;
    }
    float *mine = state + ((size_t)slots[seg] * heads + h) * dim * vdim;
    for (int i = g; i < dim; i += G) S[i * VB + j] = live ? mine[(size_t)i * vdim + j0 + j] : 0.f;
    for (int t = 0; t < n; t++) {
        const size_t row = (size_t)(r0 + t) * ld, zrow = ((size_t)(r0 + t) * heads + h) * dim;
        __syncthreads();      // the step before has read qs, ks, as and part
        for (int c = threadIdx.x; c < dim; c += kBlock) {
            qs[c] = to_f32<T>(q[row + (size_t)h * dim + c]) * query_scale;
            ks[c] = to_f32<T>(k[row + (size_t)h * dim + c]);
            as[c] = decay_of(z[zrow + c] + bias[h * dim + c], inv_tau);
        }
        const float vj = live ? to_f32<T>(v[row + (size_t)h * vdim + j0 + j]) : 0.f;
        __syncthreads();
        float acc = 0.f;
        for (int i = g; i < dim; i += G) {
            const float s = fmaf(S[i * VB + j], as[i], ks[i] * vj);
            S[i * VB + j] = s;
            acc = fmaf(s, qs[i], acc);
        }
        part[g * VB + j] = acc;
        __syncthreads();
        if (g == 0 && live) {
            float o = part[j];
            for (int a = 1; a < G; a++) o += part[a * VB + j];
            out[((size_t)(r0 + t) * heads + h) * vdim + j0 + j] = o;
        }
    }
    if (live)
        for (int i = g; i < dim; i += G) mine[(size_t)i * vdim + j0 + j] = S[i * VB + j];
}

// The same with the state in registers, for values in groups of four lanes and keys of up to 32 * RP lanes: one workgroup a
// (segment, head, slice of 32 value lanes), thread (g, j4) owns rows g, g + 32, .. of the four columns at 4 * j4.  The state is
// read once and written once behind the segment's last token; the sum over the rows is taken over the lanes of a wave and then
// over the four waves, in an order that no size of the batch changes.
constexpr int kRowsVB = 32;
template <typename T, int RP>
__global__ void __launch_bounds__(kBlock)
gated_linear_rows_kernel(const T *__restrict__ q, const T *__restrict__ k, const T *__restrict__ v, int ld, const float *__restrict__ z,
                         const float *__restrict__ bias, float inv_tau, float query_scale, float *__restrict__ state,
                         const int32_t *__restrict__ row_seg, const int32_t *__restrict__ seg_start, const int32_t *__restrict__ slots,
                         float *__restrict__ out, int heads, int dim, int vdim) {
    constexpr int G = kBlock / (kRowsVB / 4);      // 32 groups of rows
    __shared__ float qs[G * RP], ks[G * RP], as[G * RP];
    __shared__ f32x4_t part[kWaves][kRowsVB / 4];
    const int seg = blockIdx.x, h = blockIdx.y, j0 = blockIdx.z * kRowsVB;
    const int r0 = seg_start[seg], n = seg_start[seg + 1] - r0;
    if (n <= 0) return;
    const int tid = threadIdx.x, j4 = tid & 7, g = tid >> 3;
    const int col = j0 + 4 * j4;
    const bool live = col < vdim;
    const size_t out_ld = (size_t)heads * vdim;
    if (row_seg[r0] < 0) {   // padding rows: no state is touched
        if (g == 0 && live)
            for (int t = 0; t < n; t++) *(f32x4_t *)(out + (size_t)(r0 + t) * out_ld + (size_t)h * vdim + col) = f32x4_t{0.f, 0.f, 0.f, 0.f};
        return;
    }
    float *mine = state + ((size_t)slots[seg] * heads + h) * dim * vdim;
    f32x4_t S[RP];
#pragma unroll
    for (int p = 0; p < RP; p++) {
        const int i = g + G * p;
        S[p] = (live && i < dim) ? *(const f32x4_t *)(mine + (size_t)i * vdim + col) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    for (int t = 0; t < n; t++) {
        const size_t row = (size_t)(r0 + t) * ld, zrow = ((size_t)(r0 + t) * heads + h) * dim;
        if (t > 0) __syncthreads();      // the token before has read qs, ks, as and part
        for (int c = tid; c < dim; c += kBlock) {
            qs[c] = to_f32<T>(q[row + (size_t)h * dim + c]) * query_scale;
            ks[c] = to_f32<T>(k[row + (size_t)h * dim + c]);
            as[c] = decay_of(z[zrow + c] + bias[h * dim + c], inv_tau);
        }
        f32x4_t vv = {0.f, 0.f, 0.f, 0.f};
        if (live)
#pragma unroll
            for (int e = 0; e < 4; e++) vv[e] = to_f32<T>(v[row + (size_t)h * vdim + col + e]);
        __syncthreads();
        f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int p = 0; p < RP; p++) {
            const int i = g + G * p;
            if (i < dim) {
                const float kk = ks[i], qq = qs[i], aa = as[i];
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const float s = fmaf(S[p][e], aa, kk * vv[e]);
                    S[p][e] = s;
                    acc[e] = fmaf(s, qq, acc[e]);
                }
            }
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {      // the eight row groups of a wave: lanes 8, 16 and 32 apart hold the same columns
            acc[e] += __shfl_xor(acc[e], 8, kWave);
            acc[e] += __shfl_xor(acc[e], 16, kWave);
            acc[e] += __shfl_xor(acc[e], 32, kWave);
        }
        if ((tid & (kWave - 1)) < 8) part[tid / kWave][j4] = acc;
        __syncthreads();
        if (tid < 8 && live) {
            f32x4_t o = part[0][tid];
#pragma unroll
            for (int a = 1; a < kWaves; a++) o += part[a][tid];
            *(f32x4_t *)(out + (size_t)(r0 + t) * out_ld + (size_t)h * vdim + col) = o;
        }
    }
    if (live)
#pragma unroll
        for (int p = 0; p < RP; p++) {
            const int i = g + G * p;
            if (i < dim) *(f32x4_t *)(mine + (size_t)i * vdim + col) = S[p];
        }
}

// ---- minGRU ---------------------------------------------------------------------------------------------------------------------
// A token is the map S -> a S + b with a = 1 - z, b = z c, and maps compose: a part of 64 tokens is one map a lane.  A workgroup
// takes 64 lanes (one a thread of a wave) of one part; its four waves take 16 tokens each, hold their maps in registers, and
// meet in LDS.  Steps whose segments may be longer than a part run two kernels: the first leaves every part's map (and the
// state before the segment) in `carried`, the second folds the maps before its part, runs its tokens and writes the outputs; the
// last part writes the state.
constexpr int kMinPart = 64;
constexpr int kMinRun = kMinPart / kWaves;      // tokens a wave

template <typename T>
struct MinOperands {
    const T *zxg;
    int ld;
    const float *bias;
    float *state;
    const int32_t *row_seg, *seg_start, *slots;
    int num_segs, width;
    float *carried;      // [part index][3][width]: a, b, and in a segment's first part the state before the segment
};

template <typename T>
__device__ __forceinline__ void min_maps(const MinOperands<T> &p, int r, int n, int c, float (&a)[kMinRun], float (&b)[kMinRun]) {
    const float bz = p.bias[c], bx = p.bias[p.width + c];
    T zs[kMinRun], us[kMinRun];
#pragma unroll
    for (int t = 0; t < kMinRun; t++)
        if (t < n) {
            zs[t] = p.zxg[(size_t)(r + t) * p.ld + c];
            us[t] = p.zxg[(size_t)(r + t) * p.ld + p.width + c];
        }
#pragma unroll
    for (int t = 0; t < kMinRun; t++) {
        a[t] = 1.f, b[t] = 0.f;
        if (t < n) {
            const float zr = to_f32<T>(zs[t]) + bz, u = to_f32<T>(us[t]) + bx;
            const float z = sigmoid_f(zr);
            a[t] = sigmoid_f(-zr);      // 1 - z without its cancellation
            b[t] = z * (u >= 0.f ? u + 0.5f : sigmoid_f(u));
        }
    }
}

template <typename T>
__global__ void __launch_bounds__(kBlock)
min_part_kernel(const MinOperands<T> p) {
    __shared__ float sa[kWaves][kWave], sb[kWaves][kWave];
    int seg, part;
    find_part<kMinPart>(blockIdx.x, p.seg_start, p.num_segs, seg, part);
    const int seg_r0 = p.seg_start[seg], seg_n = p.seg_start[seg + 1] - seg_r0;
    if (part < 0 || seg_n <= kMinPart || seg_n <= part * kMinPart || p.row_seg[seg_r0] < 0) return;      // a segment of one part needs no map
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int c = blockIdx.y * kWave + lane;
    const bool live = c < p.width;
    const int first = part * kMinPart + wave * kMinRun;
    int n = seg_n - first;
    n = n < 0 ? 0 : (n > kMinRun ? kMinRun : n);
    float a[kMinRun], b[kMinRun];
    min_maps<T>(p, seg_r0 + first, live ? n : 0, live ? c : 0, a, b);
    float A = 1.f, B = 0.f;
#pragma unroll
    for (int t = 0; t < kMinRun; t++) B = fmaf(a[t], B, b[t]), A *= a[t];
    sa[wave][lane] = A, sb[wave][lane] = B;
    __syncthreads();
    if (wave != 0 || !live) return;
#pragma unroll
    for (int w = 1; w < kWaves; w++) B = fmaf(sa[w][lane], B, sb[w][lane]), A *= sa[w][lane];
    float *dst = p.carried + (size_t)part_index<kMinPart>(seg_r0, seg, part) * 3 * p.width;
    dst[c] = A;
    dst[p.width + c] = B;
    if (part == 0) dst[2 * p.width + c] = p.state[(size_t)p.slots[seg] * p.width + c];
}

template <typename T>
__global__ void __launch_bounds__(kBlock)
min_out_kernel(const MinOperands<T> p, T *__restrict__ out, int in_parts) {
    __shared__ float sa[kWaves][kWave], sb[kWaves][kWave];
    int seg = blockIdx.x, part = 0;
    if (in_parts) find_part<kMinPart>(blockIdx.x, p.seg_start, p.num_segs, seg, part);
    const int seg_r0 = p.seg_start[seg], seg_n = p.seg_start[seg + 1] - seg_r0;
    if (part < 0 || seg_n <= part * kMinPart) return;
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int c = blockIdx.y * kWave + lane;
    const bool live = c < p.width;
    const int first = part * kMinPart + wave * kMinRun;
    int n = seg_n - first;
    n = n < 0 ? 0 : (n > kMinRun ? kMinRun : n);
    if (!live) n = 0;
    const int r = seg_r0 + first;
    if (p.row_seg[seg_r0] < 0) {   // padding rows: no state is touched
        for (int t = 0; t < n; t++) out[(size_t)(r + t) * p.width + c] = from_f32<T>(0.f);
        return;
    }
    float a[kMinRun], b[kMinRun];
    min_maps<T>(p, r, n, live ? c : 0, a, b);
    float A = 1.f, B = 0.f;
#pragma unroll
    for (int t = 0; t < kMinRun; t++) B = fmaf(a[t], B, b[t]), A *= a[t];
    sa[wave][lane] = A, sb[wave][lane] = B;
    T gs[kMinRun];
#pragma unroll
    for (int t = 0; t < kMinRun; t++)
        if (t < n) gs[t] = p.zxg[(size_t)(r + t) * p.ld + 2 * p.width + c];
    float S = 0.f;
    if (live) {
        if (in_parts && seg_n > kMinPart) {
            const float *map = p.carried + (size_t)part_index<kMinPart>(seg_r0, seg, 0) * 3 * p.width;
            S = map[2 * p.width + c];
#pragma unroll 4
            for (int i = 0; i < part; i++, map += 3 * p.width) S = fmaf(map[c], S, map[p.width + c]);
        } else {
            S = p.state[(size_t)p.slots[seg] * p.width + c];
        }
    }
    __syncthreads();      // every wave has read the state, and the maps of all waves are there
    for (int w = 0; w < wave; w++) S = fmaf(sa[w][lane], S, sb[w][lane]);
#pragma unroll
    for (int t = 0; t < kMinRun; t++)
        if (t < n) {
            S = fmaf(a[t], S, b[t]);
            const float g = to_f32<T>(gs[t]);
            out[(size_t)(r + t) * p.width + c] = from_f32<T>(S * g * sigmoid_f(g));
        }
    if (n > 0 && first + n == seg_n) p.state[(size_t)p.slots[seg] * p.width + c] = S;      // the wave that holds the segment's last token
}

}  // namespace

extern "C" int fllm_gated_linear_attention(const void *q, const void *k, const void *v, int ld, const float *z, const float *bias, float tau,
                                           float query_scale, float *state, const int32_t *row_seg, const int32_t *seg_start,
                                           const int32_t *slots, int num_segs, float *out, int rows, int heads, int dim, int vdim, int form,
                                           int dtype, float *carried, hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && num_segs > 0 && ld > 0 && tau > 0.f,
                 "gated_linear_attention: bad sizes");
    FLLM_REQUIRE(q && k && v && z && bias && state && row_seg && seg_start && slots && out, "gated_linear_attention: operands missing");
    FLLM_REQUIRE(form >= 0 && form <= 2, "gated_linear_attention: unknown form %d", form);
    FLLM_REQUIRE(dtype == FLLM_F32 || dtype == FLLM_BF16, "gated_linear_attention: unknown dtype %d", dtype);
    if (rows == 0) return 0;
    const float inv_tau = 1.0f / tau;
    // a step that holds more rows than segments holds portions of prompts: those go over the matrix cores a chunk at a time
    if (form == 2 || (form == 0 && rows > num_segs)) {
        const int declined = fllm_gated_linear_chunked(q, k, v, ld, z, bias, inv_tau, query_scale, state, row_seg, seg_start, slots, num_segs,
                                                       out, rows, heads, dim, vdim, dtype, carried, stream);
        if (!declined) return fllm_check_launch("gated_linear_chunked");
        FLLM_REQUIRE(form != 2, "gated_linear_attention: heads of %d and %d lanes are not the chunked kernel's", dim, vdim);
    }
    if (vdim % 4 == 0 && dim <= 256) {
        const dim3 grid(num_segs, heads, (vdim + kRowsVB - 1) / kRowsVB);
#define FLLM_ROWS(T, RP)                                                                                                              \
    hipLaunchKernelGGL((gated_linear_rows_kernel<T, RP>), grid, dim3(kBlock), 0, stream, (const T *)q, (const T *)k, (const T *)v, ld, \
                       z, bias, inv_tau, query_scale, state, row_seg, seg_start, slots, out, heads, dim, vdim)
#define FLLM_ROWS_OF(T)                                                                                                               \
    do {                                                                                                                              \
        if (dim <= 32) FLLM_ROWS(T, 1);                                                                                               \
        else if (dim <= 64) FLLM_ROWS(T, 2);                                                                                          \
        else if (dim <= 128) FLLM_ROWS(T, 4);                                                                                         \
        else FLLM_ROWS(T, 8);                                                                                                         \
    } while (0)
        if (dtype == FLLM_F32) FLLM_ROWS_OF(float);
        else FLLM_ROWS_OF(bf16_t);
#undef FLLM_ROWS_OF
#undef FLLM_ROWS
        return fllm_check_launch("gated_linear_rows");
    }
    // the widest slice of value lanes whose share of the state fits into LDS beside q, k, the decays and the partial sums
    int VB = 64;
    while (VB / 2 >= vdim && VB > 1) VB >>= 1;
    while (VB > 1 && ((size_t)dim * VB + 3 * (size_t)dim + kBlock) * sizeof(float) > 64 * 1024) VB >>= 1;
    const size_t smem = ((size_t)dim * VB + 3 * (size_t)dim + kBlock) * sizeof(float);
    FLLM_REQUIRE(smem <= 64 * 1024, "gated_linear_attention: keys of %d lanes do not fit into LDS", dim);
    const int slices = (vdim + VB - 1) / VB;
    FLLM_REQUIRE(slices <= 65535, "gated_linear_attention: values of %d lanes are too many", vdim);
    const dim3 grid(num_segs, heads, slices);
    if (dtype == FLLM_F32)
        hipLaunchKernelGGL(gated_linear_kernel<float>, grid, dim3(kBlock), smem, stream, (const float *)q, (const float *)k, (const float *)v, ld,
                           z, bias, inv_tau, query_scale, state, row_seg, seg_start, slots, out, heads, dim, vdim, VB);
    else
        hipLaunchKernelGGL(gated_linear_kernel<bf16_t>, grid, dim3(kBlock), smem, stream, (const bf16_t *)q, (const bf16_t *)k, (const bf16_t *)v,
                           ld, z, bias, inv_tau, query_scale, state, row_seg, seg_start, slots, out, heads, dim, vdim, VB);
    return fllm_check_launch("gated_linear");
}

extern "C" size_t fllm_min_recurrence_carried_floats(int rows, int num_segs, int width) {
    return rows <= kMinPart ? 0 : ((size_t)rows / kMinPart + (size_t)num_segs + 1) * 3 * width;
}

extern "C" int fllm_min_recurrence(const void *zxg, int ld, const float *bias, float *state, const int32_t *row_seg, const int32_t *seg_start,
                                   const int32_t *slots, int num_segs, void *out, int rows, int width, int dtype, float *carried,
                                   hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && width > 0 && num_segs > 0 && ld >= 3 * width, "min_recurrence: bad sizes");
    FLLM_REQUIRE(zxg && bias && state && row_seg && seg_start && slots && out, "min_recurrence: operands missing");
    const int in_parts = rows > kMinPart && rows > num_segs ? 1 : 0;      // otherwise no segment is longer than a part
    FLLM_REQUIRE(!in_parts || carried, "min_recurrence: parts of segments need room for what they hand on");
    const int blocks = (width + kWave - 1) / kWave;
    FLLM_REQUIRE(blocks <= 65535, "min_recurrence: a width of %d is too large", width);
    if (rows == 0) return 0;
    const dim3 grid(in_parts ? (unsigned)(rows / kMinPart + num_segs) : (unsigned)num_segs, blocks);
#define FLLM_MIN(T)                                                                                                          \
    do {                                                                                                                     \
        MinOperands<T> p = {(const T *)zxg, ld, bias, state, row_seg, seg_start, slots, num_segs, width, carried};           \
        if (in_parts) hipLaunchKernelGGL(min_part_kernel<T>, grid, dim3(kBlock), 0, stream, p);                              \
        hipLaunchKernelGGL(min_out_kernel<T>, grid, dim3(kBlock), 0, stream, p, (T *)out, in_parts);                         \
    } while (0)
    if (dtype == FLLM_F32) FLLM_MIN(float);
    else if (dtype == FLLM_BF16) FLLM_MIN(bf16_t);
    else FLLM_REQUIRE(false, "min_recurrence: unknown dtype %d", dtype);
#undef FLLM_MIN
    return fllm_check_launch("min_recurrence");
}
