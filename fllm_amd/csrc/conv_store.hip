// Queries, keys and values behind a short convolution over time: rows of a joint product [q | k | v | ..] in; convolved, normed a
// head and rotated queries out, keys (likewise) and values (convolved alone) into the pages.
//
// Channel c of row t is y = sum_j w[c][j] u(t - taps + 1 + j), u the product's value plus the channel's bias, zero before the
// sequence's first token.  Products before the step's first row come from state[slot][i][channel], i = 0 the oldest of the last
// taps - 1; the state holds the products WITHOUT the biases, so that a slot full of zeros needs no special case: whether a tap
// exists is decided by the row's position alone.  The arithmetic is float32 up to the one rounding of what is stored.
#include "api.h"
#include "common.h"

namespace {

constexpr int kBlock = 256;
constexpr int kWaves = kBlock / kWave;
constexpr int kMaxKeep = 15;
constexpr int kMaxPer = 8;      // heads of up to 512 lanes

// grid (rows, heads in fours): a wave takes one head of q, k or v of one row.  `update` (steps of one row a segment): the wave,
// which alone reads its channels of the state, moves them on; otherwise conv_tail_kernel does behind this kernel.
template <typename T>
__global__ void __launch_bounds__(kBlock)
conv_qkv_store_kernel(const T *__restrict__ joint, int ld, const float *__restrict__ conv, int taps, const float *__restrict__ bias,
                      T *__restrict__ state, const float *__restrict__ q_weight, const float *__restrict__ k_weight, float eps,
                      T *__restrict__ q_out, const int32_t *__restrict__ row_pos, const int32_t *__restrict__ row_seg,
                      const int32_t *__restrict__ seg_start, const int32_t *__restrict__ slots, const int32_t *__restrict__ tables,
                      int table_stride, const float *__restrict__ cos_table, const float *__restrict__ sin_table, T *__restrict__ k_pages,
                      T *__restrict__ v_pages, int heads, int kv_heads, int k_dim, int v_dim, int rope_dims, int pairing, int page_size,
                      int key_chunk, int store_kv, int update) {
    extern __shared__ float smem[];
    const int r = blockIdx.x;
    const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
    const int unit = blockIdx.y * kWaves + wave;
    const int seg = row_seg[r];
    if (seg < 0 || unit >= heads + (store_kv ? 2 * kv_heads : 0)) return;   // padding row, or no such head (no barrier below)
    const int pos = row_pos[r];
    const int kind = unit < heads ? 0 : (unit < heads + kv_heads ? 1 : 2);
    const int h = kind == 0 ? unit : (kind == 1 ? unit - heads : unit - heads - kv_heads);
    const int dim = kind == 2 ? v_dim : k_dim;
    const int nq = heads * k_dim, nk = kv_heads * k_dim;
    const int channels = nq + (store_kv ? nk + kv_heads * v_dim : 0);
    const int base = kind == 0 ? h * k_dim : (kind == 1 ? nq + h * k_dim : nq + nk + h * v_dim);
    const int keep = taps - 1, t = r - seg_start[seg];
    T *mine = keep > 0 ? state + (size_t)slots[seg] * keep * channels : nullptr;
    const int page = kind > 0 ? tables[(size_t)seg * table_stride + pos / page_size] : 0, off = pos % page_size;
    float y[kMaxPer];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < kMaxPer; j++) {
        const int c = lane + j * kWave;
        if (c >= dim) break;
        const int ch = base + c;
        const float *w = conv + (size_t)ch * taps;
        const float b = bias != nullptr ? bias[ch] : 0.f;
        const T now = joint[(size_t)r * ld + ch];
        float acc = 0.f;
        if (update) {
            T held[kMaxKeep];
#pragma unroll
            for (int i = 0; i < kMaxKeep; i++)
                if (i < keep) held[i] = mine[(size_t)i * channels + ch];
#pragma unroll
            for (int i = 0; i < kMaxKeep; i++) {      // oldest first; entry i moves to i - 1
                if (i >= keep) break;
                if (pos - (keep - i) >= 0) acc = fmaf(w[i], to_f32<T>(held[i]) + b, acc);
                if (i > 0) mine[(size_t)(i - 1) * channels + ch] = held[i];
            }
            if (keep > 0) mine[(size_t)(keep - 1) * channels + ch] = now;
        } else {
            for (int d = keep; d >= 1; d--) {
                if (pos - d < 0) continue;
                const int at = t - d;
                const float u = at >= 0 ? to_f32<T>(joint[(size_t)(r - d) * ld + ch]) : to_f32<T>(mine[(size_t)(keep + at) * channels + ch]);
                acc = fmaf(w[keep - d], u + b, acc);
            }
        }
        acc = fmaf(w[keep], to_f32<T>(now) + b, acc);
        y[j] = acc;
        ss = fmaf(acc, acc, ss);
    }
    if (kind == 2) {
#pragma unroll
        for (int j = 0; j < kMaxPer; j++) {
            const int c = lane + j * kWave;
            if (c >= dim) break;
            v_pages[(((size_t)page * kv_heads + h) * v_dim + c) * page_size + off] = from_f32<T>(y[j]);
        }
        return;
    }
    const float *weight = kind == 0 ? q_weight : k_weight;
    if (weight != nullptr) {
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
        for (int j = 0; j < kMaxPer; j++) {
            const int c = lane + j * kWave;
            if (c >= dim) break;
            y[j] *= inv * weight[c];
        }
    }
    if (rope_dims > 0) {      // partners sit in other lanes: through the wave's own piece of LDS
        float *buf = smem + (size_t)wave * k_dim;
#pragma unroll
        for (int j = 0; j < kMaxPer; j++) {
            const int c = lane + j * kWave;
            if (c >= dim) break;
            buf[c] = y[j];
        }
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
        const int half = rope_dims / 2;
        const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
#pragma unroll
        for (int j = 0; j < kMaxPer; j++) {
            const int c = lane + j * kWave;
            if (c >= rope_dims) break;
            const bool first = pairing ? (c & 1) == 0 : c < half;
            const int i = pairing ? c >> 1 : (first ? c : c - half);
            const float other = buf[pairing ? c ^ 1 : (first ? c + half : c - half)];
            y[j] = first ? y[j] * cs[i] - other * sn[i] : y[j] * cs[i] + other * sn[i];
        }
    }
#pragma unroll
    for (int j = 0; j < kMaxPer; j++) {
        const int c = lane + j * kWave;
        if (c >= dim) break;
        if (kind == 0) q_out[(size_t)r * nq + base + c] = from_f32<T>(y[j]);
        else k_pages[key_offset_chunked(page, kv_heads, h, page_size, k_dim, off, c, key_chunk)] = from_f32<T>(y[j]);
    }
}

// grid (segments, blocks of channels), behind the rows: the state becomes the last taps - 1 products of the sequence.  A thread
// owns a channel: it reads what it keeps of the old entries before it writes any.
template <typename T>
__global__ void __launch_bounds__(kBlock)
conv_tail_kernel(const T *__restrict__ joint, int ld, T *__restrict__ state, const int32_t *__restrict__ row_seg,
                 const int32_t *__restrict__ seg_start, const int32_t *__restrict__ slots, int channels, int taps) {
    const int seg = blockIdx.x, c = blockIdx.y * kBlock + threadIdx.x;
    const int r0 = seg_start[seg], n = seg_start[seg + 1] - r0;
    if (n <= 0 || row_seg[r0] < 0 || c >= channels) return;
    const int keep = taps - 1;
    T *mine = state + (size_t)slots[seg] * keep * channels;
    T held[kMaxKeep];
#pragma unroll
    for (int i = 0; i < kMaxKeep; i++) {
        if (i >= keep) break;
        const int at = n - keep + i;
        held[i] = at >= 0 ? joint[(size_t)(r0 + at) * ld + c] : mine[(size_t)(keep + at) * channels + c];
    }
#pragma unroll
    for (int i = 0; i < kMaxKeep; i++) {
        if (i >= keep) break;
        mine[(size_t)i * channels + c] = held[i];
    }
}

}  // namespace

extern "C" int fllm_conv_qkv_store(const void *joint, int ld, const float *conv, int taps, const float *bias, void *state, const float *q_weight,
                                   const float *k_weight, float eps, void *q_out, const int32_t *row_pos, const int32_t *row_seg,
                                   const int32_t *seg_start, const int32_t *slots, int num_segs, const int32_t *tables, int table_stride,
                                   const float *cos_table, const float *sin_table, int table_positions, void *k_pages, void *v_pages, int rows,
                                   int heads, int kv_heads, int k_dim, int v_dim, int rope_dims, int pairing, int page_size, int key_chunk,
                                   int dtype, int store_kv, int single_rows, hipStream_t stream) {
    FLLM_REQUIRE(rows >= 0 && heads > 0 && kv_heads > 0 && k_dim > 0 && v_dim > 0 && page_size > 0 && table_stride > 0 && num_segs > 0,
                 "conv_qkv_store: bad sizes");
    const int channels = heads * k_dim + (store_kv ? kv_heads * (k_dim + v_dim) : 0);
    FLLM_REQUIRE(ld >= channels, "conv_qkv_store: rows of %d values cannot hold %d channels", ld, channels);
    FLLM_REQUIRE(taps >= 1 && taps - 1 <= kMaxKeep, "conv_qkv_store: %d taps are outside 1..%d", taps, kMaxKeep + 1);
    FLLM_REQUIRE(k_dim <= kMaxPer * kWave && v_dim <= kMaxPer * kWave, "conv_qkv_store: heads of %d and %d lanes are more than %d", k_dim, v_dim,
                 kMaxPer * kWave);
    FLLM_REQUIRE(rope_dims >= 0 && rope_dims <= k_dim && rope_dims % 2 == 0,
                 "conv_qkv_store: rope_dims %d must be even and at most the head size %d", rope_dims, k_dim);
    FLLM_REQUIRE(rope_dims == 0 || (cos_table && sin_table && table_positions > 0), "conv_qkv_store: rotary tables missing");
    FLLM_REQUIRE(pairing == 0 || pairing == 1, "conv_qkv_store: unknown pairing %d", pairing);
    FLLM_REQUIRE(key_chunk > 0 && k_dim % key_chunk == 0, "conv_qkv_store: keys of %d values in chunks of %d", k_dim, key_chunk);
    FLLM_REQUIRE(!store_kv || (k_pages && v_pages), "conv_qkv_store: pages missing");
    FLLM_REQUIRE(joint && conv && q_out && row_pos && row_seg && seg_start && slots && tables && (taps == 1 || state), "conv_qkv_store: operands missing");
    FLLM_REQUIRE(q_weight == nullptr || (eps > 0.f && (!store_kv || k_weight)), "conv_qkv_store: a norm of queries and keys needs both weights and an eps");
    FLLM_REQUIRE(!single_rows || rows == num_segs, "conv_qkv_store: %d rows of %d segments are not one each", rows, num_segs);
    if (rows == 0) return 0;
    const int units = heads + (store_kv ? 2 * kv_heads : 0), groups = (units + kWaves - 1) / kWaves;
    const int blocks = (channels + kBlock - 1) / kBlock;
    FLLM_REQUIRE(groups <= 65535 && blocks <= 65535, "conv_qkv_store: too many heads");
    const size_t smem = rope_dims > 0 ? (size_t)kWaves * k_dim * sizeof(float) : 0;
#define FLLM_CONV(T)                                                                                                                        \
    do {                                                                                                                                    \
        hipLaunchKernelGGL(conv_qkv_store_kernel<T>, dim3(rows, groups), dim3(kBlock), smem, stream, (const T *)joint, ld, conv, taps, bias, \
                           (T *)state, q_weight, k_weight, eps, (T *)q_out, row_pos, row_seg, seg_start, slots, tables, table_stride,       \
                           cos_table, sin_table, (T *)k_pages, (T *)v_pages, heads, kv_heads, k_dim, v_dim, rope_dims, pairing, page_size,  \
                           key_chunk, store_kv, single_rows);                                                                               \
        if (taps > 1 && !single_rows)                                                                                                       \
            hipLaunchKernelGGL(conv_tail_kernel<T>, dim3(num_segs, blocks), dim3(kBlock), 0, stream, (const T *)joint, ld, (T *)state,       \
                               row_seg, seg_start, slots, channels, taps);                                                                  \
    } while (0)
    if (dtype == FLLM_F32) FLLM_CONV(float);
    else if (dtype == FLLM_BF16) FLLM_CONV(bf16_t);
    else FLLM_REQUIRE(false, "conv_qkv_store: unknown dtype %d", dtype);
#undef FLLM_CONV
    return fllm_check_launch("conv_qkv_store");
}
