// Linear attention with a decay a key channel that every token chooses, over portions of prompts, on the matrix cores in float32.
//
// S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t is taken kC = 16 tokens at a time.  With L_t the sum of ln alpha over a
// chunk's tokens up to t (a vector over the key channels) and S the state before the chunk:
//     o_t = S^T (q_t e^(L_t)) + sum_{s <= t} (sum_c q_t[c] k_s[c] e^(L_t[c] - L_s[c])) v_s
//     S'  = diag(e^(L_end)) S + sum_s (k_s e^(L_end - L_s)) v_s^T
// Everything is a matrix product of float32 operands (v_mfma_f32_16x16x4_f32) whose factors are at most 1, except the scores: there
// e^(L_t - L_s) is split into e^(L_t) and e^(-L_s).  While no channel decays by more than e^-kSafe over the chunk the second factor
// stays far from overflow and the product is as exact as its parts; a chunk with a faster channel sums its scores term by term
// instead, with the difference in the exponent (one (t, s) pair a thread).
//
// v_mfma_f32_16x16x4_f32: lane l gives A[m = l%16][k = l/16] and B[k = l/16][n = l%16] and receives D[m = 4*(l/16) + r][n = l%16] in
// register r.  Register r of a result tile is at once the A operand (row n, slot l/16) of a later product over its rows, so the
// state lives in such tiles for the whole call: it is the accumulator of K^T V and the A operand of S^T Q^T.
//
// One workgroup of four waves a (part of a segment, head, 32 value lanes); wave w holds the state's rows of the key blocks w, w + 4
// (16 keys a block).  Segments of more than kPart tokens are cut into parts that run side by side, each but the first from zeros; it
// leaves its last state U, the product of its decays A and its queries times the decays since the part's first token, and the
// kernel behind it folds T_p = diag(A_(p-1)) T_(p-1) + U_(p-1) and adds T_p^T to what those queries saw.
#include "api.h"
#include "common.h"
#include "segment_parts.h"

namespace {

constexpr int kC = 16;            // tokens a chunk
constexpr int kVB = 32;           // value lanes a workgroup
constexpr int kLDV = 48;          // row stride of V in LDS: lane groups 16 banks apart
constexpr int kLDP = 17;
constexpr int kThreads = 256;
constexpr int kPart = 256;        // tokens a part
constexpr float kSafe = 40.f;

// exponentials and the logarithm of a decay: float32 operands get the library's functions, bfloat16 ones, whose own rounding is
// 2^-9, the hardware's (a few units in the last place of a float)
template <typename T> __device__ __forceinline__ float exp_of(float x);
template <> __device__ __forceinline__ float exp_of<float>(float x) { return expf(x); }
template <> __device__ __forceinline__ float exp_of<bf16_t>(float x) { return __expf(x); }
template <typename T> __device__ __forceinline__ float log_decay(float z, float inv_tau);      // ln sigmoid(z)^(1 / tau)
template <> __device__ __forceinline__ float log_decay<float>(float z, float inv_tau) {
    return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * inv_tau;
}
template <> __device__ __forceinline__ float log_decay<bf16_t>(float z, float inv_tau) {
    const float y = __expf(-fabsf(z));
    const float l = y < 1e-3f ? y - 0.5f * y * y : __logf(1.0f + y);
    return -(fmaxf(-z, 0.f) + l) * inv_tau;
}

template <typename T>
struct GatedArgs {
    const T *q, *k, *v;
    int ld;
    const float *z, *bias;
    float inv_tau, query_scale;
    float *state;
    const int32_t *row_seg, *seg_start, *slots;
    int num_segs;
    float *out;
    int rows, heads, dim, vdim;
    float *states;     // [part index][head][dim][vdim]: a part's last state
    float *decays;     // [part index][head][dim]: the product of its decays
    float *queries;    // [row][head][dim]: query_scale * q times the decays since its part's first token
    int in_parts;
};

template <typename T, int NB>     // NB: key blocks a wave (dim <= 64 * NB)
__global__ void __launch_bounds__(kThreads)
gated_linear_chunked_kernel(const GatedArgs<T> p) {
    constexpr int CW = 64 * NB, TG = kThreads / CW, TPT = kC / TG, LDQ = CW + 4;
    __shared__ float Qd[kC * LDQ], Kd[kC * LDQ], Kn[kC * LDQ], Lq[kC * LDQ], Qr[kC * LDQ];
    __shared__ float Vs[kC * kLDV], Pp[4][kC * kLDP], Part[4 * 2 * 4 * 64], sums[TG][CW], a_end[CW];

    int seg = blockIdx.x, part = 0;
    if (p.in_parts) find_part<kPart>(blockIdx.x, p.seg_start, p.num_segs, seg, part);
    const int h = blockIdx.y, j0 = blockIdx.z * kVB;
    const int seg_r0 = p.seg_start[seg], seg_n = p.seg_start[seg + 1] - seg_r0;
    if (part < 0 || seg_n <= part * kPart) return;
    const int parts = p.in_parts ? (seg_n + kPart - 1) / kPart : 1;
    const int r0 = seg_r0 + part * kPart, n = p.in_parts ? min(kPart, seg_n - part * kPart) : seg_n;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int ln = lane & 15, g = lane >> 4;
    const int dim = p.dim, vdim = p.vdim, out_ld = p.heads * vdim;
    if (p.row_seg[r0] < 0) {   // padding rows: no state is touched
        for (int i = tid; i < n * kVB; i += kThreads) {
            const int t = i / kVB, c = j0 + i % kVB;
            if (c < vdim) p.out[(size_t)(r0 + t) * out_ld + (size_t)h * vdim + c] = 0.f;
        }
        return;
    }
    const int key_blocks = dim / 16;
    const size_t head_at = (size_t)h * dim * vdim;
    float *mine = p.state + (size_t)p.slots[seg] * p.heads * dim * vdim + head_at;
    f32x4_t S[NB][2];
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int vj = 0; vj < 2; vj++) {
            const int di = wave + 4 * b, col = j0 + 16 * vj + ln;
#pragma unroll
            for (int r = 0; r < 4; r++)
                S[b][vj][r] = (part == 0 && di < key_blocks && col < vdim) ? mine[(size_t)(16 * di + 4 * g + r) * vdim + col] : 0.f;
        }
    const size_t index = p.in_parts ? part_index<kPart>(seg_r0, seg, part) : 0;
    if (parts > 1) mine = p.states + index * p.heads * dim * vdim + head_at;

    // a thread's channel and tokens of a chunk, loaded one chunk ahead
    const int c = tid % CW, tg = tid / CW;
    const bool live = c < dim;
    const float bias = live ? p.bias[h * dim + c] : 0.f;
    T rq[TPT], rk[TPT], rv[2];
    float rz[TPT];
    auto issue = [&](int c0) {
        const int nc = min(kC, n - c0);
#pragma unroll
        for (int i = 0; i < TPT; i++) {
            const int t = tg * TPT + i;
            rq[i] = rk[i] = from_f32<T>(0.f);
            rz[i] = 0.f;
            if (live && t < nc) {
                const size_t row = r0 + c0 + t;
                rq[i] = p.q[row * p.ld + (size_t)h * dim + c];
                rk[i] = p.k[row * p.ld + (size_t)h * dim + c];
                rz[i] = p.z[(row * p.heads + h) * dim + c];
            }
        }
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int t = tid / kVB + 8 * i, cv = j0 + tid % kVB;
            rv[i] = (t < nc && cv < vdim) ? p.v[(size_t)(r0 + c0 + t) * p.ld + (size_t)h * vdim + cv] : from_f32<T>(0.f);
        }
    };
    float since = 0.f;      // ln of the decays since the part's first token, up to the chunk
    issue(0);
    for (int c0 = 0; c0 < n; c0 += kC) {
        const int nc = min(kC, n - c0);
        float L[TPT];
        float run = 0.f;
#pragma unroll
        for (int i = 0; i < TPT; i++) {
            if (live && tg * TPT + i < nc) run += log_decay<T>(rz[i] + bias, p.inv_tau);
            L[i] = run;
        }
        sums[tg][c] = run;
        __syncthreads();      // ... and every wave has read the chunk before
        float before = 0.f, end = 0.f;
#pragma unroll
        for (int a = 0; a < TG; a++) {
            if (a < tg) before += sums[a][c];
            end += sums[a][c];
        }
        const bool direct = __syncthreads_or(end < -kSafe);
#pragma unroll
        for (int i = 0; i < TPT; i++) {
            const int t = tg * TPT + i, at = t * LDQ + c;
            const float l = before + L[i], qv = to_f32<T>(rq[i]) * p.query_scale, kv = to_f32<T>(rk[i]);
            Qd[at] = qv * exp_of<T>(l);
            Kd[at] = kv * exp_of<T>(end - l);
            if (direct) Kn[at] = kv, Lq[at] = l, Qr[at] = qv;
            else Kn[at] = kv * exp_of<T>(-l);
            if (part > 0 && blockIdx.z == 0 && live && t < nc)
                p.queries[((size_t)(r0 + c0 + t) * p.heads + h) * dim + c] = qv * exp_of<T>(since + l);
        }
        if (tg == 0) a_end[c] = exp_of<T>(end);
        since += end;
#pragma unroll
        for (int i = 0; i < 2; i++) Vs[(tid / kVB + 8 * i) * kLDV + tid % kVB] = to_f32<T>(rv[i]);
        if (c0 + kC < n) issue(c0 + kC);
        __syncthreads();

        // this wave's key blocks: its part of the scores, and its rows of the state times the queries
        f32x4_t sc = {0.f, 0.f, 0.f, 0.f}, po[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int b = 0; b < NB; b++) {
            const int di = wave + 4 * b;
            if (di < key_blocks) {
                const f32x4_t qa = *(const f32x4_t *)(Qd + ln * LDQ + 16 * di + 4 * g);
                if (!direct) {
                    const f32x4_t kb = *(const f32x4_t *)(Kn + ln * LDQ + 16 * di + 4 * g);
#pragma unroll
                    for (int r = 0; r < 4; r++) sc = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[r], kb[r], sc, 0, 0, 0);
                }
#pragma unroll
                for (int vj = 0; vj < 2; vj++)
#pragma unroll
                    for (int r = 0; r < 4; r++) po[vj] = __builtin_amdgcn_mfma_f32_16x16x4f32(S[b][vj][r], qa[r], po[vj], 0, 0, 0);
            }
        }
        if (!direct) {
#pragma unroll
            for (int r = 0; r < 4; r++) Pp[wave][(4 * g + r) * kLDP + ln] = sc[r];
        } else {
            const int t = tid >> 4, s = tid & 15;
            float acc = 0.f;
            if (s <= t)
                for (int i = 0; i < dim; i++) acc = fmaf(Qr[t * LDQ + i] * Kn[s * LDQ + i], exp_of<T>(Lq[t * LDQ + i] - Lq[s * LDQ + i]), acc);
            Pp[0][t * kLDP + s] = acc;
            Pp[1][t * kLDP + s] = Pp[2][t * kLDP + s] = Pp[3][t * kLDP + s] = 0.f;
        }
#pragma unroll
        for (int vj = 0; vj < 2; vj++)
#pragma unroll
            for (int r = 0; r < 4; r++) Part[((wave * 2 + vj) * 4 + r) * 64 + lane] = po[vj][r];
        __syncthreads();

        if (wave < 2) {      // output block vj: lane (ln, g), register r is o[token ln][value 16 vj + 4 g + r]
            const int vj = wave;
            f32x4_t o;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                float sum = 0.f;
#pragma unroll
                for (int w = 0; w < 4; w++) sum += Part[((w * 2 + vj) * 4 + r) * 64 + lane];
                o[r] = sum;
            }
#pragma unroll
            for (int s4 = 0; s4 < 4; s4++) {
                const int s = 4 * s4 + g, at = ln * kLDP + s;
                const float w = s <= ln ? (Pp[0][at] + Pp[1][at]) + (Pp[2][at] + Pp[3][at]) : 0.f;
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(Vs[s * kLDV + 16 * vj + ln], w, o, 0, 0, 0);
            }
            const int col = j0 + 16 * vj + 4 * g;
            if (ln < nc && col < vdim) *(f32x4_t *)(p.out + (size_t)(r0 + c0 + ln) * out_ld + (size_t)h * vdim + col) = o;
        }
        // the state behind the chunk
#pragma unroll
        for (int b = 0; b < NB; b++) {
            const int di = wave + 4 * b;
            if (di < key_blocks) {
                const f32x4_t e = *(const f32x4_t *)(a_end + 16 * di + 4 * g);
#pragma unroll
                for (int vj = 0; vj < 2; vj++) S[b][vj] *= e;
#pragma unroll
                for (int s4 = 0; s4 < 4; s4++) {
                    const int s = 4 * s4 + g;
                    const float ka = Kd[s * LDQ + 16 * di + ln];
#pragma unroll
                    for (int vj = 0; vj < 2; vj++)
                        S[b][vj] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka, Vs[s * kLDV + 16 * vj + ln], S[b][vj], 0, 0, 0);
                }
            }
        }
    }
    if (parts > 1 && blockIdx.z == 0 && live && tg == 0) p.decays[(index * p.heads + h) * dim + c] = exp_of<T>(since);
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int vj = 0; vj < 2; vj++) {
            const int di = wave + 4 * b, col = j0 + 16 * vj + ln;
            if (di < key_blocks && col < vdim)
#pragma unroll
                for (int r = 0; r < 4; r++) mine[(size_t)(16 * di + 4 * g + r) * vdim + col] = S[b][vj][r];
        }
}

// One workgroup a (segment, part > 0, head, 32 value lanes): the state before the part in registers, its product with the part's
// decayed queries added to `out`.  The workgroup of the last part also leaves the segment's state.
template <typename T, int NB>
__global__ void __launch_bounds__(kThreads)
gated_linear_carry_kernel(const GatedArgs<T> p) {
    constexpr int CW = 64 * NB, LDQ = CW + 4;
    __shared__ float Qs[2][kC * LDQ], Part[4 * 2 * 4 * 64];
    int seg, part;
    find_part<kPart>(blockIdx.x, p.seg_start, p.num_segs, seg, part);
    const int h = blockIdx.y, j0 = blockIdx.z * kVB;
    const int seg_r0 = p.seg_start[seg], seg_n = p.seg_start[seg + 1] - seg_r0;
    if (part <= 0 || seg_n <= part * kPart || p.row_seg[seg_r0] < 0) return;
    const int parts = (seg_n + kPart - 1) / kPart;
    const int r0 = seg_r0 + part * kPart, n = min(kPart, seg_n - part * kPart);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int ln = lane & 15, g = lane >> 4;
    const int dim = p.dim, vdim = p.vdim, out_ld = p.heads * vdim, key_blocks = dim / 16;
    f32x4_t S[NB][2];
    auto fold = [&](int i) {     // S = diag(A_i) S + U_i
        const size_t index = part_index<kPart>(seg_r0, seg, i);
        const float *u = p.states + (index * p.heads + h) * dim * vdim, *a = p.decays + (index * p.heads + h) * dim;
#pragma unroll
        for (int b = 0; b < NB; b++) {
            const int di = wave + 4 * b;
            if (di >= key_blocks) continue;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int row = 16 * di + 4 * g + r;
                const float ar = a[row];
#pragma unroll
                for (int vj = 0; vj < 2; vj++) {
                    const int col = j0 + 16 * vj + ln;
                    S[b][vj][r] = fmaf(S[b][vj][r], ar, col < vdim ? u[(size_t)row * vdim + col] : 0.f);
                }
            }
        }
    };
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int vj = 0; vj < 2; vj++) S[b][vj] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < part; i++) fold(i);

    constexpr int QV = kC * CW / 4 / kThreads;      // 16-byte loads a thread
    f32x4_t rq[QV];
    auto issue = [&](int c0) {
        const int nc = min(kC, n - c0);
#pragma unroll
        for (int it = 0; it < QV; it++) {
            const int i = tid + it * kThreads, t = i / (CW / 4), c = i % (CW / 4) * 4;
            rq[it] = (t < nc && c < dim) ? *(const f32x4_t *)(p.queries + ((size_t)(r0 + c0 + t) * p.heads + h) * dim + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
        }
    };
    issue(0);
    for (int c0 = 0; c0 < n; c0 += kC) {
        const int nc = min(kC, n - c0);
        float *Q = Qs[(c0 / kC) & 1];
#pragma unroll
        for (int it = 0; it < QV; it++) {
            const int i = tid + it * kThreads, t = i / (CW / 4), c = i % (CW / 4) * 4;
            *(f32x4_t *)(Q + t * LDQ + c) = rq[it];
        }
        if (c0 + kC < n) issue(c0 + kC);
        __syncthreads();
        f32x4_t po[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int b = 0; b < NB; b++) {
            const int di = wave + 4 * b;
            if (di < key_blocks) {
                const f32x4_t qa = *(const f32x4_t *)(Q + ln * LDQ + 16 * di + 4 * g);
#pragma unroll
                for (int vj = 0; vj < 2; vj++)
#pragma unroll
                    for (int r = 0; r < 4; r++) po[vj] = __builtin_amdgcn_mfma_f32_16x16x4f32(S[b][vj][r], qa[r], po[vj], 0, 0, 0);
            }
        }
#pragma unroll
        for (int vj = 0; vj < 2; vj++)
#pragma unroll
            for (int r = 0; r < 4; r++) Part[((wave * 2 + vj) * 4 + r) * 64 + lane] = po[vj][r];
        __syncthreads();
        if (wave < 2) {
            const int vj = wave, col = j0 + 16 * vj + 4 * g;
            if (ln < nc && col < vdim) {
                float *dst = p.out + (size_t)(r0 + c0 + ln) * out_ld + (size_t)h * vdim + col;
                f32x4_t o = *(const f32x4_t *)dst;
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    float sum = 0.f;
#pragma unroll
                    for (int w = 0; w < 4; w++) sum += Part[((w * 2 + vj) * 4 + r) * 64 + lane];
                    o[r] += sum;
                }
                *(f32x4_t *)dst = o;
            }
        }
        __syncthreads();      // the next chunk overwrites Part
    }
    if (part == parts - 1) {
        fold(part);
        float *mine = p.state + ((size_t)p.slots[seg] * p.heads + h) * dim * vdim;
#pragma unroll
        for (int b = 0; b < NB; b++)
#pragma unroll
            for (int vj = 0; vj < 2; vj++) {
                const int di = wave + 4 * b, col = j0 + 16 * vj + ln;
                if (di < key_blocks && col < vdim)
#pragma unroll
                    for (int r = 0; r < 4; r++) mine[(size_t)(16 * di + 4 * g + r) * vdim + col] = S[b][vj][r];
            }
    }
}

size_t part_count(int rows, int num_segs) { return (size_t)rows / kPart + (size_t)num_segs + 1; }

}  // namespace

extern "C" size_t fllm_gated_linear_carried_floats(int rows, int num_segs, int heads, int dim, int vdim) {
    if (rows <= kPart) return 0;      // no segment is longer than a part
    return part_count(rows, num_segs) * heads * dim * ((size_t)vdim + 1) + (size_t)rows * heads * dim + 8;
}

// 0: launched; 1: the sizes are not this kernel's (keys in blocks of 16 up to 128 lanes, values in blocks of 16)
int fllm_gated_linear_chunked(const void *q, const void *k, const void *v, int ld, const float *z, const float *bias, float inv_tau,
                              float query_scale, float *state, const int32_t *row_seg, const int32_t *seg_start, const int32_t *slots,
                              int num_segs, float *out, int rows, int heads, int dim, int vdim, int dtype, float *carried,
                              hipStream_t stream) {
    if (dim % 16 != 0 || dim > 128 || vdim % 16 != 0) return 1;
    const int slices = (vdim + kVB - 1) / kVB;
    if (slices > 65535 || heads > 65535) return 1;
    const int in_parts = (carried != nullptr && rows > kPart) ? 1 : 0;
    const dim3 grid(in_parts ? (unsigned)(rows / kPart + num_segs) : (unsigned)num_segs, heads, slices);
    float *states = carried, *queries = nullptr, *decays = nullptr;
    if (in_parts) {      // the queries first behind the states, on 16 bytes: dim and vdim are multiples of 16
        queries = states + part_count(rows, num_segs) * heads * dim * vdim;
        decays = queries + (size_t)rows * heads * dim;
    }
#define FLLM_GATED(T, NB)                                                                                                                  \
    do {                                                                                                                                   \
        GatedArgs<T> p = {(const T *)q, (const T *)k, (const T *)v, ld, z, bias, inv_tau, query_scale, state, row_seg, seg_start, slots,    \
                          num_segs, out, rows, heads, dim, vdim, states, decays, queries, in_parts};                                       \
        hipLaunchKernelGGL((gated_linear_chunked_kernel<T, NB>), grid, dim3(kThreads), 0, stream, p);                                      \
        if (in_parts) hipLaunchKernelGGL((gated_linear_carry_kernel<T, NB>), grid, dim3(kThreads), 0, stream, p);                          \
    } while (0)
    if (dtype == FLLM_F32) {
        if (dim <= 64) FLLM_GATED(float, 1);
        else FLLM_GATED(float, 2);
    } else if (dtype == FLLM_BF16) {
        if (dim <= 64) FLLM_GATED(bf16_t, 1);
        else FLLM_GATED(bf16_t, 2);
    } else
        return 1;
#undef FLLM_GATED
    return 0;
}
