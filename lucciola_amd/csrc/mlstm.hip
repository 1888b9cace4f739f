// The matrix memory of the xLSTM (mLSTM) around the framework's recurrence kernel.  Per head, with the state S
// [key, value], the normaliser n [key] and the reference point m (float32, all zero at a sequence's start):
//   i = cap tanh((x_i + b_i) / cap),   f = logsigmoid(cap tanh((x_f + b_f) / cap))       (logarithms of the gates)
//   m' = max(f + m, i);   S <- e^(f + m - m') S + e^(i - m') k v^T;   n <- e^(f + m - m') n + e^(i - m') k
//   o = S^T q / (max(|n . q|, e^(-m')) + floor)
// The normaliser is one more value channel, whose value is 1 in every token: with it beside the others the
// recurrence is S <- diag(decay) S + write v^T, o = S^T read without a removal term, with decay = e^(f + m - m') in
// every key channel, write = e^(i - m') k, read = q_scale q.  This file makes those inputs from a step's float32
// projections: the reference points, which tie a token to the one before it, by one workgroup per request and head that
// walks the request's tokens; the vectors by a thread an entry.  A step of lone tokens does both in one kernel.
// Behind the scan the read-out divides by the normaliser, takes each head by its root mean square, multiplies by a
// weight and sigmoid(gate) and rounds to the activation type; everything before that rounding is float32.
#include "common.h"

#include "activations.h"

namespace lc {

// What the token's gates make of the reference point before it.  The kernel of lone tokens and the one that walks a
// portion both go through these; a multiplication is not taken into a following addition, so that they give the same bits.
struct MemoryGates {
    float keep_log, write_log;
};
__device__ __forceinline__ MemoryGates memory_gates(float x_i, float b_i, float x_f, float b_f, float cap) {
#pragma clang fp contract(off)
    const float z = cap * tanhf((x_f + b_f) / cap);
    return {fminf(z, 0.f) - log1pf(expf(-fabsf(z))), cap * tanhf((x_i + b_i) / cap)};
}
__device__ __forceinline__ float next_reference(const MemoryGates& g, float m) { return fmaxf(g.keep_log + m, g.write_log); }
__device__ __forceinline__ float keep_factor(const MemoryGates& g, float before, float after) {
#pragma clang fp contract(off)
    return expf(g.keep_log + before - after);
}
__device__ __forceinline__ float write_factor(const MemoryGates& g, float after) {
#pragma clang fp contract(off)
    return expf(g.write_log - after);
}

constexpr int GATE_TOKENS = 192;       // tokens of a chunk: one for each thread behind the first wave
constexpr int CHAIN_GROUP = 16;         // tokens that the walker reads ahead

// grid (heads, requests).  proj [T, cols] with x_i at columns i_col + head and x_f at f_col + head; factors
// [3, T, heads]: keep, write and e^(-m') of every token; reference [slots, heads].
// A pipeline over chunks of tokens: while the other waves make the gates of chunk c (a token a thread) and write out
// chunk c - 2, one lane of the first wave walks the chain of maxima through chunk c - 1, one add and one max a token,
// in order, so that a token's numbers have the same bits however its request is cut into steps.
__global__ __launch_bounds__(kWave + GATE_TOKENS) void mlstm_gates_kernel(
    const float* __restrict__ proj, int cols, int i_col, int f_col, const float* __restrict__ i_bias,
    const float* __restrict__ f_bias, float cap, float* __restrict__ reference, const int* __restrict__ q_offsets,
    const int* __restrict__ slot_ids, int T, int heads, float* __restrict__ factors) {
    static_assert(GATE_TOKENS % CHAIN_GROUP == 0 && CHAIN_GROUP % 4 == 0, "whole groups of whole float4s");
    __shared__ float4 keep_log[2][GATE_TOKENS / 4], write_log[2][GATE_TOKENS / 4], found[2][GATE_TOKENS / 4];
    const int head = blockIdx.x, req = blockIdx.y, j = (int)threadIdx.x - kWave;
    const int first = q_offsets[req], last = q_offsets[req + 1];
    if (first >= last) return;
    const int chunks = (last - first + GATE_TOKENS - 1) / GATE_TOKENS;
    const size_t plane = (size_t)T * heads;
    float* home = reference + (size_t)slot_ids[req] * heads + head;
    const float b_i = i_bias[head], b_f = f_bias[head];
    float m = *home;
    for (int c = 0; c < chunks + 2; ++c) {
        const int mine = c & 1, walked = mine ^ 1;      // the chunks c and c - 2 share their places
        if (j >= 0) {
            if (c >= 2) {
                const int t = first + (c - 2) * GATE_TOKENS + j;
                if (t < last) {
                    const MemoryGates g{((const float*)keep_log[mine])[j], ((const float*)write_log[mine])[j]};
                    const float before = ((const float*)found[mine])[j], after = next_reference(g, before);
                    const size_t at = (size_t)t * heads + head;
                    factors[at] = keep_factor(g, before, after);
                    factors[plane + at] = write_factor(g, after);
                    factors[2 * plane + at] = expf(-after);
                }
            }
            if (c < chunks) {
                const int t = first + c * GATE_TOKENS + j;
                MemoryGates g = {0.f, -INFINITY};       // behind the request's end: nothing moves
                if (t < last) {
                    const float* row = proj + (size_t)t * cols;
                    g = memory_gates(row[i_col + head], b_i, row[f_col + head], b_f, cap);
                }
                ((float*)keep_log[mine])[j] = g.keep_log;
                ((float*)write_log[mine])[j] = g.write_log;
            }
        } else if (threadIdx.x == 0 && c >= 1 && c <= chunks) {
            constexpr int QUADS = CHAIN_GROUP / 4;
            const float4 *keep = keep_log[walked], *write = write_log[walked];
            const int count = min(GATE_TOKENS, last - first - (c - 1) * GATE_TOKENS);
            const int groups = (count + CHAIN_GROUP - 1) / CHAIN_GROUP;
            float4 k_now[QUADS], w_now[QUADS], k_next[QUADS], w_next[QUADS];
#pragma unroll
            for (int i = 0; i < QUADS; ++i) k_now[i] = keep[i], w_now[i] = write[i];
            for (int n = 0; n < groups; ++n) {
                const int ahead = min(n + 1, groups - 1) * QUADS;
#pragma unroll
                for (int i = 0; i < QUADS; ++i) k_next[i] = keep[ahead + i], w_next[i] = write[ahead + i];
#pragma unroll
                for (int i = 0; i < QUADS; ++i) {
                    float4 at;
                    at.x = m;
                    at.y = next_reference({k_now[i].x, w_now[i].x}, at.x);
                    at.z = next_reference({k_now[i].y, w_now[i].y}, at.y);
                    at.w = next_reference({k_now[i].z, w_now[i].z}, at.z);
                    m = next_reference({k_now[i].w, w_now[i].w}, at.w);
                    found[walked][n * QUADS + i] = at;
                }
#pragma unroll
                for (int i = 0; i < QUADS; ++i) k_now[i] = k_next[i], w_now[i] = w_next[i];
            }
            if (c == chunks) *home = m;
        }
        __syncthreads();
    }
}

// A thread per entry.  proj [T, cols]: q | k (heads x dk each) | v (heads x dv) | ...; coef [3, T, heads dk]: decay,
// write, read; v_out [T, heads (dv + 1)], a 1 behind every head's values.
__global__ void mlstm_prepare_kernel(const float* __restrict__ proj, int cols, int T, int heads, int dk, int dv,
                                     float q_scale, const float* __restrict__ factors, float* __restrict__ coef,
                                     float* __restrict__ v_out) {
    const int nk = heads * dk, nv = heads * (dv + 1);
    const size_t plane = (size_t)T * nk, total = (size_t)T * (nk + nv);
    for (size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (size_t)gridDim.x * blockDim.x) {
        const int t = (int)(idx / (nk + nv)), c = (int)(idx % (nk + nv));
        const float* row = proj + (size_t)t * cols;
        if (c < nk) {
            const size_t at = (size_t)t * nk + c, f = (size_t)t * heads + c / dk;
            coef[at] = factors[f];
            coef[plane + at] = factors[(size_t)T * heads + f] * row[nk + c];
            coef[2 * plane + at] = q_scale * row[c];
        } else {
            const int head = (c - nk) / (dv + 1), e = (c - nk) % (dv + 1);
            v_out[(size_t)t * nv + (c - nk)] = e < dv ? row[2 * nk + head * dv + e] : 1.f;
        }
    }
}

// The two above for a step whose requests bring one token each: grid (requests, heads), a workgroup per token and head.
__global__ void mlstm_lone_kernel(const float* __restrict__ proj, int cols, int i_col, int f_col,
                                  const float* __restrict__ i_bias, const float* __restrict__ f_bias, float cap,
                                  float* __restrict__ reference, const int* __restrict__ q_offsets,
                                  const int* __restrict__ slot_ids, int T, int heads, int dk, int dv, float q_scale,
                                  float* __restrict__ factors, float* __restrict__ coef, float* __restrict__ v_out) {
    const int req = blockIdx.x, head = blockIdx.y, t = q_offsets[req];
    float* home = reference + (size_t)slot_ids[req] * heads + head;
    const float* row = proj + (size_t)t * cols;
    const float m = *home;
    const MemoryGates g = memory_gates(row[i_col + head], i_bias[head], row[f_col + head], f_bias[head], cap);
    const float after = next_reference(g, m);
    const float keep = keep_factor(g, m, after), write = write_factor(g, after);
    const int nk = heads * dk;
    const size_t plane = (size_t)T * nk, at0 = (size_t)t * nk + (size_t)head * dk;
    for (int e = threadIdx.x; e < dk; e += blockDim.x) {
        coef[at0 + e] = keep;
        coef[plane + at0 + e] = write * row[nk + head * dk + e];
        coef[2 * plane + at0 + e] = q_scale * row[head * dk + e];
    }
    float* v = v_out + ((size_t)t * heads + head) * (dv + 1);
    for (int e = threadIdx.x; e <= dv; e += blockDim.x) v[e] = e < dv ? row[2 * nk + head * dv + e] : 1.f;
    __syncthreads();            // every thread has read the reference point
    if (threadIdx.x == 0) {
        *home = after;
        const size_t f = (size_t)t * heads + head, fp = (size_t)T * heads;
        factors[f] = keep;
        factors[fp + f] = write;
        factors[2 * fp + f] = expf(-after);
    }
}

constexpr int READ_WAVES = 4;

// One wave per (token, head).  o [T, heads (dv + 1)]: a head's read-outs, then its normaliser's; bottoms [T, heads]
// (e^(-m')); gates: columns gate_column .. + heads dv of [T, gate_cols]; weight [heads dv].
template <typename T>
__global__ __launch_bounds__(READ_WAVES * kWave) void mlstm_readout_kernel(
    const float* __restrict__ o, const float* __restrict__ bottoms, float floor_, const float* __restrict__ gates,
    int gate_cols, int gate_column, const float* __restrict__ weight, float eps, int rows, int heads, int dv,
    T* __restrict__ out) {
    const int row = blockIdx.x * READ_WAVES + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    if (row >= rows) return;
    const int t = row / heads, head = row % heads;
    const float* mine = o + (size_t)row * (dv + 1);
    const float inv = 1.f / (fmaxf(fabsf(mine[dv]), bottoms[row]) + floor_);
    float ss = 0.f;
    for (int e = lane; e < dv; e += kWave) {
        const float v = mine[e] * inv;
        ss = fmaf(v, v, ss);
    }
    const float by = inv / sqrtf(wave_sum(ss) / (float)dv + eps);
    for (int e = lane; e < dv; e += kWave) {
        const int c = head * dv + e;
        out[(size_t)t * heads * dv + c] =
            from_f32<T>(mine[e] * by * weight[c] * sigmoid(gates[(size_t)t * gate_cols + gate_column + c]));
    }
}

}  // namespace lc

using namespace lc;

// factors [3, T, heads], coef [3, T, heads dk], v_out [T, heads (dv + 1)].  lone: every request brings one token.
LC_API int lc_mlstm_prepare(const float* proj, int cols, int i_col, int f_col, const float* i_bias, const float* f_bias,
                            float cap, float* reference, int slots, const int* q_offsets, const int* slot_ids, int R,
                            int T, int heads, int dk, int dv, float q_scale, int lone, float* factors, float* coef,
                            float* v_out, hipStream_t stream) {
    LC_CHECK(R >= 0 && T >= R && heads > 0 && dk > 0 && dv > 0 && slots >= 0 && cap > 0.f, "mlstm prepare: bad sizes");
    LC_CHECK(i_col >= 0 && f_col >= 0 && i_col + heads <= cols && f_col + heads <= cols && heads * (2 * dk + dv) <= cols,
             "mlstm prepare: the columns do not fit the heads");
    LC_CHECK(!lone || T == R, "mlstm prepare: %d tokens are not lone tokens of %d requests", T, R);
    if (T == 0 || R == 0) return 0;
    LC_CHECK(proj && i_bias && f_bias && reference && q_offsets && slot_ids && factors && coef && v_out,
             "mlstm prepare: null pointer");
    LC_CHECK(R <= 65535 && heads <= 65535, "mlstm prepare: too many requests or heads for the grid");
    if (lone) {
        const int widest = dk > dv + 1 ? dk : dv + 1;
        const int threads = widest > 128 ? 256 : (widest > 64 ? 128 : 64);
        mlstm_lone_kernel<<<dim3(R, heads), threads, 0, stream>>>(proj, cols, i_col, f_col, i_bias, f_bias, cap, reference,
                                                                  q_offsets, slot_ids, T, heads, dk, dv, q_scale, factors,
                                                                  coef, v_out);
        LC_LAUNCH_CHECK("mlstm_lone");
        return 0;
    }
    mlstm_gates_kernel<<<dim3(heads, R), kWave + GATE_TOKENS, 0, stream>>>(proj, cols, i_col, f_col, i_bias, f_bias, cap, reference,
                                                             q_offsets, slot_ids, T, heads, factors);
    LC_LAUNCH_CHECK("mlstm_gates");
    const size_t total = (size_t)T * heads * (dk + dv + 1);
    const int blocks = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
    mlstm_prepare_kernel<<<blocks, 256, 0, stream>>>(proj, cols, T, heads, dk, dv, q_scale, factors, coef, v_out);
    LC_LAUNCH_CHECK("mlstm_prepare");
    return 0;
}

LC_API int lc_mlstm_readout(const float* o, const float* bottoms, float floor_, const float* gates, int gate_cols,
                            int gate_column, const float* weight, float eps, int T, int heads, int dv, void* out, int dt,
                            hipStream_t stream) {
    LC_CHECK(T >= 0 && heads > 0 && dv > 0 && gate_column >= 0 && gate_column + heads * dv <= gate_cols,
             "mlstm readout: bad sizes");
    if (T == 0) return 0;
    LC_CHECK(o && bottoms && gates && weight && out, "mlstm readout: null pointer");
    LC_CHECK((long long)T * heads < (1ll << 31), "mlstm readout: too many heads");
    const int rows = T * heads, blocks = (rows + READ_WAVES - 1) / READ_WAVES;
    if (dt == DT_F32)
        mlstm_readout_kernel<float><<<blocks, READ_WAVES * kWave, 0, stream>>>(o, bottoms, floor_, gates, gate_cols, gate_column,
                                                                               weight, eps, rows, heads, dv, (float*)out);
    else if (dt == DT_BF16)
        mlstm_readout_kernel<bf16><<<blocks, READ_WAVES * kWave, 0, stream>>>(o, bottoms, floor_, gates, gate_cols, gate_column,
                                                                              weight, eps, rows, heads, dv, (bf16*)out);
    else
        LC_CHECK(false, "mlstm readout: unknown dtype %d", dt);
    LC_LAUNCH_CHECK("mlstm_readout");
    return 0;
}
