// A prologue of the masked attention (masked_attention.hip) for layers whose queries and keys are normed as whole
// rows: from a step's float32 projections q | k | v (side by side, heads of d, d and dv entries) it makes q for the
// attention kernels and the rows of the cache.
//   x <- proj + bias                                                           (bias, where given)
//   q <- q / sqrt(mean of q^2 over ALL its heads' entries + eps) * q_weight    (where given; k likewise, on its own)
//   rotation of the first `rot` entries of every q and k head: entry i with i + rot / 2 (half), or 2i with 2i + 1
//   v is left in values_out as it is (where given), then v <- (1 - mix) v + mix mix_from    (where mix_from is given)
// Everything is float32; q, k and v are rounded once, to the type of the cache.  Keys lie token-major, values
// transposed inside their page.
#include "common.h"

namespace lc {

constexpr int AR_THREADS = 256;

// grid (tokens, parts): every part of a token sums the whole rows and writes its share of the entries.
template <typename T>
__global__ __launch_bounds__(AR_THREADS) void attention_rows_kernel(
    const float* __restrict__ proj, int cols, int nq, int nk, int nv, int d, int dv, const float* __restrict__ bias,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps, const float* __restrict__ table,
    int rot, int half, const int* __restrict__ positions, const float* __restrict__ mix_from, float mix,
    float* __restrict__ values_out, T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int* __restrict__ rows, int page_size) {
    __shared__ float scratch[16];
    const int t = blockIdx.x;
    const float* x = proj + (size_t)t * cols;
    const int q_cols = nq * d, qk_cols = (nq + nk) * d, v_cols = nv * dv;
    float by_q = 1.f, by_k = 1.f;
    if (q_weight) {             // the same condition in every thread
        float qq = 0.f, kk = 0.f;
        for (int c = threadIdx.x; c < qk_cols; c += AR_THREADS) {
            const float v = bias ? x[c] + bias[c] : x[c];
            if (c < q_cols) qq = fmaf(v, v, qq);
            else kk = fmaf(v, v, kk);
        }
        by_q = 1.f / sqrtf(block_sum(qq, scratch) / (float)q_cols + eps);
        by_k = 1.f / sqrtf(block_sum(kk, scratch) / (float)(nk * d) + eps);
    }
    const int turned = table ? rot / 2 : 0;          // pairs of a head that are rotated
    const int units = d - turned;                    // pairs and single entries of a head
    const float* angle = table ? table + (size_t)positions[t] * rot : nullptr;
    const int slot = rows ? rows[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, place = slot >= 0 ? slot % page_size : 0;
    auto normed = [&](int c) {
        float v = bias ? x[c] + bias[c] : x[c];
        if (q_weight) v = c < q_cols ? v * by_q * q_weight[c] : v * by_k * k_weight[c - q_cols];
        return v;
    };
    auto put = [&](int c, float v) {
        if (c < q_cols) q_out[(size_t)t * q_cols + c] = from_f32<T>(v);
        else if (slot >= 0) k_cache[(size_t)slot * nk * d + (c - q_cols)] = from_f32<T>(v);
    };
    const int qk_units = (nq + nk) * units;
    for (int idx = blockIdx.y * AR_THREADS + threadIdx.x; idx < qk_units + v_cols; idx += gridDim.y * AR_THREADS) {
        if (idx < qk_units) {
            const int head = idx / units, u = idx - head * units, base = head * d;
            if (u < turned) {
                const int c0 = base + (half ? u : 2 * u), c1 = base + (half ? u + turned : 2 * u + 1);
                const float a = normed(c0), b = normed(c1), cs = angle[u], sn = angle[turned + u];
                put(c0, a * cs - b * sn);
                put(c1, fmaf(b, cs, a * sn));
            } else {
                const int c = base + u + turned;
                put(c, normed(c));
            }
        } else {
            const int e = idx - qk_units;
            float v = bias ? x[qk_cols + e] + bias[qk_cols + e] : x[qk_cols + e];
            if (values_out) values_out[(size_t)t * v_cols + e] = v;
            if (mix_from) v = fmaf(mix, mix_from[(size_t)t * v_cols + e], (1.f - mix) * v);
            if (slot >= 0) v_cache[((size_t)page * v_cols + e) * page_size + place] = from_f32<T>(v);
        }
    }
}

typedef float quad __attribute__((ext_vector_type(4)));

__device__ __forceinline__ quad load_quad(const float* p) { return *reinterpret_cast<const quad*>(p); }
__device__ __forceinline__ void store_quad(float* p, quad v) { *reinterpret_cast<quad*>(p) = v; }
__device__ __forceinline__ void store_quad(bf16* p, quad v) {
    typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
    *reinterpret_cast<bf16x4*>(p) = bf16x4{from_f32<bf16>(v.x), from_f32<bf16>(v.y), from_f32<bf16>(v.z), from_f32<bf16>(v.w)};
}

// The same, four entries at a time, where the heads' sizes and the rotated entries come in fours.
template <typename T>
__global__ __launch_bounds__(AR_THREADS) void attention_rows_quads_kernel(
    const float* __restrict__ proj, int cols, int nq, int nk, int nv, int d, int dv, const float* __restrict__ bias,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps, const float* __restrict__ table,
    int rot, int half, const int* __restrict__ positions, const float* __restrict__ mix_from, float mix,
    float* __restrict__ values_out, T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int* __restrict__ rows, int page_size) {
    __shared__ float sums[2][AR_THREADS / kWave];
    const int t = blockIdx.x;
    const float* x = proj + (size_t)t * cols;
    const int q_cols = nq * d, qk_cols = (nq + nk) * d, v_cols = nv * dv;
    const int slot = rows ? rows[t] : -1;
    const float* angle = table ? table + (size_t)positions[t] * rot : nullptr;
    auto biased = [&](int c) {
        quad v = load_quad(x + c);
        if (bias) v += load_quad(bias + c);
        return v;
    };
    float by_q = 1.f, by_k = 1.f;
    if (q_weight) {             // the same condition in every thread
        float qq = 0.f, kk = 0.f;
#pragma unroll 4
        for (int c = 4 * threadIdx.x; c < qk_cols; c += 4 * AR_THREADS) {
            const quad v = biased(c);
            const float ss = fmaf(v.x, v.x, v.y * v.y) + fmaf(v.z, v.z, v.w * v.w);
            if (c < q_cols) qq += ss;
            else kk += ss;
        }
        qq = wave_sum(qq);
        kk = wave_sum(kk);
        if ((threadIdx.x & (kWave - 1)) == 0) sums[0][threadIdx.x / kWave] = qq, sums[1][threadIdx.x / kWave] = kk;
        __syncthreads();
        qq = kk = 0.f;
#pragma unroll
        for (int w = 0; w < AR_THREADS / kWave; ++w) qq += sums[0][w], kk += sums[1][w];
        by_q = 1.f / sqrtf(qq / (float)q_cols + eps);
        by_k = 1.f / sqrtf(kk / (float)(nk * d) + eps);
    }
    const int turned = table ? rot / 2 : 0;             // pairs of a head that are rotated
    const int pair_quads = half ? turned / 4 : 0;       // items of four pairs that lie apart
    const int units = d / 4 - pair_quads;               // items of a head
    const int page = slot >= 0 ? slot / page_size : 0, place = slot >= 0 ? slot % page_size : 0;
    auto normed = [&](int c) {
        quad v = biased(c);
        if (q_weight) v = c < q_cols ? v * by_q * load_quad(q_weight + c) : v * by_k * load_quad(k_weight + (c - q_cols));
        return v;
    };
    auto put = [&](int c, quad v) {
        if (c < q_cols) store_quad(q_out + (size_t)t * q_cols + c, v);
        else if (slot >= 0) store_quad(k_cache + (size_t)slot * nk * d + (c - q_cols), v);
    };
    const int qk_units = (nq + nk) * units, items = qk_units + v_cols / 4;
#pragma unroll 2
    for (int idx = blockIdx.y * AR_THREADS + threadIdx.x; idx < items; idx += gridDim.y * AR_THREADS) {
        if (idx < qk_units) {
            const int head = idx / units, u = idx - head * units, base = head * d;
            if (u < pair_quads) {
                const int c = base + 4 * u;
                const quad a = normed(c), b = normed(c + turned);
                const quad cs = load_quad(angle + 4 * u), sn = load_quad(angle + turned + 4 * u);
                put(c, a * cs - b * sn);
                put(c + turned, b * cs + a * sn);
            } else {
                const int e = 4 * (u + pair_quads);
                quad v = normed(base + e);
                if (!half && e < 2 * turned) {          // two pairs of neighbours
                    const float2 cs = *reinterpret_cast<const float2*>(angle + e / 2);
                    const float2 sn = *reinterpret_cast<const float2*>(angle + turned + e / 2);
                    v = quad{v.x * cs.x - v.y * sn.x, v.y * cs.x + v.x * sn.x, v.z * cs.y - v.w * sn.y,
                             v.w * cs.y + v.z * sn.y};
                }
                put(base + e, v);
            }
        } else {
            const int e = 4 * (idx - qk_units);
            quad v = biased(qk_cols + e);
            if (values_out) store_quad(values_out + (size_t)t * v_cols + e, v);
            if (mix_from) v = mix * load_quad(mix_from + (size_t)t * v_cols + e) + (1.f - mix) * v;
            if (slot >= 0) {
                T* to = v_cache + ((size_t)page * v_cols + e) * page_size + place;
                to[0] = from_f32<T>(v.x);
                to[page_size] = from_f32<T>(v.y);
                to[2 * (size_t)page_size] = from_f32<T>(v.z);
                to[3 * (size_t)page_size] = from_f32<T>(v.w);
            }
        }
    }
}

bool in_sixteens(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

template <typename T, typename... Args>
void launch_attention_rows(bool quads, dim3 grid, hipStream_t stream, Args... args) {
    if (quads) attention_rows_quads_kernel<T><<<grid, AR_THREADS, 0, stream>>>(args...);
    else attention_rows_kernel<T><<<grid, AR_THREADS, 0, stream>>>(args...);
}

}  // namespace lc

using namespace lc;

LC_API int lc_attention_rows(const float* proj, int cols, int T, int nq, int nk, int nv, int d, int dv, const float* bias,
                             const float* q_weight, const float* k_weight, float eps, const float* table, int rot,
                             int half, const int* positions, const float* mix_from, float mix, float* values_out,
                             void* q_out, void* k_cache, void* v_cache, int dt, const int* rows, int page_size,
                             hipStream_t stream) {
    LC_CHECK(T >= 0 && nq > 0 && nk > 0 && nv > 0 && d > 0 && dv > 0 && cols >= (nq + nk) * d + nv * dv,
             "attention rows: bad sizes");
    if (T == 0) return 0;
    LC_CHECK(proj && q_out, "attention rows: null pointer");
    LC_CHECK((q_weight == nullptr) == (k_weight == nullptr), "attention rows: q and k are normed together");
    LC_CHECK(!table || (rot > 0 && rot % 2 == 0 && rot <= d && positions), "attention rows: bad rotation");
    LC_CHECK(!rows || (k_cache && v_cache && page_size > 0), "attention rows: rows without a cache");
    // few tokens: several workgroups a token, so that the GPU is not left to a handful of them
    const bool quads = d % 4 == 0 && dv % 4 == 0 && cols % 4 == 0 && (!table || rot % (half ? 8 : 4) == 0) &&
                       in_sixteens(proj) && in_sixteens(bias) && in_sixteens(q_weight) && in_sixteens(k_weight) &&
                       in_sixteens(table) && in_sixteens(mix_from) && in_sixteens(values_out) && in_sixteens(q_out) &&
                       in_sixteens(k_cache);
    const int items = ((nq + nk) * d + nv * dv) / (quads ? 4 : 1);
    int parts = 1;
    while (parts < 8 && T * parts * 2 <= device_cus() && parts * AR_THREADS < items) parts *= 2;
    const dim3 grid(T, parts);
    if (dt == DT_F32)
        launch_attention_rows<float>(quads, grid, stream, proj, cols, nq, nk, nv, d, dv, bias, q_weight, k_weight, eps, table,
                                     rot, half, positions, mix_from, mix, values_out, (float*)q_out, (float*)k_cache,
                                     (float*)v_cache, rows, page_size);
    else if (dt == DT_BF16)
        launch_attention_rows<bf16>(quads, grid, stream, proj, cols, nq, nk, nv, d, dv, bias, q_weight, k_weight, eps, table,
                                    rot, half, positions, mix_from, mix, values_out, (bf16*)q_out, (bf16*)k_cache,
                                    (bf16*)v_cache, rows, page_size);
    else
        LC_CHECK(false, "attention rows: unknown dtype %d", dt);
    LC_LAUNCH_CHECK("attention_rows");
    return 0;
}
