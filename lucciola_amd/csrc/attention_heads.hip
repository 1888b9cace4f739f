// A prologue of the masked attention (masked_attention.hip) for layers that treat every head on its own: from a step's
// float32 projections q | k | v (side by side, heads of d, d and dv entries; or q | k alone, the values being the keys)
// it makes q for the attention kernels and the rows of the cache.  Per head:
//   x <- proj + bias                                                       (bias, where given)
//   values that are the keys are k at this point
//   x <- x / sqrt(mean of the head's x^2 + eps) * weight                   (q and k, where given; one weight for all heads)
//   rotation of the first `rot` entries of q and k: entry i with i + rot / 2 (half), or 2i with 2i + 1
//   q <- q (1 + coef ln(floor((p + 1) / every) + 1)) at position p         (where every > 0)
// Everything is float32; q, k and v are rounded once, to the type of the cache.  Keys lie token-major, values
// transposed inside their page.
#include "common.h"

namespace lc {

constexpr int AH_THREADS = 256;
constexpr int AH_MAX = 256;          // entries of a head at most

struct HeadsArgs {
    const float* proj;
    int cols, nq, nk, nv, d, dv, values_are_keys;
    const float* bias;
    const float* q_weight;
    const float* k_weight;
    float eps;
    const float* table;
    int rot, half;
    const int* positions;
    float coef, every;
    void* q_out;
    void* k_cache;
    void* v_cache;
    const int* rows;
    int page_size;
};

// W neighbouring entries at a time, a head on L neighbouring lanes, a lane's items L W entries apart.  A head's sum is
// added in an order that the head's size alone decides.
template <typename T, int W, int L, int ITEMS>
__global__ __launch_bounds__(AH_THREADS) void attention_heads_kernel(HeadsArgs a) {
    const int t = blockIdx.x, lane = threadIdx.x % L;
    const int u = blockIdx.y * (AH_THREADS / L) + threadIdx.x / L;         // the head of q | k | v
    const int heads = a.nq + a.nk + (a.values_are_keys ? 0 : a.nv);
    const bool on = u < heads;              // lanes without a head stay for the sums
    const bool is_q = u < a.nq, is_k = !is_q && u < a.nq + a.nk;
    const int width = is_q || is_k ? a.d : a.dv;
    const int col0 = is_q || is_k ? u * a.d : (a.nq + a.nk) * a.d + (u - a.nq - a.nk) * a.dv;
    const float* x = a.proj + (size_t)t * a.cols + col0;
    const float* bias = a.bias ? a.bias + col0 : nullptr;
    const int slot = a.rows ? a.rows[t] : -1;
    T* v_to = nullptr;                      // entry e of a value head goes to v_to[e page_size]
    if (slot >= 0 && (a.values_are_keys ? is_k : !is_q && !is_k)) {
        const int g = a.values_are_keys ? u - a.nq : u - a.nq - a.nk;
        v_to = (T*)a.v_cache + ((size_t)(slot / a.page_size) * a.nv * a.dv + (size_t)g * a.dv) * a.page_size
               + slot % a.page_size;
    }
    auto raw = [&](float (&to)[W], int e) {
        if constexpr (W == 4) {
            load4(to, x + e);
            if (bias) {
                float b[4];
                load4(b, bias + e);
#pragma unroll
                for (int i = 0; i < 4; ++i) to[i] += b[i];
            }
        } else {
            to[0] = bias ? x[e] + bias[e] : x[e];
        }
    };
    float v[ITEMS][W], ss = 0.f;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int e = (lane + L * k) * W;
#pragma unroll
        for (int i = 0; i < W; ++i) v[k][i] = 0.f;
        if (on && e < width) raw(v[k], e);
#pragma unroll
        for (int i = 0; i < W; ++i) {
            ss = fmaf(v[k][i], v[k][i], ss);
            if (v_to && on && e < width) v_to[(size_t)(e + i) * a.page_size] = from_f32<T>(v[k][i]);
        }
    }
    const float* weight = is_q ? a.q_weight : is_k ? a.k_weight : nullptr;
    float inv = 1.f;
    if (a.q_weight) {                       // the same condition in every lane
#pragma unroll
        for (int off = L / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, L);
        inv = 1.f / sqrtf(ss / (float)width + a.eps);
    }
    if (!on || (!is_q && !is_k)) return;
    float by = 1.f;
    if (is_q && a.every > 0.f)
        by = fmaf(a.coef, logf((float)(floor((double)(a.positions[t] + 1) / (double)a.every) + 1.0)), 1.f);
    const int turned = a.table ? a.rot / 2 : 0;
    const float* angle = a.table ? a.table + (size_t)a.positions[t] * a.rot : nullptr;
    auto weighed = [&](float (&to)[W], int e) {
        if (!weight) return;
        if constexpr (W == 4) {
            float w[4];
            load4(w, weight + e);
#pragma unroll
            for (int i = 0; i < 4; ++i) to[i] = to[i] * inv * w[i];
        } else {
            to[0] = to[0] * inv * weight[e];
        }
    };
    T* to = is_q ? (T*)a.q_out + (size_t)t * a.nq * a.d + col0
                 : (slot >= 0 ? (T*)a.k_cache + (size_t)slot * a.nk * a.d + (col0 - a.nq * a.d) : nullptr);
    if (!to) return;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int e = (lane + L * k) * W;
        if (e >= width) continue;
        weighed(v[k], e);
        if (e < 2 * turned) {
            if (a.half) {                   // W divides turned: all of a lane's entries are on one side
                const bool upper = e >= turned;
                float o[W];
                raw(o, upper ? e - turned : e + turned);
                weighed(o, upper ? e - turned : e + turned);
                const float* cs = angle + (upper ? e - turned : e);
#pragma unroll
                for (int i = 0; i < W; ++i) {
                    const float s = cs[turned + i];
                    v[k][i] = fmaf(v[k][i], cs[i], upper ? o[i] * s : -(o[i] * s));
                }
            } else if constexpr (W == 1) {
                float o[1];
                raw(o, e ^ 1);
                weighed(o, e ^ 1);
                const float s = angle[turned + e / 2];
                v[k][0] = fmaf(v[k][0], angle[e / 2], e & 1 ? o[0] * s : -(o[0] * s));
            } else {
#pragma unroll
                for (int i = 0; i < W; i += 2) {
                    if (e + i >= 2 * turned) continue;
                    const float c = angle[(e + i) / 2], s = angle[turned + (e + i) / 2], first = v[k][i];
                    v[k][i] = fmaf(first, c, -(v[k][i + 1] * s));
                    v[k][i + 1] = fmaf(v[k][i + 1], c, first * s);
                }
            }
        }
        if constexpr (W == 4) {
            typedef T four __attribute__((ext_vector_type(4)));
            *reinterpret_cast<four*>(to + e) = four{from_f32<T>(v[k][0] * by), from_f32<T>(v[k][1] * by),
                                                    from_f32<T>(v[k][2] * by), from_f32<T>(v[k][3] * by)};
        } else {
            to[e] = from_f32<T>(v[k][0] * by);
        }
    }
}

static bool ah_in_sixteens(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

template <typename T>
static void launch_attention_heads(const HeadsArgs& a, int T_, bool quads, hipStream_t stream) {
    const int heads = a.nq + a.nk + (a.values_are_keys ? 0 : a.nv);
    const int most = a.values_are_keys || a.d > a.dv ? a.d : a.dv;
#define LC_AH(W, L, ITEMS)                                                                                              \
    attention_heads_kernel<T, W, L, ITEMS>                                                                              \
        <<<dim3(T_, (heads + AH_THREADS / L - 1) / (AH_THREADS / L)), AH_THREADS, 0, stream>>>(a)
    if (!quads) LC_AH(1, 64, 4);
    else if (most <= 32) LC_AH(4, 8, 1);
    else if (most <= 64) LC_AH(4, 16, 1);
    else if (most <= 128) LC_AH(4, 32, 1);
    else LC_AH(4, 64, 1);
#undef LC_AH
}

}  // namespace lc

using namespace lc;

// proj [T, cols]; the rows of the cache at places rows[t] (page * page_size + place in the page; -1 or null: not written)
LC_API int lc_attention_heads(const float* proj, int cols, int T, int nq, int nk, int nv, int d, int dv,
                              int values_are_keys, const float* bias, const float* q_weight, const float* k_weight,
                              float eps, const float* table, int rot, int half, const int* positions, float coef,
                              float every, void* q_out, void* k_cache, void* v_cache, int dt, const int* rows,
                              int page_size, hipStream_t stream) {
    LC_CHECK(T >= 0 && nq > 0 && nk > 0 && nv > 0 && d > 0 && dv > 0 && d <= AH_MAX && dv <= AH_MAX,
             "attention heads: bad sizes");
    LC_CHECK(!values_are_keys || (nv == nk && dv == d), "attention heads: values that are the keys have their sizes");
    LC_CHECK(cols >= (nq + nk) * d + (values_are_keys ? 0 : nv * dv), "attention heads: %d columns are too few", cols);
    if (T == 0) return 0;
    LC_CHECK(proj && q_out, "attention heads: null pointer");
    LC_CHECK((q_weight == nullptr) == (k_weight == nullptr), "attention heads: q and k are normed together");
    LC_CHECK(!table || (rot > 0 && rot % 2 == 0 && rot <= d && positions), "attention heads: bad rotation");
    LC_CHECK(every <= 0.f || positions, "attention heads: a temperature without positions");
    LC_CHECK(!rows || (k_cache && v_cache && page_size > 0), "attention heads: rows without a cache");
    const HeadsArgs a{proj, cols, nq, nk, nv, d, dv, values_are_keys, bias, q_weight, k_weight, eps, table, rot, half,
                      positions, coef, every, q_out, k_cache, v_cache, rows, page_size};
    const bool quads = d % 4 == 0 && dv % 4 == 0 && cols % 4 == 0 && (!table || rot % (half ? 8 : 2) == 0) &&
                       ah_in_sixteens(proj) && ah_in_sixteens(bias) && ah_in_sixteens(q_weight) &&
                       ah_in_sixteens(k_weight) && ah_in_sixteens(q_out) && ah_in_sixteens(k_cache);
    if (dt == DT_F32) launch_attention_heads<float>(a, T, quads, stream);
    else if (dt == DT_BF16) launch_attention_heads<bf16>(a, T, quads, stream);
    else LC_CHECK(false, "attention heads: unknown dtype %d", dt);
    LC_LAUNCH_CHECK("attention_heads");
    return 0;
}
