// What joins a layer's branches to the residual stream where several of them wait at once, and norms the sum with one
// or two weights (a layer whose mixer and feed-forward read the same stream, each behind a norm of its own):
//   v = h + sum over the addends of scale * addend;  inv = 1 / sqrt(mean(v^2) + eps);  out_k = v inv w_k
// An addend is a tensor [T, n] (float32 or bfloat16), the float32 shares [count][T][n] of a product that was cut along
// its inner size, summed in their order, or a mixture of experts' rows: sum over a token's `count` choices of their
// weight times the row that the choice's place names.  All arithmetic is float32.
#include "common.h"

namespace lc {

enum : int { ADD_NONE = 0, ADD_F32 = 1, ADD_BF16 = 2, ADD_SHARES = 3, ADD_ROUTED = 4 };

struct Addend {
    const void* p;
    int kind, count;
    float scale;
    const float* weights;       // routed: [T, count]
    const int* places;          // routed: [T, count] rows of p
};

constexpr int ADDENDS = 3;

struct NormsArgs {
    float* h;
    const int* rows;
    Addend add[ADDENDS];
    size_t share_stride;        // T n
    const float* w1;
    const float* w2;
    float eps;
    void* out1;
    void* out2;
    int n, write_h;
};

template <int W> __device__ __forceinline__ void load_f32(float (&to)[W], const float* p) {
    if constexpr (W == 1) {
        to[0] = *p;
    } else {
        typedef float four __attribute__((ext_vector_type(4)));
#pragma unroll
        for (int i = 0; i < W; i += 4) {
            const four q = *reinterpret_cast<const four*>(p + i);
            to[i] = q.x; to[i + 1] = q.y; to[i + 2] = q.z; to[i + 3] = q.w;
        }
    }
}
template <int W> __device__ __forceinline__ void load_bf16(float (&to)[W], const bf16* p) {
    if constexpr (W == 1) {
        to[0] = to_f32(*p);
    } else {
        typedef __bf16 eight __attribute__((ext_vector_type(8)));
#pragma unroll
        for (int i = 0; i < W; i += 8) {
            const eight q = *reinterpret_cast<const eight*>(p + i);
#pragma unroll
            for (int k = 0; k < 8; ++k) to[i + k] = static_cast<float>(q[k]);
        }
    }
}

// to += scale * (entries i .. i + W - 1 of the addend's row src)
template <int W>
__device__ __forceinline__ void take_in(float (&to)[W], const Addend& a, size_t src, int n, int i, size_t share_stride) {
    float x[W];
    if (a.kind == ADD_F32) {
        load_f32<W>(x, (const float*)a.p + src * n + i);
    } else if (a.kind == ADD_BF16) {
        load_bf16<W>(x, (const bf16*)a.p + src * n + i);
    } else if (a.kind == ADD_SHARES) {
#pragma unroll
        for (int k = 0; k < W; ++k) x[k] = 0.f;
#pragma unroll 4
        for (int s = 0; s < a.count; ++s) {
            float y[W];
            load_f32<W>(y, (const float*)a.p + s * share_stride + src * n + i);
#pragma unroll
            for (int k = 0; k < W; ++k) x[k] += y[k];
        }
    } else {
#pragma unroll
        for (int k = 0; k < W; ++k) x[k] = 0.f;
#pragma unroll 4
        for (int s = 0; s < a.count; ++s) {
            float y[W];
            const float by = a.weights[src * a.count + s];
            load_f32<W>(y, (const float*)a.p + (size_t)a.places[src * a.count + s] * n + i);
#pragma unroll
            for (int k = 0; k < W; ++k) x[k] = fmaf(by, y[k], x[k]);
        }
    }
#pragma unroll
    for (int k = 0; k < W; ++k) to[k] = fmaf(a.scale, x[k], to[k]);
}

template <typename T, int W>
__device__ __forceinline__ void put(T* to, const float (&v)[W], float inv, const float (&w)[W]) {
    if constexpr (W == 1) {
        *to = from_f32<T>(v[0] * inv * w[0]);
    } else {
        constexpr int AT = 16 / sizeof(T);
        typedef T piece __attribute__((ext_vector_type(AT)));
#pragma unroll
        for (int i = 0; i < W; i += AT) {
            piece q;
#pragma unroll
            for (int k = 0; k < AT; ++k) q[k] = from_f32<T>(v[i + k] * inv * w[i + k]);
            *reinterpret_cast<piece*>(to + i) = q;
        }
    }
}

// One workgroup per output row r; src row = rows ? rows[r] : r.  A thread holds its entries in registers: THREADS W ITEMS
// entries a row at most.
template <typename T, int W, int THREADS, int ITEMS>
__global__ __launch_bounds__(THREADS) void stream_norms_kernel(NormsArgs a) {
    __shared__ float scratch[16];
    const int r = blockIdx.x, n = a.n;
    const size_t src = a.rows ? a.rows[r] : r;
    float v[ITEMS][W], ss = 0.f;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int i = (threadIdx.x + k * THREADS) * W;
        if (i < n) load_f32<W>(v[k], a.h + src * n + i);
    }
#pragma unroll
    for (int x = 0; x < ADDENDS; ++x)
        if (a.add[x].kind != ADD_NONE)
#pragma unroll
            for (int k = 0; k < ITEMS; ++k) {
                const int i = (threadIdx.x + k * THREADS) * W;
                if (i < n) take_in<W>(v[k], a.add[x], src, n, i, a.share_stride);
            }
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int i = (threadIdx.x + k * THREADS) * W;
        if (i < n)
#pragma unroll
            for (int e = 0; e < W; ++e) {
                ss = fmaf(v[k][e], v[k][e], ss);
                if (a.write_h) a.h[src * n + i + e] = v[k][e];
            }
    }
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)n + a.eps);
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int i = (threadIdx.x + k * THREADS) * W;
        if (i >= n) continue;
        float w[W];
        load_f32<W>(w, a.w1 + i);
        put<T, W>((T*)a.out1 + (size_t)r * n + i, v[k], inv, w);
        if (a.w2) {
            load_f32<W>(w, a.w2 + i);
            put<T, W>((T*)a.out2 + (size_t)r * n + i, v[k], inv, w);
        }
    }
}

// Rows of any length: a thread makes its entries anew for the second pass where the stream is not written.
template <typename T>
__global__ void stream_norms_any_kernel(NormsArgs a) {
    __shared__ float scratch[16];
    const int r = blockIdx.x, n = a.n;
    const size_t src = a.rows ? a.rows[r] : r;
    auto joined = [&](int i) {
        float v[1] = {a.h[src * n + i]};
#pragma unroll
        for (int x = 0; x < ADDENDS; ++x)
            if (a.add[x].kind != ADD_NONE) take_in<1>(v, a.add[x], src, n, i, a.share_stride);
        return v[0];
    };
    float ss = 0.f;
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const float v = joined(i);
        ss = fmaf(v, v, ss);
        if (a.write_h) a.h[src * n + i] = v;
    }
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)n + a.eps);
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const float v = a.write_h ? a.h[src * n + i] : joined(i);
        ((T*)a.out1)[(size_t)r * n + i] = from_f32<T>(v * inv * a.w1[i]);
        if (a.w2) ((T*)a.out2)[(size_t)r * n + i] = from_f32<T>(v * inv * a.w2[i]);
    }
}

static bool sn_in_sixteens(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

template <typename T>
static void launch_stream_norms(const NormsArgs& a, int R, hipStream_t stream) {
    const int n = a.n;
    bool vec = n % 8 == 0 && n <= 8192 && sn_in_sixteens(a.h) && sn_in_sixteens(a.w1) && sn_in_sixteens(a.w2) &&
               sn_in_sixteens(a.out1) && sn_in_sixteens(a.out2);
    for (const Addend& x : a.add) vec = vec && (x.kind == ADD_NONE || sn_in_sixteens(x.p));
    // the kernel's shape, and with it the grouping of a row's sum, follows from n alone
    if (!vec) stream_norms_any_kernel<T><<<R, n >= 1024 ? 256 : (n >= 256 ? 128 : 64), 0, stream>>>(a);
    else if (n <= 512) stream_norms_kernel<T, 8, 64, 1><<<R, 64, 0, stream>>>(a);
    else if (n <= 2048) stream_norms_kernel<T, 8, 256, 1><<<R, 256, 0, stream>>>(a);
    else if (n <= 4096) stream_norms_kernel<T, 8, 512, 1><<<R, 512, 0, stream>>>(a);
    else stream_norms_kernel<T, 8, 512, 2><<<R, 512, 0, stream>>>(a);
}

}  // namespace lc

using namespace lc;

// h float32 [T, n]; rows int32 [R] or null (R = T); up to three addends; w2, out2 null: one norm.  write_h: h becomes the
// sum (not with rows).
LC_API int lc_stream_norms(float* h, const int* rows, int R, int T, int n, int write_h,
                           const void* p0, int kind0, int count0, float scale0, const float* weights0, const int* places0,
                           const void* p1, int kind1, int count1, float scale1, const float* weights1, const int* places1,
                           const void* p2, int kind2, int count2, float scale2, const float* weights2, const int* places2,
                           const float* w1, const float* w2, float eps, void* out1, void* out2, int dt,
                           hipStream_t stream) {
    LC_CHECK(R >= 0 && T >= 0 && n > 0, "stream norms: bad sizes R=%d T=%d n=%d", R, T, n);
    if (R == 0) return 0;
    LC_CHECK(h && w1 && out1 && (w2 == nullptr) == (out2 == nullptr), "stream norms: null pointer");
    LC_CHECK(!(rows && write_h) && (rows || R == T), "stream norms: gathered rows cannot be written back");
    NormsArgs a{h, rows,
                {{p0, kind0, count0, scale0, weights0, places0}, {p1, kind1, count1, scale1, weights1, places1},
                 {p2, kind2, count2, scale2, weights2, places2}},
                (size_t)T * n, w1, w2, eps, out1, out2, n, write_h};
    for (const Addend& x : a.add) {
        LC_CHECK(x.kind >= ADD_NONE && x.kind <= ADD_ROUTED && (x.kind == ADD_NONE || x.p), "stream norms: bad addend");
        LC_CHECK(x.kind < ADD_SHARES || x.count > 0, "stream norms: an addend of no parts");
        LC_CHECK(x.kind != ADD_ROUTED || (x.weights && x.places), "stream norms: routed rows without their routing");
    }
    if (dt == DT_F32) launch_stream_norms<float>(a, R, stream);
    else if (dt == DT_BF16) launch_stream_norms<bf16>(a, R, stream);
    else LC_CHECK(false, "stream norms: unknown dtype %d", dt);
    LC_LAUNCH_CHECK("stream_norms");
    return 0;
}
