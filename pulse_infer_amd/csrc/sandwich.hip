// The residual update of a layer whose sublayers have a norm before AND after them, and the embedding with a norm.
//
// pulse_sandwich_step, for output row r (token t = rows ? rows[r] : r), in one pass over the row:
//   1. the sublayer's result: y = y1[t], or, as a sum of normed terms,
//          y = term_scale * sum_i y_i[t] / sqrt(mean(y_i[t]^2) + term_eps) * term_w_i          (one or two terms)
//   2. its norm:  layer norm (y - mean) / sqrt(var + eps) * w + b, RMS norm y / sqrt(mean(y^2) + eps) * w, or none
//   3. h[t] += that        (float32; not stored with a list of rows: who gathers rows reads the residual last)
//   4. the norm that reads the residual next (of the same two kinds), rounded once into out[r]   (optional)
// A row lies in the registers of one workgroup, so means and variances are formed in two passes over exact values;
// everything is float32 up to the store.
//
// pulse_embed_norm: out[t] = norm(table[ids[t]] * scale), the row's own norm included in the gather.
#include "common.h"

#include <math.h>

namespace {

enum NormKind : int { LAYER_NORM = 0, RMS_NORM = 1, NO_NORM = 2 };

struct SandwichArgs {
    int hidden;
    int terms;                 // 0: y1 as it is; 1, 2: normed terms
    float term_scale, term_eps;
    int post_kind, pre_kind;
    float post_eps, pre_eps;
    int has_out;
};

template <typename T, int VEC> struct Pack;
template <> struct Pack<float, 4> { typedef float4 type; };
template <> struct Pack<bf16_t, 4> { typedef ushort4 type; };

template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const T* p, int64_t i, float* v) {
    if constexpr (VEC == 4) {
        const typename Pack<T, 4>::type raw = reinterpret_cast<const typename Pack<T, 4>::type*>(p)[i];
        v[0] = to_f32<T>(raw.x); v[1] = to_f32<T>(raw.y); v[2] = to_f32<T>(raw.z); v[3] = to_f32<T>(raw.w);
    } else {
        v[0] = to_f32<T>(p[i]);
    }
}

template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, int64_t i, const float* v) {
    if constexpr (VEC == 4) {
        typename Pack<T, 4>::type raw;
        raw.x = from_f32<T>(v[0]); raw.y = from_f32<T>(v[1]); raw.z = from_f32<T>(v[2]); raw.w = from_f32<T>(v[3]);
        reinterpret_cast<typename Pack<T, 4>::type*>(p)[i] = raw;
    } else {
        p[i] = from_f32<T>(v[0]);
    }
}

// THREADS threads a row, each with CHUNKS pieces of VEC neighbouring values.
template <typename TY, typename TW, typename TO, int VEC, int THREADS, int CHUNKS>
__global__ __launch_bounds__(THREADS) void sandwich_step_kernel(float* __restrict__ h, const TY* __restrict__ y1,
                                                                const TY* __restrict__ y2, const TW* __restrict__ tw1,
                                                                const TW* __restrict__ tw2, const TW* __restrict__ post_w,
                                                                const TW* __restrict__ post_b, const int* __restrict__ rows,
                                                                const TW* __restrict__ pre_w, const TW* __restrict__ pre_b,
                                                                TO* __restrict__ out, SandwichArgs a) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int64_t t = rows ? rows[r] : r;
    const int nvec = a.hidden / VEC;
    const float n = static_cast<float>(a.hidden);
    float* hrow = h + t * a.hidden;
    float y[CHUNKS][VEC], z[CHUNKS][VEC];
    // the residual is asked for first: its trip lies behind the norms of the update
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * THREADS;
#pragma unroll
        for (int u = 0; u < VEC; ++u) y[c][u] = z[c][u] = 0.f;
        if (i < nvec) load_vec<float, VEC>(hrow, i, z[c]);
    }
    if (a.terms == 0) {
#pragma unroll
        for (int c = 0; c < CHUNKS; ++c) {
            const int i = threadIdx.x + c * THREADS;
            if (i < nvec) load_vec<TY, VEC>(y1 + t * a.hidden, i, y[c]);
        }
    } else {
        for (int term = 0; term < a.terms; ++term) {
            const TY* src = (term ? y2 : y1) + t * a.hidden;
            const TW* w = term ? tw2 : tw1;
            float v[CHUNKS][VEC];
            float ss = 0.f;
#pragma unroll
            for (int c = 0; c < CHUNKS; ++c) {
                const int i = threadIdx.x + c * THREADS;
                if (i < nvec) {
                    load_vec<TY, VEC>(src, i, v[c]);
#pragma unroll
                    for (int u = 0; u < VEC; ++u) ss = fmaf(v[c][u], v[c][u], ss);
                }
            }
            const float inv = a.term_scale / sqrtf(block_sum(ss, scratch) / n + a.term_eps);
#pragma unroll
            for (int c = 0; c < CHUNKS; ++c) {
                const int i = threadIdx.x + c * THREADS;
                if (i < nvec) {
                    float ww[VEC];
                    load_vec<TW, VEC>(w, i, ww);
#pragma unroll
                    for (int u = 0; u < VEC; ++u) y[c][u] = fmaf(v[c][u] * inv, ww[u], y[c][u]);
                }
            }
        }
    }
    // (mean and inverse deviation of a row in registers; an RMS norm has no mean)
    auto statistics = [&](const float (&v)[CHUNKS][VEC], int kind, float eps, float& mean, float& inv) __attribute__((always_inline)) {
        mean = 0.f;
        if (kind == LAYER_NORM) {
            float sum = 0.f;
#pragma unroll
            for (int c = 0; c < CHUNKS; ++c)
#pragma unroll
                for (int u = 0; u < VEC; ++u) sum += v[c][u];    // (places beyond the row hold zeros)
            mean = block_sum(sum, scratch) / n;
        }
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < CHUNKS; ++c) {
            const int i = threadIdx.x + c * THREADS;
            if (i < nvec) {
#pragma unroll
                for (int u = 0; u < VEC; ++u) { const float d = v[c][u] - mean; sq = fmaf(d, d, sq); }
            }
        }
        inv = 1.0f / sqrtf(block_sum(sq, scratch) / n + eps);
    };
    float mean = 0.f, inv = 1.f;
    if (a.post_kind != NO_NORM) statistics(y, a.post_kind, a.post_eps, mean, inv);
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * THREADS;
        if (i < nvec) {
            if (a.post_kind != NO_NORM) {
                float ww[VEC];
                load_vec<TW, VEC>(post_w, i, ww);
#pragma unroll
                for (int u = 0; u < VEC; ++u) y[c][u] = (y[c][u] - mean) * inv * ww[u];
                if (post_b) {
                    load_vec<TW, VEC>(post_b, i, ww);
#pragma unroll
                    for (int u = 0; u < VEC; ++u) y[c][u] += ww[u];
                }
            }
#pragma unroll
            for (int u = 0; u < VEC; ++u) z[c][u] += y[c][u];
            if (!rows) store_vec<float, VEC>(hrow, i, z[c]);
        }
    }
    if (!a.has_out) return;
    statistics(z, a.pre_kind, a.pre_eps, mean, inv);
    TO* orow = out + static_cast<int64_t>(r) * a.hidden;
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * THREADS;
        if (i < nvec) {
            float ww[VEC], o[VEC];
            load_vec<TW, VEC>(pre_w, i, ww);
#pragma unroll
            for (int u = 0; u < VEC; ++u) o[u] = (z[c][u] - mean) * inv * ww[u];
            if (pre_b) {
                load_vec<TW, VEC>(pre_b, i, ww);
#pragma unroll
                for (int u = 0; u < VEC; ++u) o[u] += ww[u];
            }
            store_vec<TO, VEC>(orow, i, o);
        }
    }
}

template <typename TT, typename TW>
__global__ __launch_bounds__(256) void embed_norm_kernel(const int* __restrict__ ids, const TT* __restrict__ table,
                                                         const TW* __restrict__ w, float* __restrict__ out, int hidden,
                                                         int vocab, int* bad_id, float scale, int kind, float eps) {
    __shared__ float scratch[16];
    const int t = blockIdx.x;
    const int id = ids[t];
    float* dst = out + static_cast<int64_t>(t) * hidden;
    if (id < 0 || id >= vocab) {   // (as in the plain gather: a row of NaN, never a silent row of zeros)
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = __builtin_nanf("");
        if (threadIdx.x == 0) *bad_id = 1;
        return;
    }
    const TT* src = table + static_cast<int64_t>(id) * hidden;
    const float n = static_cast<float>(hidden);
    float mean = 0.f;
    if (kind == LAYER_NORM) {
        float sum = 0.f;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) sum += to_f32<TT>(src[i]) * scale;
        mean = block_sum(sum, scratch) / n;
    }
    float sq = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float d = to_f32<TT>(src[i]) * scale - mean;
        sq = fmaf(d, d, sq);
    }
    const float inv = 1.0f / sqrtf(block_sum(sq, scratch) / n + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x)
        dst[i] = (to_f32<TT>(src[i]) * scale - mean) * inv * to_f32<TW>(w[i]);
}

bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

}  // namespace

// h [tokens, hidden] float32; y1, y2 [tokens, hidden] of one storage type; all weights of one storage type, biases may
// be null.  kinds: 0 layer norm, 1 RMS norm, 2 (post only) none.  out [n_rows, hidden] or null.
extern "C" int pulse_sandwich_step(float* h, int tokens, int hidden, const void* y1, const void* y2, int y_dtype, int terms,
                                   const void* term_w1, const void* term_w2, float term_scale, float term_eps, int post_kind,
                                   const void* post_w, const void* post_b, float post_eps, const int* rows, int n_rows,
                                   int pre_kind, const void* pre_w, const void* pre_b, float pre_eps, int w_dtype, void* out,
                                   int out_dtype, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && n_rows >= 0 && hidden > 0 && h && y1, "sandwich_step: bad sizes or null pointer");
    PULSE_REQUIRE(pulse_dtype_ok(y_dtype) && pulse_dtype_ok(w_dtype) && pulse_dtype_ok(out_dtype), "sandwich_step: bad dtype tag");
    PULSE_REQUIRE(terms >= 0 && terms <= 2 && (terms < 1 || term_w1) && (terms < 2 || (y2 && term_w2)),
                  "sandwich_step: a sum of %d normed terms needs as many results and weights", terms);
    PULSE_REQUIRE(post_kind >= 0 && post_kind <= 2 && (post_kind == NO_NORM || post_w), "sandwich_step: the update's norm has no weight");
    PULSE_REQUIRE(!out || ((pre_kind == 0 || pre_kind == 1) && pre_w), "sandwich_step: the next norm has no weight");
    PULSE_REQUIRE(out || !rows, "sandwich_step: an update of gathered rows is not stored, so it comes with a norm");
    PULSE_REQUIRE(rows || n_rows == tokens, "sandwich_step: %d rows of %d tokens without a list of rows", n_rows, tokens);
    if (n_rows == 0) return 0;
    SandwichArgs a;
    a.hidden = hidden; a.terms = terms; a.term_scale = term_scale; a.term_eps = term_eps; a.post_kind = post_kind;
    a.pre_kind = pre_kind; a.post_eps = post_eps; a.pre_eps = pre_eps; a.has_out = out ? 1 : 0;
    const bool vec = hidden % 4 == 0 && aligned16(h) && aligned16(y1) && aligned16(y2) && aligned16(term_w1) &&
                     aligned16(term_w2) && aligned16(post_w) && aligned16(post_b) && aligned16(pre_w) && aligned16(pre_b) &&
                     aligned16(out);
    const int pieces = vec ? hidden / 4 : hidden;
    PULSE_REQUIRE(pieces <= 1024 * 8, "sandwich_step: rows of %d values are too long", hidden);
    // few rows of a wide residual (a decoding step): wider workgroups, since there are not many of them
    const bool wide = pieces > 256 * 8 || (n_rows <= 256 && pieces >= 512);
#define PULSE_SANDWICH(VEC_, THREADS_, CHUNKS_)                                                                         \
    PULSE_DISPATCH_DTYPE(y_dtype, TY, PULSE_DISPATCH_DTYPE(w_dtype, TW, PULSE_DISPATCH_DTYPE(out_dtype, TO,             \
        hipLaunchKernelGGL((sandwich_step_kernel<TY, TW, TO, VEC_, THREADS_, CHUNKS_>), dim3(n_rows), dim3(THREADS_), 0, \
                           stream, h, static_cast<const TY*>(y1), static_cast<const TY*>(y2),                           \
                           static_cast<const TW*>(term_w1), static_cast<const TW*>(term_w2),                            \
                           static_cast<const TW*>(post_w), static_cast<const TW*>(post_b), rows,                        \
                           static_cast<const TW*>(pre_w), static_cast<const TW*>(pre_b), static_cast<TO*>(out), a))))
    if (vec) {
        if (wide && pieces <= 1024 * 2) PULSE_SANDWICH(4, 1024, 2);
        else if (wide) PULSE_SANDWICH(4, 1024, 8);
        else if (pieces <= 256 * 2) PULSE_SANDWICH(4, 256, 2);
        else if (pieces <= 256 * 4) PULSE_SANDWICH(4, 256, 4);
        else PULSE_SANDWICH(4, 256, 8);
    } else {
        if (wide) PULSE_SANDWICH(1, 1024, 8);
        else PULSE_SANDWICH(1, 256, 8);
    }
#undef PULSE_SANDWICH
    PULSE_LAUNCH_CHECK("sandwich_step");
    return 0;
}

extern "C" int pulse_embed_norm(const int* ids, const void* table, int table_dtype, const void* w, int w_dtype, int kind,
                                float eps, float* out, int tokens, int hidden, int vocab, int* bad_id, float scale,
                                hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0, "embed_norm: bad sizes T=%d H=%d V=%d", tokens, hidden, vocab);
    PULSE_REQUIRE(pulse_dtype_ok(table_dtype) && pulse_dtype_ok(w_dtype) && (kind == 0 || kind == 1), "embed_norm: bad tag");
    PULSE_REQUIRE(ids && table && w && out && bad_id, "embed_norm: null pointer");
    if (tokens == 0) return 0;
    PULSE_DISPATCH_DTYPE(table_dtype, TT, PULSE_DISPATCH_DTYPE(w_dtype, TW,
        hipLaunchKernelGGL((embed_norm_kernel<TT, TW>), dim3(tokens), dim3(256), 0, stream, ids,
                           static_cast<const TT*>(table), static_cast<const TW*>(w), out, hidden, vocab, bad_id, scale,
                           kind, eps)));
    PULSE_LAUNCH_CHECK("embed_norm");
    return 0;
}
