// The end of a layer whose sublayers read the same residual, and what reads the residual next, in one pass over the row.
//
// pulse_residual_norms, for output row r (token t = rows ? rows[r] : r):
//   v = h[t] + a[t] (the sum of `a_parts` matrices) + b[t] + row + sum_k weight[t, k] * y[t * top + k]
// (each term optional; `y` are the results of the experts a token chose, in float32, k in the order of choice; an index
// that names no expert adds nothing), h[t] = v (float32; not stored with a list of rows: who gathers rows reads the
// residual last), and up to two outputs
//   out_i[r] = v / sqrt(mean(v^2) + eps_i) * w_i        or, without a weight, v itself, rounded once
// with a row stride each, so that one of them may be columns of a wider matrix.
// A row lies in the registers of one workgroup; all arithmetic is float32.
#include "common.h"

#include <math.h>

namespace {

struct RowTerms {
    const void* a; int a_tag, a_parts; int64_t a_stride;
    const void* b; int b_tag;
    const void* row; int row_tag;
    const float* y; const int* idx; const float* weight; int experts, top;
};

struct RowOuts {
    void* out[2];
    const void* w[2];
    int64_t stride[2];
    float eps[2];
};

// VEC neighbouring values of a matrix of either storage type (the same in every lane: a uniform branch), added to v.
template <int VEC>
__device__ __forceinline__ void add_any(const void* p, int tag, int64_t at, float* v) {
    if constexpr (VEC == 4) {
        if (tag == PULSE_F32) {
            const float4 d = *reinterpret_cast<const float4*>(static_cast<const float*>(p) + at);
            v[0] += d.x; v[1] += d.y; v[2] += d.z; v[3] += d.w;
        } else {
            const ushort4 d = *reinterpret_cast<const ushort4*>(static_cast<const bf16_t*>(p) + at);
            v[0] += bf16_to_f32(d.x); v[1] += bf16_to_f32(d.y); v[2] += bf16_to_f32(d.z); v[3] += bf16_to_f32(d.w);
        }
    } else {
        v[0] += tag == PULSE_F32 ? static_cast<const float*>(p)[at] : bf16_to_f32(static_cast<const bf16_t*>(p)[at]);
    }
}

// THREADS threads a row, each with CHUNKS pieces of VEC neighbouring values.
template <typename TW, typename TO, int VEC, int THREADS, int CHUNKS>
__global__ __launch_bounds__(THREADS) void residual_norms_kernel(float* __restrict__ h, const int* __restrict__ rows,
                                                                 RowTerms in, RowOuts o, int hidden, int write_back) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int64_t t = rows ? rows[r] : r;
    const int nvec = hidden / VEC;
    const int64_t base = t * hidden;
    float v[CHUNKS][VEC];
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * THREADS;
#pragma unroll
        for (int u = 0; u < VEC; ++u) v[c][u] = 0.f;
        if (i < nvec) {
            const int64_t at = base + static_cast<int64_t>(i) * VEC;
            add_any<VEC>(h, PULSE_F32, at, v[c]);
            for (int p = 0; in.a && p < in.a_parts; ++p) add_any<VEC>(in.a, in.a_tag, p * in.a_stride + at, v[c]);
            if (in.b) add_any<VEC>(in.b, in.b_tag, at, v[c]);
            if (in.row) add_any<VEC>(in.row, in.row_tag, static_cast<int64_t>(i) * VEC, v[c]);
        }
    }
    if (in.y) {
#pragma unroll 4
        for (int k = 0; k < in.top; ++k) {
            const int64_t pair = t * in.top + k;
            const int e = in.idx[pair];
            if (e < 0 || e >= in.experts) continue;
            const float w = in.weight ? in.weight[pair] : 1.f;
            const float* yrow = in.y + pair * hidden;
#pragma unroll
            for (int c = 0; c < CHUNKS; ++c) {
                const int i = threadIdx.x + c * THREADS;
                if (i < nvec) {
                    float d[VEC];
#pragma unroll
                    for (int u = 0; u < VEC; ++u) d[u] = 0.f;
                    add_any<VEC>(yrow, PULSE_F32, static_cast<int64_t>(i) * VEC, d);
#pragma unroll
                    for (int u = 0; u < VEC; ++u) v[c][u] = fmaf(w, d[u], v[c][u]);
                }
            }
        }
    }
    float mean = 0.f;
    if (o.w[0] || o.w[1]) {
        float ss = 0.f;
#pragma unroll
        for (int c = 0; c < CHUNKS; ++c)
#pragma unroll
            for (int u = 0; u < VEC; ++u) ss = fmaf(v[c][u], v[c][u], ss);
        mean = block_sum(ss, scratch) / static_cast<float>(hidden);
    }
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * THREADS;
        if (i < nvec && write_back) {
            if constexpr (VEC == 4)
                *reinterpret_cast<float4*>(h + base + static_cast<int64_t>(i) * 4) = make_float4(v[c][0], v[c][1], v[c][2], v[c][3]);
            else
                h[base + i] = v[c][0];
        }
    }
#pragma unroll
    for (int which = 0; which < 2; ++which) {
        if (!o.out[which]) continue;
        const float inv = o.w[which] ? 1.0f / sqrtf(mean + o.eps[which]) : 1.0f;
        TO* out = static_cast<TO*>(o.out[which]) + static_cast<int64_t>(r) * o.stride[which];
        const TW* w = static_cast<const TW*>(o.w[which]);
#pragma unroll
        for (int c = 0; c < CHUNKS; ++c) {
            const int i = threadIdx.x + c * THREADS;
            if (i >= nvec) continue;
            float f[VEC], x[VEC];
#pragma unroll
            for (int u = 0; u < VEC; ++u) f[u] = 0.f;
            if (w) add_any<VEC>(w, sizeof(TW) == 4 ? PULSE_F32 : PULSE_BF16, static_cast<int64_t>(i) * VEC, f);
#pragma unroll
            for (int u = 0; u < VEC; ++u) x[u] = w ? v[c][u] * inv * f[u] : v[c][u];
            if constexpr (VEC == 4) {
                if constexpr (sizeof(TO) == 4)
                    *reinterpret_cast<float4*>(out + static_cast<int64_t>(i) * 4) = make_float4(x[0], x[1], x[2], x[3]);
                else
                    *reinterpret_cast<ushort4*>(out + static_cast<int64_t>(i) * 4) =
                        make_ushort4(f32_to_bf16(x[0]), f32_to_bf16(x[1]), f32_to_bf16(x[2]), f32_to_bf16(x[3]));
            } else {
                out[i] = from_f32<TO>(x[0]);
            }
        }
    }
}

template <typename TW, typename TO, int VEC, int THREADS>
bool launch_rows(int chunks, float* h, const int* rows, const RowTerms& in, const RowOuts& o, int out_rows, int hidden,
                 int write_back, hipStream_t stream) {
#define PULSE_ROWS_LAUNCH(C)                                                                                          \
    hipLaunchKernelGGL((residual_norms_kernel<TW, TO, VEC, THREADS, C>), dim3(out_rows), dim3(THREADS), 0, stream, h, \
                       rows, in, o, hidden, write_back)
    if (chunks <= 1) PULSE_ROWS_LAUNCH(1);
    else if (chunks <= 2) PULSE_ROWS_LAUNCH(2);
    else if (chunks <= 4) PULSE_ROWS_LAUNCH(4);
    else if (chunks <= 8) PULSE_ROWS_LAUNCH(8);
    else return false;
#undef PULSE_ROWS_LAUNCH
    return true;
}

bool aligned(const void* p, int bytes) { return reinterpret_cast<uintptr_t>(p) % bytes == 0; }

}  // namespace

// out_dtype and w_dtype are those of both outputs and both weights.
extern "C" int pulse_residual_norms(float* h, const int* rows, const void* a, int a_dtype, int a_parts, int64_t a_stride,
                                    const void* b, int b_dtype, const void* row, int row_dtype, const float* y,
                                    const int* idx, const float* weight, int experts, int top, void* out1,
                                    int64_t out1_stride, const void* w1, float eps1, void* out2, int64_t out2_stride,
                                    const void* w2, float eps2, int out_dtype, int w_dtype, int out_rows, int hidden,
                                    int write_back, hipStream_t stream) {
    PULSE_REQUIRE(out_rows >= 0 && hidden > 0 && h, "residual_norms: bad sizes rows=%d H=%d", out_rows, hidden);
    PULSE_REQUIRE(pulse_dtype_ok(a_dtype) && pulse_dtype_ok(b_dtype) && pulse_dtype_ok(row_dtype) && pulse_dtype_ok(out_dtype) &&
                  pulse_dtype_ok(w_dtype), "residual_norms: bad dtype tag");
    PULSE_REQUIRE(!(rows && write_back), "residual_norms: write_back with gathered rows is not supported");
    PULSE_REQUIRE(!a || a_parts >= 1, "residual_norms: an update has at least one part");
    PULSE_REQUIRE(!y || (idx && top > 0 && experts > 0), "residual_norms: the experts' results come with the tokens' choices");
    PULSE_REQUIRE((!w1 || out1) && (!w2 || out2), "residual_norms: a norm without an output");
    PULSE_REQUIRE((!out1 || out1_stride >= hidden) && (!out2 || out2_stride >= hidden), "residual_norms: output rows too short");
    if (out_rows == 0) return 0;
    RowTerms in{a, a_dtype, a ? a_parts : 0, a_stride, b, b_dtype, row, row_dtype, y, idx, weight, experts, top};
    RowOuts o{{out1, out2}, {w1, w2}, {out1_stride, out2_stride}, {eps1, eps2}};
    const int ob = out_dtype == PULSE_F32 ? 16 : 8;
    bool vec = hidden % 4 == 0 && a_stride % 4 == 0 && aligned(h, 16) && aligned(a, 16) && aligned(b, 16) && aligned(row, 16) &&
               aligned(y, 16) && aligned(w1, 16) && aligned(w2, 16) && aligned(out1, ob) && aligned(out2, ob) &&
               (!out1 || out1_stride % 4 == 0) && (!out2 || out2_stride % 4 == 0);
    const int nvec = vec ? hidden / 4 : hidden;
    PULSE_REQUIRE(nvec <= 8 * 1024, "residual_norms: rows of %d values are too long", hidden);
    // few rows are bound by round trips, not by bandwidth: more threads a row; long rows need them
    const bool many_threads = nvec > 8 * 256 || (out_rows <= 256 && nvec >= 512);
    bool done = false;
    PULSE_DISPATCH_DTYPE(w_dtype, TW, PULSE_DISPATCH_DTYPE(out_dtype, TO,
        if (vec && many_threads) done = launch_rows<TW, TO, 4, 1024>((nvec + 1023) / 1024, h, rows, in, o, out_rows, hidden, write_back, stream);
        else if (vec) done = launch_rows<TW, TO, 4, 256>((nvec + 255) / 256, h, rows, in, o, out_rows, hidden, write_back, stream);
        else if (many_threads) done = launch_rows<TW, TO, 1, 1024>((nvec + 1023) / 1024, h, rows, in, o, out_rows, hidden, write_back, stream);
        else done = launch_rows<TW, TO, 1, 256>((nvec + 255) / 256, h, rows, in, o, out_rows, hidden, write_back, stream)));
    PULSE_REQUIRE(done, "residual_norms: no kernel for rows of %d values", hidden);
    PULSE_LAUNCH_CHECK("residual_norms");
    return 0;
}
