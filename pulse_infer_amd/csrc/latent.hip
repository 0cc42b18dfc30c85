// Attention over one latent row a token ("latent attention"), around the paged attention kernels.
//
// A token stores c (`rank` values: the first rows of the down projection, divided by their root mean square and
// multiplied by a weight) and one turned key part (`rot` values) shared by all heads.  Head h's key is
// [W_uk,h c | turned part] and its value W_uv,h c.  Scores and weighted sums are linear in c, so the kernels work in the
// latent space: the query of head h becomes [W_uk,h^T q_plain,h | q_turned,h], the stored "key" of the one kv head is
// [c | turned part], its "value" is c, and head h's result W_uv,h (sum_j a_h(j) c_j) is expanded afterwards.
//
// pulse_latent_rows:   c and the turned key part into the pages; the queries' turned parts into their places.
// pulse_rms_rows:      some columns of every row divided by their root mean square, times a weight (a latent that queries
//                      come from)
// pulse_latent_absorb: q_abs[t, h, :] = W_uk,h^T q_plain[t, h]        (float32 sums, one rounding)
// pulse_latent_expand: y[t, h, :] = (W_uv,h o[t, h, :rank]) * sigmoid(gate[t, h, :])
// pulse_heads_product: both of these products for bfloat16 weights on the matrix cores: y[t, h, m] = sum_k
//                      w[h, m, k] x[t, h, k] (w_uk transposed once at load, w_uv as it is)
//
// Long prompt portions attend to keys and values expanded to every head instead (a third of the arithmetic where the
// latent row is much wider than a head), in pages of their own that live for one layer of one step:
// pulse_latent_queries: q[t, h, :] = [plain | turned | 0]
// pulse_latent_gather:  the cached latent rows of a list of pages, as one dense matrix (the up projections' input)
// pulse_latent_pages:   the up projections' output and the cached turned parts as keys [pages, heads, page, width] and
//                       values [pages, heads, width, page]
// pulse_latent_compact: the heads' results side by side without the channels that fill them up
#include "common.h"

#include <math.h>

namespace {

struct LatentArgs {
    int heads, d, rot, rank, stored;   // stored: channels of a stored key / value row (>= rank + rot)
    int64_t x_stride, down_stride, q_stride;
    int q0, c0;                        // first columns of the queries in a row of x and of the down projection in its
    int page_size, num_pages, bt_width;
    int pairing, write;
    float eps;
};

// One workgroup a token.
template <typename TX, typename TW, typename TC>
__global__ void latent_rows_kernel(const TX* __restrict__ x, const TX* __restrict__ down_x, TX* __restrict__ q,
                                   const TW* __restrict__ w,
                                   const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                   TC* __restrict__ kcache, TC* __restrict__ vcache, const int* __restrict__ positions,
                                   const int* __restrict__ token_entry, const int* __restrict__ block_table, LatentArgs a) {
    __shared__ float scratch[16];
    const int t = blockIdx.x;
    const TX* row = x + static_cast<int64_t>(t) * a.x_stride;
    const int half = a.rot / 2;
    const float* ct = cos_t + static_cast<int64_t>(t) * half;
    const float* st = sin_t + static_cast<int64_t>(t) * half;
    auto turned = [&](const TX* src, int e) -> float {
        int pair, freq;
        bool first;
        if (a.pairing == 1) { first = e < half; pair = first ? e + half : e - half; freq = first ? e : e - half; }
        else { first = (e & 1) == 0; pair = e ^ 1; freq = e >> 1; }
        const float v = to_f32<TX>(src[e]), o = to_f32<TX>(src[pair]);
        return first ? v * ct[freq] - o * st[freq] : v * ct[freq] + o * st[freq];
    };
    // the queries' turned parts: q[t, h, rank + e]
    TX* qrow = q + static_cast<int64_t>(t) * a.q_stride;
    const int width = a.rank + a.rot;
    for (int i = threadIdx.x; q && i < a.heads * a.rot; i += blockDim.x) {
        const int h = i / a.rot, e = i % a.rot;
        qrow[static_cast<int64_t>(h) * a.stored + a.rank + e] =
            from_f32<TX>(turned(row + a.q0 + static_cast<int64_t>(h) * (a.d + a.rot) + a.d, e));
    }
    for (int i = threadIdx.x; q && i < a.heads * (a.stored - width); i += blockDim.x) {
        const int h = i / (a.stored - width), e = i % (a.stored - width);
        qrow[static_cast<int64_t>(h) * a.stored + width + e] = from_f32<TX>(0.f);
    }
    if (!a.write) return;
    const TX* down = down_x + static_cast<int64_t>(t) * a.down_stride + a.c0;
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.rank; i += blockDim.x) { const float v = to_f32<TX>(down[i]); ss = fmaf(v, v, ss); }
    ss = block_sum(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.rank) + a.eps);
    const int pos = positions[t];
    const int pi = pos / a.page_size;
    const int page = pi < a.bt_width ? block_table[static_cast<int64_t>(token_entry[t]) * a.bt_width + pi] : -1;
    if (page < 0 || page >= a.num_pages) return;   // the host has checked the tables; a stale entry is not written through
    const int slot = pos % a.page_size;
    TC* krow = kcache + (static_cast<int64_t>(page) * a.page_size + slot) * a.stored;
    TC* vrow = vcache + static_cast<int64_t>(page) * a.stored * a.page_size + slot;
    for (int i = threadIdx.x; i < a.stored; i += blockDim.x) {
        float k = 0.f, v = 0.f;
        if (i < a.rank) k = v = to_f32<TX>(down[i]) * inv * to_f32<TW>(w[i]);
        else if (i < width) k = turned(down + a.rank, i - a.rank);
        krow[i] = from_f32<TC>(k);
        vrow[static_cast<int64_t>(i) * a.page_size] = from_f32<TC>(v);
    }
}

// out[t, i] = x[t, c0 + i] / sqrt(mean over the n columns of x^2 + eps) * w[i]; one workgroup a row.
template <typename TX, typename TW>
__global__ void rms_rows_kernel(const TX* __restrict__ x, int64_t x_stride, int c0, const TW* __restrict__ w,
                                TX* __restrict__ out, int64_t o_stride, int n, float eps) {
    __shared__ float scratch[16];
    const TX* row = x + static_cast<int64_t>(blockIdx.x) * x_stride + c0;
    float ss = 0.f;
    for (int i = threadIdx.x; i < n; i += blockDim.x) { const float v = to_f32<TX>(row[i]); ss = fmaf(v, v, ss); }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(n) + eps);
    TX* dst = out + static_cast<int64_t>(blockIdx.x) * o_stride;
    for (int i = threadIdx.x; i < n; i += blockDim.x) dst[i] = from_f32<TX>(to_f32<TX>(row[i]) * inv * to_f32<TW>(w[i]));
}

// q_abs[t, h, r] = sum_e q[t, h, e] * W_uk[h * d + e, r]; one workgroup a (token, head), a thread a latent channel.
template <typename TX, typename TW>
__global__ void latent_absorb_kernel(const TX* __restrict__ x, int64_t x_stride, int q0, int q_head, const TW* __restrict__ w,
                                     TX* __restrict__ q, int64_t q_stride, int stored, int d, int rank) {
    extern __shared__ float q_s[];
    const int t = blockIdx.x, h = blockIdx.y;
    const TX* src = x + static_cast<int64_t>(t) * x_stride + q0 + static_cast<int64_t>(h) * q_head;
    for (int e = threadIdx.x; e < d; e += blockDim.x) q_s[e] = to_f32<TX>(src[e]);
    __syncthreads();
    const TW* wh = w + static_cast<int64_t>(h) * d * rank;
    TX* dst = q + static_cast<int64_t>(t) * q_stride + static_cast<int64_t>(h) * stored;
    for (int r = threadIdx.x; r < rank; r += blockDim.x) {
        float sum = 0.f;
        for (int e = 0; e < d; ++e) sum = fmaf(q_s[e], to_f32<TW>(wh[static_cast<int64_t>(e) * rank + r]), sum);
        dst[r] = from_f32<TX>(sum);
    }
}

// y[t, h, e] = (sum_r W_uv[h * dv + e, r] * o[t, h, r]) * sigmoid(gate[t, h * dv + e]); a wavefront an output channel.
template <typename TO, typename TX, typename TW>
__global__ void latent_expand_kernel(const TO* __restrict__ o, int64_t o_stride, int stored, const TW* __restrict__ w,
                                     const TX* __restrict__ gate, int64_t gate_stride, TX* __restrict__ y,
                                     int64_t y_stride, int dv, int rank, float scale, int gate_heads) {
    extern __shared__ float o_s[];
    const int t = blockIdx.x, h = blockIdx.y;
    const TO* src = o + static_cast<int64_t>(t) * o_stride + static_cast<int64_t>(h) * stored;
    for (int r = threadIdx.x; r < rank; r += blockDim.x) o_s[r] = to_f32<TO>(src[r]);
    __syncthreads();
    const int lane = threadIdx.x % PULSE_WAVE, wave = threadIdx.x / PULSE_WAVE, waves = blockDim.x / PULSE_WAVE;
    for (int e = wave; e < dv; e += waves) {
        const TW* wr = w + (static_cast<int64_t>(h) * dv + e) * rank;
        float sum = 0.f;
        for (int r = lane; r < rank; r += PULSE_WAVE) sum = fmaf(to_f32<TW>(wr[r]), o_s[r], sum);
        sum = wave_sum(sum);
        if (lane == 0) {
            float v = sum * scale;
            if (gate) v *= 1.0f / (1.0f + expf(-to_f32<TX>(gate[static_cast<int64_t>(t) * gate_stride + (gate_heads ? h : static_cast<int64_t>(h) * dv + e)])));
            y[static_cast<int64_t>(t) * y_stride + static_cast<int64_t>(h) * dv + e] = from_f32<TX>(v);
        }
    }
}


// ------------------------------------------------------------------ a product a head, on the matrix cores
typedef __attribute__((ext_vector_type(8))) __bf16 hp_bf16x8;
typedef __attribute__((ext_vector_type(4))) float hp_f32x4;

template <typename T> __device__ __forceinline__ hp_bf16x8 load8(const T* p);
template <> __device__ __forceinline__ hp_bf16x8 load8<bf16_t>(const bf16_t* p) { return *reinterpret_cast<const hp_bf16x8*>(p); }
template <> __device__ __forceinline__ hp_bf16x8 load8<float>(const float* p) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    hp_bf16x8 out;
    out[0] = static_cast<__bf16>(a.x); out[1] = static_cast<__bf16>(a.y); out[2] = static_cast<__bf16>(a.z); out[3] = static_cast<__bf16>(a.w);
    out[4] = static_cast<__bf16>(b.x); out[5] = static_cast<__bf16>(b.y); out[6] = static_cast<__bf16>(b.z); out[7] = static_cast<__bf16>(b.w);
    return out;
}

// A workgroup takes 16 TT tokens of one head; a wavefront a tile of 16 output channels at a time, whose W operands serve
// all TT token tiles.  W rows are the matrix cores' row operand (m = output channel), the tokens' rows of x the column
// operand, so a lane ends up with four neighbouring channels of its token: one 8-byte store.
template <typename TX, int TT>
__global__ __launch_bounds__(256) void heads_product_kernel(const TX* __restrict__ x, int64_t x_stride, int x_head,
                                                            const bf16_t* __restrict__ w, const bf16_t* __restrict__ gate,
                                                            int64_t gate_stride, bf16_t* __restrict__ y, int64_t y_stride,
                                                            int y_head, int tokens, int m_out, int k_in, float scale, int gate_heads) {
    const int t0 = blockIdx.x * (16 * TT), h = blockIdx.y;
    const int lane = threadIdx.x % PULSE_WAVE, wave = threadIdx.x / PULSE_WAVE;
    const int r = lane % 16, g = lane / 16;
    const TX* xrow[TT];
#pragma unroll
    for (int u = 0; u < TT; ++u)
        xrow[u] = x + static_cast<int64_t>(min(t0 + 16 * u + r, tokens - 1)) * x_stride + static_cast<int64_t>(h) * x_head;
    const hp_bf16x8 zero = __builtin_bit_cast(hp_bf16x8, make_uint4(0u, 0u, 0u, 0u));
    for (int m0 = wave * 16; m0 < m_out; m0 += 64) {
        const int m = m0 + r;
        const bf16_t* wrow = m < m_out ? w + (static_cast<int64_t>(h) * m_out + m) * k_in : nullptr;
        hp_f32x4 acc[TT];
#pragma unroll
        for (int u = 0; u < TT; ++u) acc[u] = hp_f32x4{0.f, 0.f, 0.f, 0.f};
        for (int k0 = 0; k0 < k_in; k0 += 32) {
            const int k = k0 + 8 * g;
            const bool in = k < k_in;
            const hp_bf16x8 wa = (in && wrow) ? *reinterpret_cast<const hp_bf16x8*>(wrow + k) : zero;
#pragma unroll
            for (int u = 0; u < TT; ++u) {
                const hp_bf16x8 xb = in ? load8<TX>(xrow[u] + k) : zero;
                acc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa, xb, acc[u], 0, 0, 0);
            }
        }
        // lane: token r of every tile, channels m0 + 4 g + i
#pragma unroll
        for (int u = 0; u < TT; ++u) {
            const int tok = t0 + 16 * u + r, c0 = m0 + 4 * g;
            if (tok < tokens) {
                bf16_t* dst = y + static_cast<int64_t>(tok) * y_stride + static_cast<int64_t>(h) * y_head + c0;
                const bf16_t* gr = gate ? gate + static_cast<int64_t>(tok) * gate_stride + (gate_heads ? h : static_cast<int64_t>(h) * m_out + c0) : nullptr;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    if (c0 + i < m_out) {
                        float v = acc[u][i] * scale;
                        if (gr) v *= 1.0f / (1.0f + expf(-bf16_to_f32(gr[gate_heads ? 0 : i])));
                        dst[i] = f32_to_bf16(v);
                    }
                }
            }
        }
    }
}

// ------------------------------------------------------------------ keys and values expanded to every head
// One workgroup a token.
template <typename TX>
__global__ void latent_queries_kernel(const TX* __restrict__ x, int64_t x_stride, int q0, TX* __restrict__ q, int64_t q_stride,
                                      const float* __restrict__ cos_t, const float* __restrict__ sin_t, int heads, int d,
                                      int rot, int width, int pairing) {
    const int t = blockIdx.x, half = rot / 2, in = d + rot;
    const TX* row = x + static_cast<int64_t>(t) * x_stride + q0;
    const float* ct = cos_t + static_cast<int64_t>(t) * half;
    const float* st = sin_t + static_cast<int64_t>(t) * half;
    TX* dst = q + static_cast<int64_t>(t) * q_stride;
    for (int i = threadIdx.x; i < heads * width; i += blockDim.x) {
        const int h = i / width, c = i % width;
        const TX* src = row + static_cast<int64_t>(h) * in;
        if (c < d) { dst[i] = src[c]; continue; }
        float v = 0.f;
        if (c < in) {
            const int e = c - d;
            int pair, freq;
            bool first;
            if (pairing == 1) { first = e < half; pair = first ? e + half : e - half; freq = first ? e : e - half; }
            else { first = (e & 1) == 0; pair = e ^ 1; freq = e >> 1; }
            const float u = to_f32<TX>(src[c]), o = to_f32<TX>(src[d + pair]);
            v = first ? u * ct[freq] - o * st[freq] : u * ct[freq] + o * st[freq];
        }
        dst[i] = from_f32<TX>(v);
    }
}

struct ExpandArgs {
    int heads, d, rot, dv, rank, stored, width;   // width: channels of an expanded head
    int page, src_page, src_pages, bt_width;      // slots of an expanded page and of a cached one
};

// The cached row of (entry, position), null where there is none (behind the entry's last token, below its window).
__device__ __forceinline__ const bf16_t* cached_row(const bf16_t* __restrict__ kcache, const int* __restrict__ block_table,
                                                    int entry, int pos, int end, const ExpandArgs& a) {
    if (pos >= end) return nullptr;
    const int pi = pos / a.src_page;
    const int pg = pi < a.bt_width ? block_table[static_cast<int64_t>(entry) * a.bt_width + pi] : -1;
    if (pg < 0 || pg >= a.src_pages) return nullptr;
    return kcache + (static_cast<int64_t>(pg) * a.src_page + pos % a.src_page) * a.stored;
}

// pages: [n][4] = entry, first position, end of the entry's tokens, 0.  A wavefront a row, 16 bytes a lane.
__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16_t* __restrict__ kcache, const int* __restrict__ block_table,
                                                            const int* __restrict__ pages, bf16_t* __restrict__ rows,
                                                            ExpandArgs a) {
    const int p = blockIdx.x, slot = blockIdx.y * 4 + threadIdx.x / PULSE_WAVE, lane = threadIdx.x % PULSE_WAVE;
    if (slot >= a.page) return;
    const int* pg = pages + 4 * p;
    const bf16_t* src = cached_row(kcache, block_table, pg[0], pg[1] + slot, pg[2], a);
    uint4* dst = reinterpret_cast<uint4*>(rows + (static_cast<int64_t>(p) * a.page + slot) * a.rank);
    for (int i = lane; i < a.rank / 8; i += PULSE_WAVE)
        dst[i] = src ? reinterpret_cast<const uint4*>(src)[i] : make_uint4(0u, 0u, 0u, 0u);
}

// A workgroup a (page, head): keys as they come, values turned around through LDS.
__global__ __launch_bounds__(256) void latent_pages_kernel(const bf16_t* __restrict__ kcache, const int* __restrict__ block_table,
                                                           const int* __restrict__ pages, const bf16_t* __restrict__ up,
                                                           bf16_t* __restrict__ keys, bf16_t* __restrict__ values,
                                                           ExpandArgs a) {
    extern __shared__ bf16_t v_s[];    // [page][dv + 2]
    const int p = blockIdx.x, h = blockIdx.y;
    const int* pg = pages + 4 * p;
    const int64_t up_cols = static_cast<int64_t>(a.heads) * (a.d + a.dv);
    const bf16_t* rows = up + static_cast<int64_t>(p) * a.page * up_cols;
    bf16_t* kdst = keys + (static_cast<int64_t>(p) * a.heads + h) * a.page * a.width;
    for (int i = threadIdx.x; i < a.page * a.width; i += 256) {
        const int slot = i / a.width, c = i % a.width;
        bf16_t v = 0;
        if (c < a.d) v = rows[slot * up_cols + static_cast<int64_t>(h) * a.d + c];
        else if (c < a.d + a.rot) {
            const bf16_t* src = cached_row(kcache, block_table, pg[0], pg[1] + slot, pg[2], a);
            if (src) v = src[a.rank + c - a.d];
        }
        kdst[i] = v;
    }
    const int pitch = a.dv + 2;
    for (int i = threadIdx.x; i < a.page * a.dv; i += 256) {
        const int slot = i / a.dv, c = i % a.dv;
        v_s[slot * pitch + c] = rows[slot * up_cols + static_cast<int64_t>(a.heads) * a.d + static_cast<int64_t>(h) * a.dv + c];
    }
    __syncthreads();
    bf16_t* vdst = values + (static_cast<int64_t>(p) * a.heads + h) * a.page * a.width;
    for (int i = threadIdx.x; i < a.page * a.width; i += 256) {
        const int c = i / a.page, slot = i % a.page;
        vdst[i] = c < a.dv ? v_s[slot * pitch + c] : static_cast<bf16_t>(0);
    }
}

__global__ void latent_compact_kernel(const bf16_t* __restrict__ o, int64_t o_stride, int width, bf16_t* __restrict__ y,
                                      int64_t y_stride, int dv, int n, float scale) {
    const int t = blockIdx.x;
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const bf16_t v = o[static_cast<int64_t>(t) * o_stride + static_cast<int64_t>(i / dv) * width + i % dv];
        y[static_cast<int64_t>(t) * y_stride + i] = scale == 1.f ? v : f32_to_bf16(bf16_to_f32(v) * scale);
    }
}

}  // namespace

// x [tokens, x_stride]: queries from column q0 (heads x (d + rot), the turned part last); down_x [tokens, down_stride]:
// the down projection from column c0 (rank + rot; the two may be one matrix; without `write` down_x is not read).  q [tokens, q_stride] receives, for head h at h * stored, the turned
// part at rank .. rank + rot and zeros behind it (the first rank channels are pulse_latent_absorb's); null: no queries.  With `write`
// the token's c and turned key part go to kcache [pages, 1, page, stored] and c to vcache [pages, 1, stored, page].
extern "C" int pulse_latent_rows(const void* x, int64_t x_stride, int x_dtype, int q0, const void* down_x,
                                 int64_t down_stride, int c0, void* q, int64_t q_stride,
                                 const void* norm_w, int w_dtype, const float* cos_t, const float* sin_t, int pairing,
                                 void* kcache, void* vcache, int c_dtype, const int* positions, const int* token_entry,
                                 const int* block_table, int bt_width, int tokens, int heads, int d, int rot, int rank,
                                 int stored, int page_size, int num_pages, float eps, int write, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && d >= 0 && rank > 0 && rot > 0 && rot % 2 == 0, "latent_rows: bad sizes");
    PULSE_REQUIRE(stored >= rank + rot && (!q || q_stride >= static_cast<int64_t>(heads) * stored), "latent_rows: stored rows too narrow");
    PULSE_REQUIRE(x && (q || write) && cos_t && sin_t && positions && token_entry && (!write || (down_x && norm_w && kcache && vcache &&
                  block_table)), "latent_rows: null pointer");
    PULSE_REQUIRE(pulse_dtype_ok(x_dtype) && pulse_dtype_ok(w_dtype) && pulse_dtype_ok(c_dtype), "latent_rows: bad dtype tag");
    PULSE_REQUIRE(q0 >= 0 && c0 >= 0 && x_stride >= static_cast<int64_t>(q0) + static_cast<int64_t>(heads) * (d + rot) &&
                  (!write || down_stride >= static_cast<int64_t>(c0) + rank + rot), "latent_rows: the rows are too short");
    PULSE_REQUIRE((!write || (page_size > 0 && num_pages > 0 && bt_width > 0)) && (pairing == 0 || pairing == 1),
                  "latent_rows: bad cache geometry");
    if (tokens == 0) return 0;
    LatentArgs a;
    a.heads = heads; a.d = d; a.rot = rot; a.rank = rank; a.stored = stored; a.x_stride = x_stride;
    a.down_stride = down_stride; a.q_stride = q_stride;
    a.q0 = q0; a.c0 = c0; a.page_size = page_size; a.num_pages = num_pages; a.bt_width = bt_width; a.pairing = pairing;
    a.write = write; a.eps = eps;
    PULSE_DISPATCH_DTYPE(x_dtype, TX, PULSE_DISPATCH_DTYPE(w_dtype, TW, PULSE_DISPATCH_DTYPE(c_dtype, TC,
        hipLaunchKernelGGL((latent_rows_kernel<TX, TW, TC>), dim3(tokens), dim3(256), 0, stream, static_cast<const TX*>(x),
                           static_cast<const TX*>(down_x), static_cast<TX*>(q), static_cast<const TW*>(norm_w), cos_t, sin_t, static_cast<TC*>(kcache),
                           static_cast<TC*>(vcache), positions, token_entry, block_table, a))));
    PULSE_LAUNCH_CHECK("latent_rows");
    return 0;
}

extern "C" int pulse_rms_rows(const void* x, int64_t x_stride, int x_dtype, int c0, const void* w, int w_dtype, void* out,
                              int64_t o_stride, int tokens, int n, float eps, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && n > 0 && c0 >= 0 && x && w && out && pulse_dtype_ok(x_dtype) && pulse_dtype_ok(w_dtype),
                  "rms_rows: bad arguments");
    PULSE_REQUIRE(x_stride >= static_cast<int64_t>(c0) + n && o_stride >= n, "rms_rows: the rows are too short");
    if (tokens == 0) return 0;
    PULSE_DISPATCH_DTYPE(x_dtype, TX, PULSE_DISPATCH_DTYPE(w_dtype, TW,
        hipLaunchKernelGGL((rms_rows_kernel<TX, TW>), dim3(tokens), dim3(256), 0, stream, static_cast<const TX*>(x), x_stride,
                           c0, static_cast<const TW*>(w), static_cast<TX*>(out), o_stride, n, eps)));
    PULSE_LAUNCH_CHECK("rms_rows");
    return 0;
}

// w_uk [heads * d, rank]; q_head: columns a head takes in x (d + rot).
extern "C" int pulse_latent_absorb(const void* x, int64_t x_stride, int x_dtype, int q0, int q_head, const void* w_uk,
                                   int w_dtype, void* q, int64_t q_stride, int stored, int tokens, int heads, int d,
                                   int rank, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && d > 0 && rank > 0 && q_head >= d && stored >= rank, "latent_absorb: bad sizes");
    PULSE_REQUIRE(heads < 65536 && x && w_uk && q && pulse_dtype_ok(x_dtype) && pulse_dtype_ok(w_dtype), "latent_absorb: bad arguments");
    PULSE_REQUIRE(q_stride >= static_cast<int64_t>(heads) * stored && x_stride >= static_cast<int64_t>(q0) + static_cast<int64_t>(heads) * q_head,
                  "latent_absorb: the rows are too short");
    if (tokens == 0) return 0;
    const int threads = rank >= 256 ? 256 : (rank + 63) / 64 * 64;
    PULSE_DISPATCH_DTYPE(x_dtype, TX, PULSE_DISPATCH_DTYPE(w_dtype, TW,
        hipLaunchKernelGGL((latent_absorb_kernel<TX, TW>), dim3(tokens, heads), dim3(threads), sizeof(float) * d, stream,
                           static_cast<const TX*>(x), x_stride, q0, q_head, static_cast<const TW*>(w_uk),
                           static_cast<TX*>(q), q_stride, stored, d, rank)));
    PULSE_LAUNCH_CHECK("latent_absorb");
    return 0;
}

// o [tokens, o_stride] (float32 or the activations' type): head h's weighted latent row at h * stored; w_uv
// [heads * dv, rank]; gate [tokens, gate_stride] holds heads * dv logits a token, with gate_heads one a head (null: no
// gate).
extern "C" int pulse_latent_expand(const void* o, int64_t o_stride, int o_dtype, int stored, const void* w_uv, int w_dtype,
                                   const void* gate, int64_t gate_stride, void* y, int64_t y_stride, int x_dtype,
                                   int tokens, int heads, int dv, int rank, float scale, int gate_heads, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && dv > 0 && rank > 0 && stored >= rank, "latent_expand: bad sizes");
    PULSE_REQUIRE(heads < 65536 && o && w_uv && y && pulse_dtype_ok(o_dtype) && pulse_dtype_ok(x_dtype) && pulse_dtype_ok(w_dtype),
                  "latent_expand: bad arguments");
    PULSE_REQUIRE(o_stride >= static_cast<int64_t>(heads) * stored && y_stride >= static_cast<int64_t>(heads) * dv &&
                  (!gate || gate_stride >= static_cast<int64_t>(heads) * (gate_heads ? 1 : dv)), "latent_expand: the rows are too short");
    PULSE_REQUIRE(rank * sizeof(float) <= 60 * 1024, "latent_expand: a latent row of %d values does not fit", rank);
    if (tokens == 0) return 0;
    PULSE_DISPATCH_DTYPE(o_dtype, TO, PULSE_DISPATCH_DTYPE(x_dtype, TX, PULSE_DISPATCH_DTYPE(w_dtype, TW,
        hipLaunchKernelGGL((latent_expand_kernel<TO, TX, TW>), dim3(tokens, heads), dim3(256), sizeof(float) * rank, stream,
                           static_cast<const TO*>(o), o_stride, stored, static_cast<const TW*>(w_uv),
                           static_cast<const TX*>(gate), gate_stride, static_cast<TX*>(y), y_stride, dv, rank, scale, gate_heads))));
    PULSE_LAUNCH_CHECK("latent_expand");
    return 0;
}

// y[t, h * y_head + m] = scale * (sum_k w[h, m, k] * x[t, h * x_head + k]) * sigmoid(gate[t, h * m_out + m]) for bfloat16
// w [heads, m_out, k_in] and y, x bfloat16 or float32 (rounded to bfloat16 as it is read); k_in a multiple of 8, rows
// of x and w 16-byte aligned.  gate may be null; with gate_heads it holds one logit a head, gate[t, h].
extern "C" int pulse_heads_product(const void* x, int64_t x_stride, int x_head, int x_dtype, const void* w, const void* gate,
                                   int64_t gate_stride, void* y, int64_t y_stride, int y_head, int tokens, int heads,
                                   int m_out, int k_in, float scale, int gate_heads, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && heads < 65536 && m_out > 0 && k_in > 0 && k_in % 8 == 0, "heads_product: bad sizes");
    PULSE_REQUIRE(x && w && y && pulse_dtype_ok(x_dtype), "heads_product: bad arguments");
    const int xb = x_dtype == PULSE_F32 ? 4 : 2;
    PULSE_REQUIRE(x_head >= k_in && x_stride >= static_cast<int64_t>(heads - 1) * x_head + k_in &&
                  y_head >= m_out && y_stride >= static_cast<int64_t>(heads - 1) * y_head + m_out &&
                  (!gate || gate_stride >= static_cast<int64_t>(heads) * (gate_heads ? 1 : m_out)), "heads_product: the rows are too short");
    PULSE_REQUIRE(reinterpret_cast<uintptr_t>(x) % 16 == 0 && (x_stride * xb) % 16 == 0 && (static_cast<int64_t>(x_head) * xb) % 16 == 0 &&
                  reinterpret_cast<uintptr_t>(w) % 16 == 0, "heads_product: operands must be 16-byte aligned");
    if (tokens == 0) return 0;
#define PULSE_HEADS(TT_)                                                                                                 \
    PULSE_DISPATCH_DTYPE(x_dtype, TX,                                                                                    \
        hipLaunchKernelGGL((heads_product_kernel<TX, TT_>), dim3((tokens + 16 * TT_ - 1) / (16 * TT_), heads), dim3(256), 0, \
                           stream, static_cast<const TX*>(x), x_stride, x_head, static_cast<const bf16_t*>(w),           \
                           static_cast<const bf16_t*>(gate), gate_stride, static_cast<bf16_t*>(y), y_stride, y_head,     \
                           tokens, m_out, k_in, scale, gate_heads))
    if (tokens >= 256) PULSE_HEADS(4);
    else PULSE_HEADS(1);
#undef PULSE_HEADS
    PULSE_LAUNCH_CHECK("heads_product");
    return 0;
}

// x [tokens, x_stride] holds the queries from column q0 (heads x (d + rot)); q [tokens, q_stride] receives heads of `width`
// channels.
extern "C" int pulse_latent_queries(const void* x, int64_t x_stride, int x_dtype, int q0, void* q, int64_t q_stride,
                                    const float* cos_t, const float* sin_t, int pairing, int tokens, int heads, int d, int rot,
                                    int width, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && d > 0 && rot > 0 && rot % 2 == 0 && width >= d + rot && q0 >= 0, "latent_queries: bad sizes");
    PULSE_REQUIRE(x && q && cos_t && sin_t && pulse_dtype_ok(x_dtype) && (pairing == 0 || pairing == 1), "latent_queries: bad arguments");
    PULSE_REQUIRE(x_stride >= q0 + static_cast<int64_t>(heads) * (d + rot) && q_stride >= static_cast<int64_t>(heads) * width,
                  "latent_queries: the rows are too short");
    if (tokens == 0) return 0;
    PULSE_DISPATCH_DTYPE(x_dtype, TX,
        hipLaunchKernelGGL(latent_queries_kernel<TX>, dim3(tokens), dim3(256), 0, stream, static_cast<const TX*>(x), x_stride, q0,
                           static_cast<TX*>(q), q_stride, cos_t, sin_t, heads, d, rot, width, pairing));
    PULSE_LAUNCH_CHECK("latent_queries");
    return 0;
}

static int expand_args(ExpandArgs& a, int heads, int d, int rot, int dv, int rank, int stored, int width, int page, int src_page,
                       int src_pages, int bt_width) {
    PULSE_REQUIRE(heads > 0 && heads < 65536 && d > 0 && rot > 0 && dv > 0 && rank > 0 && stored >= rank + rot && width >= d + rot &&
                  width >= dv && page > 0 && src_page > 0 && src_pages > 0 && bt_width > 0, "latent expansion: bad sizes");
    PULSE_REQUIRE(rank % 8 == 0 && stored % 8 == 0, "latent expansion: rows must keep 16-byte alignment");
    a.heads = heads; a.d = d; a.rot = rot; a.dv = dv; a.rank = rank; a.stored = stored; a.width = width; a.page = page;
    a.src_page = src_page; a.src_pages = src_pages; a.bt_width = bt_width;
    return 0;
}

// kcache bfloat16 [src_pages, 1, src_page, stored]; pages int32 [n_pages, 4]: entry (row of block_table), first position, end
// of the entry's tokens, 0.  rows bfloat16 [n_pages * page, rank]; a row that is not cached becomes zeros.
extern "C" int pulse_latent_gather(const void* kcache, const int* block_table, int bt_width, const int* pages, int n_pages,
                                   void* rows, int rank, int rot, int stored, int page, int src_page, int src_pages,
                                   hipStream_t stream) {
    ExpandArgs a;
    if (expand_args(a, 1, 1, rot, 1, rank, stored, 1 + rot, page, src_page, src_pages, bt_width)) return 1;
    PULSE_REQUIRE(kcache && block_table && pages && rows && n_pages >= 0 && reinterpret_cast<uintptr_t>(kcache) % 16 == 0 &&
                  reinterpret_cast<uintptr_t>(rows) % 16 == 0, "latent_gather: bad arguments");
    if (n_pages == 0) return 0;
    hipLaunchKernelGGL(latent_gather_kernel, dim3(n_pages, (page + 3) / 4), dim3(256), 0, stream, static_cast<const bf16_t*>(kcache),
                       block_table, pages, static_cast<bf16_t*>(rows), a);
    PULSE_LAUNCH_CHECK("latent_gather");
    return 0;
}

// up bfloat16 [n_pages * page, heads * d + heads * dv]: the rows' keys, then values, head by head.
extern "C" int pulse_latent_pages(const void* kcache, const int* block_table, int bt_width, const int* pages, int n_pages,
                                  const void* up, void* keys, void* values, int heads, int d, int rot, int dv, int rank,
                                  int stored, int width, int page, int src_page, int src_pages, hipStream_t stream) {
    ExpandArgs a;
    if (expand_args(a, heads, d, rot, dv, rank, stored, width, page, src_page, src_pages, bt_width)) return 1;
    PULSE_REQUIRE(kcache && block_table && pages && up && keys && values && n_pages >= 0, "latent_pages: bad arguments");
    const size_t lds = sizeof(bf16_t) * static_cast<size_t>(page) * (dv + 2);
    PULSE_REQUIRE(lds <= 60 * 1024, "latent_pages: a page of %d values of %d channels does not fit", page, dv);
    if (n_pages == 0) return 0;
    hipLaunchKernelGGL(latent_pages_kernel, dim3(n_pages, heads), dim3(256), lds, stream, static_cast<const bf16_t*>(kcache),
                       block_table, pages, static_cast<const bf16_t*>(up), static_cast<bf16_t*>(keys),
                       static_cast<bf16_t*>(values), a);
    PULSE_LAUNCH_CHECK("latent_pages");
    return 0;
}

// y[t, h * dv + e] = scale * o[t, h * width + e], bfloat16.
extern "C" int pulse_latent_compact(const void* o, int64_t o_stride, int width, void* y, int64_t y_stride, int tokens, int heads,
                                    int dv, float scale, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && heads > 0 && dv > 0 && width >= dv && o && y && o_stride >= static_cast<int64_t>(heads) * width &&
                  y_stride >= static_cast<int64_t>(heads) * dv, "latent_compact: bad arguments");
    if (tokens == 0) return 0;
    hipLaunchKernelGGL(latent_compact_kernel, dim3(tokens), dim3(256), 0, stream, static_cast<const bf16_t*>(o), o_stride, width,
                       static_cast<bf16_t*>(y), y_stride, dv, heads * dv, scale);
    PULSE_LAUNCH_CHECK("latent_compact");
    return 0;
}
