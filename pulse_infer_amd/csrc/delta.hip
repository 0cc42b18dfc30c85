// Linear attention whose state is corrected towards every new value (the gated delta rule), behind short convolutions.
//
// A token's projection row holds, side by side, the raw q and k (groups x d each), the raw v (heads x dv), an output
// gate (heads x dv), and one number a head for the write strength (b) and for the decay (a).  Query head h reads q and k
// of group h / (heads / groups).  Per channel of q, k and v
//     x_t <- silu(sum_j taps[j] raw_(t - (K - 1) + j))                  zeros before the sequence's start
// then q and k become unit vectors, x / sqrt(sum(x^2) + 1e-6), q times d^(-1/2), and per head
//     beta = sigmoid(b)      g = exp(-exp(A_log) softplus(a + dt_bias))
//     D = g S                r = v - D^T k               S = D + beta k r^T    o = S^T q
//
// A request's slot holds one float32 row: S [heads, d, dv], then the last raw inputs of the convolutions as a ring
// [K, channels], the input at position p in place p % K.  A decoded token then writes a place that no other workgroup
// of its step reads.  An entry that starts at position 0 starts from zeros, whatever the slot holds.
//
// pulse_delta_prepare: convolutions, unit vectors, decays and strengths of a step's tokens, in float32 rows; a second
//                      launch moves the ring on.
// pulse_delta_walk:    the recurrence over prepared rows, token by token, entry by entry (portions, mixed batches).
// pulse_delta_chunks:  the recurrence over prepared rows of long portions, 64 tokens at a time on the matrix cores (float32).
// pulse_delta_decode:  a step of single tokens in one launch: convolution, ring, recurrence, the norm of every head's
//                      result and its gate.
// State, unit vectors, decays, strengths and all sums are float32 whatever the storage type of the rows.
#include "common.h"

#include <math.h>

namespace {

constexpr int MAX_TAPS = 16;
constexpr float UNIT_EPS = 1e-6f;

__device__ __forceinline__ float silu_f(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus_f(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

struct DeltaArgs {
    int heads, groups, d, dv, taps;
    int channels;                  // 2 groups d + heads dv
    int g0, b0, a0;                // first columns of gate, strength and decay in a projection row
    int64_t x_stride;
    int64_t slot_stride, ring0;    // floats of a slot, where its ring starts
};

// The convolution of one channel for the token at `pos` whose entry starts at position `start` with row `row0`.
template <typename TX>
__device__ __forceinline__ float conv_channel(const TX* __restrict__ x, const float* __restrict__ taps,
                                              const float* __restrict__ ring, int c, int pos, int start, int row0,
                                              const DeltaArgs& a) {
    float acc = 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int p = pos - (a.taps - 1) + j;
        float v = 0.f;
        if (p >= start) v = to_f32<TX>(x[static_cast<int64_t>(row0 + p - start) * a.x_stride + c]);
        else if (p >= 0) v = ring[static_cast<int64_t>(p % a.taps) * a.channels + c];
        acc = fmaf(taps[j * a.channels + c], v, acc);
    }
    return silu_f(acc);
}

// A workgroup a token: a wavefront takes whole heads of q and k (it needs their lengths), all threads share v.
template <typename TX>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const TX* __restrict__ x, const float* __restrict__ taps,
                                                            const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                                                            const float* __restrict__ state, float* __restrict__ rows,
                                                            float* __restrict__ gates, const int* __restrict__ positions,
                                                            const int* __restrict__ token_entry,
                                                            const int* __restrict__ entry_start,
                                                            const int* __restrict__ entry_first_row,
                                                            const int* __restrict__ entry_slot, DeltaArgs a) {
    const int t = blockIdx.x;
    const int lane = threadIdx.x % PULSE_WAVE, wave = threadIdx.x / PULSE_WAVE;
    const int e = token_entry[t];
    const int start = entry_start[e], row0 = entry_first_row[e], pos = positions[t];
    const float* ring = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride + a.ring0;
    float* dst = rows + static_cast<int64_t>(t) * a.channels;
    const int qk = 2 * a.groups * a.d;
    for (int hh = wave; hh < 2 * a.groups; hh += 4) {
        float v[4];
        float ss = 0.f;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int c = lane + u * PULSE_WAVE;
            v[u] = 0.f;
            if (c < a.d) {
                v[u] = conv_channel<TX>(x, taps, ring, hh * a.d + c, pos, start, row0, a);
                ss = fmaf(v[u], v[u], ss);
            }
        }
        float inv = 1.0f / sqrtf(wave_sum(ss) + UNIT_EPS);
        if (hh < a.groups) inv *= 1.0f / sqrtf(static_cast<float>(a.d));
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int c = lane + u * PULSE_WAVE;
            if (c < a.d) dst[hh * a.d + c] = v[u] * inv;
        }
    }
    for (int c = qk + threadIdx.x; c < a.channels; c += 256) dst[c] = conv_channel<TX>(x, taps, ring, c, pos, start, row0, a);
    const TX* row = x + static_cast<int64_t>(t) * a.x_stride;
    for (int h = threadIdx.x; h < a.heads; h += 256) {
        gates[static_cast<int64_t>(t) * 2 * a.heads + h] = -expf(a_log[h]) * softplus_f(to_f32<TX>(row[a.a0 + h]) + dt_bias[h]);
        gates[static_cast<int64_t>(t) * 2 * a.heads + a.heads + h] = sigmoid_f(to_f32<TX>(row[a.b0 + h]));
    }
}

// The same for many tokens and few taps: a wavefront takes a unit of channels (a head of q or k, or 128 channels of v) for
// RUN neighbouring tokens, two channels a lane, with the taps and the last inputs in registers: every input is read once.
constexpr int RUN = 8;

template <typename TX> __device__ __forceinline__ float2 load2(const TX* p);
template <> __device__ __forceinline__ float2 load2<float>(const float* p) { return *reinterpret_cast<const float2*>(p); }
template <> __device__ __forceinline__ float2 load2<bf16_t>(const bf16_t* p) {
    const uint32_t two = *reinterpret_cast<const uint32_t*>(p);
    return make_float2(__uint_as_float(two << 16), __uint_as_float(two & 0xffff0000u));
}

// (bfloat16 rows: the hardware's exponential and reciprocal, a few units in the last place of float32)
template <typename TX> __device__ __forceinline__ float conv_silu(float v) {
    if constexpr (sizeof(TX) == 4) return silu_f(v);
    else return v * __builtin_amdgcn_rcpf(1.0f + __expf(-v));
}

template <typename TX, int TAPS, int PASSES>
__global__ __launch_bounds__(256) void delta_prepare_runs_kernel(const TX* __restrict__ x, const float* __restrict__ taps,
                                                                 const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                                                                 const float* __restrict__ state, float* __restrict__ rows,
                                                                 float* __restrict__ gates, const int* __restrict__ positions,
                                                                 const int* __restrict__ token_entry,
                                                                 const int* __restrict__ entry_start,
                                                                 const int* __restrict__ entry_first_row,
                                                                 const int* __restrict__ entry_slot, int tokens, int units,
                                                                 DeltaArgs a) {
    const int lane = threadIdx.x % PULSE_WAVE, wave = threadIdx.x / PULSE_WAVE;
    const int t0 = blockIdx.x * RUN, t1 = min(tokens, t0 + RUN);
    if (blockIdx.y == 0) {
        for (int i = threadIdx.x; i < (t1 - t0) * a.heads; i += 256) {
            const int t = t0 + i / a.heads, h = i % a.heads;
            const TX* row = x + static_cast<int64_t>(t) * a.x_stride;
            gates[static_cast<int64_t>(t) * 2 * a.heads + h] = -expf(a_log[h]) * softplus_f(to_f32<TX>(row[a.a0 + h]) + dt_bias[h]);
            gates[static_cast<int64_t>(t) * 2 * a.heads + a.heads + h] = sigmoid_f(to_f32<TX>(row[a.b0 + h]));
        }
    }
    const int unit = blockIdx.y * 4 + wave;
    if (unit >= units) return;
    const bool qk = unit < 2 * a.groups;
    const int first = qk ? unit * a.d : 2 * a.groups * a.d + (unit - 2 * a.groups) * 128;
    const int width = qk ? a.d : min(128, a.channels - first);
    float2 w[PASSES][TAPS], in[PASSES][TAPS];
    bool ok[PASSES];
#pragma unroll
    for (int p = 0; p < PASSES; ++p) {
        const int c = 128 * p + 2 * lane;
        ok[p] = c < width;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
            w[p][j] = ok[p] ? *reinterpret_cast<const float2*>(taps + j * a.channels + first + c) : make_float2(0.f, 0.f);
            in[p][j] = make_float2(0.f, 0.f);
        }
    }
    int entry = -1;
    for (int t = t0; t < t1; ++t) {
        const int e = token_entry[t], pos = positions[t];
        const bool fresh = e != entry;        // the inputs before this token are another sequence's
        const int start = entry_start[e], row0 = entry_first_row[e];
        entry = e;
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int c = first + 128 * p + 2 * lane;
            if (fresh) {
                const float* ring = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride + a.ring0;
#pragma unroll
                for (int j = 1; j < TAPS; ++j) {      // places 1 .. TAPS - 1 become 0 .. TAPS - 2 below
                    const int q = pos - TAPS + j;
                    in[p][j] = make_float2(0.f, 0.f);
                    if (ok[p]) {
                        if (q >= start) in[p][j] = load2<TX>(x + static_cast<int64_t>(row0 + q - start) * a.x_stride + c);
                        else if (q >= 0) in[p][j] = *reinterpret_cast<const float2*>(ring + static_cast<int64_t>(q % TAPS) * a.channels + c);
                    }
                }
            }
#pragma unroll
            for (int j = 0; j + 1 < TAPS; ++j) in[p][j] = in[p][j + 1];
            in[p][TAPS - 1] = ok[p] ? load2<TX>(x + static_cast<int64_t>(t) * a.x_stride + c) : make_float2(0.f, 0.f);
        }
        float2 v[PASSES];
        float ss = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            v[p] = make_float2(0.f, 0.f);
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
                v[p].x = fmaf(w[p][j].x, in[p][j].x, v[p].x);
                v[p].y = fmaf(w[p][j].y, in[p][j].y, v[p].y);
            }
            v[p].x = conv_silu<TX>(v[p].x);
            v[p].y = conv_silu<TX>(v[p].y);
            ss = fmaf(v[p].x, v[p].x, fmaf(v[p].y, v[p].y, ss));
        }
        float f = 1.f;
        if (qk) {
            f = 1.0f / sqrtf(wave_sum(ss) + UNIT_EPS);
            if (unit < a.groups) f *= 1.0f / sqrtf(static_cast<float>(a.d));
        }
#pragma unroll
        for (int p = 0; p < PASSES; ++p)
            if (ok[p])
                *reinterpret_cast<float2*>(rows + static_cast<int64_t>(t) * a.channels + first + 128 * p + 2 * lane) =
                    make_float2(v[p].x * f, v[p].y * f);
    }
}

// The ring moves on to the end of every entry's portion: the last min(count, K) inputs go to their places.
template <typename TX>
__global__ __launch_bounds__(256) void delta_ring_kernel(const TX* __restrict__ x, float* __restrict__ state,
                                                         const int* __restrict__ entry_start,
                                                         const int* __restrict__ entry_first_row,
                                                         const int* __restrict__ entry_slot, DeltaArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x, e = blockIdx.y;
    if (c >= a.channels) return;
    const int start = entry_start[e], row0 = entry_first_row[e], count = entry_first_row[e + 1] - row0;
    float* ring = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride + a.ring0;
    for (int i = max(0, count - a.taps); i < count; ++i)
        ring[static_cast<int64_t>((start + i) % a.taps) * a.channels + c] =
            to_f32<TX>(x[static_cast<int64_t>(row0 + i) * a.x_stride + c]);
}

// A value of every lane of a group of 4 or 16 neighbouring lanes summed over the group, left in all of them.
template <int CTRL>
__device__ __forceinline__ float lane_move(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}

template <int R>
__device__ __forceinline__ float group_sum(float v) {
    v += lane_move<0xB1>(v);       // quad_perm [1, 0, 3, 2]
    v += lane_move<0x4E>(v);       // quad_perm [2, 3, 0, 1]
    if constexpr (R >= 16) {
        v += lane_move<0x124>(v);  // row_ror 4
        v += lane_move<0x128>(v);  // row_ror 8
    }
    return v;
}

constexpr int WALK_TOKENS = 16;
constexpr int WALK_THREADS = 256;

// A workgroup of four wavefronts owns 4 * 64 / R neighbouring columns of one head's state; lane l of a wavefront holds
// rows (l % R) + R j of column l / R in registers.  The columns do not depend on each other; inside one, the lanes' parts
// of S^T k and S^T q meet through lane exchanges.  16 tokens at a time lie in LDS while the next 16 are fetched.
template <int D, int R>
__global__ __launch_bounds__(WALK_THREADS) void delta_walk_kernel(const float* __restrict__ rows, const float* __restrict__ gates,
                                                                  float* __restrict__ out, float* __restrict__ state,
                                                                  const int* __restrict__ entry_first_row,
                                                                  const int* __restrict__ entry_start,
                                                                  const int* __restrict__ entry_slot,
                                                                  const int* __restrict__ which, DeltaArgs a) {
    constexpr int TB = WALK_TOKENS;
    constexpr int CW = PULSE_WAVE / R, WC = 4 * CW, DR = D / R;
    constexpr int EQ = TB * D / WALK_THREADS, EV = TB * WC / WALK_THREADS;
    static_assert(EQ >= 1 && EV >= 1 && DR >= 4 && DR % 4 == 0, "sizes");
    constexpr int SEG = DR + 4, DP = R * SEG;      // a lane's rows lie side by side, lanes set apart by 16 bytes
    __shared__ __attribute__((aligned(16))) float q_s[TB][DP];
    __shared__ __attribute__((aligned(16))) float k_s[TB][DP];
    __shared__ float v_s[TB][WC];
    __shared__ float gb_s[TB][2];
    const int e = which ? which[blockIdx.x] : blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, lane = tid % PULSE_WAVE, wave = tid / PULSE_WAVE;
    const int rg = lane % R, cl = lane / R;
    const int c = blockIdx.z * WC + wave * CW + cl;
    const bool live = c < a.dv;
    const int row0 = entry_first_row[e], n = entry_first_row[e + 1] - row0;
    const int grp = h / (a.heads / a.groups);
    const int q0 = grp * a.d, k0 = (a.groups + grp) * a.d, v0 = 2 * a.groups * a.d + h * a.dv;
    float* S = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride + static_cast<int64_t>(h) * a.d * a.dv;
    const bool fresh = entry_start[e] == 0;
    float s[DR];
#pragma unroll
    for (int j = 0; j < DR; ++j) {
        const int i = rg + R * j;
        s[j] = (!fresh && live && i < a.d) ? S[static_cast<int64_t>(i) * a.dv + c] : 0.f;
    }
    float qr[EQ], kr[EQ], vr[EV], gr = 0.f;
    auto fetch = [&](int t0) __attribute__((always_inline)) {
        const int nb = min(TB, n - t0);
#pragma unroll
        for (int u = 0; u < EQ; ++u) {
            const int idx = u * WALK_THREADS + tid;
            const int tt = idx / D, i = idx % D;
            qr[u] = kr[u] = 0.f;
            if (tt < nb && i < a.d) {
                const float* row = rows + static_cast<int64_t>(row0 + t0 + tt) * a.channels;
                qr[u] = row[q0 + i];
                kr[u] = row[k0 + i];
            }
        }
#pragma unroll
        for (int u = 0; u < EV; ++u) {
            const int idx = u * WALK_THREADS + tid;
            const int tt = idx / WC, cc = blockIdx.z * WC + idx % WC;
            vr[u] = (tt < nb && cc < a.dv) ? rows[static_cast<int64_t>(row0 + t0 + tt) * a.channels + v0 + cc] : 0.f;
        }
        if (tid < 2 * TB) {
            const int tt = tid / 2;
            gr = tt < nb ? gates[static_cast<int64_t>(row0 + t0 + tt) * 2 * a.heads + (tid % 2) * a.heads + h] : 0.f;
        }
    };
    auto step = [&](int t0, int tt) __attribute__((always_inline)) {
        const float v = v_s[tt][wave * CW + cl];
        const float g = gb_s[tt][0], beta = gb_s[tt][1];
        const float4* kp = reinterpret_cast<const float4*>(&k_s[tt][rg * SEG]);
        const float4* qp = reinterpret_cast<const float4*>(&q_s[tt][rg * SEG]);
        float kk[DR];
        float p[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j4 = 0; j4 < DR / 4; ++j4) {
            const float4 k4 = kp[j4];
            kk[4 * j4] = k4.x; kk[4 * j4 + 1] = k4.y; kk[4 * j4 + 2] = k4.z; kk[4 * j4 + 3] = k4.w;
#pragma unroll
            for (int u = 0; u < 4; ++u) { s[4 * j4 + u] *= g; p[u] = fmaf(s[4 * j4 + u], kk[4 * j4 + u], p[u]); }
        }
        const float u = beta * (v - group_sum<R>((p[0] + p[1]) + (p[2] + p[3])));
        float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j4 = 0; j4 < DR / 4; ++j4) {
            const float4 q4 = qp[j4];
            const float qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
            for (int w = 0; w < 4; ++w) {
                s[4 * j4 + w] = fmaf(kk[4 * j4 + w], u, s[4 * j4 + w]);
                o[w] = fmaf(s[4 * j4 + w], qq[w], o[w]);
            }
        }
        const float ov = group_sum<R>((o[0] + o[1]) + (o[2] + o[3]));
        if (live && rg == 0) out[static_cast<int64_t>(row0 + t0 + tt) * a.heads * a.dv + h * a.dv + c] = ov;
    };
    if (n > 0) fetch(0);
    for (int t0 = 0; t0 < n; t0 += TB) {
        __syncthreads();   // the tokens in LDS have been walked
#pragma unroll
        for (int u = 0; u < EQ; ++u) {
            const int idx = u * WALK_THREADS + tid;
            const int i = idx % D, at = (i % R) * SEG + i / R;
            q_s[idx / D][at] = qr[u];
            k_s[idx / D][at] = kr[u];
        }
#pragma unroll
        for (int u = 0; u < EV; ++u) {
            const int idx = u * WALK_THREADS + tid;
            v_s[idx / WC][idx % WC] = vr[u];
        }
        if (tid < 2 * TB) gb_s[tid / 2][tid % 2] = (tid % 2) ? gr : expf(gr);
        __syncthreads();
        if (t0 + TB < n) fetch(t0 + TB);
        const int nb = min(TB, n - t0);
        if (nb == TB) {
#pragma unroll 4
            for (int tt = 0; tt < TB; ++tt) step(t0, tt);
        } else {
            for (int tt = 0; tt < nb; ++tt) step(t0, tt);
        }
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < DR; ++j) {
            const int i = rg + R * j;
            if (i < a.d) S[static_cast<int64_t>(i) * a.dv + c] = s[j];
        }
    }
}

// ------------------------------------------------------------------ 64 tokens at a time
// With G_i the sum of the logarithms of the decays of a chunk's tokens up to i and S the state before the chunk:
//     u_i = beta_i v_i - beta_i e^(G_i) S^T k_i - sum_(j < i) A_ij u_j,      A_ij = beta_i e^(G_i - G_j) k_i . k_j
// so U = Y - W S with (I + A) [Y | W] = [diag(beta) V | diag(beta e^G) K], a forward substitution that does not know S, and
//     O = diag(e^G) Q S + P U,  P_ij = e^(G_i - G_j) q_i . k_j  (j <= i),      S <- e^(G_last) S + (diag(e^(G_last - G)) K)^T U.
// A first kernel does what needs no state, a workgroup a (chunk, head), all chunks at the same time; a second one goes
// through an entry's chunks in order, a workgroup a (entry, head, 16 columns of the state): three products of float32
// matrix instructions a chunk.  No exponent is ever positive, so nothing overflows whatever the decays.
constexpr int CHUNK = 64;
typedef __attribute__((ext_vector_type(4))) float f32x4;

// What the first kernel leaves for a (chunk, head), in floats from its place in the scratch (D: d rounded up): W [64, D],
// e^G Q [64, D], (e^(G_last - G) K)^T [D, 64], P [64, 64], Y [64, dvp], e^(G_last), 3 spare.  All matrices lie in tiles of
// 16 x 16 in the order in which the second kernel's operands want them: the four numbers of lane l of a wavefront at
// 4 l of the tile (a load is 1 KB in a row; row by row a load of 64 lanes would touch 64 pieces of 16 bytes).
//   W, Q, P:  tile (row / 16, column / 16), lane = row % 16 + 16 (column % 16 / 4), number column % 4
//   K^T:      tile (channel / 16, token / 16), lane = channel % 16 + 16 (token % 16 / 4), number token % 4
//   Y:        tile (column / 16, token / 16), lane = column % 16 + 16 (token % 16 / 4), number token % 4
__host__ __device__ inline int64_t chunk_floats(int D, int dvp) { return CHUNK * (3ll * D + CHUNK + dvp) + 4; }

__device__ __forceinline__ f32x4 load4(const float* p, bool ok) {
    return ok ? *reinterpret_cast<const f32x4*>(p) : f32x4{0.f, 0.f, 0.f, 0.f};
}

// A 4 x 4 block turned around inside every quad of lanes: lane i of a quad brings v[0 .. 3] and leaves with what lanes
// 0 .. 3 brought as their number i.
__device__ __forceinline__ f32x4 quad_transpose(f32x4 v, int lane) {
    f32x4 out;
    const int q = lane & 3;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        // what goes to lane q ^ k (and comes from there): the number with that lane's place
        const int to = q ^ k;
        float send = to == 0 ? v[0] : to == 1 ? v[1] : to == 2 ? v[2] : v[3];
        if (k == 1) send = lane_move<0xB1>(send);        // quad_perm [1, 0, 3, 2]
        else if (k == 2) send = lane_move<0x4E>(send);   // quad_perm [2, 3, 0, 1]
        else if (k == 3) send = lane_move<0x1B>(send);   // quad_perm [3, 2, 1, 0]
        if (to == 0) out[0] = send;
        else if (to == 1) out[1] = send;
        else if (to == 2) out[2] = send;
        else out[3] = send;
    }
    return out;
}

template <int D>
__global__ __launch_bounds__(256, 2) void delta_chunk_prepare_kernel(const float* __restrict__ rows, const float* __restrict__ gates,
                                                                  const int* __restrict__ chunks, float* __restrict__ scratch,
                                                                  int dvp, DeltaArgs a) {
    constexpr int B = D / 16;
    __shared__ __attribute__((aligned(16))) float A_s[CHUNK][CHUNK + 4];
    __shared__ __attribute__((aligned(16))) float K_s[CHUNK][D + 4];     // q first, then k
    __shared__ float G_s[CHUNK], beta_s[CHUNK], front_s[CHUNK], left_s[CHUNK];   // beta e^G, e^(G_last - G)
    const int h = blockIdx.y, tid = threadIdx.x, lane = tid % PULSE_WAVE, wave = tid / PULSE_WAVE;
    const int row0 = chunks[4 * blockIdx.x], n = chunks[4 * blockIdx.x + 1];
    float* item = scratch + (static_cast<int64_t>(blockIdx.x) * a.heads + h) * chunk_floats(D, dvp);
    float* W = item;
    float* Qs = W + CHUNK * D;
    float* KdT = Qs + CHUNK * D;
    float* P = KdT + CHUNK * D;
    float* Y = P + CHUNK * CHUNK;
    const int grp = h / (a.heads / a.groups);
    const int q0 = grp * a.d, k0 = (a.groups + grp) * a.d, v0 = 2 * a.groups * a.d + h * a.dv;
    if (wave == 0) {
        const float* gt = gates + static_cast<int64_t>(row0 + lane) * 2 * a.heads + h;
        float g = lane < n ? gt[0] : 0.f;
        const float beta = lane < n ? gt[a.heads] : 0.f;
#pragma unroll
        for (int off = 1; off < PULSE_WAVE; off <<= 1) {
            const float up = __shfl_up(g, off, PULSE_WAVE);
            if (lane >= off) g += up;
        }
        const float last = __shfl(g, PULSE_WAVE - 1, PULSE_WAVE);
        G_s[lane] = g;
        beta_s[lane] = beta;
        front_s[lane] = beta * expf(g);
        left_s[lane] = expf(last - g);
        if (lane == 0) Y[CHUNK * dvp] = expf(last);
    }
    auto stage = [&](int col0) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < CHUNK * D / 4 / 256; ++u) {
            const int idx = u * 256 + tid, i = idx / (D / 4), c = 4 * (idx % (D / 4));
            *reinterpret_cast<f32x4*>(&K_s[i][c]) =
                load4(rows + static_cast<int64_t>(row0 + i) * a.channels + col0 + c, i < n && c < a.d);
        }
    };
    const int m = lane % 16, kq = lane / 16;
    stage(q0);
    __syncthreads();
    f32x4 qa[B];
    {
        const float eg = expf(G_s[16 * wave + m]);
#pragma unroll
        for (int b = 0; b < B; ++b) {
            qa[b] = *reinterpret_cast<const f32x4*>(&K_s[16 * wave + m][16 * b + 4 * kq]);
            *reinterpret_cast<f32x4*>(Qs + ((wave * B + b) * PULSE_WAVE + lane) * 4) = qa[b] * eg;
        }
    }
    __syncthreads();
    stage(k0);
    __syncthreads();
    {
        f32x4 ka[B];
#pragma unroll
        for (int b = 0; b < B; ++b) ka[b] = *reinterpret_cast<const f32x4*>(&K_s[16 * wave + m][16 * b + 4 * kq]);
        for (int jt = wave + 1; jt < 4; ++jt)
            *reinterpret_cast<f32x4*>(P + ((wave * 4 + jt) * PULSE_WAVE + lane) * 4) = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int jt = 0; jt <= wave; ++jt) {
            const int j = 16 * jt + m;
            f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int b = 0; b < B; ++b) {
                const f32x4 kb = *reinterpret_cast<const f32x4*>(&K_s[j][16 * b + 4 * kq]);
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    kk = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[b][u], kb[u], kk, 0, 0, 0);
                    qk = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[b][u], kb[u], qk, 0, 0, 0);
                }
            }
            // lane: rows 16 wave + 4 kq + u, column j
            f32x4 p;
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int r = 16 * wave + 4 * kq + u;
                const float e = j <= r ? expf(G_s[r] - G_s[j]) : 0.f;
                A_s[r][j] = j < r ? beta_s[r] * e * kk[u] : 0.f;
                p[u] = e * qk[u];
            }
            // rows 4 kq .. + 3 of column m become columns 4 (m / 4) .. + 3 of row 4 kq + m % 4
            p = quad_transpose(p, lane);
            *reinterpret_cast<f32x4*>(P + ((wave * 4 + jt) * PULSE_WAVE + 16 * (m / 4) + 4 * kq + m % 4) * 4) = p;
        }
    }
    __syncthreads();
    // forward substitution, a thread a column of [W | Y] (whole wavefronts: the stores of W exchange numbers inside quads)
    for (int col = tid; col < D + dvp; col += 256) {
        const bool key = col < D;
        const int c = key ? col : col - D;
        float x[CHUNK];
        if (key) {
#pragma unroll
            for (int i = 0; i < CHUNK; ++i) x[i] = K_s[i][c];
#pragma unroll
            for (int b = 0; b < CHUNK / 4; ++b) {
                f32x4 t;
#pragma unroll
                for (int u = 0; u < 4; ++u) t[u] = x[4 * b + u] * left_s[4 * b + u];
                *reinterpret_cast<f32x4*>(KdT + (((c / 16) * 4 + b / 4) * PULSE_WAVE + 16 * (b % 4) + c % 16) * 4) = t;
            }
        } else {
            const float* src = rows + static_cast<int64_t>(row0) * a.channels + v0 + c;
#pragma unroll
            for (int i = 0; i < CHUNK; ++i) x[i] = (c < a.dv && i < n) ? src[static_cast<int64_t>(i) * a.channels] : 0.f;
        }
        int place = 0;
#pragma unroll
        for (int i = 0; i < CHUNK; ++i) {
            // a row of A is read when the row before the last has been used: all at once they need 2000 registers
            if (i > 1) asm volatile("" : "+v"(place), "+v"(x[i - 2]));
            float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int b = 0; b < (i + 3) / 4; ++b) {
                const f32x4 ar = *reinterpret_cast<const f32x4*>(&A_s[i][4 * b + place]);
#pragma unroll
                for (int u = 0; u < 4; ++u)
                    if (4 * b + u < i) s[u] = fmaf(ar[u], x[4 * b + u], s[u]);
            }
            const float f = key ? front_s[i] : beta_s[i];
            x[i] = f * x[i] - ((s[0] + s[1]) + (s[2] + s[3]));
        }
#pragma unroll
        for (int b = 0; b < CHUNK / 4; ++b) {
            f32x4 t = {x[4 * b], x[4 * b + 1], x[4 * b + 2], x[4 * b + 3]};
            if (key) {   // a row's four neighbouring columns
                t = quad_transpose(t, lane);
                const int r = 4 * b + c % 4;
                *reinterpret_cast<f32x4*>(W + (((r / 16) * B + c / 16) * PULSE_WAVE + 16 * ((c % 16) / 4) + r % 16) * 4) = t;
            } else {     // a column's four neighbouring rows
                *reinterpret_cast<f32x4*>(Y + (((c / 16) * 4 + b / 4) * PULSE_WAVE + 16 * (b % 4) + c % 16) * 4) = t;
            }
        }
    }
}

template <int D>
__global__ __launch_bounds__(256, 1) void delta_chunk_walk_kernel(float* __restrict__ scratch, const int* __restrict__ chunks,
                                                               const int* __restrict__ runs, float* __restrict__ out,
                                                               float* __restrict__ state, const int* __restrict__ entry_start,
                                                               const int* __restrict__ entry_slot, int dvp, DeltaArgs a) {
    constexpr int B = D / 16;                         // 16-channel tiles of the state
    constexpr int TW = B >= 4 ? B / 4 : 1;            // of which a wavefront keeps
    __shared__ __attribute__((aligned(16))) float S_s[16][D + 4];       // [column][channel]
    __shared__ __attribute__((aligned(16))) float U_s[16][CHUNK + 4];   // [column][token]
    const int e = runs[4 * blockIdx.x], first = runs[4 * blockIdx.x + 1], count = runs[4 * blockIdx.x + 2];
    const int h = blockIdx.y, c0 = 16 * blockIdx.z;
    const int lane = threadIdx.x % PULSE_WAVE, wave = threadIdx.x / PULSE_WAVE;
    const int m = lane % 16, kq = lane / 16;
    const int64_t size = chunk_floats(D, dvp);
    float* S = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride + static_cast<int64_t>(h) * a.d * a.dv;
    const bool fresh = entry_start[e] == 0;
    // lane: columns c0 + 4 kq + u, channel 16 tile + m
    f32x4 acc[TW];
#pragma unroll
    for (int t = 0; t < TW; ++t) {
        const int ch = 16 * (wave * TW + t) + m;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int c = c0 + 4 * kq + u;
            acc[t][u] = (!fresh && ch < a.d && c < a.dv) ? S[static_cast<int64_t>(ch) * a.dv + c] : 0.f;
            if (wave * TW + t < B) S_s[4 * kq + u][ch] = acc[t][u];
        }
    }
    // What a chunk's products read is asked for a whole chunk ahead, into one of two sets of registers.  Loads and stores
    // stand outside every branch (addresses are clamped, results that nobody may see go to a spare place behind the item's
    // last number): the compiler then knows how many are in flight and waits for the older set alone.
    struct Operands {
        f32x4 wv[B], qv[B], pv[4], kd[TW][4], yv;
        float el;
    };
    auto load = [&](int i, Operands& o) __attribute__((always_inline)) {
        const float* W = scratch + (static_cast<int64_t>(first + i) * a.heads + h) * size;
        const float* KdT = W + 2 * CHUNK * D;
        const float* P = KdT + CHUNK * D;
        const float* Y = P + CHUNK * CHUNK;
        auto tile = [&](const float* from, int t) { return *reinterpret_cast<const f32x4*>(from + (t * PULSE_WAVE + lane) * 4); };
#pragma unroll
        for (int b = 0; b < B; ++b) {
            o.wv[b] = tile(W, wave * B + b);
            o.qv[b] = tile(W + CHUNK * D, wave * B + b);
        }
        o.yv = tile(Y, blockIdx.z * 4 + wave);
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            o.pv[b] = tile(P, wave * 4 + b);
#pragma unroll
            for (int t = 0; t < TW; ++t) o.kd[t][b] = tile(KdT, min(wave * TW + t, B - 1) * 4 + b);
        }
        o.el = Y[CHUNK * dvp];
    };
    auto chunk = [&](int i, const Operands& o) __attribute__((always_inline)) {
        const int row0 = chunks[4 * (first + i)], n = chunks[4 * (first + i) + 1];
        __syncthreads();     // S_s is whole, U_s has been read
        f32x4 us = {0.f, 0.f, 0.f, 0.f}, os = {0.f, 0.f, 0.f, 0.f};
        f32x4 sb[B];
#pragma unroll
        for (int b = 0; b < B; ++b) sb[b] = *reinterpret_cast<const f32x4*>(&S_s[m][16 * b + 4 * kq]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int b = 0; b < B; ++b) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                us = __builtin_amdgcn_mfma_f32_16x16x4f32(o.wv[b][u], sb[b][u], us, 0, 0, 0);
                os = __builtin_amdgcn_mfma_f32_16x16x4f32(o.qv[b][u], sb[b][u], os, 0, 0, 0);
            }
        }
        f32x4 uv;
#pragma unroll
        for (int u = 0; u < 4; ++u) uv[u] = o.yv[u] - us[u];
        *reinterpret_cast<f32x4*>(&U_s[m][16 * wave + 4 * kq]) = uv;
        __syncthreads();
#pragma unroll
        for (int t = 0; t < TW; ++t) acc[t] *= o.el;
        f32x4 ub[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) ub[b] = *reinterpret_cast<const f32x4*>(&U_s[m][16 * b + 4 * kq]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int b = 0; b < 4; ++b) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                os = __builtin_amdgcn_mfma_f32_16x16x4f32(o.pv[b][u], ub[b][u], os, 0, 0, 0);
#pragma unroll
                for (int t = 0; t < TW; ++t)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ub[b][u], o.kd[t][b][u], acc[t], 0, 0, 0);
            }
        }
#pragma unroll
        for (int t = 0; t < TW; ++t)
            if (wave * TW + t < B) {
#pragma unroll
                for (int u = 0; u < 4; ++u) S_s[4 * kq + u][16 * (wave * TW + t) + m] = acc[t][u];
            }
        float* spare = scratch + (static_cast<int64_t>(first + i) * a.heads + h + 1) * size - 1;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int r = 16 * wave + 4 * kq + u;
            float* dst = out + static_cast<int64_t>(row0 + r) * a.heads * a.dv + h * a.dv + c0 + m;
            *(r < n && c0 + m < a.dv ? dst : spare) = os[u];
        }
    };
    Operands even, odd;
    load(0, even);
    for (int i = 0;;) {
        load(min(i + 1, count - 1), odd);
        chunk(i, even);
        if (++i == count) break;
        load(min(i + 1, count - 1), even);
        chunk(i, odd);
        if (++i == count) break;
    }
#pragma unroll
    for (int t = 0; t < TW; ++t) {
        const int ch = 16 * (wave * TW + t) + m;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int c = c0 + 4 * kq + u;
            if (wave * TW + t < B && ch < a.d && c < a.dv) S[static_cast<int64_t>(ch) * a.dv + c] = acc[t][u];
        }
    }
}

// ------------------------------------------------------------------ decoded tokens
constexpr int DEC_THREADS = 512;

__device__ __forceinline__ float4 add4(float4 x, float4 y) { return make_float4(x.x + y.x, x.y + y.y, x.z + y.z, x.w + y.w); }

// A workgroup a (token, head).  A thread holds NJ rows of four neighbouring columns of the state (rows set NG apart):
// the state is read and written once, 16 bytes a lane, and asked for before anything else.  CVP: threads side by side
// along the columns, the smallest power of two of at least dv / 4.
template <typename TX, int NJ>
__global__ __launch_bounds__(DEC_THREADS) void delta_decode_kernel(const TX* __restrict__ x, const float* __restrict__ taps,
                                                                   const float* __restrict__ a_log,
                                                                   const float* __restrict__ dt_bias,
                                                                   const float* __restrict__ norm_w, float* __restrict__ state,
                                                                   TX* __restrict__ y, int64_t y_stride,
                                                                   const int* __restrict__ positions,
                                                                   const int* __restrict__ token_entry,
                                                                   const int* __restrict__ entry_slot, int cvp, float eps,
                                                                   float out_scale, DeltaArgs a) {
    __shared__ float kq_s[2 * 256];          // q, then k
    __shared__ float v_s[512];
    __shared__ float o_s[512];
    __shared__ float4 red[512];              // [row groups of the workgroup / those inside a wavefront][cvp]
    __shared__ float small_s[4];             // 1 / |q|, 1 / |k|, decay, strength
    const int t = blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, lane = tid % PULSE_WAVE, wave = tid / PULSE_WAVE;
    const int e = token_entry[t], pos = positions[t];
    float* slot = state + static_cast<int64_t>(entry_slot[e]) * a.slot_stride;
    float4* S = reinterpret_cast<float4*>(slot + static_cast<int64_t>(h) * a.d * a.dv);
    const int nv = a.dv / 4;
    const int cv = tid % cvp, rg = tid / cvp, ng = DEC_THREADS / cvp;
    const bool col = cv < nv;
    float4 s[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = rg + ng * j;
        s[j] = (pos > 0 && col && i < a.d) ? S[static_cast<int64_t>(i) * nv + cv] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const int per = a.heads / a.groups, grp = h / per;
    const TX* row = x + static_cast<int64_t>(t) * a.x_stride;
    float* ring = slot + a.ring0;
    for (int i = tid; i < 2 * a.d + a.dv; i += DEC_THREADS) {
        int c;
        if (i < 2 * a.d) c = (i < a.d ? grp : a.groups + grp) * a.d + (i < a.d ? i : i - a.d);
        else c = 2 * a.groups * a.d + h * a.dv + i - 2 * a.d;
        float acc = 0.f;
        for (int j = 0; j + 1 < a.taps; ++j) {
            const int p = pos - (a.taps - 1) + j;
            if (p >= 0) acc = fmaf(taps[j * a.channels + c], ring[static_cast<int64_t>(p % a.taps) * a.channels + c], acc);
        }
        const float now = to_f32<TX>(row[c]);
        acc = silu_f(fmaf(taps[(a.taps - 1) * a.channels + c], now, acc));
        if (i < 2 * a.d) {
            kq_s[i] = acc;
            if (h % per == 0) ring[static_cast<int64_t>(pos % a.taps) * a.channels + c] = now;
        } else {
            v_s[i - 2 * a.d] = acc;
            ring[static_cast<int64_t>(pos % a.taps) * a.channels + c] = now;
        }
    }
    if (tid == DEC_THREADS - 1) {
        small_s[2] = expf(-expf(a_log[h]) * softplus_f(to_f32<TX>(row[a.a0 + h]) + dt_bias[h]));
        small_s[3] = sigmoid_f(to_f32<TX>(row[a.b0 + h]));
    }
    __syncthreads();
    if (wave < 2) {
        float ss = 0.f;
        for (int i = lane; i < a.d; i += PULSE_WAVE) { const float v = kq_s[wave * a.d + i]; ss = fmaf(v, v, ss); }
        ss = wave_sum(ss);
        if (lane == 0) small_s[wave] = 1.0f / sqrtf(ss + UNIT_EPS) * (wave == 0 ? 1.0f / sqrtf(static_cast<float>(a.d)) : 1.f);
    }
    __syncthreads();
    const float qn = small_s[0], kn = small_s[1], g = small_s[2], beta = small_s[3];
    // a column's sum over all rows: the wavefront's row groups by lane exchanges, the wavefronts through LDS
    auto column_sum = [&](float4 v) __attribute__((always_inline)) -> float4 {
        for (int off = cvp; off < PULSE_WAVE; off <<= 1) {
            v.x += __shfl_xor(v.x, off, PULSE_WAVE); v.y += __shfl_xor(v.y, off, PULSE_WAVE);
            v.z += __shfl_xor(v.z, off, PULSE_WAVE); v.w += __shfl_xor(v.w, off, PULSE_WAVE);
        }
        const int inside = cvp < PULSE_WAVE ? PULSE_WAVE / cvp : 1, n = ng / inside;
        __syncthreads();    // (what was summed before has been read)
        if (rg % inside == 0) red[(rg / inside) * cvp + cv] = v;
        __syncthreads();
        float4 sum = red[cv];
        for (int w = 1; w < n; ++w) sum = add4(sum, red[w * cvp + cv]);
        return sum;
    };
    float4 r = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = rg + ng * j;
        const float kv = i < a.d ? kq_s[a.d + i] * kn : 0.f;
        s[j].x *= g; s[j].y *= g; s[j].z *= g; s[j].w *= g;
        r.x = fmaf(s[j].x, kv, r.x); r.y = fmaf(s[j].y, kv, r.y); r.z = fmaf(s[j].z, kv, r.z); r.w = fmaf(s[j].w, kv, r.w);
    }
    r = column_sum(r);
    float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
    if (col) {
        u.x = beta * (v_s[4 * cv] - r.x); u.y = beta * (v_s[4 * cv + 1] - r.y);
        u.z = beta * (v_s[4 * cv + 2] - r.z); u.w = beta * (v_s[4 * cv + 3] - r.w);
    }
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = rg + ng * j;
        if (i < a.d) {
            const float kv = kq_s[a.d + i] * kn, qv = kq_s[i] * qn;
            s[j].x = fmaf(kv, u.x, s[j].x); s[j].y = fmaf(kv, u.y, s[j].y); s[j].z = fmaf(kv, u.z, s[j].z); s[j].w = fmaf(kv, u.w, s[j].w);
            o.x = fmaf(s[j].x, qv, o.x); o.y = fmaf(s[j].y, qv, o.y); o.z = fmaf(s[j].z, qv, o.z); o.w = fmaf(s[j].w, qv, o.w);
            if (col) S[static_cast<int64_t>(i) * nv + cv] = s[j];
        }
    }
    o = column_sum(o);
    if (rg == 0 && col) { o_s[4 * cv] = o.x; o_s[4 * cv + 1] = o.y; o_s[4 * cv + 2] = o.z; o_s[4 * cv + 3] = o.w; }
    __syncthreads();
    float ss = 0.f;
    for (int i = lane; i < a.dv; i += PULSE_WAVE) ss = fmaf(o_s[i], o_s[i], ss);
    const float inv = out_scale / sqrtf(wave_sum(ss) / static_cast<float>(a.dv) + eps);
    const TX* gate = row + a.g0 + h * a.dv;
    TX* dst = y + static_cast<int64_t>(t) * y_stride + h * a.dv;
    for (int i = tid; i < a.dv; i += DEC_THREADS)
        dst[i] = from_f32<TX>(o_s[i] * inv * norm_w[i] * silu_f(to_f32<TX>(gate[i])));
}

int fill_args(DeltaArgs& a, int heads, int groups, int d, int dv, int taps, int g0, int b0, int a0, int64_t x_stride,
              int64_t slot_stride) {
    PULSE_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && d > 0 && dv > 0, "delta: bad head counts or sizes");
    PULSE_REQUIRE(d <= 256, "delta: at most 256 key channels a head, got %d", d);
    PULSE_REQUIRE(taps >= 1 && taps <= MAX_TAPS, "delta: 1 to %d taps, got %d", MAX_TAPS, taps);
    a.heads = heads; a.groups = groups; a.d = d; a.dv = dv; a.taps = taps;
    a.channels = 2 * groups * d + heads * dv;
    a.g0 = g0; a.b0 = b0; a.a0 = a0; a.x_stride = x_stride; a.slot_stride = slot_stride;
    a.ring0 = static_cast<int64_t>(heads) * d * dv;
    PULSE_REQUIRE(slot_stride >= a.ring0 + static_cast<int64_t>(taps) * a.channels, "delta: the slots are too small");
    return 0;
}

}  // namespace

// x [tokens, x_stride]: raw q, k, v from column 0, the strengths (heads) from b0, the decays (heads) from a0.  taps
// float32 [n_taps, channels]; a_log, dt_bias float32 [heads]; state [slots, slot_stride] float32.  rows float32 [tokens,
// channels] and gates float32 [tokens, 2 heads] (logarithms of the decays, then the strengths) receive the results.
extern "C" int pulse_delta_prepare(const void* x, int x_dtype, int64_t x_stride, int b0, int a0, const float* taps,
                                   const float* a_log, const float* dt_bias, float* state, int slots, int64_t slot_stride,
                                   float* rows, float* gates, const int* positions, const int* token_entry,
                                   const int* entry_start, const int* entry_first_row, const int* entry_slot, int tokens,
                                   int entries, int heads, int groups, int d, int dv, int n_taps, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && entries >= 0 && entries < 65536 && slots > 0 && pulse_dtype_ok(x_dtype), "delta_prepare: bad sizes or dtype tag");
    PULSE_REQUIRE(x && taps && a_log && dt_bias && state && rows && gates && positions && token_entry && entry_start &&
                  entry_first_row && entry_slot, "delta_prepare: null pointer");
    DeltaArgs a;
    if (fill_args(a, heads, groups, d, dv, n_taps, 0, b0, a0, x_stride, slot_stride)) return 1;
    PULSE_REQUIRE(b0 >= 0 && a0 >= 0 && x_stride >= a.channels && x_stride >= b0 + heads && x_stride >= a0 + heads,
                  "delta_prepare: the rows are too short");
    if (tokens == 0 || entries == 0) return 0;
    const int xb = x_dtype == PULSE_F32 ? 4 : 2;
    const bool runs = tokens >= 64 && n_taps >= 2 && n_taps <= 4 && d % 2 == 0 && a.channels % 2 == 0 && x_stride % 2 == 0 &&
                      slot_stride % 2 == 0 && a.ring0 % 2 == 0 && reinterpret_cast<uintptr_t>(x) % (2 * xb) == 0 &&
                      reinterpret_cast<uintptr_t>(taps) % 8 == 0 && reinterpret_cast<uintptr_t>(state) % 8 == 0 &&
                      reinterpret_cast<uintptr_t>(rows) % 8 == 0;
    if (runs) {
        const int units = 2 * groups + (heads * dv + 127) / 128;
#define PULSE_RUNS(TAPS_, PASSES_)                                                                                        \
    PULSE_DISPATCH_DTYPE(x_dtype, TX,                                                                                     \
        hipLaunchKernelGGL((delta_prepare_runs_kernel<TX, TAPS_, PASSES_>), dim3((tokens + RUN - 1) / RUN, (units + 3) / 4), \
                           dim3(256), 0, stream, static_cast<const TX*>(x), taps, a_log, dt_bias, state, rows, gates,     \
                           positions, token_entry, entry_start, entry_first_row, entry_slot, tokens, units, a))
        if (d <= 128) {
            if (n_taps == 2) PULSE_RUNS(2, 1);
            else if (n_taps == 3) PULSE_RUNS(3, 1);
            else PULSE_RUNS(4, 1);
        } else {
            if (n_taps == 2) PULSE_RUNS(2, 2);
            else if (n_taps == 3) PULSE_RUNS(3, 2);
            else PULSE_RUNS(4, 2);
        }
#undef PULSE_RUNS
    } else {
        PULSE_DISPATCH_DTYPE(x_dtype, TX,
            hipLaunchKernelGGL(delta_prepare_kernel<TX>, dim3(tokens), dim3(256), 0, stream, static_cast<const TX*>(x), taps,
                               a_log, dt_bias, state, rows, gates, positions, token_entry, entry_start, entry_first_row,
                               entry_slot, a));
    }
    PULSE_LAUNCH_CHECK("delta_prepare");
    if (n_taps > 1) {
        PULSE_DISPATCH_DTYPE(x_dtype, TX,
            hipLaunchKernelGGL(delta_ring_kernel<TX>, dim3((a.channels + 255) / 256, entries), dim3(256), 0, stream,
                               static_cast<const TX*>(x), state, entry_start, entry_first_row, entry_slot, a));
        PULSE_LAUNCH_CHECK("delta_prepare (ring)");
    }
    return 0;
}

// row_groups: over how many lanes a column's rows are shared out (4, or 16 from 64 key channels a head on).  which: the
// `entries` entries that are walked (null: entries 0, 1, ...).
extern "C" int pulse_delta_walk(const float* rows, const float* gates, float* out, float* state, int slots,
                                int64_t slot_stride, const int* entry_first_row, const int* entry_start,
                                const int* entry_slot, const int* which, int entries, int heads, int groups, int d, int dv,
                                int n_taps, int row_groups, hipStream_t stream) {
    PULSE_REQUIRE(entries >= 0 && slots > 0 && heads < 65536 && dv < 65536 * 4, "delta_walk: bad sizes");
    PULSE_REQUIRE(rows && gates && out && state && entry_first_row && entry_start && entry_slot, "delta_walk: null pointer");
    DeltaArgs a;
    if (fill_args(a, heads, groups, d, dv, n_taps, 0, 0, 0, 0, slot_stride)) return 1;
    if (entries == 0) return 0;
#define PULSE_WALK(D_, R_)                                                                                              \
    hipLaunchKernelGGL((delta_walk_kernel<D_, R_>), dim3(entries, heads, (dv * R_ + 255) / 256), dim3(WALK_THREADS), 0,  \
                       stream, rows, gates, out, state, entry_first_row, entry_start, entry_slot, which, a)
    if (d <= 16) PULSE_WALK(16, 4);
    else if (d <= 32) PULSE_WALK(32, 4);
    else if (d <= 64) { if (row_groups >= 16) PULSE_WALK(64, 16); else PULSE_WALK(64, 4); }
    else if (d <= 128) { if (row_groups >= 16) PULSE_WALK(128, 16); else PULSE_WALK(128, 4); }
    else { if (row_groups >= 16) PULSE_WALK(256, 16); else PULSE_WALK(256, 4); }
#undef PULSE_WALK
    PULSE_LAUNCH_CHECK("delta_walk");
    return 0;
}

static int chunk_channels(int d) { return d <= 32 ? 32 : (d <= 64 ? 64 : 128); }

// Whether pulse_delta_chunks takes heads of these sizes.
extern "C" int pulse_delta_chunks_takes(int d, int dv) { return d >= 4 && d <= 128 && d % 4 == 0 && dv >= 4 && dv % 4 == 0; }

// Float32 values of scratch that one chunk of one head needs.
extern "C" int64_t pulse_delta_chunk_floats(int d, int dv) { return chunk_floats(chunk_channels(d), (dv + 15) / 16 * 16); }

// chunks int32 [n_chunks, 4]: first row, tokens (1 to 64), 0, 0, an entry's chunks in order and next to each other; runs int32
// [n_runs, 4]: entry, its first chunk, its number of chunks, 0.  scratch float32 [n_chunks, heads, pulse_delta_chunk_floats].
extern "C" int pulse_delta_chunks(const float* rows, const float* gates, float* out, float* state, int slots, int64_t slot_stride,
                                  const int* entry_start, const int* entry_slot, const int* chunks, int n_chunks,
                                  const int* runs, int n_runs, float* scratch, int heads, int groups, int d, int dv, int n_taps,
                                  hipStream_t stream) {
    PULSE_REQUIRE(n_chunks >= 0 && n_runs >= 0 && slots > 0 && heads < 65536, "delta_chunks: bad sizes");
    PULSE_REQUIRE(rows && gates && out && state && entry_start && entry_slot && chunks && runs && scratch, "delta_chunks: null pointer");
    PULSE_REQUIRE(pulse_delta_chunks_takes(d, dv), "delta_chunks: heads of %d x %d are not a size it takes", d, dv);
    DeltaArgs a;
    if (fill_args(a, heads, groups, d, dv, n_taps, 0, 0, 0, 0, slot_stride)) return 1;
    PULSE_REQUIRE(reinterpret_cast<uintptr_t>(rows) % 16 == 0 && reinterpret_cast<uintptr_t>(scratch) % 16 == 0,
                  "delta_chunks: rows and scratch must be 16-byte aligned");
    if (n_chunks == 0 || n_runs == 0) return 0;
    const int dvp = (dv + 15) / 16 * 16;
#define PULSE_CHUNKS(D_)                                                                                                \
    do {                                                                                                                \
        hipLaunchKernelGGL((delta_chunk_prepare_kernel<D_>), dim3(n_chunks, heads), dim3(256), 0, stream, rows, gates,  \
                           chunks, scratch, dvp, a);                                                                    \
        PULSE_LAUNCH_CHECK("delta_chunks (prepare)");                                                                   \
        hipLaunchKernelGGL((delta_chunk_walk_kernel<D_>), dim3(n_runs, heads, dvp / 16), dim3(256), 0, stream, scratch, \
                           chunks, runs, out, state, entry_start, entry_slot, dvp, a);                                  \
    } while (0)
    if (d <= 32) PULSE_CHUNKS(32);
    else if (d <= 64) PULSE_CHUNKS(64);
    else PULSE_CHUNKS(128);
#undef PULSE_CHUNKS
    PULSE_LAUNCH_CHECK("delta_chunks");
    return 0;
}

static int decode_columns(int dv) {
    int cvp = 1;
    while (cvp < dv / 4) cvp *= 2;
    return cvp;
}

// Whether pulse_delta_decode takes heads of these sizes.
extern "C" int pulse_delta_decode_takes(int d, int dv) {
    if (d < 1 || d > 256 || dv < 4 || dv % 4 != 0 || dv > 512) return 0;
    const int ng = DEC_THREADS / decode_columns(dv);
    return (d + ng - 1) / ng <= 32;
}

// A step of single tokens, row t of x the token of entry token_entry[t].  norm_w float32 [dv], shared by the heads;
// y [tokens, y_stride] of x's storage type receives (heads x dv) results: normed, gated by silu, times out_scale.
extern "C" int pulse_delta_decode(const void* x, int x_dtype, int64_t x_stride, int g0, int b0, int a0, const float* taps,
                                  const float* a_log, const float* dt_bias, const float* norm_w, float* state, int slots,
                                  int64_t slot_stride, void* y, int64_t y_stride, const int* positions,
                                  const int* token_entry, const int* entry_slot, int tokens, int heads, int groups, int d,
                                  int dv, int n_taps, float eps, float out_scale, hipStream_t stream) {
    PULSE_REQUIRE(tokens >= 0 && slots > 0 && heads < 65536 && pulse_dtype_ok(x_dtype), "delta_decode: bad sizes or dtype tag");
    PULSE_REQUIRE(x && taps && a_log && dt_bias && norm_w && state && y && positions && token_entry && entry_slot,
                  "delta_decode: null pointer");
    PULSE_REQUIRE(pulse_delta_decode_takes(d, dv), "delta_decode: heads of %d x %d are not a size it takes", d, dv);
    DeltaArgs a;
    if (fill_args(a, heads, groups, d, dv, n_taps, g0, b0, a0, x_stride, slot_stride)) return 1;
    PULSE_REQUIRE(g0 >= 0 && b0 >= 0 && a0 >= 0 && x_stride >= a.channels && x_stride >= g0 + static_cast<int64_t>(heads) * dv &&
                  x_stride >= b0 + heads && x_stride >= a0 + heads && y_stride >= static_cast<int64_t>(heads) * dv,
                  "delta_decode: the rows are too short");
    PULSE_REQUIRE(slot_stride % 4 == 0 && reinterpret_cast<uintptr_t>(state) % 16 == 0, "delta_decode: the states must be 16-byte aligned");
    if (tokens == 0) return 0;
    const int cvp = decode_columns(dv), ng = DEC_THREADS / cvp, nj = (d + ng - 1) / ng;
#define PULSE_DECODE(NJ_)                                                                                               \
    PULSE_DISPATCH_DTYPE(x_dtype, TX,                                                                                   \
        hipLaunchKernelGGL((delta_decode_kernel<TX, NJ_>), dim3(tokens, heads), dim3(DEC_THREADS), 0, stream,           \
                           static_cast<const TX*>(x), taps, a_log, dt_bias, norm_w, state, static_cast<TX*>(y), y_stride, \
                           positions, token_entry, entry_slot, cvp, eps, out_scale, a))
    if (nj <= 1) PULSE_DECODE(1);
    else if (nj <= 2) PULSE_DECODE(2);
    else if (nj <= 4) PULSE_DECODE(4);
    else if (nj <= 8) PULSE_DECODE(8);
    else if (nj <= 16) PULSE_DECODE(16);
    else PULSE_DECODE(32);
#undef PULSE_DECODE
    PULSE_LAUNCH_CHECK("delta_decode");
    return 0;
}
