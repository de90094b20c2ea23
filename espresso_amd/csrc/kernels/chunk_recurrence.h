// Blocks of a linear recurrence over matrix states in chunks of 64 tokens (gfx950), shared by the layers that have one:
//
//   S_t = decay_t S_(t-1) + u_t k_t v_t^T,   o_t = S_t^T q_t
//
// States are fp32 and kept transposed, [vdim][dim] per head.  A mixer prepares q, k, v in the layouts below; then
//   states    one wavefront per 32 x 32 tile of a head's state walks the chunks: it stores the state before the chunk, then
//             S = (decay of the chunk) S + V^T K on the matrix cores, with the decay from a token to its chunk's end already on V or K;
//   outputs   o = reach_t S^T q + sum over the chunk's keys s <= t of weight(t, s) (q . k_s) v_s; scores are computed transposed,
//             so that their accumulator is the operand of the second product and no score passes through LDS.
// A Decay says what reach and weight are:
//   float chunk(h, c, len)          decay over the chunk's len tokens
//   Query query(h, c, t)            what a query keeps (t: its place in the chunk), with float reach
//   void weights(q, h, c, t, s, w)  weights of the keys s .. s + 3, at most t (those past t are not used)
//   kScaledValues                   whether V (true) or K carries the decay to the chunk's end
// With bf16 operands, what belongs to the recurrence (states, decayed keys or values, scores) enters the products as a high and a
// low bf16.
#pragma once

#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace chunked {

using matrix::floatx16;
using matrix::Op;

constexpr int C = kRecurrenceChunk;

struct Block {
    int heads, key_share;                     // heads h of one key head (h / key_share) share q and k
    int dim_p, vdim_p;
    int rows, R, base;                        // R: rows rounded up to whole chunks
    const void *q, *k;                        // [key heads][R][dim_p]
    const void *vt;                           // [heads][vdim_p][R]
    // what enters the states: one side carries the decay to the chunk's end and has a low part (bf16)
    const void *state_k, *state_k_lo;         // [key heads][dim_p][R]
    const void *state_v, *state_v_lo;         // [heads][vdim_p][R]
    float *state;                             // the sequence's [heads][vdim_p][dim_p]
    void *states_hi, *states_lo;              // [R / 64][heads][vdim_p][dim_p], the state before each chunk
    float *o;                                 // [rows][heads * vdim_p]
    // optional: o = (o + skip[h] v) * silu(gate), gate [rows][ld_gate] in the layout of o
    const float *skip, *gate;
    int ld_gate;
};

// A fixed decay per head; powers[h][0 .. 64].
struct FixedDecay {
    static constexpr bool kScaledValues = false;
    const float *powers;
    struct Query { float reach; };
    __device__ __forceinline__ float chunk(int h, int, int len) const { return powers[h * (C + 1) + len]; }
    __device__ __forceinline__ Query query(int h, int, int t) const { return {powers[h * (C + 1) + t + 1]}; }
    __device__ __forceinline__ void weights(const Query &, int h, int, int t, int s, float (&w)[4]) const {
#pragma unroll
        for (int j = 0; j < 4; j++) w[j] = powers[h * (C + 1) + (t - s - j > 0 ? t - s - j : 0)];
    }
};

// A decay per head and token, as the logarithm summed from the chunk's start in two floats (differences of large sums stay exact),
// and a step size per head and token on the keys.
struct TokenDecay {
    static constexpr bool kScaledValues = true;
    const float *log_hi, *log_lo, *step;      // [heads][R]
    int R;
    struct Query { float reach, hi, lo; };
    __device__ __forceinline__ float chunk(int h, int c, int len) const { return expf(log_hi[(size_t)h * R + c * C + len - 1]); }
    __device__ __forceinline__ Query query(int h, int c, int t) const {
        const size_t at = (size_t)h * R + c * C + t;
        return {expf(log_hi[at]), log_hi[at], log_lo[at]};
    }
    __device__ __forceinline__ void weights(const Query &q, int h, int c, int, int s, float (&w)[4]) const {
        const size_t at = (size_t)h * R + c * C + s;
        const float4 hi = *reinterpret_cast<const float4 *>(log_hi + at), lo = *reinterpret_cast<const float4 *>(log_lo + at), u = *reinterpret_cast<const float4 *>(step + at);
        w[0] = expf((q.hi - hi.x) + (q.lo - lo.x)) * u.x;
        w[1] = expf((q.hi - hi.y) + (q.lo - lo.y)) * u.y;
        w[2] = expf((q.hi - hi.z) + (q.lo - lo.z)) * u.z;
        w[3] = expf((q.hi - hi.w) + (q.lo - lo.w)) * u.w;
    }
};

// One wavefront per tile of 32 v x 32 d of one head's state; workgroups of four tiles along d.
template <typename T, typename Decay>
__global__ __launch_bounds__(256) void states_kernel(Block a, Decay decay) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5;
    const int h = blockIdx.z, v0 = blockIdx.y * 32, d0 = (blockIdx.x * 4 + wave) * 32;
    if (d0 >= a.dim_p) return;
    const size_t tile = (size_t)v0 * a.dim_p + d0 + (lane & 31), head = (size_t)a.vdim_p * a.dim_p;
    float *state = a.state + (size_t)h * head;
    floatx16 acc = matrix::zero_accumulator();
    if (a.base > 0) {
#pragma unroll
        for (int i = 0; i < 16; i++) acc[i] = state[tile + (size_t)matrix::accumulator_row(i, half) * a.dim_p];
    }
    const size_t v_at = ((size_t)h * a.vdim_p + v0 + (lane & 31)) * a.R + 8 * half, k_at = ((size_t)(h / a.key_share) * a.dim_p + d0 + (lane & 31)) * a.R + 8 * half;
    const T *v_row = static_cast<const T *>(a.state_v) + v_at, *k_row = static_cast<const T *>(a.state_k) + k_at;
    const T *low_row = Decay::kScaledValues ? static_cast<const T *>(a.state_v_lo) + v_at : static_cast<const T *>(a.state_k_lo) + k_at;
    const int chunks = a.R / C;
    for (int c = 0; c < chunks; c++) {
        const int len = a.rows - c * C < C ? a.rows - c * C : C;
        T *hi = static_cast<T *>(a.states_hi) + ((size_t)c * a.heads + h) * head, *lo = static_cast<T *>(a.states_lo) + ((size_t)c * a.heads + h) * head;
        const float factor = decay.chunk(h, c, len);
        typename Op<T>::frag v[C / 16], k[C / 16], low[C / 16];   // on their way while the state before the chunk is stored
#pragma unroll
        for (int ks = 0; ks < C / 16; ks++) {
            v[ks] = Op<T>::load(v_row + c * C + ks * 16);
            k[ks] = Op<T>::load(k_row + c * C + ks * 16);
            if constexpr (Op<T>::kSplit) low[ks] = Op<T>::load(low_row + c * C + ks * 16);
        }
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const size_t o = tile + (size_t)matrix::accumulator_row(i, half) * a.dim_p;
            const T b = Op<T>::from_float(acc[i]);
            hi[o] = b;
            if constexpr (Op<T>::kSplit) lo[o] = Op<T>::from_float(acc[i] - Op<T>::to_float(b));
            acc[i] *= factor;
        }
#pragma unroll
        for (int ks = 0; ks < C / 16; ks++) {
            acc = Op<T>::mma(v[ks], k[ks], acc);
            if constexpr (Op<T>::kSplit) acc = Decay::kScaledValues ? Op<T>::mma(low[ks], k[ks], acc) : Op<T>::mma(v[ks], low[ks], acc);
        }
    }
#pragma unroll
    for (int i = 0; i < 16; i++) state[tile + (size_t)matrix::accumulator_row(i, half) * a.dim_p] = acc[i];
}

// grid (chunks, heads, slices of 128 v): wavefront w takes queries 32 (w % 2) .. of the chunk and 64 v from 64 (w / 2) of the slice.
template <typename T, typename Decay>
__global__ __launch_bounds__(256) void outputs_kernel(Block a, Decay decay) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5;
    const int c = blockIdx.x, h = blockIdx.y, qt = wave & 1, v0 = blockIdx.z * 128 + (wave >> 1) * 64;
    if (v0 >= a.vdim_p || c * C + qt * 32 >= a.rows) return;
    const bool two = v0 + 32 < a.vdim_p;   // a second tile of 32 v
    const int t_local = qt * 32 + (lane & 31);   // this lane's query, in the chunk
    const T *q = static_cast<const T *>(a.q) + ((size_t)(h / a.key_share) * a.R + c * C + t_local) * a.dim_p + 8 * half;
    const T *k = static_cast<const T *>(a.k) + ((size_t)(h / a.key_share) * a.R + c * C + (lane & 31)) * a.dim_p + 8 * half;
    const size_t head = (size_t)a.vdim_p * a.dim_p, s_at = ((size_t)c * a.heads + h) * head + (size_t)(v0 + (lane & 31)) * a.dim_p + 8 * half;
    const T *shi = static_cast<const T *>(a.states_hi) + s_at, *slo = static_cast<const T *>(a.states_lo) + s_at;
    const size_t next = two ? (size_t)32 * a.dim_p : 0;
    floatx16 score[2], out[2];
#pragma unroll
    for (int i = 0; i < 2; i++) score[i] = out[i] = matrix::zero_accumulator();
    constexpr int kAhead = Op<T>::kSplit ? 2 : 1;   // steps of 16 dimensions whose loads are in flight together (dim_p is a multiple of 32)
    const size_t k_next = qt ? (size_t)32 * a.dim_p : 0;
    for (int d0 = 0; d0 < a.dim_p; d0 += 16 * kAhead) {
        typename Op<T>::frag qf[kAhead], kf[kAhead][2], sf[kAhead][2], tf[kAhead][2];
#pragma unroll
        for (int u = 0; u < kAhead; u++) {
            const int d = d0 + 16 * u;
            qf[u] = Op<T>::load(q + d);
#pragma unroll
            for (int i = 0; i < 2; i++) {
                kf[u][i] = Op<T>::load(k + i * k_next + d);
                sf[u][i] = Op<T>::load(shi + i * next + d);
                if constexpr (Op<T>::kSplit) tf[u][i] = Op<T>::load(slo + i * next + d);
            }
        }
#pragma unroll
        for (int u = 0; u < kAhead; u++)
#pragma unroll
            for (int i = 0; i < 2; i++) {
                score[i] = Op<T>::mma(kf[u][i], qf[u], score[i]);
                out[i] = Op<T>::mma(sf[u][i], qf[u], out[i]);
                if constexpr (Op<T>::kSplit) out[i] = Op<T>::mma(tf[u][i], qf[u], out[i]);
            }
    }
    const typename Decay::Query mine = decay.query(h, c, t_local);
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 16; j++) out[i][j] *= mine.reach;
    const T *vt = static_cast<const T *>(a.vt) + ((size_t)h * a.vdim_p + v0 + (lane & 31)) * a.R + c * C + 4 * half;
    const size_t next_v = two ? (size_t)32 * a.R : 0;
    for (int kt = 0; kt <= qt; kt++) {
#pragma unroll
        for (int st = 0; st < 2; st++) {
            float w[8];
#pragma unroll
            for (int g = 0; g < 2; g++) {
                const int s_local = kt * 32 + matrix::accumulator_row(st * 8 + g * 4, half);
                float weight[4];
                decay.weights(mine, h, c, t_local, s_local, weight);
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    const int r = st * 8 + g * 4 + j;
                    const float x = kt ? score[1][r] : score[0][r];
                    w[g * 4 + j] = s_local + j <= t_local ? x * weight[j] : 0.0f;
                }
            }
#pragma unroll
            for (int i = 0; i < 2; i++) {
                const T *p = vt + i * next_v + kt * 32 + st * 16;
                out[i] = matrix::mma_values<T>(Op<T>::load_pair(p, p + 8), w, out[i]);
            }
        }
    }
    const int t = c * C + t_local;
    if (t >= a.rows) return;
    const size_t at = (size_t)h * a.vdim_p + v0;
    float *o = a.o + (size_t)t * a.heads * a.vdim_p + at;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        if (i && !two) break;
#pragma unroll
        for (int g = 0; g < 4; g++) {
            const int v = i * 32 + g * 8 + 4 * half;
            float4 y = make_float4(out[i][4 * g], out[i][4 * g + 1], out[i][4 * g + 2], out[i][4 * g + 3]);
            if (a.skip) {
                const float d = a.skip[h];
                const T *x = static_cast<const T *>(a.vt) + (at + v) * a.R + t;
                const float4 z = *reinterpret_cast<const float4 *>(a.gate + (size_t)t * a.ld_gate + at + v);
                y.x = (y.x + d * Op<T>::to_float(x[0])) * matrix::silu(z.x);
                y.y = (y.y + d * Op<T>::to_float(x[a.R])) * matrix::silu(z.y);
                y.z = (y.z + d * Op<T>::to_float(x[2 * (size_t)a.R])) * matrix::silu(z.z);
                y.w = (y.w + d * Op<T>::to_float(x[3 * (size_t)a.R])) * matrix::silu(z.w);
            }
            *reinterpret_cast<float4 *>(o + v) = y;
        }
    }
}

template <typename T, typename Decay>
void launch_states_and_outputs(const Block &a, const Decay &decay, hipStream_t s) {
    hipLaunchKernelGGL((states_kernel<T, Decay>), dim3((a.dim_p + 127) / 128, a.vdim_p / 32, a.heads), dim3(256), 0, s, a, decay);
    hipLaunchKernelGGL((outputs_kernel<T, Decay>), dim3(a.R / C, a.heads, (a.vdim_p + 127) / 128), dim3(256), 0, s, a, decay);
}

// Eight consecutive values in an operand's type.
template <typename T>
__device__ __forceinline__ void store8(T *p, const float (&x)[8]);
template <>
__device__ __forceinline__ void store8<uint16_t>(uint16_t *p, const float (&x)[8]) {
    *reinterpret_cast<uint4 *>(p) = make_uint4(matrix::pack_bf16(x[0], x[1]), matrix::pack_bf16(x[2], x[3]), matrix::pack_bf16(x[4], x[5]), matrix::pack_bf16(x[6], x[7]));
}
template <>
__device__ __forceinline__ void store8<float>(float *p, const float (&x)[8]) {
    reinterpret_cast<float4 *>(p)[0] = make_float4(x[0], x[1], x[2], x[3]);
    reinterpret_cast<float4 *>(p)[1] = make_float4(x[4], x[5], x[6], x[7]);
}
// The same as a high and a low part (low only where the type splits).
template <typename T>
__device__ __forceinline__ void store8_split(T *hi, T *lo, float (&x)[8]) {
    store8<T>(hi, x);
    if constexpr (Op<T>::kSplit) {
#pragma unroll
        for (int i = 0; i < 8; i++) x[i] -= Op<T>::to_float(Op<T>::from_float(x[i]));
        store8<T>(lo, x);
    }
}

}  // namespace chunked
}  // namespace esp
