// Attention of a block of rows of one sequence over gathered keys and transposed values (gfx950), shared by the attention mixers: a
// sliding window, grouped heads, optionally a second key part that all heads share, a learned sink per head in the softmax's
// denominator, and a sigmoid gate per head on the output.
//
// Tiles of 64 keys: a wavefront owns 32 queries and half of every tile; scores are computed transposed (keys as rows), so a lane holds one
// query's column, the softmax needs one exchange between the lane halves, and the weights are the B operand of the value product
// without passing through LDS.  With bf16 operands softmax weights enter the product as a high and a low bf16.
#include <hip/hip_runtime.h>

#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::floatx16;
using matrix::Op;
typedef uint32_t uintx4 __attribute__((ext_vector_type(4)));

constexpr int kQueries = 64, kKeys = 64, kValues = 128;   // per workgroup and tile
template <typename T>
struct BlockLayout {
    static constexpr int kPad = 16 / sizeof(T);
    static size_t bytes(int qk) {
        const size_t tiles = ((size_t)kKeys * (qk + kPad) + (size_t)kValues * (kKeys + kPad)) * sizeof(T), merge = (size_t)2 * 64 * 66 * 4;
        return tiles > merge ? tiles : merge;
    }
};

// grid (blocks of 64 queries, heads, slices of 128 values).  Wavefront w takes queries 32 (w % 2) .. and, of every tile of 64 keys, keys
// 32 (w / 2) ..; the two halves' softmax states meet in LDS at the end.  NQ: steps of 16 query dimensions held in registers (the next
// tile too), 0 = any number, read when needed.
template <typename T, int NQ>
__global__ __launch_bounds__(256) void block_attention_kernel(BlockAttention p, int rows_p) {
    extern __shared__ char smem[];
    constexpr int kPad = BlockLayout<T>::kPad, LDV = kKeys + kPad, kVec = sizeof(T) / 2;
    constexpr int PK = NQ ? NQ / 2 : 1, PV = kValues * kKeys / 8 / 256;   // pieces of eight per thread: keys (64 rows of 2 NQ pieces), values
    const int qk = p.dim_p + p.rot_p, ldk = qk + kPad;
    T *kt = reinterpret_cast<T *>(smem), *vt = kt + kKeys * ldk;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, half = lane >> 5, col = lane & 31, qt = wave & 1, set = wave >> 1;
    const int h = blockIdx.y, q0 = blockIdx.x * kQueries, v0 = blockIdx.z * kValues;
    const int values = p.vdim_p - v0 < kValues ? p.vdim_p - v0 : kValues;
    const int m = q0 + qt * 32 + col, at = p.before + m;   // this lane's query: row and place among the keys
    const int wave_at = p.before + q0 + qt * 32;           // the wavefront's first query
    const int block_at = p.before + q0, seen = block_at - p.window + 1;
    const int k_begin = seen > 0 ? seen / kKeys * kKeys : 0;
    const int last = q0 + kQueries < p.rows ? q0 + kQueries : p.rows, k_end = p.before + last;
    const int row_pieces = p.dim_p / 8, k_pieces = row_pieces + p.rot_p / 8;
    const int kv = h / (p.heads / p.kv_heads), ld_keys = p.kv_heads * p.dim_p;
    const T *keys = static_cast<const T *>(p.k) + kv * p.dim_p, *key_rot = static_cast<const T *>(p.key_rot);
    const T *vals = static_cast<const T *>(p.vt) + ((size_t)kv * p.vdim_p + v0) * p.keys_p;
    auto key_piece = [&](int k0, int i) {
        const int row = i / k_pieces, part = i % k_pieces;
        return reinterpret_cast<const uintx4 *>(part < row_pieces ? keys + (size_t)(k0 + row) * ld_keys + part * 8 : key_rot + (size_t)(k0 + row) * p.rot_p + (part - row_pieces) * 8);
    };
    auto value_piece = [&](int k0, int i) { return reinterpret_cast<const uintx4 *>(vals + (size_t)(i / (kKeys / 8)) * p.keys_p + k0 + i % (kKeys / 8) * 8); };
    auto key_place = [&](int i) { return reinterpret_cast<uintx4 *>(kt + i / k_pieces * ldk + i % k_pieces * 8); };
    auto value_place = [&](int i) { return reinterpret_cast<uintx4 *>(vt + i / (kKeys / 8) * LDV + i % (kKeys / 8) * 8); };
    const int n_key = kKeys * k_pieces, n_value = values * (kKeys / 8);
    uintx4 ahead_k[PK], ahead_v[NQ ? PV : 1];   // bf16 only: one word per piece
    auto fetch = [&](int k0) {
        if constexpr (NQ > 0) {
#pragma unroll
            for (int i = 0; i < PK; i++) ahead_k[i] = *key_piece(k0, tid + i * 256 < n_key ? tid + i * 256 : 0);
#pragma unroll
            for (int i = 0; i < PV; i++) ahead_v[i] = *value_piece(k0, tid + i * 256 < n_value ? tid + i * 256 : 0);
        }
    };
    fetch(k_begin);
    const T *q = static_cast<const T *>(p.q) + ((size_t)h * rows_p + (m < rows_p ? m : rows_p - 1)) * qk + 8 * half;
    typename Op<T>::frag qf[NQ ? NQ : 1];
    if constexpr (NQ > 0) {
#pragma unroll
        for (int i = 0; i < NQ; i++) qf[i] = Op<T>::load(q + (i * 16 < qk ? i * 16 : 0));
    }
    float top = p.sink ? p.sink[h] : -INFINITY, sum = p.sink && set == 0 ? 1.0f : 0.0f;   // the sink: one more term of the denominator, without a value
    floatx16 out[4];
#pragma unroll
    for (int i = 0; i < 4; i++) out[i] = matrix::zero_accumulator();
    for (int k0 = k_begin; k0 < k_end; k0 += kKeys) {
        __syncthreads();
        if constexpr (NQ > 0) {
#pragma unroll
            for (int i = 0; i < PK; i++)
                if (tid + i * 256 < n_key) *key_place(tid + i * 256) = ahead_k[i];
#pragma unroll
            for (int i = 0; i < PV; i++)
                if (tid + i * 256 < n_value) *value_place(tid + i * 256) = ahead_v[i];
            if (k0 + kKeys < k_end) fetch(k0 + kKeys);
        } else {
            for (int i = tid; i < n_key; i += 256) {
#pragma unroll
                for (int v = 0; v < kVec; v++) key_place(i)[v] = key_piece(k0, i)[v];
            }
            for (int i = tid; i < n_value; i += 256) {
#pragma unroll
                for (int v = 0; v < kVec; v++) value_place(i)[v] = value_piece(k0, i)[v];
            }
        }
        __syncthreads();
        const int ks = k0 + set * 32;
        if (ks > wave_at + 31 || ks + 31 <= wave_at - p.window) continue;   // no query of this wavefront sees these keys
        floatx16 s = matrix::zero_accumulator();
        const T *kp = kt + (set * 32 + col) * ldk + 8 * half;
        if constexpr (NQ > 0) {
#pragma unroll
            for (int i = 0; i < NQ; i++)
                if (i * 16 < qk) s = Op<T>::mma(Op<T>::load(kp + i * 16), qf[i], s);
        } else {
            for (int d = 0; d < qk; d += 16) s = Op<T>::mma(Op<T>::load(kp + d), Op<T>::load(q + d), s);
        }
        float w[16], best = -INFINITY;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int gap = at - (ks + matrix::accumulator_row(r, half));
            w[r] = gap >= 0 && gap < p.window ? s[r] * p.scale : -INFINITY;
            best = fmaxf(best, w[r]);
        }
        best = fmaxf(fmaxf(best, __shfl_xor(best, 32)), top);
        const float from = best > -INFINITY ? best : 0.0f;   // a query that has seen no key yet, without a sink: every term is zero
        const float keep = matrix::weight_exp<T>(top - from);
        float add = 0.0f;
#pragma unroll
        for (int r = 0; r < 16; r++) { w[r] = matrix::weight_exp<T>(w[r] - from); add += w[r]; }
        add += __shfl_xor(add, 32);
        sum = sum * keep + add;
        top = best;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            if (i * 32 >= values) continue;
#pragma unroll
            for (int r = 0; r < 16; r++) out[i][r] *= keep;
        }
#pragma unroll
        for (int st = 0; st < 2; st++) {
            float f[8];
#pragma unroll
            for (int j = 0; j < 8; j++) f[j] = w[st * 8 + j];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                if (i * 32 >= values) continue;
                const T *vp = vt + (i * 32 + col) * LDV + set * 32 + st * 16 + 4 * half;
                out[i] = matrix::mma_values<T>(Op<T>::load_pair(vp, vp + 8), f, out[i]);
            }
        }
    }
    // the second half of the keys joins the first: per query tile 64 lanes x (64 sums, maximum, denominator), 66 words apart
    __syncthreads();
    float *meet = reinterpret_cast<float *>(smem) + (size_t)(qt * 64 + lane) * 66;
    if (set == 1) {
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
            for (int r = 0; r < 16; r++) meet[i * 16 + r] = out[i][r];
        meet[64] = top;
        meet[65] = sum;
    }
    __syncthreads();
    if (set == 1 || m >= p.rows) return;
    const float all = fmaxf(top, meet[64]), mine = matrix::weight_exp<T>(top - all), theirs = matrix::weight_exp<T>(meet[64] - all);
    const float factor = (p.gate ? matrix::sigmoid(p.gate[(size_t)m * p.ld_gate + h]) : 1.0f) / (sum * mine + meet[65] * theirs);
    T *dst = static_cast<T *>(p.act) + (size_t)m * p.ld_act + h * p.vdim_p + v0;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        if (i * 32 >= values) continue;
#pragma unroll
        for (int g = 0; g < 4; g++)
#pragma unroll
            for (int k = 0; k < 4; k++) dst[i * 32 + g * 8 + 4 * half + k] = Op<T>::from_float((out[i][4 * g + k] * mine + meet[i * 16 + 4 * g + k] * theirs) * factor);
    }
}

template <typename T, int NQ>
hipError_t run_block(const BlockAttention &p, int rows_p, hipStream_t s) {
    const size_t lds = BlockLayout<T>::bytes(p.dim_p + p.rot_p);
    if (lds > 158 * 1024) return hipErrorInvalidValue;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&block_attention_kernel<T, NQ>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((block_attention_kernel<T, NQ>), dim3((p.rows + kQueries - 1) / kQueries, p.heads, (p.vdim_p + kValues - 1) / kValues), dim3(256), lds, s, p, rows_p);
    return hipGetLastError();
}

}  // namespace

hipError_t launch_block_attention(const BlockAttention &p, Precision type, hipStream_t s) {
    if (p.heads < 1 || p.kv_heads < 1 || p.heads % p.kv_heads || p.dim_p < 32 || p.dim_p % 32 || p.rot_p % 32 || p.vdim_p < 32 || p.vdim_p % 32 || p.window < 1 || p.rows < 1 ||
        p.before < 0 || p.keys_p % 64 || p.before + p.rows > p.keys_p || (p.rot_p > 0) != (p.key_rot != nullptr) || !p.q || !p.k || !p.vt || !p.act)
        return hipErrorInvalidValue;
    const int rows_p = (p.rows + 31) / 32 * 32, qk = p.dim_p + p.rot_p;
    if (type == Precision::f32) return run_block<float, 0>(p, rows_p, s);
    return qk <= 96 ? run_block<uint16_t, 6>(p, rows_p, s) : qk <= 192 ? run_block<uint16_t, 12>(p, rows_p, s) : run_block<uint16_t, 0>(p, rows_p, s);
}

}  // namespace esp
