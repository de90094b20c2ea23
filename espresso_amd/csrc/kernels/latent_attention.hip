// Latent attention on gfx950: keys and values of a token are projections of one cached latent, plus one rotated key part that all
// heads share; a sliding window, a learned sink per head in the softmax's denominator, a sigmoid gate per head on the output.
//
//   cached row: [latent c (rank_p) | rotated key part (rot_p)], one per token, at position % ring
//   score_h(i, j) = ((q_h . W_uk_h c_j) + q_rot_h . k_rot_j) scale,   value_h(j) = W_uv_h c_j
//
// Decode (launch_latent_step, three launches): the query goes through W_uk^T once instead of every key through W_uk, so a head's
// query is a row of rank_p + rot_p values against the cached rows themselves, and the weighted sum stays in the latent space until
// one product with W_uv.  All heads share the cached rows: 32 heads are the 32 columns of the matrix-core tile.  Slices of the
// window go to different workgroups, which leave (maximum, sum, weighted latents); the merge adds the sink once.
//
// Prompt blocks (launch_latent_block): keys and values of the visible span are products of the gathered latents (done by the
// caller as two dense products, values transposed), then attention in tiles of 64 keys: a wavefront owns 32 queries; scores are
// computed transposed (keys as rows), so a lane holds one query's column, the softmax needs one exchange between the lane halves,
// and the weights are the B operand of the value product without passing through LDS.
// With bf16 operands queries of the decode form and softmax weights enter the products as a high and a low bf16.
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::floatx16;
using matrix::Op;

// Element i of x at a position whose cosines and sines are given, rotated: pairs (2i, 2i + 1) of the first dims elements.
__device__ __forceinline__ float rotated_pairs(const float *x, int i, int dims, const float *cos, const float *sin) {
    if (i >= dims) return x[i];
    const float c = cos[i >> 1], s = sin[i >> 1], u = x[i & ~1], v = x[i | 1];
    return (i & 1) ? v * c + u * s : u * c - v * s;
}

template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(LatentShape l, const float *mixed, const int *pos, const int *seq) {
    __shared__ float red[4];
    const int m = blockIdx.x, p = pos[m], width = l.rank_p + l.rot_p;
    const float *c = mixed + (size_t)m * l.ld_mix + l.dkv_at;
    float s = 0.0f;
    for (int i = threadIdx.x; i < l.rank_p; i += 256) s += c[i] * c[i];
    const float inv = 1.0f / sqrtf(detail::workgroup_sum(s, red) / (float)l.kv_rank + l.eps);
    T *row = static_cast<T *>(l.cache) + ((size_t)seq[m] * l.ring + p % l.ring) * width;
    const size_t at = (size_t)p * (l.rot_dims / 2);
    for (int i = threadIdx.x; i < width; i += 256)
        row[i] = Op<T>::from_float(i < l.rank_p ? c[i] * inv * l.latent_norm[i] : rotated_pairs(c + l.rank_p, i - l.rank_p, l.rot_dims, l.cos + at, l.sin + at));
}

// absorbed[m][h] = scale * [W_uk_h^T q_h | rotated part]; grid (chunks of 128 ranks, heads, rows)
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentShape l, LatentStep p) {
    extern __shared__ float lds[];   // q [dim_p], partial sums [16][128]
    const int tid = threadIdx.x, c0 = blockIdx.x * 128, h = blockIdx.y, m = blockIdx.z, qk = l.dim_p + l.rot_p;
    const float *q = p.mixed + (size_t)m * l.ld_mix + h * qk;
    float *out = p.absorbed + ((size_t)m * l.heads + h) * (l.rank_p + l.rot_p);
    for (int i = tid; i < l.dim_p; i += 256) lds[i] = q[i];
    if (blockIdx.x == 0) {
        const size_t at = (size_t)p.pos[m] * (l.rot_dims / 2);
        for (int i = tid; i < l.rot_p; i += 256) out[l.rank_p + i] = l.scale * rotated_pairs(q + l.dim_p, i, l.rot_dims, l.cos + at, l.sin + at);
    }
    __syncthreads();
    const int col = c0 + (tid & 15) * 8, g = tid >> 4;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (col < l.rank_p) {
        const uint16_t *w = l.uk + (size_t)h * l.dim_p * l.rank_p + col;
        for (int d = g; d < l.dim_p; d += 16) {
            float f[8];
            matrix::unpack_bf16(*reinterpret_cast<const uint4 *>(w + (size_t)d * l.rank_p), f);
            const float x = lds[d];
#pragma unroll
            for (int i = 0; i < 8; i++) acc[i] = __builtin_fmaf(f[i], x, acc[i]);
        }
    }
    float *sums = lds + l.dim_p;
#pragma unroll
    for (int i = 0; i < 8; i++) sums[g * 128 + (tid & 15) * 8 + i] = acc[i];
    __syncthreads();
    if (tid < 128 && c0 + tid < l.rank_p) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) s += sums[i * 128 + tid];
        out[c0 + tid] = s * l.scale;
    }
}

// Keys a query at `pos` sees: first, and how many.
__device__ __forceinline__ int first_seen(int pos, int window) { return pos - window + 1 > 0 ? pos - window + 1 : 0; }

template <typename T>
struct PartialLayout {   // LDS of latent_partial_kernel
    static constexpr int kPad = 16 / sizeof(T);
    static size_t bytes(int width, bool queries) { return (size_t)32 * (width + kPad) * sizeof(T) + (size_t)4 * 32 * 33 * 4 + (queries ? (size_t)32 * (width + 4) * 4 : 0); }
};

// grid (splits, groups of 32 heads, rows); NT: tiles of 32 ranks per wavefront
template <typename T, int NT>
__global__ __launch_bounds__(256) void latent_partial_kernel(LatentShape l, LatentStep p, int queries_in_lds) {
    extern __shared__ char smem[];
    const int width = l.rank_p + l.rot_p, ldc = width + PartialLayout<T>::kPad, ldq = width + 4;
    T *tile = reinterpret_cast<T *>(smem);
    float *scores = reinterpret_cast<float *>(tile + 32 * ldc), *queries = scores + 4 * 32 * 33;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, half = lane >> 5, col = lane & 31;
    const int split = blockIdx.x, m = blockIdx.z, pos = p.pos[m];
    const int lo = first_seen(pos, l.window), tiles = (pos - lo) / 32 + 1;
    if (split >= tiles) return;
    const int head = blockIdx.y * 32 + col, head_in = head < l.heads ? head : l.heads - 1;   // columns past the heads repeat the last one
    const float *q_row = p.absorbed + ((size_t)m * l.heads + head_in) * width;
    if (queries_in_lds) {
        for (int i = tid * 4; i < 32 * width; i += 256 * 4) {
            const int hh = i / width, k = i % width, hs = blockIdx.y * 32 + hh < l.heads ? blockIdx.y * 32 + hh : l.heads - 1;
            *reinterpret_cast<float4 *>(queries + hh * ldq + k) = *reinterpret_cast<const float4 *>(p.absorbed + ((size_t)m * l.heads + hs) * width + k);
        }
        q_row = queries + col * ldq;
    }
    const T *cache = static_cast<const T *>(l.cache) + (size_t)p.seq[m] * l.ring * width;
    float top = -INFINITY, sum = 0.0f;
    floatx16 acc[NT];
#pragma unroll
    for (int i = 0; i < NT; i++) acc[i] = matrix::zero_accumulator();
    const int pieces = width / 8;
    for (int t = split; t < tiles; t += p.splits) {
        const int k0 = lo + t * 32;
        __syncthreads();
        for (int i = tid; i < 32 * pieces; i += 256) {
            const int row = i / pieces, part = i % pieces, key = k0 + row < pos ? k0 + row : pos;   // rows past the query repeat it; masked below
            const uint4 *src = reinterpret_cast<const uint4 *>(cache + (size_t)(key % l.ring) * width + part * 8);
            uint4 *dst = reinterpret_cast<uint4 *>(tile + row * ldc + part * 8);
            dst[0] = src[0];
            if constexpr (sizeof(T) == 4) dst[1] = src[1];
        }
        __syncthreads();
        floatx16 s = matrix::zero_accumulator();
        for (int ks = wave; ks < width / 16; ks += 4) {
            const float *qp = q_row + ks * 16 + 8 * half;
            const float4 q0 = reinterpret_cast<const float4 *>(qp)[0], q1 = reinterpret_cast<const float4 *>(qp)[1];
            const float f[8] = {q0.x, q0.y, q0.z, q0.w, q1.x, q1.y, q1.z, q1.w};
            s = matrix::mma_values<T>(Op<T>::load(tile + col * ldc + ks * 16 + 8 * half), f, s);
        }
#pragma unroll
        for (int r = 0; r < 16; r++) scores[(wave * 32 + matrix::accumulator_row(r, half)) * 33 + col] = s[r];
        __syncthreads();
        float w[16], best = -INFINITY;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int key = matrix::accumulator_row(r, half), at = key * 33 + col;
            const float x = (scores[at] + scores[at + 32 * 33]) + (scores[at + 64 * 33] + scores[at + 96 * 33]);
            w[r] = k0 + key <= pos ? x : -INFINITY;
            best = fmaxf(best, w[r]);
        }
        best = fmaxf(fmaxf(best, __shfl_xor(best, 32)), top);
        const float keep = expf(top - best);
        float add = 0.0f;
#pragma unroll
        for (int r = 0; r < 16; r++) { w[r] = expf(w[r] - best); add += w[r]; }
        add += __shfl_xor(add, 32);
        sum = sum * keep + add;
        top = best;
#pragma unroll
        for (int i = 0; i < NT; i++) {
            const int r0 = (wave + 4 * i) * 32;
            if (r0 >= l.rank_p) continue;
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][r] *= keep;
#pragma unroll
            for (int st = 0; st < 2; st++) {
                T e[8];
                float f[8];
#pragma unroll
                for (int j = 0; j < 8; j++) {
                    e[j] = tile[matrix::accumulator_row(st * 8 + j, half) * ldc + r0 + col];
                    f[j] = w[st * 8 + j];
                }
                acc[i] = matrix::mma_values<T>(Op<T>::from_elems(e), f, acc[i]);
            }
        }
    }
    if (head >= l.heads) return;
    const size_t at = ((size_t)m * p.splits + split) * l.heads + head;
#pragma unroll
    for (int i = 0; i < NT; i++) {
        const int r0 = (wave + 4 * i) * 32;
        if (r0 >= l.rank_p) continue;
#pragma unroll
        for (int g = 0; g < 4; g++)
            *reinterpret_cast<float4 *>(p.partial + at * l.rank_p + r0 + g * 8 + 4 * half) = make_float4(acc[i][4 * g], acc[i][4 * g + 1], acc[i][4 * g + 2], acc[i][4 * g + 3]);
    }
    if (wave == 0 && half == 0) *reinterpret_cast<float2 *>(p.partial_ml + at * 2) = make_float2(top, sum);
}

// Slices of a head merged with its sink, then 32 rows of W_uv and the gate; grid (vdim_p / 32, heads, rows)
template <typename T>
__global__ __launch_bounds__(256) void latent_merge_kernel(LatentShape l, LatentStep p) {
    extern __shared__ float lds[];   // merged latents [rank_p], weights [splits]
    const int tid = threadIdx.x, h = blockIdx.y, m = blockIdx.z, pos = p.pos[m];
    const int tiles = (pos - first_seen(pos, l.window)) / 32 + 1, live = tiles < p.splits ? tiles : p.splits;
    const size_t first = (size_t)m * p.splits * l.heads + h;   // slice s: first + s * heads
    const float sink = l.sink[h];
    float top = sink, sum = 0.0f;
    for (int s = 0; s < live; s++) top = fmaxf(top, p.partial_ml[(first + (size_t)s * l.heads) * 2]);
    for (int s = 0; s < live; s++) {
        const float2 ml = *reinterpret_cast<const float2 *>(p.partial_ml + (first + (size_t)s * l.heads) * 2);
        const float w = expf(ml.x - top);
        sum += w * ml.y;
        if (tid == 0) lds[l.rank_p + s] = w;
    }
    const float inv = 1.0f / (sum + expf(sink - top));
    __syncthreads();
    for (int r = tid; r < l.rank_p; r += 256) {
        float v = 0.0f;
        for (int s = 0; s < live; s++) v += lds[l.rank_p + s] * p.partial[(first + (size_t)s * l.heads) * l.rank_p + r];
        lds[r] = v * inv;
    }
    __syncthreads();
    const int e = tid & 7, j = blockIdx.x * 32 + (tid >> 3);
    const uint16_t *w = l.uv + ((size_t)h * l.vdim_p + j) * l.rank_p;
    float o = 0.0f;
    for (int r = e * 8; r < l.rank_p; r += 64) {
        float f[8];
        matrix::unpack_bf16(*reinterpret_cast<const uint4 *>(w + r), f);
#pragma unroll
        for (int i = 0; i < 8; i++) o = __builtin_fmaf(f[i], lds[r + i], o);
    }
    o += detail::dpp_term<0xB1, 0xF>(o);
    o += detail::dpp_term<0x4E, 0xF>(o);
    o += detail::dpp_term<0x141, 0xF>(o);
    if (e != 0) return;
    o *= matrix::sigmoid(p.mixed[(size_t)m * l.ld_mix + l.gate_at + h]);
    if (p.mix) p.mix[(size_t)m * l.heads * l.vdim_p + h * l.vdim_p + j] = o;
    else static_cast<T *>(p.act)[(size_t)m * p.ld_act + h * l.vdim_p + j] = Op<T>::from_float(o);
}

// ---- prompt blocks ---------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(128) void latent_gather_kernel(LatentShape l, LatentBlock p) {
    const int i = blockIdx.x, width = l.rank_p + l.rot_p;
    const T *row = static_cast<const T *>(l.cache) + ((size_t)p.seq * l.ring + (p.first_key + i) % l.ring) * width;
    for (int c = threadIdx.x * 4; c < width; c += 128 * 4) {   // sizes are multiples of four elements
        T *dst = c < l.rank_p ? static_cast<T *>(p.latents) + (size_t)i * l.rank_p + c : static_cast<T *>(p.key_rot) + (size_t)i * l.rot_p + c - l.rank_p;
#pragma unroll
        for (int k = 0; k < 4; k++) dst[k] = i < p.keys ? row[c + k] : (T)0;
    }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_queries_kernel(LatentShape l, LatentBlock p, int rows_p) {
    const int m = blockIdx.x, qk = l.dim_p + l.rot_p;
    const float *row = p.mixed + (size_t)m * l.ld_mix;
    const size_t at = (size_t)(p.base + m) * (l.rot_dims / 2);
    for (int i = threadIdx.x; i < l.heads * qk; i += 256) {
        const int h = i / qk, d = i % qk;
        float v = 0.0f;
        if (m < p.rows) v = d < l.dim_p ? row[i] : rotated_pairs(row + h * qk + l.dim_p, d - l.dim_p, l.rot_dims, l.cos + at, l.sin + at);
        static_cast<T *>(p.q)[((size_t)h * rows_p + m) * qk + d] = Op<T>::from_float(v);
    }
}

constexpr int kQueries = 128, kKeys = 64, kValues = 128;   // per workgroup and tile
template <typename T>
struct BlockLayout {
    static constexpr int kPad = 16 / sizeof(T);
    static size_t bytes(int qk) { return ((size_t)kKeys * (qk + kPad) + (size_t)kValues * (kKeys + kPad)) * sizeof(T); }
};

// grid (blocks of 128 queries, heads, slices of 128 values); NQ: steps of 16 query dimensions held in registers, 0 = read again
template <typename T, int NQ>
__global__ __launch_bounds__(256) void latent_block_kernel(LatentShape l, LatentBlock p, int rows_p) {
    extern __shared__ char smem[];
    constexpr int kPad = BlockLayout<T>::kPad, LDV = kKeys + kPad;
    const int qk = l.dim_p + l.rot_p, ldk = qk + kPad;
    T *kt = reinterpret_cast<T *>(smem), *vt = kt + kKeys * ldk;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, half = lane >> 5, col = lane & 31;
    const int h = blockIdx.y, q0 = blockIdx.x * kQueries, v0 = blockIdx.z * kValues;
    const int values = l.vdim_p - v0 < kValues ? l.vdim_p - v0 : kValues;
    const int m = q0 + wave * 32 + col, at = p.base - p.first_key + m;   // this lane's query: row and place among the keys
    const int wave_at = p.base - p.first_key + q0 + wave * 32;           // the wavefront's first query
    const T *q = static_cast<const T *>(p.q) + ((size_t)h * rows_p + (m < rows_p ? m : rows_p - 1)) * qk + 8 * half;
    typename Op<T>::frag qf[NQ ? NQ : 1];
    if constexpr (NQ > 0) {
#pragma unroll
        for (int i = 0; i < NQ; i++) qf[i] = Op<T>::load(q + (i * 16 < qk ? i * 16 : 0));
    }
    float top = l.sink[h], sum = 1.0f;   // the sink: one more term of the denominator, without a value
    floatx16 out[4];
#pragma unroll
    for (int i = 0; i < 4; i++) out[i] = matrix::zero_accumulator();
    const int block_at = p.base - p.first_key + q0, seen = block_at - l.window + 1;
    const int k_begin = seen > 0 ? seen / kKeys * kKeys : 0;
    const int last = q0 + kQueries < p.rows ? q0 + kQueries : p.rows, k_end = p.base - p.first_key + last;
    const int row_pieces = l.dim_p / 8, rot_pieces = l.rot_p / 8, k_pieces = row_pieces + rot_pieces;
    const T *keys = static_cast<const T *>(p.k), *key_rot = static_cast<const T *>(p.key_rot), *vals = static_cast<const T *>(p.vt);
    auto copy = [&](T *dst, const T *src) {
        reinterpret_cast<uint4 *>(dst)[0] = reinterpret_cast<const uint4 *>(src)[0];
        if constexpr (sizeof(T) == 4) reinterpret_cast<uint4 *>(dst)[1] = reinterpret_cast<const uint4 *>(src)[1];
    };
    for (int k0 = k_begin; k0 < k_end; k0 += kKeys) {
        __syncthreads();
        for (int i = tid; i < kKeys * k_pieces; i += 256) {
            const int row = i / k_pieces, part = i % k_pieces;
            copy(kt + row * ldk + part * 8, part < row_pieces ? keys + (size_t)(k0 + row) * l.heads * l.dim_p + h * l.dim_p + part * 8
                                                               : key_rot + (size_t)(k0 + row) * l.rot_p + (part - row_pieces) * 8);
        }
        for (int i = tid; i < values * (kKeys / 8); i += 256) {
            const int row = i / (kKeys / 8), part = i % (kKeys / 8);
            copy(vt + row * LDV + part * 8, vals + ((size_t)h * l.vdim_p + v0 + row) * p.keys_p + k0 + part * 8);
        }
        __syncthreads();
        if (k0 > wave_at + 31 || k0 + kKeys - 1 <= wave_at - l.window) continue;   // no query of this wavefront sees the tile
        floatx16 s[2];
        s[0] = s[1] = matrix::zero_accumulator();
        const T *kp = kt + col * ldk + 8 * half;
        if constexpr (NQ > 0) {
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                if (i * 16 < qk) {
                    s[0] = Op<T>::mma(Op<T>::load(kp + i * 16), qf[i], s[0]);
                    s[1] = Op<T>::mma(Op<T>::load(kp + 32 * ldk + i * 16), qf[i], s[1]);
                }
            }
        } else {
            for (int d = 0; d < qk; d += 16) {
                const typename Op<T>::frag f = Op<T>::load(q + d);
                s[0] = Op<T>::mma(Op<T>::load(kp + d), f, s[0]);
                s[1] = Op<T>::mma(Op<T>::load(kp + 32 * ldk + d), f, s[1]);
            }
        }
        float w[2][16], best = -INFINITY;
#pragma unroll
        for (int t = 0; t < 2; t++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int gap = at - (k0 + t * 32 + matrix::accumulator_row(r, half));
                w[t][r] = gap >= 0 && gap < l.window ? s[t][r] * l.scale : -INFINITY;
                best = fmaxf(best, w[t][r]);
            }
        best = fmaxf(fmaxf(best, __shfl_xor(best, 32)), top);
        const float keep = expf(top - best);
        float add = 0.0f;
#pragma unroll
        for (int t = 0; t < 2; t++)
#pragma unroll
            for (int r = 0; r < 16; r++) { w[t][r] = expf(w[t][r] - best); add += w[t][r]; }
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
        for (int t = 0; t < 2; t++)
#pragma unroll
            for (int st = 0; st < 2; st++) {
                float f[8];
#pragma unroll
                for (int j = 0; j < 8; j++) f[j] = w[t][st * 8 + j];
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    if (i * 32 >= values) continue;
                    const T *vp = vt + (i * 32 + col) * LDV + t * 32 + st * 16 + 4 * half;
                    out[i] = matrix::mma_values<T>(Op<T>::load_pair(vp, vp + 8), f, out[i]);
                }
            }
    }
    if (m >= p.rows) return;
    const float factor = matrix::sigmoid(p.mixed[(size_t)m * l.ld_mix + l.gate_at + h]) / sum;
    T *dst = static_cast<T *>(p.act) + (size_t)m * p.ld_act + h * l.vdim_p + v0;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        if (i * 32 >= values) continue;
#pragma unroll
        for (int g = 0; g < 4; g++)
#pragma unroll
            for (int k = 0; k < 4; k++) dst[i * 32 + g * 8 + 4 * half + k] = Op<T>::from_float(out[i][4 * g + k] * factor);
    }
}

bool shape_ok(const LatentShape &l) {
    return l.heads > 0 && l.dim_p % 32 == 0 && l.vdim_p % 32 == 0 && l.rot_p % 32 == 0 && l.rank_p % 64 == 0 && l.dim <= l.dim_p && l.vdim <= l.vdim_p && l.rot_dim <= l.rot_p &&
           l.kv_rank <= l.rank_p && l.rot_dims <= l.rot_dim && l.rot_dims % 2 == 0 && l.window >= 1 && l.ring >= 1 && l.cache && l.rank_p <= kLatentMaxRank && l.dim_p <= 4096;
}

template <typename T, int NT>
hipError_t run_partial(const LatentShape &l, const LatentStep &p, hipStream_t s) {
    const int width = l.rank_p + l.rot_p;
    const bool queries = PartialLayout<T>::bytes(width, true) <= 158 * 1024;   // otherwise they are read from memory for every tile
    const size_t lds = PartialLayout<T>::bytes(width, queries);
    if (lds > 158 * 1024) return hipErrorInvalidValue;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_partial_kernel<T, NT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_partial_kernel<T, NT>), dim3(p.splits, (l.heads + 31) / 32, p.rows), dim3(256), lds, s, l, p, queries ? 1 : 0);
    return hipGetLastError();
}

template <typename T>
hipError_t run_step(const LatentShape &l, const LatentStep &p, hipStream_t s) {
    hipLaunchKernelGGL(latent_absorb_kernel, dim3((l.rank_p + 127) / 128, l.heads, p.rows), dim3(256), (size_t)(l.dim_p + 16 * 128) * 4, s, l, p);
    const hipError_t e = l.rank_p <= 128 ? run_partial<T, 1>(l, p, s) : l.rank_p <= 256 ? run_partial<T, 2>(l, p, s) : l.rank_p <= 512 ? run_partial<T, 4>(l, p, s) : run_partial<T, 8>(l, p, s);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_merge_kernel<T>), dim3(l.vdim_p / 32, l.heads, p.rows), dim3(256), (size_t)(l.rank_p + p.splits) * 4, s, l, p);
    return hipGetLastError();
}

template <typename T, int NQ>
hipError_t run_block(const LatentShape &l, const LatentBlock &p, int rows_p, hipStream_t s) {
    const size_t lds = BlockLayout<T>::bytes(l.dim_p + l.rot_p);
    if (lds > 158 * 1024) return hipErrorInvalidValue;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_block_kernel<T, NQ>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_block_kernel<T, NQ>), dim3((p.rows + kQueries - 1) / kQueries, l.heads, (l.vdim_p + kValues - 1) / kValues), dim3(256), lds, s, l, p, rows_p);
    return hipGetLastError();
}

bool block_ok(const LatentShape &l, const LatentBlock &p) {
    return shape_ok(l) && p.rows >= 1 && p.base >= 0 && p.base + p.rows <= l.max_seq && p.first_key >= 0 && p.first_key <= p.base && p.keys == p.base + p.rows - p.first_key &&
           p.keys <= l.ring && p.keys_p % 64 == 0 && p.keys_p >= p.keys;
}
int padded_rows(int rows) { return (rows + 31) / 32 * 32; }

}  // namespace

int latent_step_splits(const LatentShape &l) {
    const int span = l.window < l.max_seq ? l.window : l.max_seq, tiles = (span + 31) / 32, groups = (l.heads + 31) / 32;
    const int most = 64 / groups > 0 ? 64 / groups : 1;
    return tiles < most ? tiles : most;
}

hipError_t launch_latent_store(const LatentShape &l, const float *mixed, const int *pos, const int *seq, int rows, Precision type, hipStream_t s) {
    if (!shape_ok(l) || l.dkv_at < 0 || rows < 1) return hipErrorInvalidValue;
    if (type == Precision::bf16) hipLaunchKernelGGL((latent_store_kernel<uint16_t>), dim3(rows), dim3(256), 0, s, l, mixed, pos, seq);
    else hipLaunchKernelGGL((latent_store_kernel<float>), dim3(rows), dim3(256), 0, s, l, mixed, pos, seq);
    return hipGetLastError();
}

hipError_t launch_latent_step(const LatentShape &l, const LatentStep &p, Precision type, hipStream_t s) {
    if (!shape_ok(l) || p.rows < 1 || p.splits < 1 || (!p.mix && !p.act)) return hipErrorInvalidValue;
    return type == Precision::bf16 ? run_step<uint16_t>(l, p, s) : run_step<float>(l, p, s);
}

hipError_t launch_latent_gather(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s) {
    if (!block_ok(l, p)) return hipErrorInvalidValue;
    if (type == Precision::bf16) hipLaunchKernelGGL((latent_gather_kernel<uint16_t>), dim3(p.keys_p), dim3(128), 0, s, l, p);
    else hipLaunchKernelGGL((latent_gather_kernel<float>), dim3(p.keys_p), dim3(128), 0, s, l, p);
    return hipGetLastError();
}

hipError_t launch_latent_queries(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s) {
    if (!block_ok(l, p)) return hipErrorInvalidValue;
    const int rows_p = padded_rows(p.rows);
    if (type == Precision::bf16) hipLaunchKernelGGL((latent_queries_kernel<uint16_t>), dim3(rows_p), dim3(256), 0, s, l, p, rows_p);
    else hipLaunchKernelGGL((latent_queries_kernel<float>), dim3(rows_p), dim3(256), 0, s, l, p, rows_p);
    return hipGetLastError();
}

hipError_t launch_latent_block(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s) {
    if (!block_ok(l, p)) return hipErrorInvalidValue;
    const int rows_p = padded_rows(p.rows), qk = l.dim_p + l.rot_p;
    if (type == Precision::f32) return run_block<float, 0>(l, p, rows_p, s);
    return qk <= 96 ? run_block<uint16_t, 6>(l, p, rows_p, s) : qk <= 192 ? run_block<uint16_t, 12>(l, p, rows_p, s) : run_block<uint16_t, 0>(l, p, rows_p, s);
}

}  // namespace esp
