// Latent attention on gfx950: keys and values of a token are projections of one cached latent, plus one rotated key part that all
// heads share; a sliding window, a learned sink per head in the softmax's denominator, a sigmoid gate per head on the output.
//
//   cached row: [latent c (rank_p) | rotated key part (rot_p)], one per token, at position % ring
//   score_h(i, j) = ((q_h . W_uk_h c_j) + q_rot_h . k_rot_j) scale,   value_h(j) = W_uv_h c_j
//
// Decode (launch_latent_step, three launches; the first also stores the row's own latent): the query goes through W_uk^T once instead of every key through W_uk, so a head's
// query is a row of rank_p + rot_p values against the cached rows themselves, and the weighted sum stays in the latent space until
// one product with W_uv.  All heads share the cached rows: 32 heads are the 32 columns of the matrix-core tile.  Slices of the
// window go to different workgroups, which leave (maximum, sum, weighted latents); the merge adds the sink once.
//
// Prompt blocks (launch_latent_block): keys and values of the visible span are products of the gathered latents (done by the
// caller as two dense products, values transposed), then attention in tiles of 64 keys (block_attention.hip).
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

// Row m's latent (normed) and rotated key part into the cache, by a workgroup of 256 threads.
template <typename T>
__device__ __forceinline__ void store_latent(const LatentShape &l, const float *mixed, const int *pos, const int *seq, int m, float *red) {
    const int p = pos[m], width = l.rank_p + l.rot_p;
    const float *c = mixed + (size_t)m * l.ld_mix + l.dkv_at;
    constexpr int kHeld = 4;
    static_assert(kHeld * 256 >= kLatentMaxRank, "a latent is held in registers");
    float held[kHeld], s = 0.0f;
#pragma unroll
    for (int k = 0; k < kHeld; k++) {
        const int i = threadIdx.x + k * 256;
        held[k] = i < l.rank_p ? c[i] : 0.0f;
    }
#pragma unroll
    for (int k = 0; k < kHeld; k++) s += held[k] * held[k];
    const float inv = 1.0f / sqrtf(detail::workgroup_sum(s, red) / (float)l.kv_rank + l.eps);
    T *row = static_cast<T *>(l.cache) + ((size_t)seq[m] * l.ring + p % l.ring) * width;
#pragma unroll
    for (int k = 0; k < kHeld; k++) {
        const int i = threadIdx.x + k * 256;
        if (i < l.rank_p) row[i] = Op<T>::from_float(held[k] * inv * l.latent_norm[i]);
    }
    const size_t at = (size_t)p * (l.rot_dims / 2);
    for (int i = threadIdx.x; i < l.rot_p; i += 256) row[l.rank_p + i] = Op<T>::from_float(rotated_pairs(c + l.rank_p, i, l.rot_dims, l.cos + at, l.sin + at));
}

template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(LatentShape l, const float *mixed, const int *pos, const int *seq) {
    __shared__ float red[4];
    store_latent<T>(l, mixed, pos, seq, blockIdx.x, red);
}

// absorbed[m][h] = scale * [W_uk_h^T q_h | rotated part]; grid (chunks of 128 ranks, heads, rows), and one more workgroup per row
// (y = heads, x = 0) that stores the row's own latent where the layer has one.
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentShape l, LatentStep p) {
    extern __shared__ float lds[];   // q [dim_p], partial sums [16][128]
    const int tid = threadIdx.x, c0 = blockIdx.x * 128, h = blockIdx.y, m = blockIdx.z, qk = l.dim_p + l.rot_p;
    if (h == l.heads) {
        if (blockIdx.x == 0) store_latent<T>(l, p.mixed, p.pos, p.seq, m, lds);
        return;
    }
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
        for (int d0 = g; d0 < l.dim_p; d0 += 16 * 4) {   // four rows of W_uk in flight
            uint4 v[4];
#pragma unroll
            for (int u = 0; u < 4; u++) v[u] = *reinterpret_cast<const uint4 *>(w + (size_t)(d0 + 16 * u < l.dim_p ? d0 + 16 * u : g) * l.rank_p);
#pragma unroll
            for (int u = 0; u < 4; u++) {
                if (d0 + 16 * u >= l.dim_p) continue;
                float f[8];
                matrix::unpack_bf16(v[u], f);
                const float x = lds[d0 + 16 * u];
#pragma unroll
                for (int i = 0; i < 8; i++) acc[i] = __builtin_fmaf(f[i], x, acc[i]);
            }
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

constexpr int kPartialWaves = 8, kPartialThreads = 64 * kPartialWaves;
template <typename T>
struct PartialLayout {   // LDS of latent_partial_kernel: a tile of 32 cached rows, the scores of its wavefronts
    static constexpr int kPad = 16 / sizeof(T);
    static size_t bytes(int width) { return (size_t)32 * (width + kPad) * sizeof(T) + (size_t)kPartialWaves * 32 * 33 * 4; }
};
typedef uint32_t uintx4 __attribute__((ext_vector_type(4)));

// grid (splits, groups of 32 heads, rows).  NT: tiles of 32 ranks per wavefront.  KS: rows of up to 128 KS values have their queries
// and the next tile in registers (KS steps of 16 per wavefront, KS pieces of eight per thread); 0: any width, from memory as needed.
template <typename T, int NT, int KS>
__global__ __launch_bounds__(kPartialThreads) void latent_partial_kernel(LatentShape l, LatentStep p) {
    extern __shared__ char smem[];
    constexpr int kVec = sizeof(T) / 2;   // 128-bit words per piece
    const int width = l.rank_p + l.rot_p, ldc = width + PartialLayout<T>::kPad;
    T *tile = reinterpret_cast<T *>(smem);
    float *scores = reinterpret_cast<float *>(tile + 32 * ldc);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, half = lane >> 5, col = lane & 31;
    const int split = blockIdx.x, m = blockIdx.z, pos = p.pos[m];
    const int lo = first_seen(pos, l.window), tiles = (pos - lo) / 32 + 1;
    if (split >= tiles) return;
    const int head = blockIdx.y * 32 + col, head_in = head < l.heads ? head : l.heads - 1;   // columns past the heads repeat the last one
    const float *q_row = p.absorbed + ((size_t)m * l.heads + head_in) * width + 8 * half;
    const T *cache = static_cast<const T *>(l.cache) + (size_t)p.seq[m] * l.ring * width;
    const int pieces = width / 8, steps = width / 16;
    constexpr int kRowThreads = kPartialThreads / 32;   // sixteen threads copy a row of the tile
    const int row = tid / kRowThreads, part = tid % kRowThreads;
    auto source_row = [&](int k0) {   // rows past the query repeat it and are masked below
        const int key = k0 + row < pos ? k0 + row : pos;
        return cache + (size_t)(key % l.ring) * width;
    };
    auto place = [&](int piece) { return reinterpret_cast<uintx4 *>(tile + row * ldc + piece * 8); };
    uintx4 ahead[KS ? KS * kVec : 1];
    auto fetch = [&](int t) {
        if constexpr (KS > 0) {
            const T *src = source_row(lo + t * 32);
#pragma unroll
            for (int k = 0; k < KS; k++) {
                const int piece = part + k * kRowThreads;
#pragma unroll
                for (int v = 0; v < kVec; v++) ahead[k * kVec + v] = reinterpret_cast<const uintx4 *>(src + (piece < pieces ? piece : 0) * 8)[v];
            }
        }
    };
    float qv[KS ? KS : 1][8];
    if constexpr (KS > 0) {
#pragma unroll
        for (int k = 0; k < KS; k++) {
            const int ks = wave + kPartialWaves * k < steps ? wave + kPartialWaves * k : 0;
            const float4 q0 = reinterpret_cast<const float4 *>(q_row + ks * 16)[0], q1 = reinterpret_cast<const float4 *>(q_row + ks * 16)[1];
            qv[k][0] = q0.x; qv[k][1] = q0.y; qv[k][2] = q0.z; qv[k][3] = q0.w; qv[k][4] = q1.x; qv[k][5] = q1.y; qv[k][6] = q1.z; qv[k][7] = q1.w;
        }
    }
    fetch(split);
    float top = -INFINITY, sum = 0.0f;
    floatx16 acc[NT];
#pragma unroll
    for (int i = 0; i < NT; i++) acc[i] = matrix::zero_accumulator();
    for (int t = split; t < tiles; t += p.splits) {
        const int k0 = lo + t * 32;
        __syncthreads();
        if constexpr (KS > 0) {
#pragma unroll
            for (int k = 0; k < KS; k++) {
                if (part + k * kRowThreads < pieces) {
#pragma unroll
                    for (int v = 0; v < kVec; v++) place(part + k * kRowThreads)[v] = ahead[k * kVec + v];
                }
            }
            if (t + p.splits < tiles) fetch(t + p.splits);
        } else {
            const T *src = source_row(k0);
            for (int i = part; i < pieces; i += kRowThreads) {
#pragma unroll
                for (int v = 0; v < kVec; v++) place(i)[v] = reinterpret_cast<const uintx4 *>(src + i * 8)[v];
            }
        }
        __syncthreads();
        floatx16 s = matrix::zero_accumulator();
        const T *key_row = tile + col * ldc + 8 * half;
        if constexpr (KS > 0) {
#pragma unroll
            for (int k = 0; k < KS; k++)
                if (wave + kPartialWaves * k < steps) s = matrix::mma_values<T>(Op<T>::load(key_row + (wave + kPartialWaves * k) * 16), qv[k], s);
        } else {
            for (int ks = wave; ks < steps; ks += kPartialWaves) {
                const float4 q0 = reinterpret_cast<const float4 *>(q_row + ks * 16)[0], q1 = reinterpret_cast<const float4 *>(q_row + ks * 16)[1];
                const float f[8] = {q0.x, q0.y, q0.z, q0.w, q1.x, q1.y, q1.z, q1.w};
                s = matrix::mma_values<T>(Op<T>::load(key_row + ks * 16), f, s);
            }
        }
#pragma unroll
        for (int r = 0; r < 16; r++) scores[(wave * 32 + matrix::accumulator_row(r, half)) * 33 + col] = s[r];
        __syncthreads();
        float w[16], best = -INFINITY;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int key = matrix::accumulator_row(r, half), at = key * 33 + col;
            float x = scores[at];
#pragma unroll
            for (int g = 1; g < kPartialWaves; g++) x += scores[at + g * 32 * 33];
            w[r] = k0 + key <= pos ? x : -INFINITY;
            best = fmaxf(best, w[r]);
        }
        best = fmaxf(fmaxf(best, __shfl_xor(best, 32)), top);
        const float keep = matrix::weight_exp<T>(top - best);
        float add = 0.0f;
#pragma unroll
        for (int r = 0; r < 16; r++) { w[r] = matrix::weight_exp<T>(w[r] - best); add += w[r]; }
        add += __shfl_xor(add, 32);
        sum = sum * keep + add;
        top = best;
#pragma unroll
        for (int i = 0; i < NT; i++) {
            const int r0 = (wave + kPartialWaves * i) * 32;
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
        const int r0 = (wave + kPartialWaves * i) * 32;
        if (r0 >= l.rank_p) continue;
#pragma unroll
        for (int g = 0; g < 4; g++)
            *reinterpret_cast<float4 *>(p.partial + at * l.rank_p + r0 + g * 8 + 4 * half) = make_float4(acc[i][4 * g], acc[i][4 * g + 1], acc[i][4 * g + 2], acc[i][4 * g + 3]);
    }
    if (wave == 0 && half == 0) *reinterpret_cast<float2 *>(p.partial_ml + at * 2) = make_float2(top, sum);
}

// Slices of a head merged with its sink, then 32 rows of W_uv and the gate; grid (vdim_p / 32, heads, rows).  splits <= 64: a lane
// of the first wavefront each.
template <typename T>
__global__ __launch_bounds__(256) void latent_merge_kernel(LatentShape l, LatentStep p) {
    extern __shared__ float lds[];   // merged latents [rank_p], weights [64]
    const int tid = threadIdx.x, h = blockIdx.y, m = blockIdx.z, pos = p.pos[m];
    const int tiles = (pos - first_seen(pos, l.window)) / 32 + 1, live = tiles < p.splits ? tiles : p.splits;
    const size_t first = (size_t)m * p.splits * l.heads + h;   // slice s: first + s * heads
    if (tid < 64) {
        const float sink = l.sink[h];
        const float2 ml = *reinterpret_cast<const float2 *>(p.partial_ml + (first + (size_t)(tid < live ? tid : 0) * l.heads) * 2);
        float top = fmaxf(ml.x, sink);
#pragma unroll
        for (int x = 32; x >= 1; x >>= 1) top = fmaxf(top, __shfl_xor(top, x));
        const float w = tid < live ? expf(ml.x - top) : 0.0f;
        const float sum = detail::wave_sum(w * ml.y) + expf(sink - top);
        lds[l.rank_p + tid] = w / sum;
    }
    // W_uv's row and the gate are on their way meanwhile
    const int e = tid & 7, j = blockIdx.x * 32 + (tid >> 3);
    const uint16_t *w = l.uv + ((size_t)h * l.vdim_p + j) * l.rank_p;
    constexpr int kHeld = 8;
    uint4 row[kHeld];
#pragma unroll
    for (int i = 0; i < kHeld; i++) row[i] = *reinterpret_cast<const uint4 *>(w + (e * 8 + i * 64 < l.rank_p ? e * 8 + i * 64 : 0));
    const float gate = p.mixed[(size_t)m * l.ld_mix + l.gate_at + h];
    __syncthreads();
    for (int r = tid * 4; r < l.rank_p; r += 256 * 4) {
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int s0 = 0; s0 < live; s0 += 8) {   // eight slices in flight
            float4 x[8];
#pragma unroll
            for (int u = 0; u < 8; u++) x[u] = *reinterpret_cast<const float4 *>(p.partial + (first + (size_t)(s0 + u < live ? s0 + u : 0) * l.heads) * l.rank_p + r);
#pragma unroll
            for (int u = 0; u < 8; u++) {
                if (s0 + u >= live) continue;
                const float f = lds[l.rank_p + s0 + u];
                v.x += f * x[u].x; v.y += f * x[u].y; v.z += f * x[u].z; v.w += f * x[u].w;
            }
        }
        *reinterpret_cast<float4 *>(lds + r) = v;
    }
    __syncthreads();
    float o = 0.0f;
    auto add = [&](const uint4 &piece, int r) {
        float f[8];
        matrix::unpack_bf16(piece, f);
#pragma unroll
        for (int i = 0; i < 8; i++) o = __builtin_fmaf(f[i], lds[r + i], o);
    };
#pragma unroll
    for (int i = 0; i < kHeld; i++)
        if (e * 8 + i * 64 < l.rank_p) add(row[i], e * 8 + i * 64);
    for (int r = e * 8 + kHeld * 64; r < l.rank_p; r += 64) add(*reinterpret_cast<const uint4 *>(w + r), r);
    o += detail::dpp_term<0xB1, 0xF>(o);
    o += detail::dpp_term<0x4E, 0xF>(o);
    o += detail::dpp_term<0x141, 0xF>(o);
    if (e != 0) return;
    o *= matrix::sigmoid(gate);
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

bool shape_ok(const LatentShape &l) {
    return l.heads > 0 && l.dim_p % 32 == 0 && l.vdim_p % 32 == 0 && l.rot_p % 32 == 0 && l.rank_p % 64 == 0 && l.dim <= l.dim_p && l.vdim <= l.vdim_p && l.rot_dim <= l.rot_p &&
           l.kv_rank <= l.rank_p && l.rot_dims <= l.rot_dim && l.rot_dims % 2 == 0 && l.window >= 1 && l.ring >= 1 && l.cache && l.rank_p <= kLatentMaxRank && l.dim_p <= 4096;
}

template <typename T, int NT, int KS>
hipError_t run_partial(const LatentShape &l, const LatentStep &p, hipStream_t s) {
    const size_t lds = PartialLayout<T>::bytes(l.rank_p + l.rot_p);
    if (lds > 158 * 1024) return hipErrorInvalidValue;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_partial_kernel<T, NT, KS>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_partial_kernel<T, NT, KS>), dim3(p.splits, (l.heads + 31) / 32, p.rows), dim3(kPartialThreads), lds, s, l, p);
    return hipGetLastError();
}

template <typename T>
hipError_t run_step(const LatentShape &l, const LatentStep &p, hipStream_t s) {
    const int width = l.rank_p + l.rot_p;
    hipLaunchKernelGGL((latent_absorb_kernel<T>), dim3((l.rank_p + 127) / 128, l.heads + (l.dkv_at >= 0 ? 1 : 0), p.rows), dim3(256), (size_t)(l.dim_p + 16 * 128) * 4, s, l, p);
    hipError_t e;
    if (l.rank_p <= 256 && width <= 128 * 3) e = run_partial<T, 1, 3>(l, p, s);
    else if (l.rank_p <= 512 && width <= 128 * 5) e = run_partial<T, 2, 5>(l, p, s);
    else e = run_partial<T, 4, 0>(l, p, s);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((latent_merge_kernel<T>), dim3(l.vdim_p / 32, l.heads, p.rows), dim3(256), (size_t)(l.rank_p + 64) * 4, s, l, p);
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
    if (!shape_ok(l) || p.rows < 1 || p.splits < 1 || p.splits > 64 || (!p.mix && !p.act)) return hipErrorInvalidValue;
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
    BlockAttention b;
    b.heads = b.kv_heads = l.heads; b.dim_p = l.dim_p; b.rot_p = l.rot_p; b.vdim_p = l.vdim_p; b.window = l.window; b.scale = l.scale;
    b.rows = p.rows; b.before = p.base - p.first_key; b.keys_p = p.keys_p;
    b.q = p.q; b.k = p.k; b.key_rot = p.key_rot; b.vt = p.vt; b.sink = l.sink; b.gate = p.mixed + l.gate_at; b.ld_gate = l.ld_mix; b.act = p.act; b.ld_act = p.ld_act;
    return launch_block_attention(b, type, s);
}

}  // namespace esp
