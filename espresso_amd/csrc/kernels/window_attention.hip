// Attention with grouped heads over a ring of cached keys and values, a sliding window, root-mean-square norms over the whole query and
// key projections, and rotation of the first dimensions of a head (gfx950).
//
//   mixed row   [q: heads | k: kv_heads | v: kv_heads], heads padded; a layer that reads another one's cache has q alone
//   cached row  [k: kv_heads x dim_p | v: kv_heads x vdim_p], one per token, at position % ring, keys normed and rotated
//
// A decode step is two launches.  partial: a workgroup takes a slice of the window for the query heads of one key head; it norms and
// rotates their queries itself (the norm's sum runs over the whole projection, which every workgroup reads), and the workgroup whose
// slice holds the row's own token puts its key and value into the cache first.  Eight lanes share a key, so a key is read once for all
// query heads of the group.  merge: the slices' (maximum, sum, weighted values) joined.
//
// A prompt block is three: prepare (queries, and keys and values into the ring), gather (the visible span, values transposed), and
// attention in tiles of 64 keys (block_attention.hip).
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::Op;

__host__ __device__ __forceinline__ int cached_row(const AttentionShape &l) { return l.kv_heads * (l.dim_p + l.vdim_p); }
__device__ __forceinline__ int first_seen(int pos, int window) { return pos - window + 1 > 0 ? pos - window + 1 : 0; }

// Element d of a head x, normed (scale inv, weights w) and rotated: pairs (i, i + dims / 2) of the first dims elements.
__device__ __forceinline__ float normed_rotated(const float *x, const float *w, float inv, int d, int dims, const float *cos, const float *sin) {
    if (d >= dims) return x[d] * inv * w[d];
    const int half = dims / 2, i = d < half ? d : d - half;
    const float c = cos[i], s = sin[i], u = x[i] * inv * w[i], v = x[i + half] * inv * w[i + half];
    return d < half ? u * c - v * s : v * c + u * s;
}

__device__ __forceinline__ float squares(const float *x, int count) {   // this thread's share; count is a multiple of four
    float s = 0.0f;
    for (int i = threadIdx.x * 4; i < count; i += 256 * 4) {
        const float4 v = *reinterpret_cast<const float4 *>(x + i);
        s += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
    }
    return s;
}

// Eight consecutive cached elements.
__device__ __forceinline__ void load8(const uint16_t *p, float (&f)[8]) { matrix::unpack_bf16(*reinterpret_cast<const uint4 *>(p), f); }
__device__ __forceinline__ void load8(const float *p, float (&f)[8]) {
    const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}

// The same eight as they are loaded, to be unpacked later.
template <typename T>
struct Piece;
template <>
struct Piece<uint16_t> {
    uint4 v;
    __device__ __forceinline__ void load(const uint16_t *p) { v = *reinterpret_cast<const uint4 *>(p); }
    __device__ __forceinline__ void unpack(float (&f)[8]) const { matrix::unpack_bf16(v, f); }
};
template <>
struct Piece<float> {
    float4 a, b;
    __device__ __forceinline__ void load(const float *p) { a = reinterpret_cast<const float4 *>(p)[0]; b = reinterpret_cast<const float4 *>(p)[1]; }
    __device__ __forceinline__ void unpack(float (&f)[8]) const { f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w; }
};

constexpr int kTile = 32;   // keys per pass of a workgroup: eight lanes each

constexpr int kKeyPieces = 4, kValuePieces = 2;   // pieces of eight per thread that are requested ahead; longer heads read the rest when needed

// grid (splits, key heads x chunks of Q query heads, rows).  LDS: queries [Q][dim_p], scores [Q][kTile], running (maximum, sum, rescale)
// [Q][4], the row's own key [dim_p] and value [vdim_p], and for the end the value sums [parts][vdim_p].  A tile's keys and values are
// requested a tile ahead, the first ones before the norms.
template <typename T, int Q>
__global__ __launch_bounds__(256) void attention_partial_kernel(AttentionShape l, AttentionStep p) {
    extern __shared__ float lds[];
    __shared__ float red[8];
    float *q = lds, *scores = q + Q * l.dim_p, *running = scores + Q * kTile, *own_key = running + Q * 4, *own_value = own_key + l.dim_p, *meet = own_value + l.vdim_p;
    const int tid = threadIdx.x, lane = tid & 63, split = blockIdx.x, m = blockIdx.z, pos = p.pos[m], seq = p.seq[m];
    const int share = l.heads / l.kv_heads, chunks = (share + Q - 1) / Q, kv = blockIdx.y / chunks, h0 = kv * share + blockIdx.y % chunks * Q;
    const int live = (kv + 1) * share - h0 < Q ? (kv + 1) * share - h0 : Q;
    const int lo = first_seen(pos, l.window), tiles = (pos - lo) / kTile + 1;
    if (split >= tiles) return;
    const float *row = p.mixed + (size_t)m * l.ld_mix;
    const float *cos = l.cos + (size_t)pos * (l.rot_dims / 2), *sin = l.sin + (size_t)pos * (l.rot_dims / 2);
    const int width = cached_row(l);
    T *cache = static_cast<T *>(l.cache) + (size_t)seq * l.ring * width;
    const bool owner = l.k_at >= 0 && split == (tiles - 1) % p.splits;   // the last tile holds the row's own token
    const int e = tid & 7, key_in = tid >> 3;
    const int pieces = l.vdim_p / 8, parts = 256 / pieces < kTile ? 256 / pieces : kTile, piece = tid % pieces, part = tid / pieces;   // value phase: eight values, every parts-th key
    const T *keys = cache + kv * l.dim_p, *values = cache + l.kv_heads * l.dim_p + kv * l.vdim_p + piece * 8;
    auto row_of = [&](int key) { return (size_t)((key < pos ? key : pos) % l.ring) * width; };   // keys past the query repeat it and weigh nothing
    Piece<T> key_ahead[kKeyPieces], value_ahead[kValuePieces];
    auto request = [&](int t) {
        const int k0 = lo + t * kTile;
        const T *from = keys + row_of(k0 + key_in);
#pragma unroll
        for (int i = 0; i < kKeyPieces; i++) key_ahead[i].load(from + (e * 8 + i * 64 < l.dim_p ? e * 8 + i * 64 : 0));
#pragma unroll
        for (int i = 0; i < kValuePieces; i++) value_ahead[i].load(values + row_of(k0 + (part + i * parts < kTile ? part + i * parts : 0)));
    };
    {
        float sq = squares(row, l.heads * l.dim_p), sk = owner ? squares(row + l.k_at, l.kv_heads * l.dim_p) : 0.0f;
        request(split);
        sq = detail::wave_sum(sq);
        sk = detail::wave_sum(sk);
        if (lane == 0) { red[tid >> 6] = sq; red[4 + (tid >> 6)] = sk; }
        __syncthreads();
        sq = (red[0] + red[1]) + (red[2] + red[3]);
        sk = (red[4] + red[5]) + (red[6] + red[7]);
        const float inv_q = 1.0f / sqrtf(sq / ((float)l.heads * (float)l.dim) + l.eps), inv_k = 1.0f / sqrtf(sk / ((float)l.kv_heads * (float)l.dim) + l.eps);
        for (int i = tid; i < Q * l.dim_p; i += 256) {
            const int r = i / l.dim_p, d = i - r * l.dim_p, at = (h0 + (r < live ? r : 0)) * l.dim_p;   // heads past the group repeat its first
            q[i] = l.scale * normed_rotated(row + at, l.q_norm + at, inv_q, d, l.rot_dims, cos, sin);
        }
        if (owner) {   // every chunk of the group's heads writes the same; here they are read from LDS
            T *own = cache + (size_t)(pos % l.ring) * width;
            for (int d = tid; d < l.dim_p; d += 256) {
                const int at = kv * l.dim_p;
                const T k = Op<T>::from_float(normed_rotated(row + l.k_at + at, l.k_norm + at, inv_k, d, l.rot_dims, cos, sin));
                own[at + d] = k;
                own_key[d] = Op<T>::to_float(k);
            }
            const float *v = row + l.k_at + l.kv_heads * l.dim_p + kv * l.vdim_p;
            for (int d = tid; d < l.vdim_p; d += 256) {
                const T x = Op<T>::from_float(v[d]);
                own[l.kv_heads * l.dim_p + kv * l.vdim_p + d] = x;
                own_value[d] = Op<T>::to_float(x);
            }
        }
        if (tid < Q) { running[tid * 4] = -INFINITY; running[tid * 4 + 1] = 0.0f; }
    }
    __syncthreads();
    float acc[Q][8];
#pragma unroll
    for (int r = 0; r < Q; r++)
#pragma unroll
        for (int i = 0; i < 8; i++) acc[r][i] = 0.0f;
    for (int t = split; t < tiles; t += p.splits) {
        const int k0 = lo + t * kTile;
        const bool in = k0 + key_in <= pos, mine = owner && k0 + key_in >= pos;
        float s[Q];
#pragma unroll
        for (int r = 0; r < Q; r++) s[r] = 0.0f;
        auto score = [&](float (&k)[8], int d) {
            if (mine) load8(own_key + d, k);
#pragma unroll
            for (int r = 0; r < Q; r++) {
                float x[8];
                load8(q + r * l.dim_p + d, x);
#pragma unroll
                for (int i = 0; i < 8; i++) s[r] = __builtin_fmaf(k[i], x[i], s[r]);
            }
        };
#pragma unroll
        for (int i = 0; i < kKeyPieces; i++) {
            float k[8];
            key_ahead[i].unpack(k);
            if (e * 8 + i * 64 < l.dim_p) score(k, e * 8 + i * 64);
        }
        for (int d = e * 8 + kKeyPieces * 64; d < l.dim_p; d += 64) {
            float k[8];
            load8(keys + row_of(k0 + key_in) + d, k);
            score(k, d);
        }
#pragma unroll
        for (int r = 0; r < Q; r++) {   // the eight lanes of a key
            s[r] += detail::dpp_term<0xB1, 0xF>(s[r]);
            s[r] += detail::dpp_term<0x4E, 0xF>(s[r]);
            s[r] += detail::dpp_term<0x141, 0xF>(s[r]);
            if (e == 0) scores[r * kTile + key_in] = in ? s[r] : -INFINITY;
        }
        __syncthreads();
        for (int r = tid / kTile; r < Q; r += 256 / kTile) {   // 32 lanes per head
            const float x = scores[r * kTile + (tid & 31)], was = running[r * 4];
            float top = fmaxf(x, was);
#pragma unroll
            for (int d = 16; d >= 1; d >>= 1) top = fmaxf(top, __shfl_xor(top, d));
            const float w = matrix::weight_exp<T>(x - top), keep = matrix::weight_exp<T>(was - top);
            float sum = w;
#pragma unroll
            for (int d = 16; d >= 1; d >>= 1) sum += __shfl_xor(sum, d);
            scores[r * kTile + (tid & 31)] = w;
            if ((tid & 31) == 0) { running[r * 4] = top; running[r * 4 + 1] = running[r * 4 + 1] * keep + sum; running[r * 4 + 2] = keep; }
        }
        __syncthreads();
        if (part < parts) {
#pragma unroll
            for (int r = 0; r < Q; r++) {
                const float keep = running[r * 4 + 2];
#pragma unroll
                for (int i = 0; i < 8; i++) acc[r][i] *= keep;
            }
            auto add = [&](float (&v)[8], int k) {
                if (owner && k0 + k >= pos) load8(own_value + piece * 8, v);
#pragma unroll
                for (int r = 0; r < Q; r++) {
                    const float w = scores[r * kTile + k];
#pragma unroll
                    for (int i = 0; i < 8; i++) acc[r][i] = __builtin_fmaf(w, v[i], acc[r][i]);
                }
            };
#pragma unroll
            for (int i = 0; i < kValuePieces; i++) {
                float v[8];
                value_ahead[i].unpack(v);
                if (part + i * parts < kTile) add(v, part + i * parts);
            }
            for (int k = part + kValuePieces * parts; k < kTile; k += parts) {
                float v[8];
                load8(values + row_of(k0 + k), v);
                add(v, k);
            }
        }
        if (t + p.splits < tiles) request(t + p.splits);
        __syncthreads();
    }
    const size_t first = ((size_t)m * p.splits + split) * l.heads + h0;
#pragma unroll
    for (int r = 0; r < Q; r++) {
        if (r >= live) break;
        if (part < parts) {
            reinterpret_cast<float4 *>(meet + part * l.vdim_p + piece * 8)[0] = make_float4(acc[r][0], acc[r][1], acc[r][2], acc[r][3]);
            reinterpret_cast<float4 *>(meet + part * l.vdim_p + piece * 8)[1] = make_float4(acc[r][4], acc[r][5], acc[r][6], acc[r][7]);
        }
        __syncthreads();
        for (int v = tid; v < l.vdim_p; v += 256) {
            float s = 0.0f;
            for (int i = 0; i < parts; i++) s += meet[i * l.vdim_p + v];
            p.partial[(first + r) * l.vdim_p + v] = s;
        }
        if (tid == 0) *reinterpret_cast<float2 *>(p.partial_ml + (first + r) * 2) = make_float2(running[r * 4], running[r * 4 + 1]);
        __syncthreads();
    }
}

// grid (heads, rows).  splits <= 64: a lane of the first wavefront each.
template <typename T>
__global__ __launch_bounds__(256) void attention_merge_kernel(AttentionShape l, AttentionStep p) {
    __shared__ float weight[64];
    const int tid = threadIdx.x, h = blockIdx.x, m = blockIdx.y, pos = p.pos[m];
    const int tiles = (pos - first_seen(pos, l.window)) / kTile + 1, live = tiles < p.splits ? tiles : p.splits;
    const size_t first = (size_t)m * p.splits * l.heads + h;   // slice s: first + s * heads
    if (tid < 64) {
        const float2 ml = *reinterpret_cast<const float2 *>(p.partial_ml + (first + (size_t)(tid < live ? tid : 0) * l.heads) * 2);
        float top = ml.x;
#pragma unroll
        for (int x = 32; x >= 1; x >>= 1) top = fmaxf(top, __shfl_xor(top, x));
        const float w = tid < live ? expf(ml.x - top) : 0.0f;
        weight[tid] = w / detail::wave_sum(w * ml.y);
    }
    __syncthreads();
    for (int v = tid; v < l.vdim_p; v += 256) {
        float o = 0.0f;
        for (int s0 = 0; s0 < live; s0 += 8) {   // eight slices in flight
            float x[8];
#pragma unroll
            for (int u = 0; u < 8; u++) x[u] = p.partial[(first + (size_t)(s0 + u < live ? s0 + u : 0) * l.heads) * l.vdim_p + v];
#pragma unroll
            for (int u = 0; u < 8; u++) o += s0 + u < live ? weight[s0 + u] * x[u] : 0.0f;
        }
        if (p.mix) p.mix[(size_t)m * l.heads * l.vdim_p + h * l.vdim_p + v] = o;
        else static_cast<T *>(p.act)[(size_t)m * p.ld_act + h * l.vdim_p + v] = Op<T>::from_float(o);
    }
}

// ---- prompt blocks ---------------------------------------------------------------------------------------
// One workgroup per row: queries normed and rotated to [heads][rows_p][dim_p] (rows past the block are zero), keys and values to the ring.
template <typename T>
__global__ __launch_bounds__(256) void attention_prepare_kernel(AttentionShape l, AttentionBlock p, int rows_p) {
    __shared__ float red[8];
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63;
    T *out = static_cast<T *>(p.q) + (size_t)m * l.dim_p;
    if (m >= p.rows) {
        for (int i = tid; i < l.heads * l.dim_p; i += 256) out[(size_t)(i / l.dim_p) * rows_p * l.dim_p + i % l.dim_p] = Op<T>::from_float(0.0f);
        return;
    }
    const int pos = p.base + m, kv = l.kv_heads * l.dim_p;
    const float *row = p.mixed + (size_t)m * l.ld_mix;
    const float *cos = l.cos + (size_t)pos * (l.rot_dims / 2), *sin = l.sin + (size_t)pos * (l.rot_dims / 2);
    float sq = detail::wave_sum(squares(row, l.heads * l.dim_p)), sk = l.k_at >= 0 ? detail::wave_sum(squares(row + l.k_at, kv)) : 0.0f;
    if (lane == 0) { red[tid >> 6] = sq; red[4 + (tid >> 6)] = sk; }
    __syncthreads();
    sq = (red[0] + red[1]) + (red[2] + red[3]);
    sk = (red[4] + red[5]) + (red[6] + red[7]);
    const float inv_q = 1.0f / sqrtf(sq / ((float)l.heads * (float)l.dim) + l.eps), inv_k = 1.0f / sqrtf(sk / ((float)l.kv_heads * (float)l.dim) + l.eps);
    for (int i = tid; i < l.heads * l.dim_p; i += 256) {
        const int h = i / l.dim_p, d = i - h * l.dim_p, at = h * l.dim_p;
        out[(size_t)h * rows_p * l.dim_p + d] = Op<T>::from_float(normed_rotated(row + at, l.q_norm + at, inv_q, d, l.rot_dims, cos, sin));
    }
    if (l.k_at < 0) return;
    T *own = static_cast<T *>(l.cache) + ((size_t)p.seq * l.ring + pos % l.ring) * cached_row(l);
    for (int i = tid; i < kv; i += 256) {
        const int at = i / l.dim_p * l.dim_p;
        own[i] = Op<T>::from_float(normed_rotated(row + l.k_at + at, l.k_norm + at, inv_k, i - at, l.rot_dims, cos, sin));
    }
    for (int i = tid; i < l.kv_heads * l.vdim_p; i += 256) own[kv + i] = Op<T>::from_float(row[l.k_at + kv + i]);
}

// The keys a block sees as rows, their values transposed; grid (tiles of 64 keys, slabs of 32 elements: keys, then values).
template <typename T>
__global__ __launch_bounds__(256) void attention_gather_kernel(AttentionShape l, AttentionBlock p) {
    __shared__ T slab[32][64 + 8];
    const int tid = threadIdx.x, i0 = blockIdx.x * 64, c0 = blockIdx.y * 32, kv = l.kv_heads * l.dim_p, width = cached_row(l);
    const T *cache = static_cast<const T *>(l.cache) + (size_t)p.seq * l.ring * width;
    const bool values = c0 >= kv;
#pragma unroll
    for (int k = 0; k < 8; k++) {
        const int i = (tid >> 5) + 8 * k, c = tid & 31;
        const T x = i0 + i < p.keys ? cache[(size_t)((p.first_key + i0 + i) % l.ring) * width + c0 + c] : (T)0;
        if (values) slab[c][i] = x;
        else static_cast<T *>(p.k)[(size_t)(i0 + i) * kv + c0 + c] = x;
    }
    if (!values) return;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 8; k++) {
        const int c = (tid >> 6) + 4 * k, i = tid & 63;
        static_cast<T *>(p.vt)[(size_t)(c0 - kv + c) * p.keys_p + i0 + i] = slab[c][i];
    }
}

bool shape_ok(const AttentionShape &l) {
    return l.heads > 0 && l.kv_heads > 0 && l.heads % l.kv_heads == 0 && l.dim_p % 32 == 0 && l.vdim_p % 32 == 0 && l.dim > 0 && l.vdim > 0 && l.dim <= l.dim_p && l.vdim <= l.vdim_p &&
           l.rot_dims >= 0 && l.rot_dims <= l.dim && l.rot_dims % 2 == 0 && l.window >= 1 && l.ring >= 1 && l.cache && l.vdim_p <= kAttentionMaxHead && l.dim_p <= kAttentionMaxHead &&
           (l.k_at < 0 || (l.k_at >= l.heads * l.dim_p && l.k_norm && l.k_at + cached_row(l) <= l.ld_mix)) && l.q_norm && l.heads * l.dim_p <= l.ld_mix;
}

int heads_together(const AttentionShape &l) {
    const int share = l.heads / l.kv_heads;
    return share <= 1 ? 1 : share <= 2 ? 2 : share <= 4 ? 4 : 8;
}

template <typename T, int Q>
hipError_t run_partial(const AttentionShape &l, const AttentionStep &p, hipStream_t s) {
    const int chunks = (l.heads / l.kv_heads + Q - 1) / Q, parts = 256 / (l.vdim_p / 8) < kTile ? 256 / (l.vdim_p / 8) : kTile;
    const size_t lds = (size_t)(Q * (l.dim_p + kTile + 4) + l.dim_p + l.vdim_p + parts * l.vdim_p) * 4;
    if (lds > 62 * 1024) return hipErrorInvalidValue;
    hipLaunchKernelGGL((attention_partial_kernel<T, Q>), dim3(p.splits, l.kv_heads * chunks, p.rows), dim3(256), lds, s, l, p);
    return hipGetLastError();
}

template <typename T>
hipError_t run_step(const AttentionShape &l, const AttentionStep &p, hipStream_t s) {
    hipError_t e;
    switch (heads_together(l)) {
        case 1: e = run_partial<T, 1>(l, p, s); break;
        case 2: e = run_partial<T, 2>(l, p, s); break;
        case 4: e = run_partial<T, 4>(l, p, s); break;
        default: e = run_partial<T, 8>(l, p, s); break;
    }
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL((attention_merge_kernel<T>), dim3(l.heads, p.rows), dim3(256), 0, s, l, p);
    return hipGetLastError();
}

template <typename T>
hipError_t run_block(const AttentionShape &l, const AttentionBlock &p, hipStream_t s) {
    const int rows_p = (p.rows + 31) / 32 * 32;
    hipLaunchKernelGGL((attention_prepare_kernel<T>), dim3(rows_p), dim3(256), 0, s, l, p, rows_p);
    hipLaunchKernelGGL((attention_gather_kernel<T>), dim3(p.keys_p / 64, cached_row(l) / 32), dim3(256), 0, s, l, p);
    return hipGetLastError();
}

}  // namespace

int attention_step_splits(const AttentionShape &l) {
    const int span = l.window < l.max_seq ? l.window : l.max_seq, tiles = (span + kTile - 1) / kTile;
    const int groups = l.kv_heads * ((l.heads / l.kv_heads + heads_together(l) - 1) / heads_together(l)), wanted = (512 + groups - 1) / groups, most = wanted < 64 ? wanted : 64;
    return tiles < most ? tiles : most;
}

hipError_t launch_attention_step(const AttentionShape &l, const AttentionStep &p, Precision type, hipStream_t s) {
    if (!shape_ok(l) || p.rows < 1 || p.splits < 1 || p.splits > 64 || (!p.mix && !p.act)) return hipErrorInvalidValue;
    return type == Precision::bf16 ? run_step<uint16_t>(l, p, s) : run_step<float>(l, p, s);
}

hipError_t launch_attention_block(const AttentionShape &l, const AttentionBlock &p, Precision type, hipStream_t s) {
    if (!shape_ok(l) || p.rows < 1 || p.base < 0 || p.base + p.rows > l.max_seq || p.first_key < 0 || p.first_key > p.base || p.keys != p.base + p.rows - p.first_key || p.keys > l.ring ||
        p.keys_p % 64 || p.keys_p < p.keys)
        return hipErrorInvalidValue;
    const hipError_t e = type == Precision::bf16 ? run_block<uint16_t>(l, p, s) : run_block<float>(l, p, s);
    if (e != hipSuccess) return e;
    BlockAttention b;
    b.heads = l.heads; b.kv_heads = l.kv_heads; b.dim_p = l.dim_p; b.vdim_p = l.vdim_p; b.window = l.window; b.scale = l.scale;
    b.rows = p.rows; b.before = p.base - p.first_key; b.keys_p = p.keys_p; b.q = p.q; b.k = p.k; b.vt = p.vt; b.act = p.act; b.ld_act = p.ld_act;
    return launch_block_attention(b, type, s);
}

}  // namespace esp
