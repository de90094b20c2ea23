// Retention (linear attention with a fixed decay per head, no softmax, no denominator) on gfx950.
//
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   then o_t over its root mean square per head, times SiLU(gate)
//
// States are fp32 and kept transposed, [vdim][dim] per head, so that a row of them meets q and k lane by lane.
//
// A decode step (retention_step_kernel) reads and writes every state once: eight lanes share a row of a state, a wavefront takes
// eight rows; q and k are rotated by every workgroup of the head.  The norm of the output needs the whole head, so a workgroup
// leaves the sum of squares of its part and the output product's staging finishes it.
//
// A prompt block runs in chunks of 64 tokens, three launches:
//   prepare   rotates q and k, writes them and v in the layouts the products read (k and v transposed, k times the decay that is
//             left at the end of its chunk);
//   states    one wavefront per 32 x 32 tile of a head's state walks the chunks: it stores the state before the chunk, then
//             S = decay^64 S + V^T K' on the matrix cores;
//   outputs   o = decay^(t + 1) S^T q + sum over the chunk's keys s <= t of decay^(t - s) (q . k_s) v_s; scores are computed transposed,
//             so that their accumulator is the operand of the second product and no score passes through LDS.
// With bf16 operands, what belongs to the recurrence (states, decayed keys, scores) enters the products as a high and a low bf16.
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::floatx16;
using matrix::Op;

constexpr int kStepRows = 32;   // rows of a transposed state per workgroup of a step
constexpr int C = kRetentionChunk;

// Element i of a head's q or k at `position`, rotated: pairs (i, i + dims / 2) of the first dims elements.
__device__ __forceinline__ float rotated_half(const float *x, int i, int dims, const float *cos, const float *sin) {
    const int half = dims / 2;
    if (i >= dims) return x[i];
    const int p = i < half ? i : i - half;
    const float c = cos[p], s = sin[p], u = x[p], v = x[p + half];
    return i < half ? u * c - v * s : v * c + u * s;
}

__global__ __launch_bounds__(256) void retention_step_kernel(RetentionShape r, RetentionStep p) {
    extern __shared__ float lds[];   // q [dim_p], k [dim_p]
    __shared__ float red[4];
    const int part = blockIdx.x, h = blockIdx.y, m = blockIdx.z, tid = threadIdx.x;
    const int pos = p.pos[m], seq = p.seq[m];
    const bool again = p.halt && *p.halt, fresh = pos == 0 && !again;
    const int e = tid & 7, v = part * kStepRows + (tid >> 3);
    float *state = r.state + (((size_t)seq * r.heads + h) * r.vdim_p + v) * r.dim_p + e * 4;
    // up to eight pieces of the row are on their way while q and k are rotated
    constexpr int kHeld = 8;
    float4 held[kHeld];
#pragma unroll
    for (int i = 0; i < kHeld; i++) held[i] = *reinterpret_cast<const float4 *>(state + (i * 32 < r.dim_p ? i * 32 : 0));
    const float *row = p.mixed + (size_t)m * r.ld_mix;
    const float *cos = r.cos + (size_t)pos * (r.rot_dims / 2), *sin = r.sin + (size_t)pos * (r.rot_dims / 2);
    const float k_scale = 1.0f / sqrtf((float)r.dim);
    for (int i = tid; i < r.dim_p; i += 256) {
        lds[i] = rotated_half(row + h * r.dim_p, i, r.rot_dims, cos, sin);
        lds[r.dim_p + i] = rotated_half(row + (r.heads + h) * r.dim_p, i, r.rot_dims, cos, sin) * k_scale;
    }
    const float value = row[2 * r.heads * r.dim_p + h * r.vdim_p + v], decay = r.decay[h];
    __syncthreads();
    float o = 0.0f;
    auto piece = [&](int d0, float4 s) {
        if (fresh) s = make_float4(0.f, 0.f, 0.f, 0.f);
        const float4 q = *reinterpret_cast<const float4 *>(lds + d0 + e * 4), k = *reinterpret_cast<const float4 *>(lds + r.dim_p + d0 + e * 4);
        if (!again) {
            s.x = decay * s.x + k.x * value; s.y = decay * s.y + k.y * value; s.z = decay * s.z + k.z * value; s.w = decay * s.w + k.w * value;
            *reinterpret_cast<float4 *>(state + d0) = s;
        }
        o += s.x * q.x + s.y * q.y + s.z * q.z + s.w * q.w;
    };
#pragma unroll
    for (int i = 0; i < kHeld; i++)
        if (i * 32 < r.dim_p) piece(i * 32, held[i]);
    for (int d0 = kHeld * 32; d0 < r.dim_p; d0 += 32) piece(d0, *reinterpret_cast<const float4 *>(state + d0));
    o += detail::dpp_term<0xB1, 0xF>(o);    // the eight lanes of a row
    o += detail::dpp_term<0x4E, 0xF>(o);
    o += detail::dpp_term<0x141, 0xF>(o);
    if (e == 0) p.o[(size_t)m * r.heads * r.vdim_p + h * r.vdim_p + v] = o;
    const float total = detail::workgroup_sum(e == 0 ? o * o : 0.0f, red);
    if (tid == 0) p.squares[((size_t)m * r.heads + h) * gridDim.x + part] = total;
}

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

struct BlockArgs {
    RetentionShape r;
    const float *mixed;
    int rows, R, base, seq;
    void *q, *k, *kt_hi, *kt_lo, *vt, *states_hi, *states_lo;
    float *o;
};

// grid (chunks, heads, slabs of 32 columns: first those of q and k, then those of v).  What is needed transposed goes through LDS.
template <typename T>
__global__ __launch_bounds__(256) void retention_prepare_kernel(BlockArgs a) {
    __shared__ float slab[32][C + 1];
    const RetentionShape &r = a.r;
    const int chunk = blockIdx.x, h = blockIdx.y, t0 = chunk * C, tid = threadIdx.x, slabs = r.dim_p / 32;
    const int len = a.rows - t0 < C ? a.rows - t0 : C, c = tid & 31;
    const bool values = (int)blockIdx.z >= slabs;
    const int d = (values ? (int)blockIdx.z - slabs : (int)blockIdx.z) * 32 + c;
    if (values) {
        const float *v = a.mixed + 2 * r.heads * r.dim_p + h * r.vdim_p + d;
#pragma unroll
        for (int i = 0; i < C / 8; i++) {
            const int t = (tid >> 5) + 8 * i;
            slab[c][t] = t < len ? v[(size_t)(t0 + t) * r.ld_mix] : 0.0f;
        }
    } else {
        const float k_scale = 1.0f / sqrtf((float)r.dim);
        const float *powers = r.powers + h * (C + 1);
#pragma unroll
        for (int i = 0; i < C / 8; i++) {
            const int t = (tid >> 5) + 8 * i;
            float q = 0.0f, k = 0.0f;
            if (t < len) {
                const float *row = a.mixed + (size_t)(t0 + t) * r.ld_mix;
                const size_t at = (size_t)(a.base + t0 + t) * (r.rot_dims / 2);
                q = rotated_half(row + h * r.dim_p, d, r.rot_dims, r.cos + at, r.sin + at);
                k = rotated_half(row + (r.heads + h) * r.dim_p, d, r.rot_dims, r.cos + at, r.sin + at) * k_scale;
            }
            const size_t o = ((size_t)h * a.R + t0 + t) * r.dim_p + d;
            static_cast<T *>(a.q)[o] = Op<T>::from_float(q);
            static_cast<T *>(a.k)[o] = Op<T>::from_float(k);
            slab[c][t] = t < len ? k * powers[len - 1 - t] : 0.0f;
        }
    }
    __syncthreads();
    // eight tokens of one column per thread
    const int col = tid >> 3, part = (tid & 7) * 8;
    const int first = (values ? (int)blockIdx.z - slabs : (int)blockIdx.z) * 32 + col;
    float x[8];
#pragma unroll
    for (int i = 0; i < 8; i++) x[i] = slab[col][part + i];
    if (values) {
        store8<T>(static_cast<T *>(a.vt) + ((size_t)h * r.vdim_p + first) * a.R + t0 + part, x);
    } else {
        const size_t o = ((size_t)h * r.dim_p + first) * a.R + t0 + part;
        store8<T>(static_cast<T *>(a.kt_hi) + o, x);
        if constexpr (Op<T>::kSplit) {
#pragma unroll
            for (int i = 0; i < 8; i++) x[i] -= Op<T>::to_float(Op<T>::from_float(x[i]));
            store8<T>(static_cast<T *>(a.kt_lo) + o, x);
        }
    }
}

// One wavefront per tile of 32 v x 32 d of one head's state; workgroups of four tiles along d.
template <typename T>
__global__ __launch_bounds__(256) void retention_states_kernel(BlockArgs a) {
    const RetentionShape &r = a.r;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5;
    const int h = blockIdx.z, v0 = blockIdx.y * 32, d0 = (blockIdx.x * 4 + wave) * 32;
    if (d0 >= r.dim_p) return;
    const size_t tile = (size_t)v0 * r.dim_p + d0 + (lane & 31), head = (size_t)r.vdim_p * r.dim_p;
    float *state = r.state + ((size_t)a.seq * r.heads + h) * head;
    floatx16 acc = matrix::zero_accumulator();
    if (a.base > 0) {
#pragma unroll
        for (int i = 0; i < 16; i++) acc[i] = state[tile + (size_t)matrix::accumulator_row(i, half) * r.dim_p];
    }
    const T *vt = static_cast<const T *>(a.vt) + ((size_t)h * r.vdim_p + v0 + (lane & 31)) * a.R + 8 * half;
    const T *kh = static_cast<const T *>(a.kt_hi) + ((size_t)h * r.dim_p + d0 + (lane & 31)) * a.R + 8 * half;
    const T *kl = static_cast<const T *>(a.kt_lo) + ((size_t)h * r.dim_p + d0 + (lane & 31)) * a.R + 8 * half;
    const int chunks = a.R / C;
    for (int c = 0; c < chunks; c++) {
        const int len = a.rows - c * C < C ? a.rows - c * C : C;
        T *hi = static_cast<T *>(a.states_hi) + ((size_t)c * r.heads + h) * head, *lo = static_cast<T *>(a.states_lo) + ((size_t)c * r.heads + h) * head;
        const float factor = r.powers[h * (C + 1) + len];
        typename Op<T>::frag v[C / 16], w[C / 16], x[C / 16];   // on their way while the state before the chunk is stored
#pragma unroll
        for (int ks = 0; ks < C / 16; ks++) {
            v[ks] = Op<T>::load(vt + c * C + ks * 16);
            w[ks] = Op<T>::load(kh + c * C + ks * 16);
            if constexpr (Op<T>::kSplit) x[ks] = Op<T>::load(kl + c * C + ks * 16);
        }
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const size_t o = tile + (size_t)matrix::accumulator_row(i, half) * r.dim_p;
            const T b = Op<T>::from_float(acc[i]);
            hi[o] = b;
            if constexpr (Op<T>::kSplit) lo[o] = Op<T>::from_float(acc[i] - Op<T>::to_float(b));
            acc[i] *= factor;
        }
#pragma unroll
        for (int ks = 0; ks < C / 16; ks++) {
            acc = Op<T>::mma(v[ks], w[ks], acc);
            if constexpr (Op<T>::kSplit) acc = Op<T>::mma(v[ks], x[ks], acc);
        }
    }
#pragma unroll
    for (int i = 0; i < 16; i++) state[tile + (size_t)matrix::accumulator_row(i, half) * r.dim_p] = acc[i];
}

// grid (chunks, heads, slices of 128 v): wavefront w takes queries 32 (w % 2) .. of the chunk and 64 v from 64 (w / 2) of the slice.
template <typename T>
__global__ __launch_bounds__(256) void retention_outputs_kernel(BlockArgs a) {
    const RetentionShape &r = a.r;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5;
    const int c = blockIdx.x, h = blockIdx.y, qt = wave & 1, v0 = blockIdx.z * 128 + (wave >> 1) * 64;
    if (v0 >= r.vdim_p || c * C + qt * 32 >= a.rows) return;
    const bool two = v0 + 32 < r.vdim_p;   // a second tile of 32 v
    const int t_local = qt * 32 + (lane & 31);   // this lane's query, in the chunk
    const T *q = static_cast<const T *>(a.q) + ((size_t)h * a.R + c * C + t_local) * r.dim_p + 8 * half;
    const T *k = static_cast<const T *>(a.k) + ((size_t)h * a.R + c * C + (lane & 31)) * r.dim_p + 8 * half;
    const size_t head = (size_t)r.vdim_p * r.dim_p, s_at = ((size_t)c * r.heads + h) * head + (size_t)(v0 + (lane & 31)) * r.dim_p + 8 * half;
    const T *shi = static_cast<const T *>(a.states_hi) + s_at, *slo = static_cast<const T *>(a.states_lo) + s_at;
    const size_t next = two ? (size_t)32 * r.dim_p : 0;
    floatx16 score[2], out[2];
#pragma unroll
    for (int i = 0; i < 2; i++) score[i] = out[i] = matrix::zero_accumulator();
    constexpr int kAhead = Op<T>::kSplit ? 2 : 1;   // steps of 16 dimensions whose loads are in flight together (dim_p is a multiple of 32)
    const size_t k_next = qt ? (size_t)32 * r.dim_p : 0;
    for (int d0 = 0; d0 < r.dim_p; d0 += 16 * kAhead) {
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
    const float *powers = r.powers + h * (C + 1);
    const float reach = powers[t_local + 1];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 16; j++) out[i][j] *= reach;
    const T *vt = static_cast<const T *>(a.vt) + ((size_t)h * r.vdim_p + v0 + (lane & 31)) * a.R + c * C + 4 * half;
    const size_t next_v = two ? (size_t)32 * a.R : 0;
    for (int kt = 0; kt <= qt; kt++) {
#pragma unroll
        for (int st = 0; st < 2; st++) {
            float w[8];
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const int s_local = kt * 32 + matrix::accumulator_row(st * 8 + j, half), gap = t_local - s_local;
                const float x = kt ? score[1][st * 8 + j] : score[0][st * 8 + j];
                w[j] = gap >= 0 ? x * powers[gap] : 0.0f;
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
    float *o = a.o + (size_t)t * r.heads * r.vdim_p + h * r.vdim_p + v0;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        if (i && !two) break;
#pragma unroll
        for (int g = 0; g < 4; g++)
            *reinterpret_cast<float4 *>(o + i * 32 + g * 8 + 4 * half) = make_float4(out[i][4 * g], out[i][4 * g + 1], out[i][4 * g + 2], out[i][4 * g + 3]);
    }
}

// One wavefront per (row, head).
template <typename T>
__global__ __launch_bounds__(256) void retention_gate_kernel(RetentionShape r, const float *o, const float *mixed, int rows, float eps, void *act, int ld_act) {
    const int lane = threadIdx.x & 63, at = blockIdx.x * 4 + (threadIdx.x >> 6), m = at / r.heads, h = at % r.heads;
    if (m >= rows) return;
    const float *x = o + (size_t)m * r.heads * r.vdim_p + h * r.vdim_p;
    const float *g = mixed + (size_t)m * r.ld_mix + 2 * r.heads * r.dim_p + r.heads * r.vdim_p + h * r.vdim_p;
    float s = 0.0f;
    for (int i = lane; i < r.vdim_p; i += 64) s += x[i] * x[i];
    const float inv = 1.0f / sqrtf(detail::wave_sum(s) / (float)r.vdim + eps);
    T *dst = static_cast<T *>(act) + (size_t)m * ld_act + h * r.vdim_p;
    for (int i = lane; i < r.vdim_p; i += 64) dst[i] = Op<T>::from_float(x[i] * inv * matrix::silu(g[i]));
}

bool shape_ok(const RetentionShape &r) {
    return r.heads > 0 && r.dim > 0 && r.vdim > 0 && r.dim_p % 32 == 0 && r.vdim_p % 32 == 0 && r.dim <= r.dim_p && r.vdim <= r.vdim_p && r.rot_dims <= r.dim && r.rot_dims % 2 == 0 &&
           r.ld_mix >= 2 * r.heads * (r.dim_p + r.vdim_p) && r.dim_p <= 4096 && r.state;
}

template <typename T>
hipError_t run_block(const BlockArgs &a, hipStream_t s) {
    const RetentionShape &r = a.r;
    const int chunks = a.R / C;
    hipLaunchKernelGGL((retention_prepare_kernel<T>), dim3(chunks, r.heads, (r.dim_p + r.vdim_p) / 32), dim3(256), 0, s, a);
    hipLaunchKernelGGL((retention_states_kernel<T>), dim3((r.dim_p + 127) / 128, r.vdim_p / 32, r.heads), dim3(256), 0, s, a);
    hipLaunchKernelGGL((retention_outputs_kernel<T>), dim3(chunks, r.heads, (r.vdim_p + 127) / 128), dim3(256), 0, s, a);
    return hipGetLastError();
}

}  // namespace

int retention_step_parts(int vdim_p) { return vdim_p / kStepRows; }

hipError_t launch_retention_step(const RetentionShape &r, const RetentionStep &p, hipStream_t s) {
    if (!shape_ok(r) || p.rows < 1) return hipErrorInvalidValue;
    hipLaunchKernelGGL(retention_step_kernel, dim3(retention_step_parts(r.vdim_p), r.heads, p.rows), dim3(256), (size_t)r.dim_p * 8, s, r, p);
    return hipGetLastError();
}

hipError_t launch_retention_block(const RetentionShape &r, const RetentionBlock &p, Precision type, hipStream_t s) {
    if (!shape_ok(r) || p.rows < 1 || p.base < 0 || p.base + p.rows > r.max_seq) return hipErrorInvalidValue;
    BlockArgs a{r, p.mixed, p.rows, (p.rows + C - 1) / C * C, p.base, p.seq, p.q, p.k, p.kt_hi, p.kt_lo, p.vt, p.states_hi, p.states_lo, p.o};
    return type == Precision::bf16 ? run_block<uint16_t>(a, s) : run_block<float>(a, s);
}

hipError_t launch_retention_gate(const RetentionShape &r, const float *o, const float *mixed, int rows, float eps, void *act, int ld_act, Precision type, hipStream_t s) {
    if (!shape_ok(r) || rows < 1 || ld_act < r.heads * r.vdim_p) return hipErrorInvalidValue;
    const dim3 grid((rows * r.heads + 3) / 4);
    if (type == Precision::bf16) hipLaunchKernelGGL((retention_gate_kernel<uint16_t>), grid, dim3(256), 0, s, r, o, mixed, rows, eps, act, ld_act);
    else hipLaunchKernelGGL((retention_gate_kernel<float>), grid, dim3(256), 0, s, r, o, mixed, rows, eps, act, ld_act);
    return hipGetLastError();
}

}  // namespace esp
