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
// A prompt block runs in chunks of 64 tokens (chunk_recurrence.h) after one launch of its own: prepare rotates q and k, writes them and
// v in the layouts the products read (k and v transposed, k times the decay that is left at the end of its chunk).
#include <hip/hip_runtime.h>

#include "chunk_recurrence.h"
#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using chunked::C;
using matrix::Op;

constexpr int kStepRows = 32;   // rows of a transposed state per workgroup of a step

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
        chunked::store8<T>(static_cast<T *>(a.vt) + ((size_t)h * r.vdim_p + first) * a.R + t0 + part, x);
    } else {
        const size_t o = ((size_t)h * r.dim_p + first) * a.R + t0 + part;
        chunked::store8_split<T>(static_cast<T *>(a.kt_hi) + o, static_cast<T *>(a.kt_lo) + o, x);
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
    chunked::Block c{};
    c.heads = r.heads; c.key_share = 1; c.dim_p = r.dim_p; c.vdim_p = r.vdim_p; c.rows = a.rows; c.R = a.R; c.base = a.base;
    c.q = a.q; c.k = a.k; c.vt = c.state_v = a.vt; c.state_k = a.kt_hi; c.state_k_lo = a.kt_lo;
    c.state = r.state + (size_t)a.seq * r.heads * r.vdim_p * r.dim_p; c.states_hi = a.states_hi; c.states_lo = a.states_lo; c.o = a.o;
    chunked::launch_states_and_outputs<T>(c, chunked::FixedDecay{r.powers}, s);
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
