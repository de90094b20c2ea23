// Mamba-2 mixers (state-space duality) on gfx950.  Per head, with the B and C of the head's group:
//
//   x, B, C  pass a causal convolution per channel and SiLU;   dt <- softplus(dt + bias)
//   S_t = exp(-rate dt) S_(t-1) + dt B x^T,   y = (S_t^T C + skip x) SiLU(z)
//
// and y over the root mean square of its part of all heads' values, times a weight, is what the output product reads.
//
// Mixed rows and the values are laid out by padded heads, z | x | B | C | dt; zeros fill up heads and groups, and padded channels have
// no weights and no bias, so they stay zero.  What a sequence keeps: fp32 states, transposed ([vdim][state] per head), and a ring of its
// last inputs of the convolution, position p at row p % taps, so that a step that is run again writes what is there already.
//
// A decode step (mamba2_step_kernel) reads and writes every state once: eight lanes share a row of a state, a wavefront takes eight rows;
// the convolution of the group's B and C is done by every workgroup that needs it.
//
// A prompt block runs in chunks (chunk_recurrence.h) after one launch of its own: prepare convolves, sums the logarithms of the decays
// (double, kept as two floats), and writes B, C and x in the layouts the products read, x also times dt and the decay that is left at
// the end of its chunk.
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

__host__ __device__ __forceinline__ int values_of(const Mamba2Shape &r) { return r.heads * r.vdim_p; }
__host__ __device__ __forceinline__ int channels_of(const Mamba2Shape &r) { return values_of(r) + 2 * r.groups * r.state_p; }
__device__ __forceinline__ float softplus(float v) { return v > 20.0f ? v : log1pf(expf(v)); }

// TAPS: taps of the convolution, 0 = any number.  Every load that needs no other is requested before the first is used.
template <int TAPS>
__global__ __launch_bounds__(256) void mamba2_step_kernel(Mamba2Shape r, Mamba2Step p) {
    extern __shared__ float lds[];   // B [state_p], C [state_p]
    const int part = blockIdx.x, h = blockIdx.y, m = blockIdx.z, tid = threadIdx.x;
    const int pos = p.pos[m], seq = p.seq[m];
    const int e = tid & 7, v = part * kStepRows + (tid >> 3), values = values_of(r), channels = channels_of(r);
    const float *row = p.mixed + (size_t)m * r.ld_mix, *inputs = row + values;
    float *past = r.inputs + (size_t)seq * r.taps * channels;
    constexpr int kTaps = TAPS ? TAPS : 1;
    struct Window {   // what one channel's convolution reads
        float in[kTaps], w[kTaps], bias;
    };
    auto request = [&](int channel) {
        Window g;
        g.bias = r.conv_bias[channel];
        g.in[0] = inputs[channel];
        g.w[0] = r.conv[(size_t)(r.taps - 1) * channels + channel];
#pragma unroll
        for (int j = 1; j < kTaps; j++) {
            const int at = pos - j;
            g.w[j] = r.conv[(size_t)(kTaps - 1 - j) * channels + channel];
            g.in[j] = past[(size_t)(at > 0 ? at % kTaps : 0) * channels + channel];
        }
        return g;
    };
    auto convolved = [&](const Window &g, int channel) {
        float s = g.bias + g.w[0] * g.in[0];
#pragma unroll
        for (int j = 1; j < kTaps; j++) s += pos >= j ? g.w[j] * g.in[j] : 0.0f;
        if constexpr (TAPS == 0) {
            const int reach = pos < r.taps - 1 ? pos : r.taps - 1;
            for (int j = 1; j <= reach; j++) s += r.conv[(size_t)(r.taps - 1 - j) * channels + channel] * past[(size_t)((pos - j) % r.taps) * channels + channel];
        }
        return matrix::silu(s);
    };
    const int share = r.heads / r.groups, group = h / share;
    auto shared_channel = [&](int i) { return values + (i < r.state_p ? group * r.state_p + i : (r.groups + group) * r.state_p + i - r.state_p); };
    const int x_channel = h * r.vdim_p + v, first = tid < 2 * r.state_p ? shared_channel(tid) : values;
    const Window of_x = request(x_channel), of_shared = request(first);
    const float z = row[h * r.vdim_p + v], raw_dt = inputs[channels + h], dt_bias = r.dt_bias[h], rate = r.rate[h], skip = r.skip[h];
    float *state = r.state_of + (((size_t)seq * r.heads + h) * r.vdim_p + v) * r.state_p + e * 4;
    constexpr int kHeld = 8;   // pieces of the state's row
    float4 held[kHeld];
#pragma unroll
    for (int i = 0; i < kHeld; i++) held[i] = *reinterpret_cast<const float4 *>(state + (i * 32 < r.state_p ? i * 32 : 0));
    const bool again = p.halt && *p.halt, fresh = pos == 0 && !again;
    const bool keeps = part == 0 && h % share == 0;   // the workgroup that keeps the group's inputs
    float *now = past + (size_t)(pos % r.taps) * channels;
    if (tid < 2 * r.state_p) {
        lds[tid] = convolved(of_shared, first);
        if (keeps) now[first] = of_shared.in[0];
    }
    for (int i = tid + 256; i < 2 * r.state_p; i += 256) {
        const int channel = shared_channel(i);
        const Window g = request(channel);
        lds[i] = convolved(g, channel);
        if (keeps) now[channel] = g.in[0];
    }
    const float x = convolved(of_x, x_channel);
    if (e == 0) now[x_channel] = of_x.in[0];
    const float dt = softplus(raw_dt + dt_bias), decay = expf(-rate * dt), value = dt * x;
    __syncthreads();
    float o = 0.0f;
    auto piece = [&](int d0, float4 s) {
        if (fresh) s = make_float4(0.f, 0.f, 0.f, 0.f);
        const float4 b = *reinterpret_cast<const float4 *>(lds + d0 + e * 4), c = *reinterpret_cast<const float4 *>(lds + r.state_p + d0 + e * 4);
        if (!again) {
            s.x = decay * s.x + b.x * value; s.y = decay * s.y + b.y * value; s.z = decay * s.z + b.z * value; s.w = decay * s.w + b.w * value;
            *reinterpret_cast<float4 *>(state + d0) = s;
        }
        o += s.x * c.x + s.y * c.y + s.z * c.z + s.w * c.w;
    };
#pragma unroll
    for (int i = 0; i < kHeld; i++)
        if (i * 32 < r.state_p) piece(i * 32, held[i]);
    for (int d0 = kHeld * 32; d0 < r.state_p; d0 += 32) piece(d0, *reinterpret_cast<const float4 *>(state + d0));
    o += detail::dpp_term<0xB1, 0xF>(o);    // the eight lanes of a row
    o += detail::dpp_term<0x4E, 0xF>(o);
    o += detail::dpp_term<0x141, 0xF>(o);
    if (e == 0) p.y[(size_t)m * values + h * r.vdim_p + v] = (o + skip * x) * matrix::silu(z);
}

struct BlockArgs {
    Mamba2Shape r;
    Mamba2Block p;
    int R;
};

// grid (chunks, slabs of 32 channels: those of x head by head, of B and of C group by group).  LDS: the slab's inputs from taps - 1 tokens
// ahead of the chunk, and its convolved values, which are read back transposed.
template <typename T>
__global__ __launch_bounds__(256) void mamba2_prepare_kernel(BlockArgs a) {
    extern __shared__ float lds[];   // inputs [C + taps - 1][33]
    __shared__ float slab[32][C + 1], left[C];
    const Mamba2Shape &r = a.r;
    const int chunk = blockIdx.x, t0 = chunk * C, tid = threadIdx.x, c = tid & 31;
    const int len = a.p.rows - t0 < C ? a.p.rows - t0 : C, values = values_of(r), channels = channels_of(r);
    const int first = blockIdx.y * 32, channel = first + c, before = r.taps - 1;
    const float *inputs = a.p.mixed + values + channel;
    const float *past = r.inputs + (size_t)a.p.seq * r.taps * channels + channel;
    for (int i = tid >> 5; i < before + len; i += 8) {
        const int t = t0 + i - before, pos = a.p.base + t;   // inputs ahead of the block come from the ring, ahead of the sequence are zero
        lds[i * 33 + c] = t >= 0 ? inputs[(size_t)t * r.ld_mix] : pos >= 0 ? past[(size_t)(pos % r.taps) * channels] : 0.0f;
    }
    const bool is_x = first < values;
    const int h = is_x ? first / r.vdim_p : 0;
    if (is_x && tid < 64) {
        const float dt = tid < len ? softplus(a.p.mixed[(size_t)(t0 + tid) * r.ld_mix + values + channels + h] + r.dt_bias[h]) : 0.0f;
        double sum = -(double)r.rate[h] * dt;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const double other = __shfl_up(sum, d);
            if (tid >= d) sum += other;
        }
        const double end = __shfl(sum, 63);
        left[tid] = dt * expf((float)(end - sum));
        if (first % r.vdim_p == 0) {
            const size_t at = (size_t)h * a.R + t0 + tid;
            const float hi = (float)sum;
            a.p.log_hi[at] = hi;
            a.p.log_lo[at] = (float)(sum - (double)hi);
            a.p.step[at] = dt;
        }
    }
    __syncthreads();
    const float bias = r.conv_bias[channel];
    float y[C / 8];
#pragma unroll
    for (int i = 0; i < C / 8; i++) y[i] = bias;
    for (int j = 0; j < r.taps; j++) {
        const float f = r.conv[(size_t)j * channels + channel];
#pragma unroll
        for (int i = 0; i < C / 8; i++) {
            const int t = (tid >> 5) + 8 * i;
            y[i] += f * lds[(t < len ? t + j : 0) * 33 + c];
        }
    }
    const bool is_b = !is_x && first < values + r.groups * r.state_p;
    const int at_group = is_x ? 0 : first - values - (is_b ? 0 : r.groups * r.state_p), g = at_group / r.state_p, d0 = at_group % r.state_p;
    T *rows = is_x ? nullptr : static_cast<T *>(is_b ? a.p.k : a.p.q) + ((size_t)g * a.R + t0) * r.state_p + d0 + c;
#pragma unroll
    for (int i = 0; i < C / 8; i++) {
        const int t = (tid >> 5) + 8 * i;
        const float v = t < len ? matrix::silu(y[i]) : 0.0f;
        slab[c][t] = v;
        if (rows) rows[(size_t)t * r.state_p] = Op<T>::from_float(v);
    }
    if (!is_x && !is_b) return;
    __syncthreads();
    // eight tokens of one channel per thread
    const int col = tid >> 3, part = (tid & 7) * 8;
    float x[8];
#pragma unroll
    for (int i = 0; i < 8; i++) x[i] = slab[col][part + i];
    if (is_b) {
        chunked::store8<T>(static_cast<T *>(a.p.kt) + ((size_t)g * r.state_p + d0 + col) * a.R + t0 + part, x);
        return;
    }
    const size_t o = (size_t)(first + col) * a.R + t0 + part;
    chunked::store8<T>(static_cast<T *>(a.p.vt) + o, x);
#pragma unroll
    for (int i = 0; i < 8; i++) x[i] *= left[part + i];
    chunked::store8_split<T>(static_cast<T *>(a.p.vs_hi) + o, static_cast<T *>(a.p.vs_lo) + o, x);
}

// One workgroup per row: parts of the row over their root mean squares; and a block's last inputs into the sequence's ring.
constexpr int kNormWaves = 8;
__device__ __forceinline__ void store4(uint16_t *p, const float4 &v) { *reinterpret_cast<uint2 *>(p) = make_uint2(matrix::pack_bf16(v.x, v.y), matrix::pack_bf16(v.z, v.w)); }
__device__ __forceinline__ void store4(float *p, const float4 &v) { *reinterpret_cast<float4 *>(p) = v; }
template <typename T>
__global__ __launch_bounds__(64 * kNormWaves) void mamba2_norm_kernel(Mamba2Shape r, Mamba2Norm p) {
    extern __shared__ float lds[];   // [norm_groups * pieces] sums, then scales [norm_groups]
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, values = values_of(r), pieces = p.pieces;
    const float *y = p.y + (size_t)m * values;
    if (p.block_rows && m >= p.block_rows - (r.taps - 1)) {
        const int channels = channels_of(r), pos = p.base + m;
        float *now = r.inputs + ((size_t)p.seq * r.taps + pos % r.taps) * channels;
        const float *inputs = p.mixed + (size_t)m * r.ld_mix + values;
        for (int i = tid; i < channels; i += 64 * kNormWaves) now[i] = inputs[i];
    }
    for (int i = wave; i < r.norm_groups * pieces; i += kNormWaves) {
        const int g = i / pieces, at = (i % pieces) * 64 + lane, from = r.norm_starts[g], to = r.norm_starts[g + 1];
        float s = 0.0f;
        if (r.norm_by_eight) {
#pragma unroll 4
            for (int k = from + at * 4; k < to; k += 256 * pieces) {
                const float4 v = *reinterpret_cast<const float4 *>(y + k);
                s += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
            }
        } else {
            for (int k = from + at; k < to; k += 64 * pieces) s += y[k] * y[k];
        }
        s = detail::wave_sum(s);
        if (lane == 0) lds[i] = s;
    }
    __syncthreads();
    float *scale = lds + r.norm_groups * pieces;
    const float size = (float)r.heads * (float)r.vdim / (float)r.norm_groups;
    for (int g = tid; g < r.norm_groups; g += 64 * kNormWaves) {
        float s = 0.0f;
        for (int i = 0; i < pieces; i++) s += lds[g * pieces + i];
        scale[g] = 1.0f / sqrtf(s / size + p.eps);
    }
    __syncthreads();
    T *dst = static_cast<T *>(p.act) + (size_t)m * p.ld_act;
#pragma unroll 4
    for (int k = tid * 4; k < values; k += 256 * kNormWaves) {
        const float4 v = *reinterpret_cast<const float4 *>(y + k), n = *reinterpret_cast<const float4 *>(r.norm + k);
        const int4 g = *reinterpret_cast<const int4 *>(r.norm_part + k);
        store4(dst + k, make_float4(v.x * scale[g.x] * n.x, v.y * scale[g.y] * n.y, v.z * scale[g.z] * n.z, v.w * scale[g.w] * n.w));
    }
}

bool shape_ok(const Mamba2Shape &r) {
    return r.heads > 0 && r.vdim > 0 && r.state > 0 && r.groups > 0 && r.heads % r.groups == 0 && r.vdim_p % 32 == 0 && r.state_p % 32 == 0 && r.vdim <= r.vdim_p && r.state <= r.state_p &&
           r.taps >= 1 && r.taps <= kMamba2MaxTaps && r.state_p <= kMamba2MaxState && r.norm_groups >= 1 && r.norm_groups <= kMamba2MaxNormGroups &&
           r.ld_mix >= values_of(r) + channels_of(r) + r.heads && r.state_of && r.inputs && r.norm_part && r.norm_starts;
}

template <typename T>
hipError_t run_block(const BlockArgs &a, hipStream_t s) {
    const Mamba2Shape &r = a.r;
    hipLaunchKernelGGL((mamba2_prepare_kernel<T>), dim3(a.R / C, channels_of(r) / 32), dim3(256), (size_t)(C + r.taps - 1) * 33 * 4, s, a);
    chunked::Block c{};
    c.heads = r.heads; c.key_share = r.heads / r.groups; c.dim_p = r.state_p; c.vdim_p = r.vdim_p; c.rows = a.p.rows; c.R = a.R; c.base = a.p.base;
    c.q = a.p.q; c.k = a.p.k; c.vt = a.p.vt; c.state_k = a.p.kt; c.state_v = a.p.vs_hi; c.state_v_lo = a.p.vs_lo;
    c.state = r.state_of + (size_t)a.p.seq * r.heads * r.vdim_p * r.state_p; c.states_hi = a.p.states_hi; c.states_lo = a.p.states_lo; c.o = a.p.y;
    c.skip = r.skip; c.gate = a.p.mixed; c.ld_gate = r.ld_mix;
    chunked::launch_states_and_outputs<T>(c, chunked::TokenDecay{a.p.log_hi, a.p.log_lo, a.p.step, a.R}, s);
    return hipGetLastError();
}

}  // namespace

hipError_t launch_mamba2_step(const Mamba2Shape &r, const Mamba2Step &p, hipStream_t s) {
    if (!shape_ok(r) || p.rows < 1) return hipErrorInvalidValue;
    const dim3 grid(r.vdim_p / kStepRows, r.heads, p.rows);
    const size_t lds = (size_t)r.state_p * 8;
    switch (r.taps) {
        case 2: hipLaunchKernelGGL((mamba2_step_kernel<2>), grid, dim3(256), lds, s, r, p); break;
        case 3: hipLaunchKernelGGL((mamba2_step_kernel<3>), grid, dim3(256), lds, s, r, p); break;
        case 4: hipLaunchKernelGGL((mamba2_step_kernel<4>), grid, dim3(256), lds, s, r, p); break;
        default: hipLaunchKernelGGL((mamba2_step_kernel<0>), grid, dim3(256), lds, s, r, p); break;
    }
    return hipGetLastError();
}

hipError_t launch_mamba2_block(const Mamba2Shape &r, const Mamba2Block &p, Precision type, hipStream_t s) {
    if (!shape_ok(r) || p.rows < 1 || p.base < 0 || p.base + p.rows > r.max_seq) return hipErrorInvalidValue;
    const BlockArgs a{r, p, (p.rows + C - 1) / C * C};
    return type == Precision::bf16 ? run_block<uint16_t>(a, s) : run_block<float>(a, s);
}

hipError_t launch_mamba2_norm(const Mamba2Shape &r, const Mamba2Norm &given, int rows, Precision type, hipStream_t s) {
    if (!shape_ok(r) || rows < 1 || given.ld_act < values_of(r) || (given.block_rows && given.block_rows != rows)) return hipErrorInvalidValue;
    Mamba2Norm p = given;
    p.pieces = r.norm_groups >= kNormWaves ? 1 : kNormWaves / r.norm_groups;
    const size_t lds = (size_t)r.norm_groups * (p.pieces + 1) * 4;
    if (type == Precision::bf16) hipLaunchKernelGGL((mamba2_norm_kernel<uint16_t>), dim3(rows), dim3(64 * kNormWaves), lds, s, r, p);
    else hipLaunchKernelGGL((mamba2_norm_kernel<float>), dim3(rows), dim3(64 * kNormWaves), lds, s, r, p);
    return hipGetLastError();
}

}  // namespace esp
