// One activation row against bf16 weights (gfx950): the decode products of the layered models.
//
//   y[r] = sum_k x[k] W[r][k],   fp32 activations, exact bf16 -> fp32 weights, fp32 sums in a fixed order
//
// The kernels are bound by HBM: a weight is read once with 128-bit loads and costs a shift and a fused multiply-add.
//   * a workgroup of eight wavefronts stages the whole activation row in LDS (fp32, the two halves of every eight values in planes
//     of their own, so that a lane's two 128-bit reads are free of bank conflicts) and then walks units of 32 weight rows, four per
//     wavefront; two workgroups fit a compute unit, which keeps 64 KB of weights on their way to it;
//   * what surrounds the product lives in the staging and the epilogue: RMS norm (its scale factors out of the dot product), the
//     per-head norm and gate of a retention output, SiLU(gate) * up, the residual sum, the soft cap of the logits;
//   * the input side of a parallel layer is one launch over two activation rows: workgroups are dealt to the mixer's rows (norm1)
//     and the feed-forward's (norm2) in proportion.
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using detail::wave_sum;

constexpr int kGemvThreads = 512, kGemvWaves = 8, kRowsPerWave = 4, kUnitRows = kGemvWaves * kRowsPerWave;
constexpr int kStep = 512;   // columns a wavefront takes per step: 64 lanes x 8
enum GemvKind : int { KIND_IN, KIND_OUT, KIND_HEAD };

struct DenseGemvArgs {
    const uint16_t *w;
    int ld, k_pad;                      // columns, and columns rounded up to kStep
    int units_a, units_b, blocks_a;     // KIND_IN: units of the mixer and of the feed-forward; workgroups of the mixer
    int mix_rows;
    const float *x, *norm_a, *norm_b;
    int width;
    float eps;
    float *y, *act_out;
    const float *mix, *act, *squares, *gate;
    int mix_cols, act_at, act_cols, parts, heads, vdim, vdim_p;
    float mult, cap;
    const float *residual;
    int vocab;
};

// The place of column k in the staged row: groups of eight, the two fours of a group in separate planes.
__device__ __forceinline__ int staged_at(int k, int k_pad) { return (k >> 3) * 4 + (k & 3) + ((k & 4) ? k_pad / 2 : 0); }

template <int KIND>
__global__ __launch_bounds__(kGemvThreads) void dense_gemv_kernel(DenseGemvArgs a) {
    extern __shared__ float xs[];   // [k_pad], then [heads]
    __shared__ float red[kGemvWaves];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const bool second = KIND == KIND_IN && (int)blockIdx.x >= a.blocks_a;
    float scale = 1.0f;
    if constexpr (KIND == KIND_OUT) {
        float *head_inv = xs + a.k_pad;
        if (a.squares) {
            for (int h = tid; h < a.heads; h += kGemvThreads) {
                float s = 0.0f;
                for (int i = 0; i < a.parts; i++) s += a.squares[h * a.parts + i];
                head_inv[h] = 1.0f / sqrtf(s / (float)a.vdim + a.eps);
            }
            __syncthreads();
        }
        for (int k = tid * 4; k < a.k_pad; k += kGemvThreads * 4) {
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (k < a.mix_cols) {
                v = *reinterpret_cast<const float4 *>(a.mix + k);
                if (a.squares) {
                    const float4 g = *reinterpret_cast<const float4 *>(a.gate + k);
                    const float inv = head_inv[k / a.vdim_p];
                    v.x = v.x * inv * matrix::silu(g.x); v.y = v.y * inv * matrix::silu(g.y);
                    v.z = v.z * inv * matrix::silu(g.z); v.w = v.w * inv * matrix::silu(g.w);
                }
            } else if (k >= a.act_at && k < a.act_at + a.act_cols) {
                v = *reinterpret_cast<const float4 *>(a.act + (k - a.act_at));
            }
            *reinterpret_cast<float4 *>(xs + staged_at(k, a.k_pad)) = v;
        }
        __syncthreads();
    } else {
        const float *norm = second ? a.norm_b : a.norm_a;
        float s = 0.0f;
        for (int k = tid * 4; k < a.k_pad; k += kGemvThreads * 4) {
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (k < a.ld) {
                const float4 x = *reinterpret_cast<const float4 *>(a.x + k), g = *reinterpret_cast<const float4 *>(norm + k);
                s += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
                v = make_float4(x.x * g.x, x.y * g.y, x.z * g.z, x.w * g.w);
            }
            *reinterpret_cast<float4 *>(xs + staged_at(k, a.k_pad)) = v;
        }
        s = wave_sum(s);
        if (lane == 0) red[wave] = s;
        __syncthreads();
        const float total = ((red[0] + red[1]) + (red[2] + red[3])) + ((red[4] + red[5]) + (red[6] + red[7]));
        scale = 1.0f / sqrtf(total / (float)a.width + a.eps);
    }

    const int first = second ? (int)blockIdx.x - a.blocks_a : (int)blockIdx.x;
    const int stride = KIND == KIND_IN ? (second ? (int)gridDim.x - a.blocks_a : a.blocks_a) : (int)gridDim.x;
    const int units = second ? a.units_b : a.units_a, base_row = second ? a.mix_rows : 0;
    const int steps = a.k_pad / kStep;
    for (int u = first; u < units; u += stride) {
        const int row0 = base_row + u * kUnitRows + wave * kRowsPerWave;
        const uint16_t *wr = a.w + (size_t)row0 * a.ld;
        float acc[kRowsPerWave] = {0.f, 0.f, 0.f, 0.f};
        uint4 next[kRowsPerWave];
        auto fetch = [&](int step) {
            const int k = step * kStep + lane * 8, kc = k < a.ld ? k : 0;   // columns past the end meet staged zeros
#pragma unroll
            for (int r = 0; r < kRowsPerWave; r++) next[r] = *reinterpret_cast<const uint4 *>(wr + (size_t)r * a.ld + kc);
        };
        fetch(0);
        for (int step = 0; step < steps; step++) {
            uint4 cur[kRowsPerWave];
#pragma unroll
            for (int r = 0; r < kRowsPerWave; r++) cur[r] = next[r];
            if (step + 1 < steps) fetch(step + 1);
            const float4 x0 = reinterpret_cast<const float4 *>(xs)[step * 64 + lane];
            const float4 x1 = reinterpret_cast<const float4 *>(xs + a.k_pad / 2)[step * 64 + lane];
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int r = 0; r < kRowsPerWave; r++) {
                float w[8];
                matrix::unpack_bf16(cur[r], w);
#pragma unroll
                for (int i = 0; i < 8; i++) acc[r] = __builtin_fmaf(w[i], x[i], acc[r]);
            }
        }
#pragma unroll
        for (int r = 0; r < kRowsPerWave; r++) acc[r] = wave_sum(acc[r]) * scale;
        if (lane != 0) continue;
        if constexpr (KIND == KIND_IN) {
            if (!second) {
                *reinterpret_cast<float4 *>(a.y + row0) = make_float4(acc[0], acc[1], acc[2], acc[3]);
            } else {
                const int i = (row0 - a.mix_rows) / 2;
                *reinterpret_cast<float2 *>(a.act_out + i) = make_float2(matrix::silu(acc[0]) * acc[1], matrix::silu(acc[2]) * acc[3]);
            }
        } else if constexpr (KIND == KIND_OUT) {
            const float4 x = *reinterpret_cast<const float4 *>(a.residual + row0);
            *reinterpret_cast<float4 *>(a.y + row0) = make_float4(x.x + a.mult * acc[0], x.y + a.mult * acc[1], x.z + a.mult * acc[2], x.w + a.mult * acc[3]);
        } else {
#pragma unroll
            for (int r = 0; r < kRowsPerWave; r++)
                if (row0 + r < a.vocab) a.y[row0 + r] = a.cap > 0.0f ? a.cap * tanhf(acc[r] / a.cap) : acc[r];
        }
    }
}

int resident_workgroups() {
    static const int n = [] {
        int dev = 0, cus = 0;
        if (hipGetDevice(&dev) != hipSuccess || hipDeviceGetAttribute(&cus, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || cus <= 0) cus = 256;
        return 2 * cus;
    }();
    return n;
}

template <int KIND>
hipError_t run(const DenseGemvArgs &a, int grid, hipStream_t s) {
    const size_t lds = (size_t)(a.k_pad + a.heads) * 4;
    if (lds > 150 * 1024 || grid < 1) return hipErrorInvalidValue;
    static size_t allowed = 0;
    if (lds > 48 * 1024 && lds > allowed) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&dense_gemv_kernel<KIND>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
        allowed = lds;
    }
    hipLaunchKernelGGL((dense_gemv_kernel<KIND>), dim3(grid), dim3(kGemvThreads), lds, s, a);
    return hipGetLastError();
}
int round_up(int v, int to) { return (v + to - 1) / to * to; }

}  // namespace

hipError_t launch_dense_gemv_in(const DenseGemvIn &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.mix_rows % kUnitRows || p.w.rows % kUnitRows || p.w.rows < p.mix_rows || p.mix_rows < kUnitRows) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep);
    a.units_a = p.mix_rows / kUnitRows; a.units_b = (p.w.rows - p.mix_rows) / kUnitRows; a.mix_rows = p.mix_rows;
    const int units = a.units_a + a.units_b, wanted = units < resident_workgroups() ? units : resident_workgroups();
    a.blocks_a = (int)((long long)wanted * a.units_a / units);
    if (a.blocks_a < 1) a.blocks_a = 1;
    int grid = wanted;
    if (a.units_b == 0) a.blocks_a = grid;
    else if (a.blocks_a >= grid) grid = a.blocks_a + 1;
    a.x = p.x; a.norm_a = p.norm1; a.norm_b = p.norm2; a.width = p.width; a.eps = p.eps; a.y = p.y; a.act_out = p.act;
    return run<KIND_IN>(a, grid, s);
}

hipError_t launch_dense_gemv_out(const DenseGemvOut &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.rows % kUnitRows || p.w.rows < p.rows || p.mix_cols % 32 || p.act_cols % 32 || p.act_at < p.mix_cols || p.act_at + p.act_cols > p.w.ld || p.rows < kUnitRows)
        return hipErrorInvalidValue;
    if (p.squares && (p.vdim_p <= 0 || p.mix_cols % p.vdim_p || !p.gate)) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep); a.units_a = p.rows / kUnitRows;
    a.mix = p.mix; a.act = p.act; a.squares = p.squares; a.gate = p.gate; a.mix_cols = p.mix_cols; a.act_at = p.act_at; a.act_cols = p.act_cols; a.parts = p.parts;
    a.heads = p.squares ? p.mix_cols / p.vdim_p : 0; a.vdim = p.vdim; a.vdim_p = p.vdim_p; a.eps = p.eps; a.mult = p.mult; a.residual = p.residual; a.y = p.out;
    return run<KIND_OUT>(a, a.units_a < resident_workgroups() ? a.units_a : resident_workgroups(), s);
}

hipError_t launch_dense_gemv_head(const DenseGemvHead &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.w.rows % kUnitRows || p.vocab > p.w.rows || p.vocab < 1) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep); a.units_a = p.w.rows / kUnitRows;
    a.x = p.x; a.norm_a = p.norm; a.width = p.width; a.eps = p.eps; a.vocab = p.vocab; a.cap = p.cap; a.y = p.logits;
    return run<KIND_HEAD>(a, a.units_a < resident_workgroups() ? a.units_a : resident_workgroups(), s);
}

}  // namespace esp
