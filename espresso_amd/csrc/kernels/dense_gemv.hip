// One activation row against bf16 weights (gfx950): the decode products of the layered models.
//
//   y[r] = sum_k x[k] W[r][k],   fp32 activations, exact bf16 -> fp32 weights, fp32 sums in a fixed order
//
// The kernels are bound by HBM: a weight is read once with 128-bit loads and costs a shift and a fused multiply-add.
//   * a workgroup of eight wavefronts stages the whole activation row in LDS (fp32, the two halves of every eight values in planes
//     of their own, so that a lane's two 128-bit reads are free of bank conflicts) and then walks units of weight rows: four rows per
//     wavefront, two or one where the matrix has too few rows to give every compute unit work (the loads run further ahead then);
//   * what surrounds the product lives in the staging and the epilogue: RMS norm (its scale factors out of the dot product), the
//     per-head norm and gate of a retention output, the norm by parts of a Mamba-2 output, f(gate) * up, the residual sum, the soft cap
//     of the logits; where branches are normed as they join the stream, that sum too (the first workgroup keeps it);
//   * the input side of a parallel layer is one launch over two activation rows: workgroups are dealt to the mixer's rows (norm1)
//     and the feed-forward's (norm2) in proportion.
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using detail::wave_sum;

constexpr int kGemvThreads = 512, kGemvWaves = 8, kRowAlign = 32;
constexpr int kStep = 512;   // columns a wavefront takes per step: 64 lanes x 8
// What a workgroup stages, and what becomes of a row's sum: the input side of a layer over normed rows, and over the stream itself (with
// the branch that joins it); the output side, and the same with a norm by parts; the head.
enum GemvKind : int { KIND_IN, KIND_IN_STREAM, KIND_OUT, KIND_OUT_PARTS, KIND_HEAD };
__host__ __device__ constexpr bool is_in(int kind) { return kind == KIND_IN || kind == KIND_IN_STREAM; }

struct DenseGemvArgs {
    const uint16_t *w;
    int ld, k_pad;                      // columns, and columns rounded up to kStep
    int units_a, units_b, blocks_a;     // KIND_IN: units of the mixer and of the feed-forward; workgroups of the mixer
    int mix_rows;
    const float *x, *norm_a, *norm_b;
    const float *branch, *branch_norm;
    float *x_out;
    int gate_function;
    int width;
    float eps;
    float *y, *act_out;
    const float *mix, *act, *squares, *gate;
    int mix_cols, act_at, act_cols, parts, heads, vdim, vdim_p;
    const int *part_of, *part_starts;   // KIND_OUT: norm by parts
    const float *part_norm;
    int part_count, part_pieces;
    bool part_by_eight;                 // every part starts at a multiple of eight columns
    float part_size;
    float mult, cap;
    const float *residual;
    int vocab;
    float *best_value;                  // KIND_HEAD: the workgroup's largest logit and its lowest row
    int *best_index;
};

// The place of column k in the staged row: groups of eight, the two fours of a group in separate planes.
__device__ __forceinline__ int staged_at(int k, int k_pad) { return (k >> 3) * 4 + (k & 3) + ((k & 4) ? k_pad / 2 : 0); }

// RPW weight rows per wavefront, AHEAD steps of loads in flight
template <int KIND, int RPW, int AHEAD>
__global__ __launch_bounds__(kGemvThreads) void dense_gemv_kernel(DenseGemvArgs a) {
    constexpr int kUnitRows = kGemvWaves * RPW;
    extern __shared__ float xs[];   // [k_pad], then [heads] or [part_count * part_pieces]
    __shared__ float red[kGemvWaves];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const bool second = is_in(KIND) && (int)blockIdx.x >= a.blocks_a;
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
    } else if constexpr (KIND == KIND_OUT_PARTS) {
        // parts over their root mean squares: the values times the norm's weights wait in registers (up to four loads per thread, the rest is
        // read again) while the values as they are pass through LDS and every part's squares are summed in part_pieces shares
        constexpr int kHeld = 4, kSpan = kGemvThreads * 4;
        float *sums = xs + a.k_pad;
        float4 held[kHeld];
        int4 part[kHeld];
        auto at = [](const float *p, int k) { return *reinterpret_cast<const float4 *>(p + k); };
        auto place = [&](int k, const float4 &v) { *reinterpret_cast<float4 *>(xs + staged_at(k, a.k_pad)) = v; };
        auto squared = [](const float4 &v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; };
        auto value = [&](int k) {
            const bool act = k >= a.act_at && k < a.act_at + a.act_cols;
            const float4 v = act ? at(a.act, k - a.act_at) : at(a.mix, k < a.mix_cols ? k : 0);
            const float keep = act || k < a.mix_cols ? 1.0f : 0.0f;
            return make_float4(v.x * keep, v.y * keep, v.z * keep, v.w * keep);
        };
        {
            float4 weight[kHeld];
#pragma unroll
            for (int c = 0; c < kHeld; c++) {
                const int k = c * kSpan + tid * 4, in = k < a.mix_cols ? k : 0;
                held[c] = value(k);
                weight[c] = at(a.part_norm, in);
                part[c] = *reinterpret_cast<const int4 *>(a.part_of + in);
            }
#pragma unroll
            for (int c = 0; c < kHeld; c++) {
                if (c * kSpan + tid * 4 < a.k_pad) place(c * kSpan + tid * 4, held[c]);
                held[c].x *= weight[c].x; held[c].y *= weight[c].y; held[c].z *= weight[c].z; held[c].w *= weight[c].w;
            }
        }
        for (int k = kHeld * kSpan + tid * 4; k < a.k_pad; k += kSpan) place(k, value(k));
        __syncthreads();
        for (int i = wave; i < a.part_count * a.part_pieces; i += kGemvWaves) {
            const int g = i / a.part_pieces, piece = i % a.part_pieces, from = a.part_starts[g], to = a.part_starts[g + 1];
            float s = 0.0f;
            if (a.part_by_eight) {   // both halves of every eight, four at a time
                for (int k = from / 2 + (piece * 64 + lane) * 4; k < to / 2; k += 256 * a.part_pieces) s += squared(at(xs, k)) + squared(at(xs + a.k_pad / 2, k));
            } else {
                for (int k = from + piece * 64 + lane; k < to; k += 64 * a.part_pieces) {
                    const float v = xs[staged_at(k, a.k_pad)];
                    s += v * v;
                }
            }
            s = wave_sum(s);
            if (lane == 0) sums[i] = s;
        }
        __syncthreads();
        auto scale_of = [&](int g) {
            float s = 0.0f;
            for (int i = 0; i < a.part_pieces; i++) s += sums[g * a.part_pieces + i];
            return 1.0f / sqrtf(s / a.part_size + a.eps);
        };
        auto put = [&](int k, float4 v, const int4 &g) {   // part indices ascend
            const float f = scale_of(g.x), l = g.w == g.x ? f : scale_of(g.w);
            v.x *= f;
            v.y *= g.y == g.x ? f : g.y == g.w ? l : scale_of(g.y);
            v.z *= g.z == g.x ? f : g.z == g.w ? l : scale_of(g.z);
            v.w *= l;
            place(k, v);
        };
#pragma unroll
        for (int c = 0; c < kHeld; c++)
            if (c * kSpan + tid * 4 < a.mix_cols) put(c * kSpan + tid * 4, held[c], part[c]);
        for (int k = kHeld * kSpan + tid * 4; k < a.mix_cols; k += kSpan) {
            float4 v = value(k);
            const float4 w = at(a.part_norm, k);
            v.x *= w.x; v.y *= w.y; v.z *= w.z; v.w *= w.w;
            put(k, v, *reinterpret_cast<const int4 *>(a.part_of + k));
        }
        __syncthreads();
    } else if constexpr (KIND == KIND_IN_STREAM) {
        // the stream as it is, or with a branch that is normed as it joins; both are kept in registers up to 8192 columns
        constexpr int kHeld = 4;
        float4 x[kHeld], b[kHeld], g[kHeld];
        const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
        auto at = [](const float *p, int k) { return *reinterpret_cast<const float4 *>(p + k); };
        float s = 0.0f, inv = 0.0f;
#pragma unroll
        for (int c = 0; c < kHeld; c++) {
            const int k = (tid + c * kGemvThreads) * 4;
            const bool in = k < a.ld;
            x[c] = in ? at(a.x, k) : zero;
            b[c] = in && a.branch ? at(a.branch, k) : zero;
            g[c] = in && a.branch ? at(a.branch_norm, k) : zero;
        }
        if (a.branch) {
#pragma unroll
            for (int c = 0; c < kHeld; c++) s += b[c].x * b[c].x + b[c].y * b[c].y + b[c].z * b[c].z + b[c].w * b[c].w;
            for (int k = (tid + kHeld * kGemvThreads) * 4; k < a.ld; k += kGemvThreads * 4) {
                const float4 v = at(a.branch, k);
                s += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
            }
            s = wave_sum(s);
            if (lane == 0) red[wave] = s;
            __syncthreads();
            const float total = ((red[0] + red[1]) + (red[2] + red[3])) + ((red[4] + red[5]) + (red[6] + red[7]));
            inv = 1.0f / sqrtf(total / (float)a.width + a.eps);
        }
        auto put = [&](int k, float4 v, const float4 &y, const float4 &w) {
            v.x += y.x * inv * w.x; v.y += y.y * inv * w.y; v.z += y.z * inv * w.z; v.w += y.w * inv * w.w;
            *reinterpret_cast<float4 *>(xs + staged_at(k, a.k_pad)) = v;
            if (a.branch && blockIdx.x == 0 && k < a.ld) *reinterpret_cast<float4 *>(a.x_out + k) = v;
        };
#pragma unroll
        for (int c = 0; c < kHeld; c++) {
            const int k = (tid + c * kGemvThreads) * 4;
            if (k < a.k_pad) put(k, x[c], b[c], g[c]);
        }
        for (int k = (tid + kHeld * kGemvThreads) * 4; k < a.k_pad; k += kGemvThreads * 4) {
            const bool in = k < a.ld;
            put(k, in ? at(a.x, k) : zero, in && a.branch ? at(a.branch, k) : zero, in && a.branch ? at(a.branch_norm, k) : zero);
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
    const int stride = is_in(KIND) ? (second ? (int)gridDim.x - a.blocks_a : a.blocks_a) : (int)gridDim.x;
    const int units = second ? a.units_b : a.units_a, base_row = second ? a.mix_rows : 0;
    const int steps = a.k_pad / kStep;
    float best = -INFINITY;
    int best_row = 0x7FFFFFFF;
    for (int u = first; u < units; u += stride) {
        const int row0 = base_row + u * kUnitRows + wave * RPW;
        const uint16_t *wr = a.w + (size_t)row0 * a.ld;
        float acc[RPW];
#pragma unroll
        for (int r = 0; r < RPW; r++) acc[r] = 0.0f;
        uint4 ring[AHEAD][RPW];
        auto fetch = [&](uint4 (&slot)[RPW], int step) {
            const int k = step * kStep + lane * 8, kc = k < a.ld ? k : 0;   // columns past the end meet staged zeros
#pragma unroll
            for (int r = 0; r < RPW; r++) slot[r] = *reinterpret_cast<const uint4 *>(wr + (size_t)r * a.ld + kc);
        };
        auto use = [&](const uint4 (&slot)[RPW], int step) {
            const float4 x0 = reinterpret_cast<const float4 *>(xs)[step * 64 + lane];
            const float4 x1 = reinterpret_cast<const float4 *>(xs + a.k_pad / 2)[step * 64 + lane];
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int r = 0; r < RPW; r++) {
                float w[8];
                matrix::unpack_bf16(slot[r], w);
#pragma unroll
                for (int i = 0; i < 8; i++) acc[r] = __builtin_fmaf(w[i], x[i], acc[r]);
            }
        };
#pragma unroll
        for (int i = 0; i < AHEAD; i++) fetch(ring[i], i);   // steps past the end read the row's first columns; never used
        int step = 0;
        for (; step + AHEAD <= steps; step += AHEAD) {
#pragma unroll
            for (int i = 0; i < AHEAD; i++) {
                use(ring[i], step + i);
                fetch(ring[i], step + i + AHEAD);
            }
        }
#pragma unroll
        for (int i = 0; i < AHEAD; i++)
            if (step + i < steps) use(ring[i], step + i);
#pragma unroll
        for (int r = 0; r < RPW; r++) acc[r] = wave_sum(acc[r]) * scale;
        if (lane != 0) continue;
        if constexpr (is_in(KIND)) {
            if (!second) {
#pragma unroll
                for (int r = 0; r < RPW; r++) a.y[row0 + r] = acc[r];
            } else {
                const int i = (row0 - a.mix_rows) / 2;
#pragma unroll
                for (int r = 0; r + 1 < RPW; r += 2) a.act_out[i + r / 2] = matrix::gated(a.gate_function, acc[r], acc[r + 1]);
            }
        } else if constexpr (KIND != KIND_HEAD) {
#pragma unroll
            for (int r = 0; r < RPW; r++) a.y[row0 + r] = a.residual ? a.residual[row0 + r] + a.mult * acc[r] : acc[r];
        } else {
#pragma unroll
            for (int r = 0; r < RPW; r++) {
                if (row0 + r >= a.vocab) continue;
                const float v = a.cap > 0.0f ? a.cap * tanhf(acc[r] / a.cap) : acc[r];
                if (a.y) a.y[row0 + r] = v;
                if (v > best) { best = v; best_row = row0 + r; }   // rows ascend: the first of equal logits stays
            }
        }
    }
    if constexpr (KIND == KIND_HEAD) {
        __shared__ float bv[kGemvWaves];
        __shared__ int bi[kGemvWaves];
        if (!a.best_value) return;
        if (lane == 0) { bv[wave] = best; bi[wave] = best_row; }
        __syncthreads();
        if (tid == 0) {
            for (int w = 1; w < kGemvWaves; w++)
                if (bv[w] > best || (bv[w] == best && bi[w] < best_row)) { best = bv[w]; best_row = bi[w]; }
            a.best_value[blockIdx.x] = best;
            a.best_index[blockIdx.x] = best_row;
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

template <int KIND, int RPW, int AHEAD>
hipError_t run(DenseGemvArgs a, int grid, hipStream_t s) {
    const size_t lds = (size_t)(a.k_pad + a.heads + a.part_count * a.part_pieces) * 4;
    if (lds > 150 * 1024 || grid < 1) return hipErrorInvalidValue;
    static size_t allowed = 0;
    if (lds > 48 * 1024 && lds > allowed) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&dense_gemv_kernel<KIND, RPW, AHEAD>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
        allowed = lds;
    }
    hipLaunchKernelGGL((dense_gemv_kernel<KIND, RPW, AHEAD>), dim3(grid), dim3(kGemvThreads), lds, s, a);
    return hipGetLastError();
}
int round_up(int v, int to) { return (v + to - 1) / to * to; }
int at_most(int units) { return units < resident_workgroups() ? units : resident_workgroups(); }

}  // namespace

hipError_t launch_dense_gemv_in(const DenseGemvIn &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.mix_rows % kRowAlign || p.w.rows % kRowAlign || p.w.rows < p.mix_rows || p.w.rows < kRowAlign || p.mix_rows < 0) return hipErrorInvalidValue;
    if ((p.branch && (!p.branch_norm || !p.x_out || p.x_out == p.x || p.norm1)) || (p.mix_rows && p.norm2 && !p.norm1) || (p.w.rows > p.mix_rows && p.norm1 && !p.norm2)) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep); a.mix_rows = p.mix_rows;
    a.x = p.x; a.norm_a = p.norm1; a.norm_b = p.norm2; a.width = p.width; a.eps = p.eps; a.y = p.y; a.act_out = p.act;
    a.branch = p.branch; a.branch_norm = p.branch_norm; a.x_out = p.x_out; a.gate_function = (int)p.gate_function;
    const int unit = p.w.rows >= resident_workgroups() * kGemvWaves * 4 ? kGemvWaves * 4 : kGemvWaves * 2;   // (gate, up) pairs stay together
    a.units_a = p.mix_rows / unit; a.units_b = (p.w.rows - p.mix_rows) / unit;
    const int units = a.units_a + a.units_b, wanted = at_most(units);
    a.blocks_a = (int)((long long)wanted * a.units_a / units);
    if (a.blocks_a < 1 && a.units_a) a.blocks_a = 1;
    int grid = wanted;
    if (a.units_b == 0) a.blocks_a = grid;
    else if (a.units_a && a.blocks_a >= grid) grid = a.blocks_a + 1;
    if (!p.norm1 && !p.norm2) return unit == kGemvWaves * 4 ? run<KIND_IN_STREAM, 4, 2>(a, grid, s) : run<KIND_IN_STREAM, 2, 3>(a, grid, s);
    return unit == kGemvWaves * 4 ? run<KIND_IN, 4, 2>(a, grid, s) : run<KIND_IN, 2, 3>(a, grid, s);
}

template <int KIND>
static hipError_t run_out(DenseGemvArgs a, int rows, hipStream_t s) {
    const int cus = resident_workgroups() / 2;   // long rows: a workgroup per compute unit
    if (rows >= cus * kGemvWaves * 4) { a.units_a = rows / (kGemvWaves * 4); return run<KIND, 4, 2>(a, at_most(a.units_a), s); }
    if (rows >= cus * kGemvWaves * 2) { a.units_a = rows / (kGemvWaves * 2); return run<KIND, 2, 4>(a, at_most(a.units_a), s); }
    a.units_a = rows / kGemvWaves;
    return run<KIND, 1, 6>(a, at_most(a.units_a), s);
}

hipError_t launch_dense_gemv_out(const DenseGemvOut &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.rows % kRowAlign || p.w.rows < p.rows || p.mix_cols % 32 || p.act_cols % 32 || p.act_at < p.mix_cols || p.act_at + p.act_cols > p.w.ld || p.rows < kRowAlign)
        return hipErrorInvalidValue;
    if (p.squares && (p.vdim_p <= 0 || p.mix_cols % p.vdim_p || !p.gate)) return hipErrorInvalidValue;
    if (p.part_of && (p.squares || p.part_count < 1 || !p.part_starts || !p.part_norm || !(p.part_size > 0))) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep);
    a.part_of = p.part_of; a.part_starts = p.part_starts; a.part_norm = p.part_norm; a.part_count = p.part_of ? p.part_count : 0; a.part_size = p.part_size;
    a.part_by_eight = p.part_by_eight;
    a.part_pieces = !p.part_of || p.part_count >= kGemvWaves ? 1 : kGemvWaves / p.part_count;
    a.mix = p.mix; a.act = p.act; a.squares = p.squares; a.gate = p.gate; a.mix_cols = p.mix_cols; a.act_at = p.act_at; a.act_cols = p.act_cols; a.parts = p.parts;
    a.heads = p.squares ? p.mix_cols / p.vdim_p : 0; a.vdim = p.vdim; a.vdim_p = p.vdim_p; a.eps = p.eps; a.mult = p.mult; a.residual = p.residual; a.y = p.out;
    return p.part_of ? run_out<KIND_OUT_PARTS>(a, p.rows, s) : run_out<KIND_OUT>(a, p.rows, s);
}

int dense_gemv_head_workgroups(const DenseMatrix &w) { return at_most(w.rows / (kGemvWaves * 4)); }

hipError_t launch_dense_gemv_head(const DenseGemvHead &p, hipStream_t s) {
    if (!p.w.w || p.w.ld % 64 || p.w.rows % kRowAlign || p.vocab > p.w.rows || p.vocab < 1 || (!p.logits && !p.best_value) || (p.best_value && !p.best_index)) return hipErrorInvalidValue;
    DenseGemvArgs a{};
    a.w = p.w.w; a.ld = p.w.ld; a.k_pad = round_up(p.w.ld, kStep); a.units_a = p.w.rows / (kGemvWaves * 4);
    a.x = p.x; a.norm_a = p.norm; a.width = p.width; a.eps = p.eps; a.vocab = p.vocab; a.cap = p.cap; a.y = p.logits;
    a.best_value = p.best_value; a.best_index = p.best_index;
    return run<KIND_HEAD, 4, 2>(a, dense_gemv_head_workgroups(p.w), s);
}

}  // namespace esp
