// Embedding, residual stream and RMS norms of the layered models (gfx950).  One workgroup per row; fp32 throughout.
#include <hip/hip_runtime.h>

#include "gemv_device.h"
#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::Op;

constexpr int kBlock = 256;

constexpr int kEmbedBlock = 1024;
__global__ __launch_bounds__(kEmbedBlock) void embed_norm_kernel(const uint16_t *table, int ld_table, const int *tokens, const float *weight, float eps, int width, int ld, float *x) {
    __shared__ float red[kEmbedBlock / 64];
    const int m = blockIdx.x;
    const uint16_t *row = table + (size_t)tokens[m] * ld_table;
    constexpr int kHeld = 8;   // values per thread kept in registers: rows up to 8192 wide are read once, with every load in flight
    uint16_t bits[kHeld];
    float gain[kHeld], s = 0.0f;
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kEmbedBlock, in = i < width ? i : width - 1;
        bits[c] = row[in];
        gain[c] = weight ? weight[in] : 1.0f;
    }
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const float v = matrix::bf16_bits_to_float(bits[c]);
        s += (int)threadIdx.x + c * kEmbedBlock < width ? v * v : 0.0f;
    }
    for (int i = threadIdx.x + kHeld * kEmbedBlock; i < width; i += kEmbedBlock) { const float v = matrix::bf16_bits_to_float(row[i]); s += v * v; }
    s = detail::wave_sum(s);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = s;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < kEmbedBlock / 64; w++) total += red[w];
    const float inv = weight ? 1.0f / sqrtf(total / (float)width + eps) : 1.0f;
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kEmbedBlock;
        if (i < ld) x[(size_t)m * ld + i] = i < width ? matrix::bf16_bits_to_float(bits[c]) * inv * gain[c] : 0.0f;
    }
    for (int i = threadIdx.x + kHeld * kEmbedBlock; i < ld; i += kEmbedBlock)
        x[(size_t)m * ld + i] = i < width ? matrix::bf16_bits_to_float(row[i]) * inv * (weight ? weight[i] : 1.0f) : 0.0f;
}

struct ResidualNormArgs {
    float *x, *final_x;
    int width, ld, splits;
    const float *planes;
    size_t plane;
    float mult, eps;
    const float *norm1, *norm2;
    void *out1, *out2;
};

__device__ __forceinline__ void store4(float *p, float4 v) { *reinterpret_cast<float4 *>(p) = v; }
__device__ __forceinline__ void store4(uint16_t *p, float4 v) { *reinterpret_cast<uint2 *>(p) = make_uint2(matrix::pack_bf16(v.x, v.y), matrix::pack_bf16(v.z, v.w)); }

template <typename T>
__global__ __launch_bounds__(kBlock) void residual_norm_kernel(ResidualNormArgs a) {
    __shared__ float red[4];
    const size_t row = (size_t)blockIdx.x * a.ld;
    float s = 0.0f;
    constexpr int kHeld = 8;   // float4 per thread kept in registers: rows up to 8192 wide are read once
    const int n4 = a.ld / 4;
    float4 held[kHeld];
    auto value = [&](int i) {
        float4 v = reinterpret_cast<const float4 *>(a.x + row)[i];
        if (a.splits > 0) {
            float4 t = reinterpret_cast<const float4 *>(a.planes + row)[i];
            for (int k = 1; k < a.splits; k++) {
                const float4 u = reinterpret_cast<const float4 *>(a.planes + k * a.plane + row)[i];
                t.x += u.x; t.y += u.y; t.z += u.z; t.w += u.w;
            }
            v.x += a.mult * t.x; v.y += a.mult * t.y; v.z += a.mult * t.z; v.w += a.mult * t.w;
        }
        return v;
    };
    float *dst = (a.final_x ? a.final_x : a.x) + row;
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kBlock;
        if (i < n4) {
            held[c] = value(i);
            s += held[c].x * held[c].x + held[c].y * held[c].y + held[c].z * held[c].z + held[c].w * held[c].w;
            if (a.splits > 0) store4(dst + 4 * i, held[c]);
        }
    }
    for (int i = threadIdx.x + kHeld * kBlock; i < n4; i += kBlock) {   // wider rows: the rest is read back for the norms
        const float4 v = value(i);
        s += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        if (a.splits > 0) store4(dst + 4 * i, v);
    }
    if (!a.norm1) return;
    const float inv = 1.0f / sqrtf(detail::workgroup_sum(s, red) / (float)a.width + a.eps);
    auto emit = [&](int i, const float4 &v) {
        const float4 g = reinterpret_cast<const float4 *>(a.norm1)[i];
        store4(static_cast<T *>(a.out1) + row + 4 * i, make_float4(v.x * inv * g.x, v.y * inv * g.y, v.z * inv * g.z, v.w * inv * g.w));
        if (a.norm2) {
            const float4 h = reinterpret_cast<const float4 *>(a.norm2)[i];
            store4(static_cast<T *>(a.out2) + row + 4 * i, make_float4(v.x * inv * h.x, v.y * inv * h.y, v.z * inv * h.z, v.w * inv * h.w));
        }
    };
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kBlock;
        if (i < n4) emit(i, held[c]);
    }
    for (int i = threadIdx.x + kHeld * kBlock; i < n4; i += kBlock) emit(i, reinterpret_cast<const float4 *>(dst)[i]);
}

struct BranchNormArgs {
    float *x, *final_x;
    int width, ld, splits;
    const float *planes;
    size_t plane;
    float eps;
    const float *norm;
    void *out;
};

template <typename T>
__global__ __launch_bounds__(kBlock) void branch_norm_kernel(BranchNormArgs a) {
    __shared__ float red[4];
    const size_t row = (size_t)blockIdx.x * a.ld;
    constexpr int kHeld = 8;   // float4 per thread kept in registers: rows up to 8192 wide are read once
    const int n4 = a.ld / 4;
    float4 held[kHeld], x[kHeld], g[kHeld];
    auto branch = [&](int i) {
        float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int k = 0; k < a.splits; k++) {
            const float4 u = reinterpret_cast<const float4 *>(a.planes + k * a.plane + row)[i];
            t.x += u.x; t.y += u.y; t.z += u.z; t.w += u.w;
        }
        return t;
    };
    auto square = [](const float4 &v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; };
    float s = 0.0f;
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kBlock;
        if (i < n4) {
            x[c] = reinterpret_cast<const float4 *>(a.x + row)[i];
            if (a.splits > 0) g[c] = reinterpret_cast<const float4 *>(a.norm)[i];
            held[c] = branch(i);
            s += square(held[c]);
        }
    }
    for (int i = threadIdx.x + kHeld * kBlock; i < n4; i += kBlock) s += square(branch(i));   // wider rows: the rest is read twice
    const float inv = a.splits > 0 ? 1.0f / sqrtf(detail::workgroup_sum(s, red) / (float)a.width + a.eps) : 0.0f;
    float *dst = (a.final_x ? a.final_x : a.x) + row;
    auto emit = [&](int i, float4 v, const float4 &b, const float4 &w) {
        if (a.splits > 0) {
            v.x += b.x * inv * w.x; v.y += b.y * inv * w.y; v.z += b.z * inv * w.z; v.w += b.w * inv * w.w;
            store4(dst + 4 * i, v);
        }
        if (a.out) store4(static_cast<T *>(a.out) + row + 4 * i, v);
    };
#pragma unroll
    for (int c = 0; c < kHeld; c++) {
        const int i = threadIdx.x + c * kBlock;
        if (i < n4) emit(i, x[c], held[c], g[c]);
    }
    for (int i = threadIdx.x + kHeld * kBlock; i < n4; i += kBlock)
        emit(i, reinterpret_cast<const float4 *>(a.x + row)[i], branch(i), a.splits > 0 ? reinterpret_cast<const float4 *>(a.norm)[i] : make_float4(0.f, 0.f, 0.f, 0.f));
}

}  // namespace

hipError_t launch_embed_norm(const uint16_t *table, int ld_table, const int *tokens, const float *weight, float eps, int rows, int width, int ld, float *x, hipStream_t s) {
    if (!table || rows < 1 || width < 1 || ld < width || ld_table < width) return hipErrorInvalidValue;
    hipLaunchKernelGGL(embed_norm_kernel, dim3(rows), dim3(kEmbedBlock), 0, s, table, ld_table, tokens, weight, eps, width, ld, x);
    return hipGetLastError();
}

hipError_t launch_residual_norm(const ResidualNorm &p, Precision type, hipStream_t s) {
    if (!p.x || p.rows < 1 || p.ld % 64 || p.width > p.ld || (p.splits > 0 && !p.planes) || (p.norm1 && !p.out1) || (p.norm2 && !p.out2)) return hipErrorInvalidValue;
    if (p.splits == 0 && p.final_x) return hipErrorInvalidValue;
    ResidualNormArgs a{p.x, p.final_x, p.width, p.ld, p.splits, p.planes, p.plane, p.mult, p.eps, p.norm1, p.norm2, p.out1, p.out2};
    if (type == Precision::bf16) hipLaunchKernelGGL((residual_norm_kernel<uint16_t>), dim3(p.rows), dim3(kBlock), 0, s, a);
    else hipLaunchKernelGGL((residual_norm_kernel<float>), dim3(p.rows), dim3(kBlock), 0, s, a);
    return hipGetLastError();
}

hipError_t launch_branch_norm(const BranchNorm &p, Precision type, hipStream_t s) {
    if (!p.x || p.rows < 1 || p.ld % 64 || p.width > p.ld || (p.splits > 0 && (!p.planes || !p.norm)) || (p.splits == 0 && (p.final_x || !p.out))) return hipErrorInvalidValue;
    BranchNormArgs a{p.x, p.final_x, p.width, p.ld, p.splits, p.planes, p.plane, p.eps, p.norm, p.out};
    if (type == Precision::bf16) hipLaunchKernelGGL((branch_norm_kernel<uint16_t>), dim3(p.rows), dim3(kBlock), 0, s, a);
    else hipLaunchKernelGGL((branch_norm_kernel<float>), dim3(p.rows), dim3(kBlock), 0, s, a);
    return hipGetLastError();
}

}  // namespace esp
