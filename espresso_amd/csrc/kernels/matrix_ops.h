// Matrix-core operands of the layered models' kernels (gfx950, wave64), in two precisions with one register layout.
//
// A fragment is eight consecutive k of one row (A: lane % 32 = row of A; B: lane % 32 = column of B); lanes 0..31 hold k 0..7 of a
// step of sixteen, lanes 32..63 k 8..15.  bf16: one v_mfma_f32_32x32x16_bf16 per step.  fp32: eight v_mfma_f32_32x32x2_f32,
// the j-th over element j of both halves - the order of k inside a sum is free as long as A and B agree.
// Accumulator register r of lane l: row 8 * (r / 4) + 4 * (l / 32) + r % 4, column l % 32.
// An accumulator is also the B fragment of the next product over its rows: registers 8t .. 8t + 7 are the step whose k are rows
// 16t + 4 half + 0..3 and 16t + 8 + 4 half + 0..3, so the A operand is read at those k.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace esp {
namespace matrix {

typedef float floatx16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ float bf16_bits_to_float(uint32_t b) { return __builtin_bit_cast(float, b << 16); }
// round to nearest even; NaN keeps its sign and stays NaN
__device__ __forceinline__ uint16_t float_to_bf16_bits(float v) { return __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ uint32_t pack_bf16(float lo, float hi) { return (uint32_t)float_to_bf16_bits(lo) | ((uint32_t)float_to_bf16_bits(hi) << 16); }
__device__ __forceinline__ void unpack_bf16(const uint4 &v, float (&f)[8]) {
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int i = 0; i < 4; i++) {
        f[2 * i] = __builtin_bit_cast(float, w[i] << 16);
        f[2 * i + 1] = __builtin_bit_cast(float, w[i] & 0xFFFF0000u);
    }
}

struct F32Fragment { float v[8]; };

template <typename T>
struct Op;

template <>
struct Op<uint16_t> {   // bf16
    typedef uint16_t elem;
    typedef bf16x8 frag;
    static constexpr bool kSplit = true;   // fp32 values travel as a high and a low part
    static __device__ __forceinline__ frag load(const elem *p) { return *reinterpret_cast<const bf16x8 *>(p); }
    static __device__ __forceinline__ frag load_pair(const elem *p, const elem *q) {   // four elements from each
        const uint2 a = *reinterpret_cast<const uint2 *>(p), b = *reinterpret_cast<const uint2 *>(q);
        return __builtin_bit_cast(bf16x8, make_uint4(a.x, a.y, b.x, b.y));
    }
    static __device__ __forceinline__ frag from_elems(const elem (&e)[8]) {
        uint4 v;
        v.x = (uint32_t)e[0] | ((uint32_t)e[1] << 16); v.y = (uint32_t)e[2] | ((uint32_t)e[3] << 16);
        v.z = (uint32_t)e[4] | ((uint32_t)e[5] << 16); v.w = (uint32_t)e[6] | ((uint32_t)e[7] << 16);
        return __builtin_bit_cast(bf16x8, v);
    }
    static __device__ __forceinline__ frag high(const float (&f)[8]) {
        frag r;
#pragma unroll
        for (int i = 0; i < 8; i++) r[i] = (__bf16)f[i];
        return r;
    }
    static __device__ __forceinline__ frag low(const float (&f)[8], const frag &hi) {
        frag r;
#pragma unroll
        for (int i = 0; i < 8; i++) r[i] = (__bf16)(f[i] - (float)hi[i]);
        return r;
    }
    static __device__ __forceinline__ floatx16 mma(const frag &a, const frag &b, floatx16 c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }
    static __device__ __forceinline__ elem from_float(float v) { return float_to_bf16_bits(v); }
    static __device__ __forceinline__ float to_float(elem v) { return bf16_bits_to_float(v); }
};

template <>
struct Op<float> {
    typedef float elem;
    typedef F32Fragment frag;
    static constexpr bool kSplit = false;
    static __device__ __forceinline__ frag load(const elem *p) { return load_pair(p, p + 4); }
    static __device__ __forceinline__ frag load_pair(const elem *p, const elem *q) {
        const float4 a = *reinterpret_cast<const float4 *>(p), b = *reinterpret_cast<const float4 *>(q);
        return frag{{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w}};
    }
    static __device__ __forceinline__ frag from_elems(const elem (&e)[8]) {
        frag r;
#pragma unroll
        for (int i = 0; i < 8; i++) r.v[i] = e[i];
        return r;
    }
    static __device__ __forceinline__ frag high(const float (&f)[8]) { return from_elems(f); }
    static __device__ __forceinline__ frag low(const float (&)[8], const frag &hi) { return hi; }   // never used
    static __device__ __forceinline__ floatx16 mma(const frag &a, const frag &b, floatx16 c) {
#pragma unroll
        for (int i = 0; i < 8; i++) c = __builtin_amdgcn_mfma_f32_32x32x2f32(a.v[i], b.v[i], c, 0, 0, 0);
        return c;
    }
    static __device__ __forceinline__ elem from_float(float v) { return v; }
    static __device__ __forceinline__ float to_float(elem v) { return v; }
};

__device__ __forceinline__ int accumulator_row(int r, int half) { return 8 * (r >> 2) + 4 * half + (r & 3); }
__device__ __forceinline__ floatx16 zero_accumulator() {
    floatx16 z;
#pragma unroll
    for (int i = 0; i < 16; i++) z[i] = 0.0f;
    return z;
}
// The B fragment of fp32 values times an A fragment: two products where fp32 values are split, one otherwise.
template <typename T>
__device__ __forceinline__ floatx16 mma_values(const typename Op<T>::frag &a, const float (&f)[8], floatx16 c) {
    const typename Op<T>::frag hi = Op<T>::high(f);
    c = Op<T>::mma(a, hi, c);
    if constexpr (Op<T>::kSplit) c = Op<T>::mma(a, Op<T>::low(f, hi), c);
    return c;
}

__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh u) = z / (1 + exp(-2 u)), u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh(float z) { return z / (1.0f + expf(-1.5957691216057308f * (z + 0.044715f * z * z * z))); }
// A gated feed-forward's value (function: GateFunction).
__device__ __forceinline__ float gated(int function, float gate, float up) { return (function ? gelu_tanh(gate) : silu(gate)) * up; }
// Exponentials of scores: bf16 models use the hardware's exponential directly.
template <typename T>
__device__ __forceinline__ float weight_exp(float x) {
    if constexpr (Op<T>::kSplit) return __expf(x);
    else return expf(x);
}

}  // namespace matrix
}  // namespace esp
