// Blocks of rows against dense matrices on the matrix cores (gfx950): the prompt products of the layered models.
//
//   y[m][n] = sum_k a[m][k] b[n][k],   bf16 operands (or fp32 ones: v_mfma_f32_32x32x2_f32), fp32 accumulation
//
//   * a workgroup of four wavefronts owns a BM x BN tile of y and walks k in tiles of 128 bytes per row (64 bf16 or 32 fp32
//     values); LDS holds two tiles of both operands, so one barrier per tile is enough, and two more are on their way in registers;
//   * rows of LDS are 144 bytes apart: the 128-bit fragment reads of eight rows cover all banks;
//   * a bf16 operand of an fp32 product (weights under fp32 activations) is widened on its way to LDS;
//   * block index -> tile: the tiles of y that share rows of b follow each other on the same die (workgroups are dealt round robin
//     over the eight dies), so a tile of weights comes from HBM once and from that die's L2 afterwards;
//   * short grids split k over grid.y and leave partial planes, which launch_residual_norm adds in order.
#include <hip/hip_runtime.h>

#include <type_traits>

#include "layer_ops.h"
#include "matrix_ops.h"

namespace esp {
namespace {

using matrix::floatx16;
using matrix::Op;

constexpr int kDies = 8;

struct DenseGemmArgs {
    const void *a, *a2, *b;
    int lda, ldb, m, n, tiles, tiles_per_split, m_tiles, n_tiles;
    int out;
    void *y;
    int ldy, mix_cols;
    void *act;
    int ld_act, gate_function, n_store;
    float cap;
};

// Eight consecutive values of an operand row on their way to LDS.
typedef uint32_t uintx4 __attribute__((ext_vector_type(4)));
typedef float floatx4 __attribute__((ext_vector_type(4)));
typedef float floatx8 __attribute__((ext_vector_type(8)));
template <typename T>
struct PieceOf { typedef uintx4 type; };
template <>
struct PieceOf<float> { typedef floatx8 type; };
__device__ __forceinline__ uintx4 fetch_piece(const uint16_t *p) { return *reinterpret_cast<const uintx4 *>(p); }
__device__ __forceinline__ floatx8 fetch_piece(const float *p) {
    const floatx4 a = reinterpret_cast<const floatx4 *>(p)[0], b = reinterpret_cast<const floatx4 *>(p)[1];
    return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}
__device__ __forceinline__ void store_piece(uintx4 d, uint16_t *lds) { *reinterpret_cast<uintx4 *>(lds) = d; }
__device__ __forceinline__ void store_piece(floatx8 d, float *lds) {
    reinterpret_cast<floatx4 *>(lds)[0] = __builtin_shufflevector(d, d, 0, 1, 2, 3);
    reinterpret_cast<floatx4 *>(lds)[1] = __builtin_shufflevector(d, d, 4, 5, 6, 7);
}
__device__ __forceinline__ void store_piece(uintx4 d, float *lds) {
    const uintx4 lo = d << 16, hi = d & 0xFFFF0000u;
    reinterpret_cast<floatx4 *>(lds)[0] = __builtin_bit_cast(floatx4, __builtin_shufflevector(lo, hi, 0, 4, 1, 5));
    reinterpret_cast<floatx4 *>(lds)[1] = __builtin_bit_cast(floatx4, __builtin_shufflevector(lo, hi, 2, 6, 3, 7));
}

template <typename TA, typename TB, int WM, int WN, int TM, int TN>
__global__ __launch_bounds__(64 * WM * WN) void dense_gemm_kernel(DenseGemmArgs a) {
    using E = typename std::conditional<std::is_same<TA, float>::value || std::is_same<TB, float>::value, float, uint16_t>::type;
    constexpr int THREADS = 64 * WM * WN, BM = 32 * WM * TM, BN = 32 * WN * TN;
    constexpr int KT = 128 / sizeof(E), LDK = 144 / sizeof(E), NCH = KT / 8;   // values per tile row, per LDS row; pieces per tile row
    constexpr int XA = BM * NCH / THREADS, XB = BN * NCH / THREADS;
    static_assert(XA >= 1 && XB >= 1, "tile too small for the copy loop");
    __shared__ E at[2][BM * LDK];
    __shared__ E bt[2][BN * LDK];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave / WN, wn = wave % WN;
    // the m tiles of one n tile follow each other on one die
    const int die = blockIdx.x % kDies, at_die = blockIdx.x / kDies, mt = at_die % a.m_tiles, nt = at_die / a.m_tiles * kDies + die;
    if (nt >= a.n_tiles) return;
    const int m0 = mt * BM, n0 = nt * BN;
    const int t_begin = blockIdx.y * a.tiles_per_split;
    const int t_end = t_begin + a.tiles_per_split < a.tiles ? t_begin + a.tiles_per_split : a.tiles, t_last = t_end - 1;
    const bool after_mix = a.out == (int)GemmOut::mix_gated && n0 >= a.mix_cols;
    const TA *ap = static_cast<const TA *>(after_mix ? a.a2 : a.a);
    const TB *bp = static_cast<const TB *>(a.b);

    floatx16 acc[TM][TN];
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++) acc[i][j] = matrix::zero_accumulator();

    typedef typename PieceOf<TA>::type PA;
    typedef typename PieceOf<TB>::type PB;
    PA pa0[XA], pa1[XA];   // even and odd tiles
    PB pb0[XB], pb1[XB];
    const TA *ar[XA];
    const TB *br[XB];
#pragma unroll
    for (int i = 0; i < XA; i++) {
        const int piece = tid + i * THREADS, row = m0 + piece / NCH;
        ar[i] = ap + (size_t)(row < a.m ? row : a.m - 1) * a.lda + (piece % NCH) * 8;   // rows past the end repeat the last one; never stored
    }
#pragma unroll
    for (int i = 0; i < XB; i++) {
        const int piece = tid + i * THREADS, row = n0 + piece / NCH;
        br[i] = bp + (size_t)(row < a.n ? row : a.n - 1) * a.ldb + (piece % NCH) * 8;
    }
    auto fetch = [&](PA (&pa)[XA], PB (&pb)[XB], int tile) {   // tiles past the end repeat the last one
        const size_t k = (size_t)(tile < t_last ? tile : t_last) * KT;
#pragma unroll
        for (int i = 0; i < XA; i++) pa[i] = fetch_piece(ar[i] + k);
#pragma unroll
        for (int i = 0; i < XB; i++) pb[i] = fetch_piece(br[i] + k);
    };
    auto stage = [&](const PA (&pa)[XA], const PB (&pb)[XB], int buf) {
#pragma unroll
        for (int i = 0; i < XA; i++) {
            const int piece = tid + i * THREADS;
            store_piece(pa[i], at[buf] + piece / NCH * LDK + (piece % NCH) * 8);
        }
#pragma unroll
        for (int i = 0; i < XB; i++) {
            const int piece = tid + i * THREADS;
            store_piece(pb[i], bt[buf] + piece / NCH * LDK + (piece % NCH) * 8);
        }
    };
    fetch(pa0, pb0, t_begin);
    fetch(pa1, pb1, t_begin + 1);
    stage(pa0, pb0, 0);
    fetch(pa0, pb0, t_begin + 2);
    __syncthreads();
    auto multiply = [&](int buf) {
#pragma unroll
        for (int ks = 0; ks < KT / 16; ks++) {
            const int kk = ks * 16 + 8 * (lane >> 5);
            typename Op<E>::frag af[TM], bf[TN];
#pragma unroll
            for (int i = 0; i < TM; i++) af[i] = Op<E>::load(at[buf] + ((wm * TM + i) * 32 + (lane & 31)) * LDK + kk);
#pragma unroll
            for (int j = 0; j < TN; j++) bf[j] = Op<E>::load(bt[buf] + ((wn * TN + j) * 32 + (lane & 31)) * LDK + kk);
#pragma unroll
            for (int i = 0; i < TM; i++)
#pragma unroll
                for (int j = 0; j < TN; j++) acc[i][j] = Op<E>::mma(af[i], bf[j], acc[i][j]);
        }
    };
    int t0 = t_begin;
    for (; t0 + 1 < t_end; t0 += 2) {
        multiply(0);
        stage(pa1, pb1, 1);
        fetch(pa1, pb1, t0 + 3);
        __syncthreads();
        multiply(1);
        stage(pa0, pb0, 0);
        fetch(pa0, pb0, t0 + 4);
        __syncthreads();
    }
    if (t0 < t_end) multiply(0);

    const int half = lane >> 5;
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++) {
            const int n = n0 + (wn * TN + j) * 32 + (lane & 31);
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int m = m0 + (wm * TM + i) * 32 + matrix::accumulator_row(r, half);
                const float v = acc[i][j][r];
                if (after_mix) {   // even lanes hold gates, their right neighbours the ups
                    const float up = __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, false));   // quad_perm [1,0,3,2]
                    if (!(lane & 1) && m < a.m && n < a.n)
                        static_cast<E *>(a.act)[(size_t)m * a.ld_act + (n - a.mix_cols) / 2] = Op<E>::from_float(matrix::gated(a.gate_function, v, up));
                    continue;
                }
                if (m >= a.m || n >= a.n) continue;
                if (a.out == (int)GemmOut::planes) static_cast<float *>(a.y)[((size_t)blockIdx.y * a.m + m) * a.ldy + n] = v;
                else if (a.out == (int)GemmOut::mix_gated) static_cast<float *>(a.y)[(size_t)m * a.ldy + n] = v;
                else if (a.out == (int)GemmOut::elems) static_cast<E *>(a.y)[(size_t)m * a.ldy + n] = Op<E>::from_float(v);
                else if (n < a.n_store) static_cast<float *>(a.y)[(size_t)m * a.ldy + n] = a.cap > 0.0f ? a.cap * tanhf(v / a.cap) : v;
            }
        }
}

struct TileShape { int bm, bn; };
// Tall tiles unless they leave compute units without one (a launch that may split k fills the chip that way instead).
TileShape tile_for(int m, int n, bool f32, bool splits) {
    if (m <= 32 && !f32) return TileShape{32, 128};
    if (m <= 64 || (!splits && ((m + 127) / 128) * ((n + 127) / 128) < 200)) return TileShape{64, 128};
    return TileShape{128, 128};
}
int ceil_div(int a, int b) { return (a + b - 1) / b; }

template <typename TA, typename TB>
hipError_t run(const DenseGemm &p, hipStream_t s) {
    constexpr bool f32 = std::is_same<TA, float>::value || std::is_same<TB, float>::value;
    constexpr int KT = f32 ? 32 : 64;
    const TileShape t = tile_for(p.m, p.n, f32, p.out == GemmOut::planes);
    DenseGemmArgs a{};
    a.a = p.a; a.a2 = p.a2; a.b = p.b; a.lda = p.lda; a.ldb = p.ldb; a.m = p.m; a.n = p.n;
    a.tiles = p.k / KT;
    a.tiles_per_split = ceil_div(a.tiles, p.splits);
    if ((p.splits - 1) * a.tiles_per_split >= a.tiles) return hipErrorInvalidValue;   // a split without work would leave its plane unwritten
    a.m_tiles = ceil_div(p.m, t.bm); a.n_tiles = ceil_div(p.n, t.bn);
    a.out = (int)p.out; a.y = p.y; a.ldy = p.ldy; a.mix_cols = p.mix_cols; a.act = p.act; a.ld_act = p.ld_act; a.gate_function = (int)p.gate_function; a.n_store = p.n_store; a.cap = p.cap;
    const dim3 grid(ceil_div(a.n_tiles, kDies) * kDies * a.m_tiles, p.splits);
    if constexpr (!f32) {
        if (t.bm == 32) {
            hipLaunchKernelGGL((dense_gemm_kernel<TA, TB, 1, 4, 1, 1>), grid, dim3(256), 0, s, a);
            return hipGetLastError();
        }
    }
    if (t.bm == 64) hipLaunchKernelGGL((dense_gemm_kernel<TA, TB, 2, 2, 1, 2>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((dense_gemm_kernel<TA, TB, 2, 2, 2, 2>), grid, dim3(256), 0, s, a);
    return hipGetLastError();
}

}  // namespace

// Enough workgroups for two per compute unit, at least four tiles of 64 per split, planes within the workspace.
int gemm_planes_splits(int m, int n, int k, size_t workspace_floats) {
    const TileShape t = tile_for(m, n, false, true);
    const int tiles = ceil_div(m, t.bm) * ceil_div(n, t.bn), k_tiles = k / 64;
    int splits = 1;
    for (int s = 2; s <= 16; s++) {
        const int per = ceil_div(k_tiles, s);
        if (tiles * s > 640 || per < 4 || (size_t)s * m * n > workspace_floats) break;
        if ((s - 1) * per < k_tiles) splits = s;
    }
    return splits;
}

hipError_t launch_dense_gemm(const DenseGemm &p, hipStream_t s) {
    const bool gated_only = p.out == GemmOut::mix_gated && p.mix_cols == 0;
    if (!p.a || !p.b || (!p.y && !gated_only) || p.m < 1 || p.n < 1 || p.k < 64 || p.k % 64 || p.splits < 1 || p.lda < p.k || p.ldb < p.k || p.lda % 8 || p.ldb % 8) return hipErrorInvalidValue;
    if (p.out != GemmOut::planes && p.splits != 1) return hipErrorInvalidValue;
    if (p.out == GemmOut::mix_gated && (p.mix_cols % 128 || p.n % 2 || (p.n > p.mix_cols && (!p.a2 || !p.act)))) return hipErrorInvalidValue;
    if (p.a_type == Precision::bf16 && p.b_type == Precision::bf16) return run<uint16_t, uint16_t>(p, s);
    if (p.a_type == Precision::f32 && p.b_type == Precision::bf16) return run<float, uint16_t>(p, s);
    if (p.a_type == Precision::bf16 && p.b_type == Precision::f32) return run<uint16_t, float>(p, s);
    return hipErrorInvalidValue;
}

}  // namespace esp
