// C = A W^T on the matrix cores for weights in bfloat16 (v_mfma_f32_32x32x16_bf16) or float
// (v_mfma_f32_32x32x2_f32: true 32-bit products and sums).
//
// A workgroup of four waves takes a BM x BN tile, a wave a quarter of it in 32 x 32 pieces.  K goes in steps of
// 128 bytes per row; a step's rows are copied global -> LDS by direct 16-byte loads, two stages, the next step's
// copies in flight while the current one is multiplied.  In LDS chunk c of row r sits at place c ^ (r & 7), so that
// the 32 rows a wave reads at one chunk column spread over the banks.  A fragment is the same 16 bytes per lane for
// both types: lane l holds row l & 31, chunk 2 kk + (l >> 5).
#include "dense_common.h"

namespace a81w41 {
namespace {

__device__ __forceinline__ void mma(f32x16& acc, const uint4& a, const uint4& b, bf16*) {
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(&a), *reinterpret_cast<const bf16x8*>(&b), acc, 0, 0, 0);
}
__device__ __forceinline__ void mma(f32x16& acc, const uint4& a, const uint4& b, float*) {
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(__uint_as_float(a.x), __uint_as_float(b.x), acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(__uint_as_float(a.y), __uint_as_float(b.y), acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(__uint_as_float(a.z), __uint_as_float(b.z), acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(__uint_as_float(a.w), __uint_as_float(b.w), acc, 0, 0, 0);
}

struct NoHeads {};

// X: HeadRows<T> with the epilogue kHeads, NoHeads with the others
template <typename T, int BM, int BN, Epilogue EPI, typename X>
__global__ __launch_bounds__(256, 2) void dense_gemm_kernel(GemmArgs g, X heads) {
    constexpr int WM = BM / 2, WN = BN / 2, FM = WM / 32, FN = WN / 32;
    constexpr int LA = BM / 32, LB = BN / 32;  // direct copies per thread and stage
    constexpr int kStage = (BM + BN) * 128;
    __shared__ __attribute__((aligned(128))) uint8_t lds[2 * kStage];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int l31 = lane & 31, half = lane >> 5;
    // Tiles in the order (column panel, row tile), dealt to the XCDs in contiguous runs: a panel's weights then come
    // into one L2.
    const int n_nt = (g.N + BN - 1) / BN, n_mt = gridDim.x / n_nt;
    const int q = gridDim.x >> 3, r8 = gridDim.x & 7, xcd = blockIdx.x & 7, idx = blockIdx.x >> 3;
    const int t = xcd < r8 ? xcd * (q + 1) + idx : r8 * (q + 1) + (xcd - r8) * q + idx;
    const int mt = t % n_mt, nt = t / n_mt;
    int m0 = mt * BM, rows = g.M - m0;
    long long batch = blockIdx.y;
    if (g.tiles) {
        if (mt >= *g.n_tiles) return;
        const GroupTile gt = g.tiles[mt];
        m0 = gt.row0;
        rows = gt.rows;
        batch = gt.expert;
    }
    const int n0 = nt * BN;
    const uint8_t* A = reinterpret_cast<const uint8_t*>(static_cast<const T*>(g.A) + (g.tiles ? 0 : batch * g.a_step));
    const uint8_t* W = reinterpret_cast<const uint8_t*>(static_cast<const T*>(g.W) + batch * g.w_step);
    const uint8_t *a_src[LA], *b_src[LB];
#pragma unroll
    for (int i = 0; i < LA; i++) {
        const int c = i * 256 + tid, r = c >> 3;
        int row = m0 + min(r, rows - 1);
        if (g.a_rows) row = g.a_rows[row];
        a_src[i] = A + (size_t)row * g.lda * sizeof(T) + (((c & 7) ^ (r & 7)) << 4);
    }
#pragma unroll
    for (int i = 0; i < LB; i++) {
        const int c = i * 256 + tid, r = c >> 3;
        b_src[i] = W + (size_t)min(n0 + r, g.N - 1) * g.ldw * sizeof(T) + (((c & 7) ^ (r & 7)) << 4);
    }
    auto copy_step = [&](int step, int stage) {
        uint8_t* base = lds + stage * kStage + wave * 1024;
#pragma unroll
        for (int i = 0; i < LA; i++) copy16_to_lds(a_src[i] + (size_t)step * 128, base + i * 4096);
#pragma unroll
        for (int i = 0; i < LB; i++) copy16_to_lds(b_src[i] + (size_t)step * 128, base + BM * 128 + i * 4096);
    };
    f32x16 acc[FM][FN];
#pragma unroll
    for (int i = 0; i < FM; i++)
#pragma unroll
        for (int j = 0; j < FN; j++)
#pragma unroll
            for (int v = 0; v < 16; v++) acc[i][j][v] = 0.f;
    const int wm = (wave & 1) * WM, wn = (wave >> 1) * WN;
    const int n_steps = g.K * (int)sizeof(T) / 128;
    copy_step(0, 0);
    for (int step = 0; step < n_steps; step++) {
        // this wave's copies of the step are in LDS, then everybody's; and nobody still reads the other stage
        __builtin_amdgcn_s_waitcnt(0x0070);
        __syncthreads();
        if (step + 1 < n_steps) copy_step(step + 1, (step + 1) & 1);
        const uint8_t* sa = lds + (step & 1) * kStage;
        const uint8_t* sb = sa + BM * 128;
#pragma unroll
        for (int kk = 0; kk < 4; kk++) {
            uint4 a[FM], b[FN];
#pragma unroll
            for (int i = 0; i < FM; i++) {
                const int r = wm + i * 32 + l31;
                a[i] = *reinterpret_cast<const uint4*>(sa + r * 128 + (((2 * kk + half) ^ (r & 7)) << 4));
            }
#pragma unroll
            for (int j = 0; j < FN; j++) {
                const int r = wn + j * 32 + l31;
                b[j] = *reinterpret_cast<const uint4*>(sb + r * 128 + (((2 * kk + half) ^ (r & 7)) << 4));
            }
#pragma unroll
            for (int i = 0; i < FM; i++)
#pragma unroll
                for (int j = 0; j < FN; j++) mma(acc[i][j], a[i], b[j], static_cast<T*>(nullptr));
        }
    }
    [[maybe_unused]] int pos = 0;
    if constexpr (EPI == Epilogue::kHeads) pos = min(max(heads.pos_dev[0], 0), heads.max_seq - 1);
    // register v of lane l holds row 8 (v / 4) + 4 (l / 32) + v % 4, column l % 32 of a piece
#pragma unroll
    for (int i = 0; i < FM; i++)
#pragma unroll
        for (int j = 0; j < FN; j++) {
            const int col = n0 + wn + j * 32 + l31;
#pragma unroll
            for (int v = 0; v < 16; v++) {
                const int r = wm + i * 32 + 8 * (v >> 2) + 4 * half + (v & 3);
                const size_t row = m0 + r;
                if constexpr (EPI == Epilogue::kGatedPair) {
                    const float up = __shfl_xor(acc[i][j][v], 16, 64);
                    if (r < rows && col < g.N && !(lane & 16))
                        static_cast<T*>(g.C)[row * g.ldc + (col >> 5) * 16 + (col & 15)] = (T)gated_unit(g.unit, acc[i][j][v], up);
                } else if constexpr (EPI == Epilogue::kHeads) {
                    const float other = __shfl_xor(acc[i][j][v], 1, 64);
                    if (r < rows && col < g.N) store_head_column(heads, pos, (int)row, col, acc[i][j][v], other);
                } else if (r < rows && col < g.N) {
                    if constexpr (EPI == Epilogue::kFloat) {
                        (static_cast<float*>(g.C) + (g.tiles ? 0 : batch * g.c_step))[row * g.ldc + col] = acc[i][j][v];
                    } else {
                        float f = acc[i][j][v];
                        if constexpr (EPI == Epilogue::kHeadGate) f *= sigmoid(g.head_gate[row * g.ld_gate + batch]);
                        (static_cast<T*>(g.C) + (g.tiles ? 0 : batch * g.c_step))[row * g.ldc + col] = (T)f;
                    }
                }
            }
        }
}

template <typename T, int BM, int BN, Epilogue EPI, typename X>
hipError_t launch_kernel(const GemmArgs& g, const X& heads, hipStream_t s) {
    const int n_mt = g.tiles ? g.max_tiles : (g.M + BM - 1) / BM, n_nt = (g.N + BN - 1) / BN;
    hipLaunchKernelGGL((dense_gemm_kernel<T, BM, BN, EPI, X>), dim3(n_mt * n_nt, g.batches), dim3(256), 0, s, g, heads);
    return hipGetLastError();
}

template <typename T, Epilogue EPI, typename X>
hipError_t launch_by_size(const GemmArgs& g, const X& heads, hipStream_t s) {
    // large tiles where they still give every CU work; a grouped product's row tiles are kGroupTileRows high
    const long long big = (long long)((g.M + 127) / 128) * ((g.N + 127) / 128) * g.batches;
    if (!g.tiles && g.M > 64 && big >= 192) return launch_kernel<T, 128, 128, EPI>(g, heads, s);
    if (g.tiles && g.N >= 1024) return launch_kernel<T, kGroupTileRows, 128, EPI>(g, heads, s);
    return launch_kernel<T, 64, 64, EPI>(g, heads, s);
}

}  // namespace

template <typename T>
hipError_t launch_dense_gemm(const GemmArgs& g, Epilogue epi, hipStream_t s) {
    switch (epi) {
        case Epilogue::kFloat: return launch_by_size<T, Epilogue::kFloat>(g, NoHeads{}, s);
        case Epilogue::kElement: return launch_by_size<T, Epilogue::kElement>(g, NoHeads{}, s);
        case Epilogue::kGatedPair: return launch_by_size<T, Epilogue::kGatedPair>(g, NoHeads{}, s);
        case Epilogue::kHeadGate: return launch_by_size<T, Epilogue::kHeadGate>(g, NoHeads{}, s);
        case Epilogue::kHeads: break;  // has a launcher of its own
    }
    return hipErrorInvalidValue;
}
template <typename T>
hipError_t launch_dense_gemm_heads(const GemmArgs& g, const HeadRows<T>& heads, hipStream_t s) {
    return launch_by_size<T, Epilogue::kHeads>(g, heads, s);
}
#define INSTANTIATE(T)                                                              \
    template hipError_t launch_dense_gemm<T>(const GemmArgs&, Epilogue, hipStream_t); \
    template hipError_t launch_dense_gemm_heads<T>(const GemmArgs&, const HeadRows<T>&, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
