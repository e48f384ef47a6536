// Row kernels around the dense matrix products: norms in groups, the residual step between two norms with an
// optional weighted mean over depth, the choice of experts by a router, and the sorting of tokens by expert.  One workgroup
// per row; the row sits in LDS as fp32.
#include "dense_common.h"

namespace a81w41 {
namespace {

constexpr int kThreads = 256;

template <typename T>
__global__ __launch_bounds__(kThreads) void group_norm_kernel(const float* __restrict__ x, int width, GroupNorm norm, T* __restrict__ out,
                                                             int ld_out) {
    extern __shared__ float smem[];
    float* inv = smem;
    float* red = inv + norm.groups;
    const float* row = x + (size_t)blockIdx.x * width;
    group_inverse_rms<kThreads>([&](int i) { return row[i]; }, width, norm.groups, norm.eps, inv, red);
    const int size = width / norm.groups;
    T* dst = out + (size_t)blockIdx.x * ld_out;
    for (int i = threadIdx.x; i < width; i += kThreads) dst[i] = (T)(row[i] * inv[i / size] * norm.w[i]);
}

// Any sizes.
template <typename T>
__global__ __launch_bounds__(kThreads) void residual_norm_any_kernel(const float* x, SublayerOut y, GroupNorm norm_y, DepthAverage depth,
                                                                float* x_out, GroupNorm norm_h, T* __restrict__ h, int ld_h,
                                                                int width, const float* __restrict__ add) {
    extern __shared__ float smem[];
    float* v = smem;
    float* inv = v + width;
    float* red = inv + max(norm_y.groups, norm_h.groups);
    const size_t m = blockIdx.x, base = m * width;
    const int t = threadIdx.x;
    if (y.y) {
        const float share = y.slot_rows ? 1.0f / (float)y.top : 0.f;
        for (int i = t; i < width; i += kThreads) {
            float s;
            if (y.slot_rows) {
                s = 0.f;
                for (int k = 0; k < y.top; k++) {
                    const float w = y.weights ? y.weights[m * y.top + k] : share;
                    s = fmaf(w, y.y[(size_t)y.slot_rows[m * y.top + k] * width + i], s);
                }
                if (y.shared) s += y.shared[base + i];
            } else {
                s = y.y[base + i];
            }
            v[i] = s;
        }
        __syncthreads();
        if (norm_y.w) group_inverse_rms<kThreads>([&](int i) { return v[i]; }, width, norm_y.groups, norm_y.eps, inv, red);
    }
    const int size_y = width / max(norm_y.groups, 1);
    for (int i = t; i < width; i += kThreads) {  // every element of v is read and written by the same thread from here on
        float r = x[base + i];
        if (y.y) r = norm_y.w ? r + v[i] * inv[i / size_y] * norm_y.w[i] : fmaf(norm_y.scale, v[i], r);
        if (depth.states) depth.states[depth.n * depth.state_step + base + i] = r;
        if (depth.coef) {
            float s = 0.f;
            for (int j = 0; j < depth.n; j++) s = fmaf(depth.coef[j], depth.states[j * depth.state_step + base + i], s);
            r = fmaf(depth.coef[depth.n], r, s);
        }
        if (add) r += add[i];
        x_out[base + i] = r;
        v[i] = r;
    }
    __syncthreads();
    group_inverse_rms<kThreads>([&](int i) { return v[i]; }, width, norm_h.groups, norm_h.eps, inv, red);
    const int size_h = width / norm_h.groups;
    T* dst = h + m * ld_h;
    for (int i = t; i < width; i += kThreads) dst[i] = (T)(v[i] * inv[i / size_h] * norm_h.w[i]);
}

// The same for rows that RowParts can hold: every operand is read once, sixteen bytes at a time, and the row stays in
// registers between the two norms.
template <typename T>
__global__ __launch_bounds__(kThreads) void residual_norm_kernel(const float* x, SublayerOut y, GroupNorm norm_y, DepthAverage depth,
                                                                float* x_out, GroupNorm norm_h, T* __restrict__ h, int ld_h,
                                                                int width, const float* __restrict__ add) {
    constexpr int P = RowParts<kThreads>::kParts;
    __shared__ float red[kThreads / 64];
    const RowParts<kThreads> parts(width, norm_h.groups);
    const size_t m = blockIdx.x, base = m * width;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 r[P], v[P];
#pragma unroll
    for (int k = 0; k < P; k++) {
        const int i = parts.place(k);
        r[k] = i >= 0 ? load4(x + base + i) : zero;
        v[k] = zero;
        if (i < 0 || !y.y) continue;
        if (y.slot_rows) {
            const float share = 1.0f / (float)y.top;
            if (y.shared) v[k] = load4(y.shared + base + i);
            for (int s = 0; s < y.top; s++)
                v[k] = fma4(y.weights ? y.weights[m * y.top + s] : share, load4(y.y + (size_t)y.slot_rows[m * y.top + s] * width + i), v[k]);
        } else {
            v[k] = load4(y.y + base + i);
        }
    }
    if (y.y && norm_y.w) {
        const float inv = parts.inverse_rms(v, norm_y.eps, red);
#pragma unroll
        for (int k = 0; k < P; k++) {
            const int i = parts.place(k);
            if (i >= 0) r[k] = add4(r[k], scale4(v[k], inv, load4(norm_y.w + i)));
        }
    } else if (y.y) {
#pragma unroll
        for (int k = 0; k < P; k++) r[k] = fma4(norm_y.scale, v[k], r[k]);
    }
    if (depth.states) {
#pragma unroll
        for (int k = 0; k < P; k++) {
            const int i = parts.place(k);
            v[k] = zero;
            if (i < 0) continue;
            store4(depth.states + depth.n * depth.state_step + base + i, r[k]);
            if (!depth.coef) continue;
            const float* st = depth.states + base + i;
            int j = 0;
            for (; j + 4 <= depth.n; j += 4) {
                float4 a[4];
#pragma unroll
                for (int u = 0; u < 4; u++) a[u] = load4(st + (j + u) * depth.state_step);
#pragma unroll
                for (int u = 0; u < 4; u++) v[k] = fma4(depth.coef[j + u], a[u], v[k]);
            }
            for (; j < depth.n; j++) v[k] = fma4(depth.coef[j], load4(st + j * depth.state_step), v[k]);
            r[k] = fma4(depth.coef[depth.n], r[k], v[k]);
        }
    }
#pragma unroll
    for (int k = 0; k < P; k++) {
        const int i = parts.place(k);
        if (i < 0) continue;
        if (add) r[k] = add4(r[k], load4(add + i));
        store4(x_out + base + i, r[k]);
    }
    const float inv = parts.inverse_rms(r, norm_h.eps, red);
#pragma unroll
    for (int k = 0; k < P; k++) {
        const int i = parts.place(k);
        if (i < 0) continue;
        const float4 o = scale4(r[k], inv, load4(norm_h.w + i));
        T* dst = h + m * ld_h + i;  // i and the row stride are multiples of 4
        alignas(16) T packed[4] = {(T)o.x, (T)o.y, (T)o.z, (T)o.w};
        if constexpr (sizeof(T) == 2)
            *reinterpret_cast<uint2*>(dst) = *reinterpret_cast<const uint2*>(packed);
        else
            *reinterpret_cast<uint4*>(dst) = *reinterpret_cast<const uint4*>(packed);
    }
}

// Exclusive prefix sum of a[0..n) in place, total returned to every thread; 1024 threads, tmp: 16 ints of LDS.
__device__ int block_exclusive_scan(int* a, int n, int* tmp) {
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    int carry = 0;
    for (int base = 0; base < n; base += 1024) {
        const int own = base + t < n ? a[base + t] : 0;
        int upto = own;
        for (int off = 1; off < 64; off <<= 1) {
            const int add = __shfl_up(upto, off, 64);
            if (lane >= off) upto += add;
        }
        if (lane == 63) tmp[wave] = upto;
        __syncthreads();
        int before = 0, all = 0;
        for (int w = 0; w < 16; w++) {
            if (w < wave) before += tmp[w];
            all += tmp[w];
        }
        if (base + t < n) a[base + t] = carry + before + upto - own;
        carry += all;
        __syncthreads();
    }
    return carry;
}

// One wave per token.  An expert's rank is the number of experts before it; ranks below `top` are the choice.  A row of
// logits sits in LDS.
constexpr int kRouterWaves = 4;
__global__ __launch_bounds__(64 * kRouterWaves) void router_kernel(const float* __restrict__ logits, int ld, const float* __restrict__ bias,
                                                                  int experts, int top, int M, int* __restrict__ chosen,
                                                                  float* __restrict__ weights) {
    extern __shared__ float smem[];
    __shared__ float best[kRouterWaves][kMaxTop];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = blockIdx.x * kRouterWaves + wave;
    float* z = smem + wave * experts;
    const bool real = m < M;
    if (real)
        for (int e = lane; e < experts; e += 64) z[e] = logits[(size_t)m * ld + e] + bias[e];
    __syncthreads();
    if (real)
        for (int e = lane; e < experts; e += 64) {
            const int rank = expert_rank(z, experts, e);
            if (rank < top) {
                chosen[(size_t)m * top + rank] = e;
                best[wave][rank] = z[e];
            }
        }
    __syncthreads();
    if (!real) return;
    const float w = lane < top ? expf(best[wave][lane] - best[wave][0]) : 0.f, sum = dense_wave_sum(w);
    if (lane < top) weights[(size_t)m * top + lane] = w / sum;
}
static_assert(kMaxTop <= 64, "one weight per lane");

__global__ __launch_bounds__(1024) void expert_rows_kernel(const int* __restrict__ ids, const int* __restrict__ table, int vocab,
                                                         int top, int experts, int M, int* __restrict__ src_rows,
                                                         int* __restrict__ slot_rows, GroupTile* __restrict__ tiles,
                                                         int* __restrict__ n_tiles) {
    extern __shared__ int cnt[];  // [experts] counts, [experts] first rows, [experts] first tiles, [16]
    int *first = cnt + experts, *tile0 = first + experts, *tmp = tile0 + experts;
    const int t = threadIdx.x, total = M * top;
    for (int e = t; e < experts; e += 1024) cnt[e] = 0;
    __syncthreads();
    auto expert_of = [&](int i) {
        if (!ids) return min(max(table[i], 0), experts - 1);
        const int id = min(max(ids[i / top], 0), vocab - 1);
        return min(max(table[(size_t)id * top + i % top], 0), experts - 1);
    };
    constexpr int U = 4;
    for (int i0 = t; i0 < total; i0 += U * 1024) {  // slot_rows keeps the expert until the row is known
        int e[U];
#pragma unroll
        for (int u = 0; u < U; u++) e[u] = i0 + u * 1024 < total ? expert_of(i0 + u * 1024) : 0;
#pragma unroll
        for (int u = 0; u < U; u++)
            if (i0 + u * 1024 < total) {
                slot_rows[i0 + u * 1024] = e[u];
                atomicAdd(&cnt[e[u]], 1);
            }
    }
    __syncthreads();
    for (int e = t; e < experts; e += 1024) {
        first[e] = cnt[e];
        tile0[e] = (cnt[e] + kGroupTileRows - 1) / kGroupTileRows;
    }
    __syncthreads();
    block_exclusive_scan(first, experts, tmp);
    const int all_tiles = block_exclusive_scan(tile0, experts, tmp);
    if (t == 0) *n_tiles = all_tiles;
    for (int e = t; e < experts; e += 1024) {
        const int n = cnt[e];
        for (int k = 0; k * kGroupTileRows < n; k++)
            tiles[tile0[e] + k] = GroupTile{e, first[e] + k * kGroupTileRows, min(kGroupTileRows, n - k * kGroupTileRows)};
    }
    __syncthreads();
    // where a token's row lands among its expert's rows does not matter: a row's result does not depend on its place
    for (int i0 = t; i0 < total; i0 += U * 1024) {
        int e[U];
#pragma unroll
        for (int u = 0; u < U; u++) e[u] = i0 + u * 1024 < total ? slot_rows[i0 + u * 1024] : 0;
#pragma unroll
        for (int u = 0; u < U; u++)
            if (i0 + u * 1024 < total) {
                const int r = atomicAdd(&first[e[u]], 1);
                src_rows[r] = (i0 + u * 1024) / top;
                slot_rows[i0 + u * 1024] = r;
            }
    }
}

}  // namespace

template <typename T>
hipError_t launch_group_norm(const float* x, int M, int width, const GroupNorm& norm, T* out, int ld_out, hipStream_t s) {
    const size_t lds = (norm.groups + kThreads / 64) * sizeof(float);
    hipLaunchKernelGGL(group_norm_kernel<T>, dim3(M), dim3(kThreads), lds, s, x, width, norm, out, ld_out);
    return hipGetLastError();
}

template <typename T>
hipError_t launch_residual_norm(const float* x, const SublayerOut& y, const GroupNorm& norm_y, const DepthAverage& depth, float* x_out,
                                const GroupNorm& norm_h, T* h, int ld_h, int M, int width, hipStream_t s, const float* add) {
    const int groups = norm_y.groups > norm_h.groups ? norm_y.groups : norm_h.groups;
    int per = 1;  // what RowParts holds
    while (per < norm_h.groups && per < kThreads) per <<= 1;
    const int size = width / norm_h.groups;
    if ((!y.y || !norm_y.w || norm_y.groups == norm_h.groups) && norm_h.groups <= kThreads && size % 4 == 0 &&
        size / 4 <= RowParts<kThreads>::kParts * (kThreads / per)) {
        hipLaunchKernelGGL(residual_norm_kernel<T>, dim3(M), dim3(kThreads), 0, s, x, y, norm_y, depth, x_out, norm_h, h, ld_h, width, add);
    } else {
        const size_t lds = (width + groups + kThreads / 64) * sizeof(float);
        hipLaunchKernelGGL(residual_norm_any_kernel<T>, dim3(M), dim3(kThreads), lds, s, x, y, norm_y, depth, x_out, norm_h, h, ld_h, width, add);
    }
    return hipGetLastError();
}

hipError_t launch_router(const float* logits, int ld, const float* bias, int experts, int top, int M, int* chosen, float* weights,
                         hipStream_t s) {
    hipLaunchKernelGGL(router_kernel, dim3((M + kRouterWaves - 1) / kRouterWaves), dim3(64 * kRouterWaves),
                       (size_t)kRouterWaves * experts * sizeof(float), s, logits, ld, bias, experts, top, M, chosen, weights);
    return hipGetLastError();
}

hipError_t launch_expert_rows(const int* ids, const int* table, int vocab, int top, int experts, int M, int* src_rows,
                              int* slot_rows, GroupTile* tiles, int* n_tiles, hipStream_t s) {
    const size_t lds = (3 * (size_t)experts + 16) * sizeof(int);
    hipLaunchKernelGGL(expert_rows_kernel, dim3(1), dim3(1024), lds, s, ids, table, vocab, top, experts, M, src_rows, slot_rows,
                       tiles, n_tiles);
    return hipGetLastError();
}

#define INSTANTIATE(T)                                                                                                          \
    template hipError_t launch_group_norm<T>(const float*, int, int, const GroupNorm&, T*, int, hipStream_t);                     \
    template hipError_t launch_residual_norm<T>(const float*, const SublayerOut&, const GroupNorm&, const DepthAverage&, float*, \
                                                const GroupNorm&, T*, int, int, int, hipStream_t, const float*);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
