// One-token products for dense weights, with the row work around them fused in: every workgroup forms the input row in
// LDS (fp32) in its prologue -- residual step and norm, the norm of a latent, the attention output -- and its waves
// then stream weight rows in pairs, 16 bytes per lane and load, eight loads of a pair in flight.  A row's sum is formed
// in an order that depends on the row's length only.
#include "dense_common.h"

namespace a81w41 {
namespace {

constexpr int kThreads = 256;

__device__ __forceinline__ float dot16(const uint4& w, const float* x, bf16*) {
    const float4 a = *reinterpret_cast<const float4*>(x), b = *reinterpret_cast<const float4*>(x + 4);
    float s = __uint_as_float(w.x << 16) * a.x;
    s = fmaf(__uint_as_float(w.x & 0xffff0000u), a.y, s);
    s = fmaf(__uint_as_float(w.y << 16), a.z, s);
    s = fmaf(__uint_as_float(w.y & 0xffff0000u), a.w, s);
    s = fmaf(__uint_as_float(w.z << 16), b.x, s);
    s = fmaf(__uint_as_float(w.z & 0xffff0000u), b.y, s);
    s = fmaf(__uint_as_float(w.w << 16), b.z, s);
    return fmaf(__uint_as_float(w.w & 0xffff0000u), b.w, s);
}
__device__ __forceinline__ float dot16(const uint4& w, const float* x, float*) {
    const float4 a = *reinterpret_cast<const float4*>(x);
    float s = __uint_as_float(w.x) * a.x;
    s = fmaf(__uint_as_float(w.y), a.y, s);
    s = fmaf(__uint_as_float(w.z), a.z, s);
    return fmaf(__uint_as_float(w.w), a.w, s);
}

// How rows are dealt: `lanes` lanes (a power of two) share a pair of rows; `group` counts the lane groups of the launch.
struct Deal {
    int lanes, group, groups, at;
};
template <typename T>
__device__ __forceinline__ Deal deal_rows(int chunks) {
    Deal d;
    d.lanes = 1;
    while (d.lanes < 64 && 2 * d.lanes <= chunks) d.lanes <<= 1;
    const int per_wg = kThreads / d.lanes;
    d.group = blockIdx.x * per_wg + threadIdx.x / d.lanes;
    d.groups = gridDim.x * per_wg;
    d.at = threadIdx.x & (d.lanes - 1);
    return d;
}

// The dot products of two weight rows with xs (LDS, zero-padded to whole chunks); every lane of the group gets both.
template <typename T>
__device__ __forceinline__ void two_row_dots(const T* w0, const T* w1, const float* xs, int chunks, const Deal& d, float& s0, float& s1) {
    constexpr int U = 4, E = 16 / (int)sizeof(T);
    const uint4* p0 = reinterpret_cast<const uint4*>(w0);
    const uint4* p1 = reinterpret_cast<const uint4*>(w1);
    s0 = s1 = 0.f;
    for (int c = d.at; c < chunks; c += U * d.lanes) {
        uint4 a[U], b[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int cc = min(c + u * d.lanes, chunks - 1);
            a[u] = p0[cc];
            b[u] = p1[cc];
        }
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int cc = c + u * d.lanes;
            if (cc < chunks) {
                s0 += dot16(a[u], xs + cc * E, static_cast<T*>(nullptr));
                s1 += dot16(b[u], xs + cc * E, static_cast<T*>(nullptr));
            }
        }
    }
    s0 = dense_wave_sum(s0, d.lanes);
    s1 = dense_wave_sum(s1, d.lanes);
}

// xs[0 .. padded) = f(i), zero from n on
template <typename F>
__device__ __forceinline__ void fill_row(float* xs, int n, int padded, F f) {
    for (int i = threadIdx.x; i < padded; i += kThreads) xs[i] = i < n ? f(i) : 0.f;
}

// The residual step and the norm of RowStep into xs; workgroup 0 of the launch also writes the stream.
template <typename T>
__device__ __forceinline__ void row_step(const RowStep& p, float* xs, int padded, float* inv, float* red) {
    const int t = threadIdx.x, W = p.width;
    const bool writer = blockIdx.x == 0 && blockIdx.y == 0;
    if (p.y) {
        group_inverse_rms<kThreads>([&](int i) { return p.y[i]; }, W, p.norm_y.groups, p.norm_y.eps, inv, red);
    }
    const float coef = p.before ? *p.coef : 0.f;
    const int size_y = p.y ? W / p.norm_y.groups : 1;
    for (int i = t; i < padded; i += kThreads) {
        float r = 0.f;
        if (i < W) {
            r = p.x[i];
            if (p.y) r += p.y[i] * inv[i / size_y] * p.norm_y.w[i];
            if (writer && p.state) p.state[i] = r;
            if (p.before) r = fmaf(coef, r, p.before[i]);
            if (writer && p.x_out) p.x_out[i] = r;
        }
        xs[i] = r;
    }
    __syncthreads();
    group_inverse_rms<kThreads>([&](int i) { return xs[i]; }, W, p.norm_h.groups, p.norm_h.eps, inv, red);
    const int size_h = W / p.norm_h.groups;
    for (int i = t; i < W; i += kThreads) xs[i] = xs[i] * inv[i / size_h] * p.norm_h.w[i];
    __syncthreads();
}

// C[n] = W[n] . row
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_step_kernel(RowStep p, const T* __restrict__ w, int ld, int N, float* __restrict__ C) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *xs = smem, *red = xs + ld, *inv = red + kThreads / 64;
    row_step<T>(p, xs, ld, inv, red);
    const int chunks = ld * (int)sizeof(T) / 16;
    const Deal d = deal_rows<T>(chunks);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        float s0, s1;
        two_row_dots<T>(w + (size_t)n * ld, w + (size_t)min(n + 1, N - 1) * ld, xs, chunks, d, s0, s1);
        if (d.at == 0) {
            C[n] = s0;
            if (n + 1 < N) C[n + 1] = s1;
        }
    }
}

// C[n] = W[n] . x
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_plain_kernel(const float* __restrict__ x, int K, const T* __restrict__ w, int ld, int N,
                                                             float* __restrict__ C) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    fill_row(smem, K, ld, [&](int i) { return x[i]; });
    __syncthreads();
    const int chunks = ld * (int)sizeof(T) / 16;
    const Deal d = deal_rows<T>(chunks);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        float s0, s1;
        two_row_dots<T>(w + (size_t)n * ld, w + (size_t)min(n + 1, N - 1) * ld, smem, chunks, d, s0, s1);
        if (d.at == 0) {
            C[n] = s0;
            if (n + 1 < N) C[n + 1] = s1;
        }
    }
}

// Queries from their normed latent.  The last workgroups of the launch do other work of the same stage: one appends the
// token's cache row, the others sum the states of the layers so far for the mean over depth.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_query_kernel(LatentRows in, LatentShape sh, const T* __restrict__ w, int ld, int N,
                                                             float* __restrict__ q, T* __restrict__ cache, DepthAverage depth,
                                                             int width, float* __restrict__ before, int main_groups) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *xs = smem, *red = xs + ld, *inv = red + kThreads / 64;
    const int t = threadIdx.x;
    if ((int)blockIdx.x >= main_groups) {
        int extra = blockIdx.x - main_groups;
        if (cache && extra-- == 0) {
            const float* c = in.down + sh.q_rank;
            group_inverse_rms<kThreads>([&](int i) { return c[i]; }, sh.rank, 1, in.eps, inv, red);
            const int p = min(max(in.pos_dev[0], 0), in.max_seq - 1);
            T* dst = cache + (size_t)p * sh.ld_cache;
            for (int i = t; i < sh.rank; i += kThreads) dst[i] = (T)(c[i] * inv[0] * in.kv_norm[i]);
            const int half = sh.rot >> 1;
            const float* k = c + sh.rank;
            for (int i = t; i < half; i += kThreads) {
                const float cs = in.cos_t[(size_t)p * half + i], sn = in.sin_t[(size_t)p * half + i];
                dst[sh.rank + i] = (T)(k[i] * cs - k[i + half] * sn);
                dst[sh.rank + half + i] = (T)(k[i + half] * cs + k[i] * sn);
            }
        } else {
            const int i = extra * kThreads + t;
            if (i < width) {
                float s = 0.f;
                for (int j = 0; j < depth.n; j++) s = fmaf(depth.coef[j], depth.states[j * depth.state_step + i], s);
                before[i] = s;
            }
        }
        return;
    }
    group_inverse_rms<kThreads>([&](int i) { return in.down[i]; }, sh.q_rank, 1, in.eps, inv, red);
    fill_row(xs, sh.q_rank, ld, [&](int i) { return in.down[i] * inv[0] * in.q_norm[i]; });
    __syncthreads();
    const int chunks = ld * (int)sizeof(T) / 16;
    Deal d = deal_rows<T>(chunks);
    d.groups = main_groups * (kThreads / d.lanes);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        float s0, s1;
        two_row_dots<T>(w + (size_t)n * ld, w + (size_t)min(n + 1, N - 1) * ld, xs, chunks, d, s0, s1);
        if (d.at == 0) {
            q[n] = s0;
            if (n + 1 < N) q[n + 1] = s1;
        }
    }
}

// Query rows in latent space, one head per blockIdx.y: columns 0..rank from the unrotated part through the transposed key
// up-projection, then the rotated part (first workgroup of the head).
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_absorb_kernel(const float* __restrict__ q, LatentRows in, LatentShape sh,
                                                              const T* __restrict__ uk_t, int ld, T* __restrict__ q_lat) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int h = blockIdx.y, half = sh.rot >> 1;
    const float* src = q + (size_t)h * (sh.dim + sh.rot);
    T* dst = q_lat + (size_t)h * sh.ld_cache;
    if (blockIdx.x == 0) {
        const int p = min(max(in.pos_dev[0], 0), in.max_seq - 1);
        for (int j = threadIdx.x; j < half; j += kThreads) {
            const float u = src[sh.dim + j], v = src[sh.dim + half + j];
            const float cs = in.cos_t[(size_t)p * half + j], sn = in.sin_t[(size_t)p * half + j];
            dst[sh.rank + j] = (T)(u * cs - v * sn);
            dst[sh.rank + half + j] = (T)(v * cs + u * sn);
        }
    }
    fill_row(smem, sh.dim, ld, [&](int i) { return src[i]; });
    __syncthreads();
    const T* w = uk_t + (size_t)h * sh.rank * ld;
    const int chunks = ld * (int)sizeof(T) / 16, N = sh.rank;
    const Deal d = deal_rows<T>(chunks);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        float s0, s1;
        two_row_dots<T>(w + (size_t)n * ld, w + (size_t)min(n + 1, N - 1) * ld, smem, chunks, d, s0, s1);
        if (d.at == 0) {
            dst[n] = (T)s0;
            if (n + 1 < N) dst[n + 1] = (T)s1;
        }
    }
}

// Values of a head (blockIdx.y) from its weighted latent, times the head's gate.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_values_kernel(const float* __restrict__ o_lat, int ld_o, LatentShape sh,
                                                              const T* __restrict__ uv, int ld, const float* __restrict__ gates,
                                                              float* __restrict__ attn) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int h = blockIdx.y;
    const float* src = o_lat + (size_t)h * ld_o;
    fill_row(smem, sh.rank, ld, [&](int i) { return src[i]; });
    __syncthreads();
    const T* w = uv + (size_t)h * sh.vdim * ld;
    const float gate = sigmoid(gates[h]);
    const int chunks = ld * (int)sizeof(T) / 16, N = sh.vdim;
    const Deal d = deal_rows<T>(chunks);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        float s0, s1;
        two_row_dots<T>(w + (size_t)n * ld, w + (size_t)min(n + 1, N - 1) * ld, smem, chunks, d, s0, s1);
        if (d.at == 0) {
            attn[(size_t)h * N + n] = s0 * gate;
            if (n + 1 < N) attn[(size_t)h * N + n + 1] = s1 * gate;
        }
    }
}

__device__ __forceinline__ int expert_of(const ExpertRows& e, int slot) {
    const int id = min(max(e.ids[0], 0), e.vocab - 1);
    return min(max(e.table[(size_t)id * e.top + slot], 0), e.experts - 1);
}

// act = silu(gate) * up for the token's experts (blockIdx.y < top) and the dense or shared feed-forward (the last).
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_gate_up_kernel(RowStep p, ExpertRows e, const T* __restrict__ experts,
                                                               const T* __restrict__ dense, int ld, float* __restrict__ act) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *xs = smem, *red = xs + ld, *inv = red + kThreads / 64;
    const int slot = blockIdx.y;
    const T* w = slot < e.top ? experts + (size_t)expert_of(e, slot) * e.pair_rows * ld : dense;
    const int ff = slot < e.top ? e.ff : e.dense_ff;
    row_step<T>(p, xs, ld, inv, red);
    const int chunks = ld * (int)sizeof(T) / 16;
    const Deal d = deal_rows<T>(chunks);
    float* dst = act + (size_t)slot * e.ld_act;
    for (int j = d.group; j < ff; j += d.groups) {
        const T* row = w + (size_t)((j >> 4) * 32 + (j & 15)) * ld;
        float gate, up;
        two_row_dots<T>(row, row + (size_t)16 * ld, xs, chunks, d, gate, up);
        if (d.at == 0) dst[j] = silu(gate) * up;
    }
}

// y[n] = mean over the token's experts of W_e[n] . act_e, plus the dense or shared feed-forward's.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_ff_down_kernel(ExpertRows e, const float* __restrict__ act, const T* __restrict__ experts,
                                                               int ld, const T* __restrict__ dense, int ld_dense, int N,
                                                               float* __restrict__ y) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ int chosen[64];
    for (int k = 0; k < e.top; k++) fill_row(smem + k * ld, e.ff, ld, [&](int i) { return act[(size_t)k * e.ld_act + i]; });
    float* xs_dense = smem + e.top * ld;
    if (e.dense_ff) fill_row(xs_dense, e.dense_ff, ld_dense, [&](int i) { return act[(size_t)e.top * e.ld_act + i]; });
    if ((int)threadIdx.x < e.top) chosen[threadIdx.x] = expert_of(e, threadIdx.x);
    __syncthreads();
    const int chunks = ld * (int)sizeof(T) / 16, chunks_dense = ld_dense * (int)sizeof(T) / 16;
    const Deal d = deal_rows<T>(e.dense_ff ? chunks_dense : chunks);
    const float share = 1.0f / (float)max(e.top, 1);
    for (int n = 2 * d.group; n < N; n += 2 * d.groups) {
        const int n1 = min(n + 1, N - 1);
        float a0 = 0.f, a1 = 0.f, s0, s1;
        for (int k = 0; k < e.top; k++) {
            const T* w = experts + (size_t)chosen[k] * N * ld;
            two_row_dots<T>(w + (size_t)n * ld, w + (size_t)n1 * ld, smem + k * ld, chunks, d, s0, s1);
            a0 += s0;
            a1 += s1;
        }
        a0 *= share;
        a1 *= share;
        if (e.dense_ff) {
            two_row_dots<T>(dense + (size_t)n * ld_dense, dense + (size_t)n1 * ld_dense, xs_dense, chunks_dense, d, s0, s1);
            a0 += s0;
            a1 += s1;
        }
        if (d.at == 0) {
            y[n] = a0;
            if (n + 1 < N) y[n + 1] = a1;
        }
    }
}

// Workgroups for N rows of `ld` elements: a pair of rows per lane group and turn, at most `limit`.
template <typename T>
int workgroups(int N, int ld, int limit) {
    const int chunks = ld * (int)sizeof(T) / 16;
    int lanes = 1;
    while (lanes < 64 && 2 * lanes <= chunks) lanes <<= 1;
    const int per_wg = 2 * (kThreads / lanes), n = (N + per_wg - 1) / per_wg;
    return n < 1 ? 1 : n > limit ? limit : n;
}
constexpr int kMaxGrid = 1024;

size_t step_lds(int ld, const RowStep& p) {
    const int groups = p.norm_y.groups > p.norm_h.groups ? p.norm_y.groups : p.norm_h.groups;
    return (ld + kThreads / 64 + groups) * sizeof(float);
}

}  // namespace

template <typename T>
hipError_t launch_gemv_step(const RowStep& p, const T* w, int ld, int N, float* C, hipStream_t s) {
    hipLaunchKernelGGL(gemv_step_kernel<T>, dim3(workgroups<T>(N, ld, kMaxGrid)), dim3(kThreads), step_lds(ld, p), s, p, w, ld, N, C);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_plain(const float* x, int K, const T* w, int ld, int N, float* C, hipStream_t s) {
    hipLaunchKernelGGL(gemv_plain_kernel<T>, dim3(workgroups<T>(N, ld, kMaxGrid)), dim3(kThreads), ld * sizeof(float), s, x, K, w, ld, N, C);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_query(const LatentRows& in, const LatentShape& sh, const T* w, int ld, float* q, T* cache, const DepthAverage& depth,
                             int width, float* before, hipStream_t s) {
    const int N = sh.heads * (sh.dim + sh.rot), main_groups = workgroups<T>(N, ld, kMaxGrid);
    const int extra = (cache ? 1 : 0) + (width + kThreads - 1) / kThreads;
    hipLaunchKernelGGL(gemv_query_kernel<T>, dim3(main_groups + extra), dim3(kThreads), (ld + kThreads / 64 + 1) * sizeof(float), s, in, sh,
                       w, ld, N, q, cache, depth, width, before, main_groups);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_absorb(const float* q, const LatentRows& in, const LatentShape& sh, const T* uk_t, int ld, T* q_lat, hipStream_t s) {
    hipLaunchKernelGGL(gemv_absorb_kernel<T>, dim3(workgroups<T>(sh.rank, ld, 64), sh.heads), dim3(kThreads), ld * sizeof(float), s, q, in,
                       sh, uk_t, ld, q_lat);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_values(const float* o_lat, int ld_o, const LatentShape& sh, const T* uv, int ld, const float* gates, float* attn,
                              hipStream_t s) {
    hipLaunchKernelGGL(gemv_values_kernel<T>, dim3(workgroups<T>(sh.vdim, ld, 64), sh.heads), dim3(kThreads), ld * sizeof(float), s, o_lat,
                       ld_o, sh, uv, ld, gates, attn);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_gate_up(const RowStep& p, const ExpertRows& e, const T* experts, const T* dense, int ld, float* act, hipStream_t s) {
    const int most = e.top && e.ff > e.dense_ff ? e.ff : e.dense_ff;
    const int slots = e.top + (e.dense_ff ? 1 : 0);
    hipLaunchKernelGGL(gemv_gate_up_kernel<T>, dim3(workgroups<T>(2 * most, ld, kMaxGrid), slots), dim3(kThreads), step_lds(ld, p), s, p, e,
                       experts, dense, ld, act);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_ff_down(const ExpertRows& e, const float* act, const T* experts, int ld, const T* dense, int ld_dense, int N,
                               float* y, hipStream_t s) {
    const size_t lds = ((size_t)e.top * ld + (e.dense_ff ? ld_dense : 0)) * sizeof(float);
    hipLaunchKernelGGL(gemv_ff_down_kernel<T>, dim3(workgroups<T>(N, e.dense_ff ? ld_dense : ld, kMaxGrid)), dim3(kThreads), lds, s, e, act,
                       experts, ld, dense, ld_dense, N, y);
    return hipGetLastError();
}

#define INSTANTIATE(T)                                                                                                            \
    template hipError_t launch_gemv_step<T>(const RowStep&, const T*, int, int, float*, hipStream_t);                              \
    template hipError_t launch_gemv_plain<T>(const float*, int, const T*, int, int, float*, hipStream_t);                          \
    template hipError_t launch_gemv_query<T>(const LatentRows&, const LatentShape&, const T*, int, float*, T*, const DepthAverage&, \
                                             int, float*, hipStream_t);                                                           \
    template hipError_t launch_gemv_absorb<T>(const float*, const LatentRows&, const LatentShape&, const T*, int, T*, hipStream_t); \
    template hipError_t launch_gemv_values<T>(const float*, int, const LatentShape&, const T*, int, const float*, float*,          \
                                              hipStream_t);                                                                       \
    template hipError_t launch_gemv_gate_up<T>(const RowStep&, const ExpertRows&, const T*, const T*, int, float*, hipStream_t);   \
    template hipError_t launch_gemv_ff_down<T>(const ExpertRows&, const float*, const T*, int, const T*, int, int, float*,         \
                                               hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
