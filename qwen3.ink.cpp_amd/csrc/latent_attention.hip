// Latent attention: per token the cache holds one normed latent and one rotated key part, shared by all heads.  A
// head's unrotated key is W_uk c, so q . (W_uk c) = (W_uk^T q) . c: with the up-projection moved into the query, a
// query row has the layout of a cache row and the score is one dot product; the value is W_uv sum_j p_j c_j.
// Positions come from device memory; every index that depends on them is clamped into its array.
#include "dense_common.h"

namespace a81w41 {
namespace {

constexpr int kThreads = 256;

// One workgroup per token.
template <typename T>
__global__ __launch_bounds__(kThreads) void latent_rows_kernel(LatentRows in, LatentShape sh, T* __restrict__ q_latent, int ld_q,
                                                              T* __restrict__ cache) {
    __shared__ float inv[2], red[kThreads / 64];
    const int m = blockIdx.x, t = threadIdx.x;
    const float* row = in.down + (size_t)m * in.ld_down;
    group_inverse_rms<kThreads>([&](int i) { return row[i]; }, sh.q_rank, 1, in.eps, inv, red);
    for (int i = t; i < sh.q_rank; i += kThreads) q_latent[(size_t)m * ld_q + i] = (T)(row[i] * inv[0] * in.q_norm[i]);
    if (!cache) return;
    const float* c = row + sh.q_rank;
    group_inverse_rms<kThreads>([&](int i) { return c[i]; }, sh.rank, 1, in.eps, inv + 1, red);
    const int p = min(max(in.pos_dev[0] + m, 0), in.max_seq - 1);
    T* dst = cache + (size_t)p * sh.ld_cache;
    for (int i = t; i < sh.rank; i += kThreads) dst[i] = (T)(c[i] * inv[1] * in.kv_norm[i]);
    const int half = sh.rot >> 1;
    const float* k = c + sh.rank;
    for (int i = t; i < half; i += kThreads) {
        const float cs = in.cos_t[(size_t)p * half + i], sn = in.sin_t[(size_t)p * half + i];
        dst[sh.rank + i] = (T)(k[i] * cs - k[i + half] * sn);
        dst[sh.rank + half + i] = (T)(k[i + half] * cs + k[i] * sn);
    }
}

// One workgroup per token.
template <typename T>
__global__ __launch_bounds__(kThreads) void rotate_queries_kernel(const float* __restrict__ q, int ld_q, LatentRows in, LatentShape sh,
                                                                 T* __restrict__ nope, int ld_nope, T* __restrict__ rot_out,
                                                                 int ld_rot) {
    const int m = blockIdx.x, t = threadIdx.x, half = sh.rot >> 1, per = sh.dim + half;
    const int p = min(max(in.pos_dev[0] + m, 0), in.max_seq - 1);
    const float* row = q + (size_t)m * ld_q;
    for (int i = t; i < sh.heads * per; i += kThreads) {
        const int h = i / per, d = i % per;
        const float* src = row + h * (sh.dim + sh.rot);
        const size_t o = (size_t)m * sh.heads + h;
        if (d < sh.dim) {
            nope[o * ld_nope + d] = (T)src[d];
        } else {
            const int j = d - sh.dim;
            const float u = src[sh.dim + j], v = src[sh.dim + half + j];
            const float cs = in.cos_t[(size_t)p * half + j], sn = in.sin_t[(size_t)p * half + j];
            rot_out[o * ld_rot + j] = (T)(u * cs - v * sn);
            rot_out[o * ld_rot + half + j] = (T)(v * cs + u * sn);
        }
    }
}

}  // namespace

template <typename T>
hipError_t launch_latent_rows(const LatentRows& in, const LatentShape& sh, int M, T* q_latent, int ld_q, T* cache, hipStream_t s) {
    hipLaunchKernelGGL(latent_rows_kernel<T>, dim3(M), dim3(kThreads), 0, s, in, sh, q_latent, ld_q, cache);
    return hipGetLastError();
}

template <typename T>
hipError_t launch_rotate_queries(const float* q, int ld_q, const LatentRows& in, const LatentShape& sh, int M, T* nope, int ld_nope,
                                 T* rot_out, int ld_rot, hipStream_t s) {
    hipLaunchKernelGGL(rotate_queries_kernel<T>, dim3(M), dim3(kThreads), 0, s, q, ld_q, in, sh, nope, ld_nope, rot_out, ld_rot);
    return hipGetLastError();
}

#define INSTANTIATE(T)                                                                                                           \
    template hipError_t launch_latent_rows<T>(const LatentRows&, const LatentShape&, int, T*, int, T*, hipStream_t);               \
    template hipError_t launch_rotate_queries<T>(const float*, int, const LatentRows&, const LatentShape&, int, T*, int, T*, int, \
                                                 hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
