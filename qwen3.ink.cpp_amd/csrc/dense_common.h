// Device helpers of the dense-weight kernels.
#pragma once
#include "dense.h"

namespace a81w41 {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((address_space(3))) void* dense_lds_ptr;

__device__ __forceinline__ float dense_wave_sum(float v, int width = 64) {
    for (int off = width >> 1; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}
__device__ __forceinline__ float dense_wave_max(float v, int width = 64) {
    for (int off = width >> 1; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, 64));
    return v;
}
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }

// One direct copy global -> LDS of 16 bytes per lane: lane l's bytes land at lds_base + 16 l (lds_base uniform).
__device__ __forceinline__ void copy16_to_lds(const void* global_src, void* lds_base) {
    __builtin_amdgcn_global_load_lds(global_src, (dense_lds_ptr)lds_base, 16, 0, 0);
}

// 1 / sqrt(mean of squares + eps) of `groups` equal consecutive parts of a row, into inv[0..groups) (LDS).
// x(i) is element i.  red: THREADS / 64 floats of LDS.  Ends with a barrier.
template <int THREADS, typename F>
__device__ __forceinline__ void group_inverse_rms(F x, int width, int groups, float eps, float* inv, float* red) {
    const int t = threadIdx.x, size = width / groups;
    int per = 1;  // groups worked on at a time
    while (per < groups && per < THREADS) per <<= 1;
    const int tpg = THREADS / per;  // threads per group, a power of two
    for (int g0 = 0; g0 < groups; g0 += per) {
        const int g = g0 + t / tpg, at = t % tpg;
        float sum = 0.f;
        if (g < groups)
            for (int i = at; i < size; i += tpg) {
                const float v = x(g * size + i);
                sum = fmaf(v, v, sum);
            }
        sum = dense_wave_sum(sum, tpg < 64 ? tpg : 64);
        if (tpg > 64) {
            if ((t & 63) == 0) red[t >> 6] = sum;
            __syncthreads();
            sum = 0.f;
            const int w0 = (t / tpg) * (tpg >> 6);
            for (int w = 0; w < (tpg >> 6); w++) sum += red[w0 + w];
        }
        if (g < groups && at == 0) inv[g] = 1.0f / sqrtf(sum / (float)size + eps);
        __syncthreads();
    }
}

}  // namespace a81w41
