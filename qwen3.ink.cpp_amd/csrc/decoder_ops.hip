// Kernels of the loop around every decoder model: embedding rows, the first maximum of the logits, the position.
//   embed_rows      Embedding::forward                     src/ops/embedding.cc:13-26
//   argmax_token    sample_token_greedy (first maximum)    Pipeline.cc:54-62
// Every index that depends on device data is clamped into its array.
#include <hip/hip_fp16.h>

#include "decoder_session.h"

namespace a81w41 {
namespace {

struct Bf16Bits {
    uint16_t bits;
};
__device__ __forceinline__ float to_float(__half h) { return __half2float(h); }
__device__ __forceinline__ float to_float(Bf16Bits b) { return __uint_as_float((unsigned)b.bits << 16); }
__device__ __forceinline__ float to_float(float f) { return f; }

// Eight values per load where the rows allow it (hidden and the row stride multiples of 8, 16-byte aligned).
template <typename E>
__global__ __launch_bounds__(256) void embed_rows_kernel(const int* __restrict__ ids, const E* __restrict__ table, int ld,
                                                       float* __restrict__ out, int hidden, int vocab) {
    const int m = blockIdx.x;
    const int id = min(max(ids[m], 0), vocab - 1);
    const E* row = table + (size_t)id * ld;
    float* dst = out + (size_t)m * hidden;
    if (sizeof(E) == 2 && ((hidden | ld) & 7) == 0) {
        const uint4* row4 = reinterpret_cast<const uint4*>(row);
        float4* dst4 = reinterpret_cast<float4*>(dst);
        for (int j = threadIdx.x; j < (hidden >> 3); j += 256) {
            const uint4 u = row4[j];
            const E* e = reinterpret_cast<const E*>(&u);
            dst4[2 * j] = make_float4(to_float(e[0]), to_float(e[1]), to_float(e[2]), to_float(e[3]));
            dst4[2 * j + 1] = make_float4(to_float(e[4]), to_float(e[5]), to_float(e[6]), to_float(e[7]));
        }
    } else {
        for (int j = threadIdx.x; j < hidden; j += 256) dst[j] = to_float(row[j]);
    }
}

// First index of the maximum of logits[0..n); written to next_id[0] and to history[*step], then
// the step counter and the position advance (the token just consumed is now in the cache).
__global__ __launch_bounds__(1024) void argmax_token_kernel(const float* __restrict__ logits, int n, int* __restrict__ next_id,
                                                          int* __restrict__ history, int history_len, int* __restrict__ step_dev) {
    __shared__ float best_v[1024];
    __shared__ int best_i[1024];
    const int t = threadIdx.x;
    float bv = -3.402823466e38f;
    int bi = 0x7fffffff;
    // logits are 16-byte aligned: scan float4s, four in flight, then the up to three left over
    const float4* l4 = reinterpret_cast<const float4*>(logits);
    const int n4 = n >> 2;
    for (int j0 = t; j0 < n4; j0 += 4 * 1024) {
        float4 v[4];
#pragma unroll
        for (int u = 0; u < 4; u++) {
            const int j = j0 + u * 1024;
            v[u] = j < n4 ? l4[j] : make_float4(-3.402823466e38f, -3.402823466e38f, -3.402823466e38f, -3.402823466e38f);
        }
#pragma unroll
        for (int u = 0; u < 4; u++) {
            const int i = 4 * (j0 + u * 1024);  // indices rise within a thread, so '>' keeps the first maximum
            const float e[4] = {v[u].x, v[u].y, v[u].z, v[u].w};
#pragma unroll
            for (int k = 0; k < 4; k++)
                if (e[k] > bv) {
                    bv = e[k];
                    bi = i + k;
                }
        }
    }
    if (t < (n & 3)) {
        const float e = logits[4 * n4 + t];
        if (e > bv) {
            bv = e;
            bi = 4 * n4 + t;
        }
    }
    best_v[t] = bv;
    best_i[t] = bi;
    __syncthreads();
    for (int s = 512; s > 0; s >>= 1) {
        if (t < s) {
            const float ov = best_v[t + s];
            const int oi = best_i[t + s];
            if (ov > best_v[t] || (ov == best_v[t] && oi < best_i[t])) {
                best_v[t] = ov;
                best_i[t] = oi;
            }
        }
        __syncthreads();
    }
    if (t == 0) {
        const int id = best_i[0] == 0x7fffffff ? 0 : best_i[0];
        next_id[0] = id;
        const int st = step_dev[0];
        if (st >= 0 && st < history_len) history[st] = id;
        step_dev[0] = st + 1;
    }
}

__global__ void advance_kernel(int* __restrict__ pos_dev, int by) {
    if (threadIdx.x == 0 && blockIdx.x == 0) pos_dev[0] += by;
}

}  // namespace

hipError_t launch_embed_rows(const int* ids, const void* table, TableType type, int ld, float* out, int M, int hidden, int vocab,
                             hipStream_t s) {
    switch (type) {
        case TableType::kFp16:
            hipLaunchKernelGGL(embed_rows_kernel<__half>, dim3(M), dim3(256), 0, s, ids, static_cast<const __half*>(table), ld, out,
                               hidden, vocab);
            break;
        case TableType::kBf16:
            hipLaunchKernelGGL(embed_rows_kernel<Bf16Bits>, dim3(M), dim3(256), 0, s, ids, static_cast<const Bf16Bits*>(table), ld,
                               out, hidden, vocab);
            break;
        case TableType::kFp32:
            hipLaunchKernelGGL(embed_rows_kernel<float>, dim3(M), dim3(256), 0, s, ids, static_cast<const float*>(table), ld, out,
                               hidden, vocab);
            break;
    }
    return hipGetLastError();
}
hipError_t launch_argmax_token(const float* logits, int n, int* next_id, int* history, int history_len, int* step_dev,
                               hipStream_t s) {
    hipLaunchKernelGGL(argmax_token_kernel, dim3(1), dim3(1024), 0, s, logits, n, next_id, history, history_len, step_dev);
    return hipGetLastError();
}
hipError_t launch_advance(int* pos_dev, int by, hipStream_t s) {
    hipLaunchKernelGGL(advance_kernel, dim3(1), dim3(64), 0, s, pos_dev, by);
    return hipGetLastError();
}

}  // namespace a81w41
