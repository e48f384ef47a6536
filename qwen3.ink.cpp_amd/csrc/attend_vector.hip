// Causal attention in 32-bit arithmetic for rows of any sizes that hold key and value together (shared and rows form).
#include "dense_common.h"

namespace a81w41 {
namespace {

constexpr int kThreads = 256, kBlock = 64;

// One workgroup per (query row, head).  Keys in blocks of kBlock: every wave scores a quarter of the block's keys, the
// block's maximum rescales what is there, then every thread owns some of the output's elements.
template <typename T, typename O>
__global__ __launch_bounds__(kThreads) void attend_vector_kernel(AttendArgs<T> a, O* __restrict__ out) {
    extern __shared__ float smem[];
    float* qs = smem;                    // k_own_width
    float* acc = qs + a.k_own_width;     // dv
    float* p = acc + a.dv;               // kBlock
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, width = a.k_own_width, z = blockIdx.y;
    const int token = blockIdx.x / a.rows_per_token, sub = blockIdx.x - token * a.rows_per_token;
    const int last = min(max(a.pos_dev[0] + token, 0), a.max_seq - 1);
    const T* qr = a.q + z * a.q_head + (size_t)token * a.q_token + sub * a.ld_q;
    const T* rows = a.k_own + z * a.k_own_head;
    for (int i = t; i < width; i += kThreads) qs[i] = (float)qr[i];
    for (int i = t; i < a.dv; i += kThreads) acc[i] = 0.f;
    float mx = a.sink ? 0.f : -3.402823466e38f, sum = a.sink ? 1.f : 0.f;
    __syncthreads();
    for (int k0 = a.chunk ? last - last % a.chunk : 0; k0 <= last; k0 += kBlock) {
        const int nk = min(kBlock, last + 1 - k0);
        for (int k = wave; k < nk; k += kThreads / 64) {
            const T* row = rows + (size_t)(k0 + k) * a.ld_k_own + a.v_width;
            float s = 0.f;
            for (int i = lane; i < width; i += 64) s = fmaf(qs[i], (float)row[i], s);
            s = dense_wave_sum(s) * a.scale;
            if (lane == 0) p[k] = s;
        }
        __syncthreads();
        float bm = -3.402823466e38f;
        for (int k = 0; k < nk; k++) bm = fmaxf(bm, p[k]);
        const float nm = fmaxf(mx, bm), keep = expf(mx - nm);
        __syncthreads();
        if (t < nk) p[t] = expf(p[t] - nm);
        __syncthreads();
        float bs = 0.f;
        for (int k = 0; k < nk; k++) bs += p[k];
        sum = sum * keep + bs;
        mx = nm;
        for (int i = t; i < a.dv; i += kThreads) {
            float v = acc[i] * keep;
            for (int k = 0; k < nk; k++) v = fmaf(p[k], (float)rows[(size_t)(k0 + k) * a.ld_k_own + i], v);
            acc[i] = v;
        }
        __syncthreads();
    }
    O* dst = out + z * a.out_head + (size_t)token * a.out_token + sub * a.ld_out;
    for (int i = t; i < a.dv; i += kThreads) dst[i] = (O)(acc[i] / sum);
}

}  // namespace

template <typename T, typename O>
hipError_t launch_attend_vector(const AttendArgs<T>& a, int heads, O* out, hipStream_t s) {
    const size_t lds = (a.k_own_width + a.dv + kBlock) * sizeof(float);
    hipLaunchKernelGGL((attend_vector_kernel<T, O>), dim3(a.rows, heads), dim3(kThreads), lds, s, a, out);
    return hipGetLastError();
}
template hipError_t launch_attend_vector<bf16, bf16>(const AttendArgs<bf16>&, int, bf16*, hipStream_t);
template hipError_t launch_attend_vector<bf16, float>(const AttendArgs<bf16>&, int, float*, hipStream_t);
template hipError_t launch_attend_vector<float, float>(const AttendArgs<float>&, int, float*, hipStream_t);

}  // namespace a81w41
