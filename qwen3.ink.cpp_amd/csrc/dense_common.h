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
__device__ __forceinline__ float gated_unit(const GatedUnit& p, float gate, float up) {
    const float g = fminf(gate, p.limit), u = fminf(fmaxf(up, -p.limit), p.limit);
    return g / (1.0f + expf(-p.slope * g)) * (u + p.shift);
}

// How many of z[0 .. n) come before z[e]: the larger ones, and the equal ones with lower numbers.
__device__ __forceinline__ int expert_rank(const float* z, int n, int e) {
    const float own = z[e];
    int rank = 0;
#pragma unroll 4
    for (int j = 0; j < n; j++) rank += (z[j] > own || (z[j] == own && j < e)) ? 1 : 0;
    return rank;
}

// One column of a HeadRows product for row m: `own` is its value, `other` that of its pair's other column.
template <typename T>
__device__ __forceinline__ void store_head_column(const HeadRows<T>& p, int pos, int m, int col, float own, float other) {
    const int nq = p.heads * p.dim, nk = p.kv_heads * p.dim, nv = p.kv_heads * p.vdim;
    if (col >= nq + nk + nv) {
        p.rest[(size_t)m * p.ld_rest + col - nq - nk - nv] = own;
        return;
    }
    const int at = min(pos + m, p.max_seq - 1);
    if (col >= nq + nk) {
        const int c = col - nq - nk, h = c / p.vdim;
        p.cache[(size_t)at * p.ld_cache + h * (p.vdim + p.dim) + (c - h * p.vdim)] = (T)own;
        return;
    }
    const bool key = col >= nq;
    const int c = key ? col - nq : col, h = c / p.dim, d = c - h * p.dim;
    if ((d >> 1) < p.rot_pairs) {
        const size_t i = (size_t)at * p.rot_pairs + (d >> 1);
        const float cs = p.cos_t[i], sn = p.sin_t[i];
        own = (d & 1) ? own * cs + other * sn : own * cs - other * sn;
    }
    if (key)
        p.cache[(size_t)at * p.ld_cache + h * (p.vdim + p.dim) + p.vdim + d] = (T)own;
    else
        p.q[(size_t)m * nq + c] = (T)own;
}

// One direct copy global -> LDS of 16 bytes per lane: lane l's bytes land at lds_base + 16 l (lds_base uniform).
__device__ __forceinline__ void copy16_to_lds(const void* global_src, void* lds_base) {
    __builtin_amdgcn_global_load_lds(global_src, (dense_lds_ptr)lds_base, 16, 0, 0);
}

// A barrier that orders LDS only: requested global loads stay in flight.
__device__ __forceinline__ void dense_lds_barrier() {
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt = 0; vector-memory and export counters left alone
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_sched_barrier(0);
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

// A row whose norm groups are whole float4s, dealt to a workgroup so that a group's threads are neighbours and a thread
// holds at most kParts float4s, all of one group: the row stays in registers between its norms.
template <int THREADS>
class RowParts {
   public:
    static constexpr int kParts = 4;
    __device__ __forceinline__ RowParts(int width, int groups) : groups_(groups), size_(width / groups) {
        int per = 1;
        while (per < groups && per < THREADS) per <<= 1;
        log_tpg_ = 31 - __builtin_clz((unsigned)(THREADS / per));
        group_ = threadIdx.x >> log_tpg_;
        at_ = threadIdx.x & ((1 << log_tpg_) - 1);
    }
    __device__ __forceinline__ bool fits() const {
        return groups_ <= THREADS && (size_ & 3) == 0 && (size_ >> 2) <= (kParts << log_tpg_);
    }
    // first element of this thread's k-th float4, -1 if it has none
    __device__ __forceinline__ int place(int k) const {
        const int c = at_ + (k << log_tpg_);
        return group_ < groups_ && 4 * c < size_ ? group_ * size_ + 4 * c : -1;
    }
    // of this thread's group; v: the thread's parts (absent ones zero), red: THREADS / 64 floats of LDS
    __device__ __forceinline__ float inverse_rms(const float4* v, float eps, float* red) const {
        float sum = 0.f;
#pragma unroll
        for (int k = 0; k < kParts; k++) {
            sum = fmaf(v[k].x, v[k].x, sum), sum = fmaf(v[k].y, v[k].y, sum);
            sum = fmaf(v[k].z, v[k].z, sum), sum = fmaf(v[k].w, v[k].w, sum);
        }
        sum = dense_wave_sum(sum, log_tpg_ < 6 ? 1 << log_tpg_ : 64);
        if (log_tpg_ > 6) {
            dense_lds_barrier();  // nobody still reads red
            if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = sum;
            dense_lds_barrier();
            sum = 0.f;
            const int waves = 1 << (log_tpg_ - 6);
            for (int w = 0; w < waves; w++) sum += red[group_ * waves + w];
        }
        return 1.0f / sqrtf(sum / (float)size_ + eps);
    }

   private:
    int groups_, size_, log_tpg_, group_, at_;
};
__device__ __forceinline__ float4 load4(const float* a) { return *reinterpret_cast<const float4*>(a); }
__device__ __forceinline__ void store4(float* a, float4 v) { *reinterpret_cast<float4*>(a) = v; }
__device__ __forceinline__ float4 fma4(float a, float4 b, float4 c) {
    return make_float4(fmaf(a, b.x, c.x), fmaf(a, b.y, c.y), fmaf(a, b.z, c.z), fmaf(a, b.w, c.w));
}
__device__ __forceinline__ float4 scale4(float4 v, float s, float4 w) {
    return make_float4(v.x * s * w.x, v.y * s * w.y, v.z * s * w.z, v.w * s * w.w);
}
__device__ __forceinline__ float4 add4(float4 a, float4 b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }

}  // namespace a81w41
