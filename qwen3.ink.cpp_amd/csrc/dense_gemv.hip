// One-token products for dense weights, with the row work around them fused in: every workgroup forms the input row in
// LDS (fp32) in its prologue -- residual step and norm, the norm of a latent, the attention output -- and its waves
// then stream weight rows in pairs, 16 bytes per lane and load, the next eight loads in flight while eight are used; the
// first ones are requested before the prologue.  A row's sum is formed
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

constexpr int kAhead = 4;  // 16-byte chunks of a row that a lane requests at once
__host__ __device__ constexpr int lanes_of(int chunks) {
    int lanes = 1;
    while (lanes < 64 && lanes * kAhead < chunks) lanes <<= 1;
    return lanes;
}
// How rows are dealt: `lanes` lanes (a power of two) share a pair of rows; `group` counts the lane groups of the launch.
struct Deal {
    int lanes, group, groups, at;
};
template <typename T>
__device__ __forceinline__ Deal deal_rows(int chunks, int workgroups) {
    Deal d;
    d.lanes = lanes_of(chunks);
    const int per_wg = kThreads / d.lanes;
    d.group = blockIdx.x * per_wg + threadIdx.x / d.lanes;
    d.groups = workgroups * per_wg;
    d.at = threadIdx.x & (d.lanes - 1);
    return d;
}

// Up to kAhead chunks per lane of two weight rows.
struct Pair {
    uint4 a[kAhead], b[kAhead];
};
struct RowPair {
    const void *w0, *w1;
};
__device__ __forceinline__ void load_pair(Pair& p, const RowPair& r, int c, int lanes, int chunks) {
    const uint4 *p0 = static_cast<const uint4*>(r.w0), *p1 = static_cast<const uint4*>(r.w1);
#pragma unroll
    for (int u = 0; u < kAhead; u++) {
        const int cc = min(c + u * lanes, chunks - 1);
        p.a[u] = p0[cc];
        p.b[u] = p1[cc];
    }
}
template <typename T>
__device__ __forceinline__ void use_pair(const Pair& p, const float* xs, int c, int lanes, int chunks, float& s0, float& s1) {
    constexpr int E = 16 / (int)sizeof(T);
#pragma unroll
    for (int u = 0; u < kAhead; u++) {
        const int cc = c + u * lanes;
        if (cc < chunks) {
            s0 += dot16(p.a[u], xs + cc * E, static_cast<T*>(nullptr));
            s1 += dot16(p.b[u], xs + cc * E, static_cast<T*>(nullptr));
        }
    }
}

// The lane group's share of `pairs` row pairs: rows(n) names pair n, emit(n, s0, s1) gets the dot products with xs (LDS,
// zero-padded to whole chunks).  The loads run one step ahead; `ahead` holds the first one's, requested by
// request_first before the caller's prologue.
template <typename Rows>
__device__ __forceinline__ void request_first(Pair& ahead, Rows rows, int pairs, int chunks, const Deal& d) {
    if (d.group < pairs) load_pair(ahead, rows(d.group), d.at, d.lanes, chunks);
}
template <typename T, typename Rows, typename Emit>
__device__ __forceinline__ void stream_pairs(Pair& ahead, Rows rows, Emit emit, int pairs, const float* xs, int chunks, const Deal& d) {
    const int per_step = kAhead * d.lanes, steps = (chunks + per_step - 1) / per_step;
    for (int n = d.group; n < pairs; n += d.groups) {
        float s0 = 0.f, s1 = 0.f;
        for (int step = 0; step < steps; step++) {
            const int c = d.at + step * per_step;
            const Pair now = ahead;
            if (step + 1 < steps)
                load_pair(ahead, rows(n), c + per_step, d.lanes, chunks);
            else if (n + d.groups < pairs)
                load_pair(ahead, rows(n + d.groups), d.at, d.lanes, chunks);
            use_pair<T>(now, xs, c, d.lanes, chunks, s0, s1);
        }
        s0 = dense_wave_sum(s0, d.lanes);
        s1 = dense_wave_sum(s1, d.lanes);
        if (d.at == 0) emit(n, s0, s1);
    }
}
// Rows 2 n and 2 n + 1 of a plain matrix.
template <typename T>
struct PlainRows {
    const T* w;
    int ld, N;
    __device__ RowPair operator()(int n) const { return {w + (size_t)(2 * n) * ld, w + (size_t)min(2 * n + 1, N - 1) * ld}; }
};
struct PlainEmit {
    float* C;
    int N;
    float factor;
    __device__ void operator()(int n, float s0, float s1) const {
        C[2 * n] = s0 * factor;
        if (2 * n + 1 < N) C[2 * n + 1] = s1 * factor;
    }
};

// xs[0 .. padded) = f(i), zero from n on
template <typename F>
__device__ __forceinline__ void fill_row(float* xs, int n, int padded, F f) {
    for (int i = threadIdx.x; i < padded; i += kThreads) xs[i] = i < n ? f(i) : 0.f;
}

// xs[0 .. padded) = src[0 .. n), zero from n on; sixteen bytes per load where the row is made of whole float4s
__device__ __forceinline__ void copy_row(float* xs, const float* src, int n, int padded) {
    if (((n & 3) | (int)(reinterpret_cast<uintptr_t>(src) & 15)) == 0) {
#pragma unroll 4
        for (int i = 4 * threadIdx.x; i < n; i += 4 * kThreads) store4(xs + i, load4(src + i));
        for (int i = n + threadIdx.x; i < padded; i += kThreads) xs[i] = 0.f;
    } else {
        fill_row(xs, n, padded, [&](int i) { return src[i]; });
    }
}

// The residual step and the norm of RowStep into xs; workgroup 0 of the launch also writes the stream.  Rows whose parts
// are whole float4s and fit four of them per thread are requested at once by load() and stay in registers (a part's
// threads are neighbours); other rows are read when they are needed.
class StepRow {
   public:
    __device__ __forceinline__ explicit StepRow(const RowStep& p) : p_(p), parts_(p.width, p.norm_h.groups), fast_(parts_.fits()) {}
    __device__ __forceinline__ void load() {
        if (!fast_) return;
#pragma unroll
        for (int k = 0; k < kParts; k++) {
            const int i = parts_.place(k);
            const bool in = i >= 0;
            const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
            x_[k] = in ? load4(p_.x + i) : zero;
            y_[k] = in && p_.y ? load4(p_.y + i) : zero;
            wy_[k] = in && p_.norm_y.w ? load4(p_.norm_y.w + i) : zero;
            before_[k] = in && p_.before ? load4(p_.before + i) : zero;
            wh_[k] = in ? load4(p_.norm_h.w + i) : zero;
        }
    }
    __device__ __forceinline__ void finish(float* xs, int padded, float* inv, float* red) {
        if (!fast_) return slow(xs, padded, inv, red);
        const bool writer = blockIdx.x == 0 && blockIdx.y == 0;
        const float coef = p_.before && p_.coef ? *p_.coef : 1.f;
        const bool normed = p_.y && p_.norm_y.w;
        const float inv_y = normed ? parts_.inverse_rms(y_, p_.norm_y.eps, red) : 0.f;
#pragma unroll
        for (int k = 0; k < kParts; k++) {
            const int i = parts_.place(k);
            float4 r = normed ? add4(x_[k], scale4(y_[k], inv_y, wy_[k])) : fma4(p_.norm_y.scale, y_[k], x_[k]);
            if (i >= 0 && writer && p_.state) store4(p_.state + i, r);
            if (p_.before) r = fma4(coef, r, before_[k]);
            if (i >= 0 && writer && p_.x_out) store4(p_.x_out + i, r);
            x_[k] = r;
        }
        const float inv_h = parts_.inverse_rms(x_, p_.norm_h.eps, red);
#pragma unroll
        for (int k = 0; k < kParts; k++) {
            const int i = parts_.place(k);
            if (i < 0) continue;
            const float4 h = scale4(x_[k], inv_h, wh_[k]);
            store4(xs + i, h);
            if (writer && p_.h_out) store4(p_.h_out + i, h);
        }
        for (int i = p_.width + threadIdx.x; i < padded; i += kThreads) xs[i] = 0.f;
        dense_lds_barrier();
    }

   private:
    static constexpr int kParts = RowParts<kThreads>::kParts;
    __device__ void slow(float* xs, int padded, float* inv, float* red) const {
        const RowStep& p = p_;
        const int t = threadIdx.x, W = p.width;
        const bool writer = blockIdx.x == 0 && blockIdx.y == 0;
        const bool normed = p.y && p.norm_y.w;
        if (normed) group_inverse_rms<kThreads>([&](int i) { return p.y[i]; }, W, p.norm_y.groups, p.norm_y.eps, inv, red);
        const float coef = p.before && p.coef ? *p.coef : 1.f;
        const int size_y = normed ? W / p.norm_y.groups : 1;
        for (int i = t; i < padded; i += kThreads) {
            float r = 0.f;
            if (i < W) {
                r = p.x[i];
                if (p.y) r = normed ? r + p.y[i] * inv[i / size_y] * p.norm_y.w[i] : fmaf(p.norm_y.scale, p.y[i], r);
                if (writer && p.state) p.state[i] = r;
                if (p.before) r = fmaf(coef, r, p.before[i]);
                if (writer && p.x_out) p.x_out[i] = r;
            }
            xs[i] = r;
        }
        __syncthreads();
        group_inverse_rms<kThreads>([&](int i) { return xs[i]; }, W, p.norm_h.groups, p.norm_h.eps, inv, red);
        const int size_h = W / p.norm_h.groups;
        for (int i = t; i < W; i += kThreads) {
            xs[i] = xs[i] * inv[i / size_h] * p.norm_h.w[i];
            if (writer && p.h_out) p.h_out[i] = xs[i];
        }
        __syncthreads();
    }
    const RowStep& p_;
    RowParts<kThreads> parts_;
    bool fast_;
    float4 x_[kParts], y_[kParts], wy_[kParts], before_[kParts], wh_[kParts];
};

template <typename T>
struct HeadsEmit {
    HeadRows<T> heads;
    int N;
    __device__ void operator()(int n, float s0, float s1) const {
        const int pos = min(max(heads.pos_dev[0], 0), heads.max_seq - 1);
        store_head_column(heads, pos, 0, 2 * n, s0, s1);
        if (2 * n + 1 < N) store_head_column(heads, pos, 0, 2 * n + 1, s1, s0);
    }
};

// emit gets W[n] . row, in pairs of n
template <typename T, typename Emit>
__global__ __launch_bounds__(kThreads) void gemv_step_kernel(RowStep p, const T* __restrict__ w, int ld, int N, Emit emit) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *xs = smem, *red = xs + ld, *inv = red + kThreads / 64;
    StepRow row(p);
    row.load();
    const int chunks = ld * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    const PlainRows<T> rows{w, ld, N};
    Pair ahead;
    request_first(ahead, rows, pairs, chunks, d);
    row.finish(xs, ld, inv, red);
    stream_pairs<T>(ahead, rows, emit, pairs, xs, chunks, d);
}

// C[n] = W[n] . x
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_plain_kernel(const float* __restrict__ x, int K, const T* __restrict__ w, int ld, int N,
                                                             float* __restrict__ C) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int chunks = ld * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    const PlainRows<T> rows{w, ld, N};
    Pair ahead;
    request_first(ahead, rows, pairs, chunks, d);
    copy_row(smem, x, K, ld);
    dense_lds_barrier();
    stream_pairs<T>(ahead, rows, PlainEmit{C, N, 1.f}, pairs, smem, chunks, d);
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
    const int chunks = ld * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    const Deal d = deal_rows<T>(chunks, main_groups);
    const PlainRows<T> rows{w, ld, N};
    Pair ahead;
    request_first(ahead, rows, pairs, chunks, d);
    fill_row(xs, sh.q_rank, ld, [&](int i) { return in.down[i]; });
    float sum = 0.f;  // of this thread's own elements
    for (int i = t; i < sh.q_rank; i += kThreads) sum = fmaf(xs[i], xs[i], sum);
    sum = dense_wave_sum(sum);
    if ((t & 63) == 0) red[t >> 6] = sum;
    dense_lds_barrier();
    sum = 0.f;
    for (int k = 0; k < kThreads / 64; k++) sum += red[k];
    const float scale = 1.0f / sqrtf(sum / (float)sh.q_rank + in.eps);
    for (int i = t; i < sh.q_rank; i += kThreads) xs[i] *= scale * in.q_norm[i];
    dense_lds_barrier();
    stream_pairs<T>(ahead, rows, PlainEmit{q, N, 1.f}, pairs, xs, chunks, d);
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
    const int N = sh.rank, chunks = ld * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    const PlainRows<T> rows{uk_t + (size_t)h * N * ld, ld, N};
    Pair ahead;
    request_first(ahead, rows, pairs, chunks, d);
    copy_row(smem, src, sh.dim, ld);
    dense_lds_barrier();
    stream_pairs<T>(
        ahead, rows,
        [&](int n, float s0, float s1) {
            dst[2 * n] = (T)s0;
            if (2 * n + 1 < N) dst[2 * n + 1] = (T)s1;
        },
        pairs, smem, chunks, d);
}

// Values of a head (blockIdx.y) from its weighted latent, times the head's gate.  The latent is a row of o_lat, or is
// merged here from the shares of the attention: sum_k w_k share_k / sum_k w_k sum_k, w_k = 2^(maximum_k - largest).
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_values_kernel(const float* __restrict__ o_lat, int ld_o, LatentShares shares,
                                                              LatentShape sh, const T* __restrict__ uv, int ld,
                                                              const float* __restrict__ gates, float* __restrict__ attn) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ float weight[kAttendMaxSplits];
    const int h = blockIdx.y, t = threadIdx.x;
    const int N = sh.vdim, chunks = ld * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    const PlainRows<T> rows{uv + (size_t)h * N * ld, ld, N};
    const float gate = sigmoid(gates[h]);
    Pair ahead;
    if (shares.part) {
        // a thread takes four columns of every `teams`-th share; the teams' sums meet in LDS.  Requested in the order of use.
        constexpr int U = 16;
        const int n = shares.splits, quads = shares.ld >> 2, teams = max(1, kThreads / quads);
        const int l63 = min(t & 63, n - 1);
        const float maximum = shares.stats[2 * ((size_t)l63 * sh.heads + h)], total = shares.stats[2 * ((size_t)l63 * sh.heads + h) + 1];
        const float* part = shares.part + (size_t)h * shares.ld;
        const size_t step = (size_t)sh.heads * shares.ld;
        float4 v[U];
        auto request = [&](int q, int k) {
#pragma unroll
            for (int u = 0; u < U; u++) v[u] = load4(part + min(k + u * teams, n - 1) * step + 4 * (q % quads));
        };
        if (t < quads * teams) request(t, t / quads);
        request_first(ahead, rows, pairs, chunks, d);
        {   // every wave forms the shares' weights
            const bool real = (t & 63) < n;
            const float largest = dense_wave_max(real ? maximum : -3.402823466e38f), w = real ? exp2f(maximum - largest) : 0.f;
            const float all = dense_wave_sum(w * total);
            if (t < 64) weight[t] = w / all;
        }
        dense_lds_barrier();
        float* sums = smem + ld;
        for (int q = t; q < quads * teams; q += kThreads) {
            const int team = q / quads;
            if (q != t) request(q, team);
            float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int k = team; k < n; k += U * teams) {
                if (k != team) request(q, k);
#pragma unroll
                for (int u = 0; u < U; u++)
                    if (k + u * teams < n) s = fma4(weight[k + u * teams], v[u], s);
            }
            store4(sums + team * shares.ld + 4 * (q % quads), s);
        }
        dense_lds_barrier();
        fill_row(smem, sh.rank, ld, [&](int i) {
            float s = 0.f;
            for (int k = 0; k < teams; k++) s += sums[k * shares.ld + i];
            return s;
        });
    } else {
        request_first(ahead, rows, pairs, chunks, d);
        copy_row(smem, o_lat + (size_t)h * ld_o, sh.rank, ld);
    }
    dense_lds_barrier();
    stream_pairs<T>(ahead, rows, PlainEmit{attn + (size_t)h * N, N, gate}, pairs, smem, chunks, d);
}

__device__ __forceinline__ int expert_of(const ExpertRows& e, int slot) {
    const int id = min(max(e.ids[0], 0), e.vocab - 1);
    return min(max(e.table[(size_t)id * e.top + slot], 0), e.experts - 1);
}

// The router's choice for one token, formed by a whole workgroup from its logits (z, best: LDS): ids[0 .. top).
__device__ __forceinline__ void choose_experts(const ExpertRows& e, float* z, int* ids, float* best) {
    for (int i = threadIdx.x; i < e.experts; i += kThreads) z[i] = e.logits[i] + e.bias[i];
    __syncthreads();
    for (int i = threadIdx.x; i < e.experts; i += kThreads) {
        const int rank = expert_rank(z, e.experts, i);
        if (rank < e.top) {
            ids[rank] = i;
            best[rank] = z[i];
        }
    }
    __syncthreads();
    if (blockIdx.x == 0 && blockIdx.y == 0 && threadIdx.x < 64) {
        const int k = threadIdx.x;
        const float w = k < e.top ? expf(best[k] - best[0]) : 0.f, sum = dense_wave_sum(w);
        if (k < e.top) {
            e.chosen[k] = ids[k];
            e.weights[k] = w / sum;
        }
    }
}

// act = unit(gate, up) for the token's experts (blockIdx.y < top) and the dense or shared feed-forward (the last).
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_gate_up_kernel(RowStep p, const float* __restrict__ h, ExpertRows e,
                                                               const T* __restrict__ experts, const T* __restrict__ dense, int ld,
                                                               float* __restrict__ act) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ int ids[kMaxTop];
    __shared__ float best[kMaxTop];
    float *xs = smem, *red = xs + ld, *inv = red + kThreads / 64;
    const int slot = blockIdx.y;
    StepRow row(p);
    if (!h) row.load();
    if (e.logits) choose_experts(e, red, ids, best);  // the places of red and inv are free until the row is formed
    const T* w = slot < e.top ? experts + (size_t)(e.logits ? ids[slot] : expert_of(e, slot)) * e.pair_rows * ld : dense;
    const int ff = slot < e.top ? e.ff : e.dense_ff;
    const int chunks = ld * (int)sizeof(T) / 16;
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    auto rows = [&](int j) {  // the gate and the up row of column j
        const T* r = w + (size_t)((j >> 4) * 32 + (j & 15)) * ld;
        return RowPair{r, r + (size_t)16 * ld};
    };
    Pair ahead;
    request_first(ahead, rows, ff, chunks, d);
    if (h) {
        copy_row(xs, h, p.width, ld);
        dense_lds_barrier();
    } else {
        if (e.logits) __syncthreads();
        row.finish(xs, ld, inv, red);
    }
    float* dst = act + (size_t)slot * e.ld_act;
    stream_pairs<T>(ahead, rows, [&](int j, float gate, float up) { dst[j] = gated_unit(e.unit, gate, up); }, ff, xs, chunks, d);
}

// y[n] = mean over the token's experts of W_e[n] . act_e, plus the dense or shared feed-forward's.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_ff_down_kernel(ExpertRows e, const float* __restrict__ act, const T* __restrict__ experts,
                                                               int ld, const T* __restrict__ dense, int ld_dense, int N,
                                                               float* __restrict__ y) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ int chosen[64];
    const int chunks = ld * (int)sizeof(T) / 16, chunks_dense = ld_dense * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    float* xs_dense = smem + e.top * ld;
    auto fill = [&]() {
        for (int k = 0; k < e.top; k++) copy_row(smem + k * ld, act + (size_t)k * e.ld_act, e.ff, ld);
        if (e.dense_ff) copy_row(xs_dense, act + (size_t)e.top * e.ld_act, e.dense_ff, ld_dense);
    };
    if (!e.top) {
        const Deal d = deal_rows<T>(chunks_dense, gridDim.x);
        const PlainRows<T> rows{dense, ld_dense, N};
        Pair ahead;
        request_first(ahead, rows, pairs, chunks_dense, d);
        fill();
        dense_lds_barrier();
        stream_pairs<T>(ahead, rows, PlainEmit{y, N, 1.f}, pairs, xs_dense, chunks_dense, d);
        return;
    }
    // a pair of rows of every expert in turn, then of the shared feed-forward; the loads run one step ahead
    const Deal d = deal_rows<T>(chunks, gridDim.x);
    if ((int)threadIdx.x < e.top) chosen[threadIdx.x] = expert_of(e, threadIdx.x);
    fill();
    __syncthreads();
    const int parts = e.top + (e.dense_ff ? 1 : 0), per_step = kAhead * d.lanes;
    const float share = 1.0f / (float)e.top;
    auto rows_of = [&](int n, int k) {
        return k < e.top ? PlainRows<T>{experts + (size_t)chosen[k] * N * ld, ld, N}(n) : PlainRows<T>{dense, ld_dense, N}(n);
    };
    Pair ahead;
    if (d.group < pairs) load_pair(ahead, rows_of(d.group, 0), d.at, d.lanes, chunks);
    for (int n = d.group; n < pairs; n += d.groups) {
        float a0 = 0.f, a1 = 0.f;
        for (int k = 0; k < parts; k++) {
            const bool expert = k < e.top;
            const int all = expert ? chunks : chunks_dense, steps = (all + per_step - 1) / per_step;
            const float* xs = expert ? smem + k * ld : xs_dense;
            float s0 = 0.f, s1 = 0.f;
            for (int step = 0; step < steps; step++) {
                const int c = d.at + step * per_step;
                const Pair now = ahead;
                if (step + 1 < steps)
                    load_pair(ahead, rows_of(n, k), c + per_step, d.lanes, all);
                else if (k + 1 < parts)
                    load_pair(ahead, rows_of(n, k + 1), d.at, d.lanes, k + 1 < e.top ? chunks : chunks_dense);
                else if (n + d.groups < pairs)
                    load_pair(ahead, rows_of(n + d.groups, 0), d.at, d.lanes, chunks);
                use_pair<T>(now, xs, c, d.lanes, all, s0, s1);
            }
            a0 = fmaf(expert ? share : 1.f, s0, a0);
            a1 = fmaf(expert ? share : 1.f, s1, a1);
        }
        a0 = dense_wave_sum(a0, d.lanes);
        a1 = dense_wave_sum(a1, d.lanes);
        if (d.at == 0) PlainEmit{y, N, 1.f}(n, a0, a1);
    }
}

// The mixer's row into xs (LDS, zero-padded).  inv: a float for every head, or for every head and share.
__device__ __forceinline__ void form_mixer_row(const MixerRow& m, float* xs, int padded, float* inv, float* red) {
    const int t = threadIdx.x;
    if (m.shares.part) {  // per head sum_k w_k share_k / sum_k w_k sum_k, w_k = 2^(maximum_k - largest)
        const int n = m.shares.splits, H = m.heads;
        for (int h = t; h < H; h += kThreads) {
            float top = -3.402823466e38f;
            for (int k = 0; k < n; k++) top = fmaxf(top, m.shares.stats[2 * ((size_t)k * H + h)]);
            float all = 0.f;
            for (int k = 0; k < n; k++) {
                const float w = exp2f(m.shares.stats[2 * ((size_t)k * H + h)] - top);
                inv[h * n + k] = w;
                all = fmaf(w, m.shares.stats[2 * ((size_t)k * H + h) + 1], all);
            }
            for (int k = 0; k < n; k++) inv[h * n + k] /= all;
        }
        __syncthreads();
        fill_row(xs, m.width, padded, [&](int i) {
            const int h = i / m.vdim, d = i - h * m.vdim;
            float s = 0.f;
            for (int k = 0; k < n; k++) s = fmaf(inv[h * n + k], m.shares.part[((size_t)k * H + h) * m.shares.ld + d], s);
            return s;
        });
    } else if (m.norm) {
        group_inverse_rms<kThreads>([&](int i) { return m.row[i]; }, m.width, m.heads, m.eps, inv, red);
        fill_row(xs, m.width, padded, [&](int i) { return m.row[i] * inv[i / m.vdim] * m.norm[i] * sigmoid(m.gates[i]); });
    } else {
        copy_row(xs, m.row, m.width, padded);
    }
}

// y[n] = W_o[n] . mixer row + sum_k weights[k] W_e(k)[n] . act_k: a pair of rows of every expert in turn, then of W_o; the
// loads run one step ahead.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_mixer_down_kernel(MixerRow m, const T* __restrict__ wo, int ld_wo, ExpertRows e,
                                                                  const float* __restrict__ act, const T* __restrict__ experts, int ld,
                                                                  int N, float* __restrict__ y) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ int chosen[kMaxTop];
    __shared__ float weights[kMaxTop];
    const int chunks = ld * (int)sizeof(T) / 16, chunks_wo = ld_wo * (int)sizeof(T) / 16, pairs = (N + 1) / 2;
    float *xs_mixer = smem, *xs = xs_mixer + ld_wo, *red = xs + e.top * ld, *inv = red + kThreads / 64;
    const Deal d = deal_rows<T>(chunks_wo, gridDim.x);
    if ((int)threadIdx.x < e.top) {
        chosen[threadIdx.x] = min(max(e.chosen[threadIdx.x], 0), e.experts - 1);
        weights[threadIdx.x] = e.weights[threadIdx.x];
    }
    const int parts = e.top + 1, per_step = kAhead * d.lanes;
    auto rows_of = [&](int n, int k) {
        return k == 0 ? PlainRows<T>{wo, ld_wo, N}(n) : PlainRows<T>{experts + (size_t)chosen[k - 1] * N * ld, ld, N}(n);
    };
    Pair ahead;
    if (d.group < pairs) load_pair(ahead, rows_of(d.group, 0), d.at, d.lanes, chunks_wo);
    for (int k = 0; k < e.top; k++) copy_row(xs + k * ld, act + (size_t)k * e.ld_act, e.ff, ld);
    form_mixer_row(m, xs_mixer, ld_wo, inv, red);
    __syncthreads();
    for (int n = d.group; n < pairs; n += d.groups) {
        float a0 = 0.f, a1 = 0.f;
        for (int k = 0; k < parts; k++) {
            const int all = k ? chunks : chunks_wo, steps = (all + per_step - 1) / per_step;
            const float* row = k ? xs + (k - 1) * ld : xs_mixer;
            float s0 = 0.f, s1 = 0.f;
            for (int step = 0; step < steps; step++) {
                const int c = d.at + step * per_step;
                const Pair now = ahead;
                if (step + 1 < steps)
                    load_pair(ahead, rows_of(n, k), c + per_step, d.lanes, all);
                else if (k + 1 < parts)
                    load_pair(ahead, rows_of(n, k + 1), d.at, d.lanes, chunks);
                else if (n + d.groups < pairs)
                    load_pair(ahead, rows_of(n + d.groups, 0), d.at, d.lanes, chunks_wo);
                use_pair<T>(now, row, c, d.lanes, all, s0, s1);
            }
            a0 = fmaf(k ? weights[k - 1] : 1.f, s0, a0);
            a1 = fmaf(k ? weights[k - 1] : 1.f, s1, a1);
        }
        a0 = dense_wave_sum(a0, d.lanes);
        a1 = dense_wave_sum(a1, d.lanes);
        if (d.at == 0) PlainEmit{y, N, 1.f}(n, a0, a1);
    }
}

// Workgroups for N rows of `ld` elements: at most `limit`, and as many as give every lane group the same number of pairs.
template <typename T>
int workgroups(int N, int ld, int limit) {
    const int per_wg = kThreads / lanes_of(ld * (int)sizeof(T) / 16), pairs = (N + 1) / 2;
    const int rounds = (pairs + per_wg * limit - 1) / (per_wg * limit);
    return (pairs + per_wg * rounds - 1) / (per_wg * rounds);
}
constexpr int kMaxGrid = 1024;

size_t step_lds(int ld, const RowStep& p) {
    const int groups = p.norm_y.groups > p.norm_h.groups ? p.norm_y.groups : p.norm_h.groups;
    return (ld + kThreads / 64 + groups) * sizeof(float);
}

}  // namespace

template <typename T>
hipError_t launch_gemv_step(const RowStep& p, const T* w, int ld, int N, float* C, hipStream_t s) {
    hipLaunchKernelGGL((gemv_step_kernel<T, PlainEmit>), dim3(workgroups<T>(N, ld, kMaxGrid)), dim3(kThreads), step_lds(ld, p), s, p, w, ld,
                       N, PlainEmit{C, N, 1.f});
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_step_heads(const RowStep& p, const T* w, int ld, int N, const HeadRows<T>& heads, hipStream_t s) {
    hipLaunchKernelGGL((gemv_step_kernel<T, HeadsEmit<T>>), dim3(workgroups<T>(N, ld, kMaxGrid)), dim3(kThreads), step_lds(ld, p), s, p, w,
                       ld, N, HeadsEmit<T>{heads, N});
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
hipError_t launch_gemv_values(const float* o_lat, int ld_o, const LatentShares& shares, const LatentShape& sh, const T* uv, int ld,
                              const float* gates, float* attn, hipStream_t s) {
    // every workgroup of a head repeats the merge of its shares
    const int teams = shares.part ? (kThreads * 4 > shares.ld ? kThreads * 4 / shares.ld : 1) : 0;
    hipLaunchKernelGGL(gemv_values_kernel<T>, dim3(workgroups<T>(sh.vdim, ld, shares.part ? 4 : 64), sh.heads), dim3(kThreads),
                       (ld + teams * shares.ld) * sizeof(float), s, o_lat, ld_o, shares, sh, uv, ld, gates, attn);
    return hipGetLastError();
}
template <typename T>
hipError_t launch_gemv_gate_up(const RowStep& p, const float* h, const ExpertRows& e, const T* experts, const T* dense, int ld, float* act,
                               hipStream_t s) {
    const int most = e.top && e.ff > e.dense_ff ? e.ff : e.dense_ff;
    const int slots = e.top + (e.dense_ff ? 1 : 0);
    const size_t router = e.logits ? (ld + e.experts) * sizeof(float) : 0, lds = step_lds(ld, p);
    hipLaunchKernelGGL(gemv_gate_up_kernel<T>, dim3(workgroups<T>(2 * most, ld, kMaxGrid), slots), dim3(kThreads), lds > router ? lds : router,
                       s, p, h, e, experts, dense, ld, act);
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

template <typename T>
hipError_t launch_gemv_mixer_down(const MixerRow& m, const T* wo, int ld_wo, const ExpertRows& e, const float* act, const T* experts,
                                  int ld, int N, float* y, hipStream_t s) {
    const int inv = m.shares.part ? m.heads * m.shares.splits : m.heads;
    const size_t lds = (ld_wo + (size_t)e.top * ld + kThreads / 64 + inv) * sizeof(float);
    hipLaunchKernelGGL(gemv_mixer_down_kernel<T>, dim3(workgroups<T>(N, ld_wo, kMaxGrid)), dim3(kThreads), lds, s, m, wo, ld_wo, e, act,
                       experts, ld, N, y);
    return hipGetLastError();
}

#define INSTANTIATE(T)                                                                                                            \
    template hipError_t launch_gemv_step<T>(const RowStep&, const T*, int, int, float*, hipStream_t);                              \
    template hipError_t launch_gemv_plain<T>(const float*, int, const T*, int, int, float*, hipStream_t);                          \
    template hipError_t launch_gemv_query<T>(const LatentRows&, const LatentShape&, const T*, int, float*, T*, const DepthAverage&, \
                                             int, float*, hipStream_t);                                                           \
    template hipError_t launch_gemv_absorb<T>(const float*, const LatentRows&, const LatentShape&, const T*, int, T*, hipStream_t); \
    template hipError_t launch_gemv_values<T>(const float*, int, const LatentShares&, const LatentShape&, const T*, int,           \
                                              const float*, float*, hipStream_t);                                                                       \
    template hipError_t launch_gemv_gate_up<T>(const RowStep&, const float*, const ExpertRows&, const T*, const T*, int, float*,    \
                                               hipStream_t);                                                                       \
    template hipError_t launch_gemv_step_heads<T>(const RowStep&, const T*, int, int, const HeadRows<T>&, hipStream_t);             \
    template hipError_t launch_gemv_mixer_down<T>(const MixerRow&, const T*, int, const ExpertRows&, const float*, const T*, int,   \
                                                  int, float*, hipStream_t);                                                       \
    template hipError_t launch_gemv_ff_down<T>(const ExpertRows&, const float*, const T*, int, const T*, int, int, float*,         \
                                               hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
