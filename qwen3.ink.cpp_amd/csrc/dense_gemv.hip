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

// The mixer's row: load() requests what a thread will need of it, finish() puts it into xs (LDS, zero-padded; ends without
// a barrier).  inv: LDS, a float for every head, or for every head and share.
class MixerPrologue {
   public:
    __device__ __forceinline__ explicit MixerPrologue(const MixerRow& m)
        : m_(m), parts_(m.width, m.norm ? m.heads : 1), quads_(m.shares.part && m.vdim % 4 == 0), normed_(m.norm && parts_.fits()) {}
    __device__ __forceinline__ void load() {
        const int t = threadIdx.x;
        if (quads_) {
            if (t < m_.heads) {
#pragma unroll
                for (int k = 0; k < kShares; k++) stats_[k] = stat(min(k, m_.shares.splits - 1), t);
            }
            request_shares(0);
        } else if (normed_) {
#pragma unroll
            for (int k = 0; k < RowParts<kThreads>::kParts; k++) {
                const int i = parts_.place(k);
                const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
                row_[k] = i >= 0 ? load4(m_.row + i) : zero;
                norm_[k] = i >= 0 ? load4(m_.norm + i) : zero;
                gate_[k] = i >= 0 ? load4(m_.gates + i) : zero;
            }
        }
    }
    __device__ __forceinline__ void finish(float* xs, int padded, float* inv, float* red) {
        const int t = threadIdx.x, n = m_.shares.splits, H = m_.heads;
        if (m_.shares.part) {
            for (int h = t; h < H; h += kThreads) {  // weights w_k / sum_k w_k sum_k, w_k = 2^(maximum_k - largest)
                if (!quads_ || h != t) {
#pragma unroll
                    for (int k = 0; k < kShares; k++) stats_[k] = stat(min(k, n - 1), h);
                }
                float largest = stats_[0].x, all = 0.f, w[kShares];
#pragma unroll
                for (int k = 1; k < kShares; k++) largest = fmaxf(largest, stats_[k].x);
#pragma unroll
                for (int k = 0; k < kShares; k++) {
                    w[k] = k < n ? exp2f(stats_[k].x - largest) : 0.f;
                    all = fmaf(w[k], stats_[k].y, all);
                }
                const float share = 1.0f / all;
#pragma unroll
                for (int k = 0; k < kShares; k++) inv[h * kShares + k] = w[k] * share;
            }
            dense_lds_barrier();
            if (quads_) {
                for (int q0 = 0; 4 * q0 < m_.width; q0 += kQuads * kThreads) {
                    if (q0) request_shares(q0);
#pragma unroll
                    for (int u = 0; u < kQuads; u++) {
                        const int i = 4 * (q0 + u * kThreads + t), h = i / m_.vdim;
                        if (i >= m_.width) continue;
                        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                        for (int k = 0; k < kShares; k++) s = fma4(inv[h * kShares + k], shares_[u][k], s);
                        store4(xs + i, s);
                    }
                }
                for (int i = m_.width + t; i < padded; i += kThreads) xs[i] = 0.f;
            } else {
                fill_row(xs, m_.width, padded, [&](int i) {
                    const int h = i / m_.vdim, d = i - h * m_.vdim;
                    float s = 0.f;
                    for (int k = 0; k < n; k++) s = fmaf(inv[h * kShares + k], share_row(k, h)[d], s);
                    return s;
                });
            }
        } else if (normed_) {
            const float scale = parts_.inverse_rms(row_, m_.eps, red);
#pragma unroll
            for (int k = 0; k < RowParts<kThreads>::kParts; k++) {
                const int i = parts_.place(k);
                if (i < 0) continue;
                const float4 r = row_[k], w = norm_[k], g = gate_[k], v = scale4(r, scale, w);
                store4(xs + i, make_float4(v.x * sigmoid(g.x), v.y * sigmoid(g.y), v.z * sigmoid(g.z), v.w * sigmoid(g.w)));
            }
            for (int i = m_.width + t; i < padded; i += kThreads) xs[i] = 0.f;
        } else if (m_.norm) {
            group_inverse_rms<kThreads>([&](int i) { return m_.row[i]; }, m_.width, H, m_.eps, inv, red);
            fill_row(xs, m_.width, padded, [&](int i) { return m_.row[i] * inv[i / m_.vdim] * m_.norm[i] * sigmoid(m_.gates[i]); });
        } else {
            copy_row(xs, m_.row, m_.width, padded);
        }
    }

   private:
    static constexpr int kShares = kMixerShares, kQuads = 2;
    __device__ __forceinline__ float2 stat(int k, int h) const {
        return *reinterpret_cast<const float2*>(m_.shares.stats + 2 * ((size_t)k * m_.heads + h));
    }
    __device__ __forceinline__ const float* share_row(int k, int h) const {
        return m_.shares.part + ((size_t)k * m_.heads + h) * m_.shares.ld;
    }
    __device__ __forceinline__ void request_shares(int q0) {
#pragma unroll
        for (int u = 0; u < kQuads; u++) {
            const int i = min(4 * (q0 + u * kThreads + (int)threadIdx.x), m_.width - 4), h = i / m_.vdim;
#pragma unroll
            for (int k = 0; k < kShares; k++) shares_[u][k] = load4(share_row(min(k, m_.shares.splits - 1), h) + (i - h * m_.vdim));
        }
    }
    const MixerRow& m_;
    RowParts<kThreads> parts_;
    bool quads_, normed_;
    float2 stats_[kShares];
    float4 shares_[kQuads][kShares], row_[RowParts<kThreads>::kParts], norm_[RowParts<kThreads>::kParts], gate_[RowParts<kThreads>::kParts];
};

// y[n] = W_o[n] . mixer row + sum_k weights[k] W_e(k)[n] . act_k, as one row of W_o's and the chosen experts' chunks in turn;
// the experts' weights are in the activations.
template <typename T>
__global__ __launch_bounds__(kThreads) void gemv_mixer_down_kernel(MixerRow m, const T* __restrict__ wo, int ld_wo, ExpertRows e,
                                                                  const float* __restrict__ act, const T* __restrict__ experts, int ld,
                                                                  int N, float* __restrict__ y) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ int chosen[kMaxTop];
    const int t = threadIdx.x;
    const int chunks = ld * (int)sizeof(T) / 16, chunks_wo = ld_wo * (int)sizeof(T) / 16, all = chunks_wo + e.top * chunks;
    const int pairs = (N + 1) / 2;
    float *xs = smem, *xs_experts = xs + ld_wo, *red = xs_experts + e.top * ld, *inv = red + kThreads / 64;
    const Deal d = deal_rows<T>(all, gridDim.x);
    const float per_chunk = 1.0f / (float)max(chunks, 1);
    auto load = [&](Pair& p, int n, int c) __attribute__((always_inline)) {
        const int second = 2 * n + 1 < N ? 1 : 0;
#pragma unroll
        for (int u = 0; u < kAhead; u++) {
            int at = min(c + u * d.lanes, all - 1);
            size_t row = 2 * (size_t)n;
            const T* w = wo;
            int stride = ld_wo;
            if (at >= chunks_wo) {
                at -= chunks_wo;
                const int k = (int)(((float)at + 0.5f) * per_chunk);
                at -= k * chunks;
                row += (size_t)chosen[k] * N;
                w = experts;
                stride = ld;
            }
            const uint4* src = reinterpret_cast<const uint4*>(w + row * stride) + at;
            p.a[u] = *src;
            p.b[u] = *reinterpret_cast<const uint4*>(reinterpret_cast<const T*>(src) + (second ? stride : 0));
        }
    };
    Pair ahead;
    MixerPrologue row(m);
    row.load();
    const bool early = kAhead * d.lanes <= chunks_wo;  // the first step is W_o's alone
    if (early && d.group < pairs) load(ahead, d.group, d.at);
    if (t < e.top) chosen[t] = min(max(e.chosen[t], 0), e.experts - 1);
    if ((e.ff & 3) == 0) {
        for (int i = t; i < e.top * (e.ff >> 2); i += kThreads) {
            const int k = i / (e.ff >> 2), c = 4 * (i - k * (e.ff >> 2));
            const float w = e.weights[k];
            const float4 v = load4(act + (size_t)k * e.ld_act + c);
            store4(xs_experts + k * ld + c, make_float4(w * v.x, w * v.y, w * v.z, w * v.w));
        }
        for (int i = t; i < e.top * (ld - e.ff); i += kThreads) {
            const int k = i / (ld - e.ff);
            xs_experts[k * ld + e.ff + (i - k * (ld - e.ff))] = 0.f;
        }
    } else {
        for (int k = 0; k < e.top; k++) {
            const float w = e.weights[k];
            fill_row(xs_experts + k * ld, e.ff, ld, [&](int i) { return w * act[(size_t)k * e.ld_act + i]; });
        }
    }
    if (!early) {
        dense_lds_barrier();
        if (d.group < pairs) load(ahead, d.group, d.at);
    }
    row.finish(xs, ld_wo, inv, red);
    dense_lds_barrier();
    const int per_step = kAhead * d.lanes, steps = (all + per_step - 1) / per_step;
    for (int n = d.group; n < pairs; n += d.groups) {
        float s0 = 0.f, s1 = 0.f;
        for (int step = 0; step < steps; step++) {
            const int c = d.at + step * per_step;
            const Pair now = ahead;
            if (step + 1 < steps)
                load(ahead, n, c + per_step);
            else if (n + d.groups < pairs)
                load(ahead, n + d.groups, d.at);
            use_pair<T>(now, xs, c, d.lanes, all, s0, s1);
        }
        s0 = dense_wave_sum(s0, d.lanes);
        s1 = dense_wave_sum(s1, d.lanes);
        if (d.at == 0) PlainEmit{y, N, 1.f}(n, s0, s1);
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
    // behind a router a workgroup first has to learn its expert: two rounds of rows for each of the 512 that fit the chip at once
    const int limit = e.logits && slots < 16 ? 512 / slots : e.logits ? 32 : kMaxGrid;
    hipLaunchKernelGGL(gemv_gate_up_kernel<T>, dim3(workgroups<T>(2 * most, ld, limit), slots), dim3(kThreads), lds > router ? lds : router, s,
                       p, h, e, experts, dense, ld, act);
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
    const int row = ld_wo + e.top * ld, inv = m.shares.part ? m.heads * kMixerShares : m.heads;
    const size_t lds = (row + kThreads / 64 + inv) * sizeof(float);
    hipLaunchKernelGGL(gemv_mixer_down_kernel<T>, dim3(workgroups<T>(N, row, kMaxGrid)), dim3(kThreads), lds, s, m, wo, ld_wo, e, act,
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
