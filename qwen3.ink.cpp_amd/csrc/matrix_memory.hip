// Matrix memory with exponential gates: a recurrence over tokens whose state per head is a matrix S, a vector n and a
// scale m (dense.h has the equations).  Everything here is fp32, gate sums fp64.
//
// A prompt goes in chunks of 64 tokens.  With f_t, i_t the gates' logarithms, b_t = f_1 + .. + f_t inside the chunk,
// a_s = i_s - b_s and m_0, S_0, n_0 the state before the chunk, the recurrence unrolls to
//   M_t = max(m_0, max_{s <= t} a_s),   m_t = b_t + M_t
//   S_t = e^(m_0 - M_t) S_0 + sum_{s <= t} e^(a_s - M_t) k_s v_s^T          (n_t likewise)
//   S_t^T q_t = e^(m_0 - M_t) S_0^T q_t + sum_{s <= t} e^(a_s - M_t) (q_t . k_s) v_s
// so that a chunk needs S only at its start.  Three launches: every chunk's own sum over s for t = its last token (outer
// products, all chunks at once); the chain over chunks, element by element; the outputs of all chunks.
#include "dense_common.h"

namespace a81w41 {
namespace {

constexpr int kThreads = 256, C = kMemoryChunk;
static_assert(C == 64, "the lanes of a wave hold a chunk's gates");

__device__ __forceinline__ float soft_cap(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
struct Gates {
    float log_in, log_keep;
};
__device__ __forceinline__ Gates gates_of(const MemoryArgs& a, int m, int h) {
    const float* row = a.in + (size_t)m * a.ld_in;
    Gates g;
    g.log_in = soft_cap(row[a.sh.at_i + h] + a.bias_i[h], a.sh.cap);
    g.log_keep = log_sigmoid(soft_cap(row[a.sh.at_f + h] + a.bias_f[h], a.sh.cap));
    return g;
}

__device__ __forceinline__ double shfl_up(double v, int by) {
    const long long u = __double_as_longlong(v);
    const int lo = __shfl_up((int)u, by, 64), hi = __shfl_up((int)(u >> 32), by, 64);
    return __longlong_as_double(((long long)hi << 32) | (unsigned)lo);
}
// One wave, lane t = token t of the chunk: b_t, a_t and max_{s <= t} a_s; tokens from `count` on change nothing.
struct ChunkGates {
    double b, a, most;
};
__device__ __forceinline__ ChunkGates chunk_gates(const MemoryArgs& p, int m0, int count, int h) {
    const int t = threadIdx.x & 63;
    const Gates g = gates_of(p, m0 + min(t, count - 1), h);
    ChunkGates c;
    c.b = t < count ? (double)g.log_keep : 0.0;
    for (int off = 1; off < 64; off <<= 1) {
        const double other = shfl_up(c.b, off);
        if (t >= off) c.b += other;
    }
    c.a = t < count ? (double)g.log_in - c.b : -1e300;
    c.most = c.a;
    for (int off = 1; off < 64; off <<= 1) {
        const double other = shfl_up(c.most, off);
        if (t >= off) c.most = fmax(c.most, other);
    }
    return c;
}

__device__ __forceinline__ float* state_nm(const MemoryArgs& a, int parity) {
    return a.state + a.sh.s_size() + (size_t)(parity & 1) * a.sh.heads * (a.sh.dim + 1);
}

// Token by token.  A workgroup has kSlice columns of one head's S; W columns and every (kThreads W / kSlice)-th row of them
// are a thread's, in registers only while a token uses them.  n and m are formed by every workgroup of the head; the first
// writes them to the copy that nobody reads.
constexpr int kSlice = 32;
template <int W>
__global__ __launch_bounds__(kThreads) void memory_steps_kernel(MemoryArgs a, float* __restrict__ o) {
    constexpr int kPer = kSlice / W, kRows = kThreads / kPer;  // threads of a row of the slice, rows worked on at a time
    extern __shared__ float smem[];
    const MemoryShape sh = a.sh;
    float *n = smem, *q = n + sh.dim, *k = q + sh.dim, *sums = k + sh.dim, *red = sums + kRows * kSlice;
    const int t = threadIdx.x, h = blockIdx.y, pos = max(a.pos_dev[0], 0);
    const int c = blockIdx.x * kSlice + (t % kPer) * W, r0 = t / kPer;
    const bool mine = c < sh.vdim;  // W > 1: vdim is a multiple of W
    float* S = a.state + (size_t)h * sh.dim * sh.vdim;
    const float* nm = state_nm(a, pos) + (size_t)h * (sh.dim + 1);
    for (int d = t; d < sh.dim; d += kThreads) n[d] = nm[d];
    float m = nm[sh.dim];
    for (int token = 0; token < a.M; token++) {
        const float* row = a.in + (size_t)token * a.ld_in;
        const Gates g = gates_of(a, token, h);
        const float next = fmaxf(g.log_keep + m, g.log_in), keep = expf(g.log_keep + m - next), add = expf(g.log_in - next);
        m = next;
        float nq = 0.f;
        for (int d = t; d < sh.dim; d += kThreads) {
            q[d] = row[sh.at_q + h * sh.dim + d] * sh.q_scale;
            k[d] = add * row[sh.at_k + h * sh.dim + d];
            n[d] = fmaf(keep, n[d], k[d]);
            nq = fmaf(n[d], q[d], nq);
        }
        nq = dense_wave_sum(nq);
        if ((t & 63) == 0) red[t >> 6] = nq;
        __syncthreads();
        float acc[W], v[W];
#pragma unroll
        for (int w = 0; w < W; w++) {
            acc[w] = 0.f;
            v[w] = mine ? row[sh.at_v + h * sh.vdim + c + w] : 0.f;
        }
        if (mine) {
#pragma unroll 8
            for (int d = r0; d < sh.dim; d += kRows) {
                float* at = S + (size_t)d * sh.vdim + c;
                float s[W];
                if constexpr (W == 4)
                    *reinterpret_cast<float4*>(s) = load4(at);
                else
                    s[0] = at[0];
#pragma unroll
                for (int w = 0; w < W; w++) {
                    s[w] = fmaf(keep, s[w], k[d] * v[w]);
                    acc[w] = fmaf(s[w], q[d], acc[w]);
                }
                if constexpr (W == 4)
                    store4(at, *reinterpret_cast<const float4*>(s));
                else
                    at[0] = s[0];
            }
        }
#pragma unroll
        for (int w = 0; w < W; w++) sums[r0 * kSlice + (t % kPer) * W + w] = acc[w];
        __syncthreads();
        const int col = blockIdx.x * kSlice + t;
        if (t < kSlice && col < sh.vdim) {
            float s = 0.f, den = 0.f;
            for (int r = 0; r < kRows; r++) s += sums[r * kSlice + t];
            for (int w = 0; w < kThreads / 64; w++) den += red[w];
            o[((size_t)token * sh.heads + h) * sh.vdim + col] = s / (fmaxf(fabsf(den), expf(-m)) + kMemoryFloor);
        }
        __syncthreads();
    }
    if (blockIdx.x == 0) {
        float* out = state_nm(a, pos + a.M) + (size_t)h * (sh.dim + 1);
        for (int d = t; d < sh.dim; d += kThreads) out[d] = n[d];
        if (t == 0) out[sh.dim] = m;
    }
}

// One workgroup per token.
template <typename T>
__global__ __launch_bounds__(kThreads) void memory_norm_kernel(MemoryArgs a, const float* __restrict__ o, T* __restrict__ out, int ld_out) {
    extern __shared__ float smem[];
    const int width = a.sh.heads * a.sh.vdim;
    float *inv = smem, *red = inv + a.sh.heads;
    const float *row = o + (size_t)blockIdx.x * width, *gate = a.in + (size_t)blockIdx.x * a.ld_in + a.sh.at_g;
    group_inverse_rms<kThreads>([&](int i) { return row[i]; }, width, a.sh.heads, a.sh.eps, inv, red);
    T* dst = out + (size_t)blockIdx.x * ld_out;
    for (int i = threadIdx.x; i < width; i += kThreads) dst[i] = (T)(row[i] * inv[i / a.sh.vdim] * a.norm[i] * sigmoid(gate[i]));
}

__device__ __forceinline__ f32x16 mfma32(float a, float b, f32x16 c) { return __builtin_amdgcn_mfma_f32_32x32x2f32(a, b, c, 0, 0, 0); }

// W floats (4: aligned to 16 bytes), zeros where there are none
template <int W>
__device__ __forceinline__ void read_part(float* part, const float* src, bool real) {
    if constexpr (W == 4) {
        const float4 v = real ? load4(src) : make_float4(0.f, 0.f, 0.f, 0.f);
        part[0] = v.x, part[1] = v.y, part[2] = v.z, part[3] = v.w;
    } else {
        part[0] = real ? src[0] : 0.f;
    }
}
template <int W>
__device__ __forceinline__ void write_part(float* dst, const float* part) {
    if constexpr (W == 4)
        store4(dst, make_float4(part[0], part[1], part[2], part[3]));
    else
        dst[0] = part[0];
}

// A chunk's own sums for its last token: sum_s w_s k_s v_s^T and sum_s w_s k_s with w_s = e^(a_s - max a).  A workgroup has
// a 128 x 128 tile of a head's S; its waves take the 32 x 32 pieces in turn.  K and V sit in LDS as [token][column], column
// c of token s at place c ^ 32 (s & 1): the two tokens a matrix operand takes at a time lie in different banks.
constexpr int kOuter = 128;
template <int W>
__global__ __launch_bounds__(kThreads) void memory_outer_kernel(MemoryArgs a) {
    constexpr int kPer = kOuter / W, kLoads = C * kPer / kThreads, kBatch = W == 4 ? kLoads : 8;
    __shared__ __attribute__((aligned(16))) float ks[C * kOuter], vs[C * kOuter], weight[C];
    const MemoryShape sh = a.sh;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l31 = lane & 31, half = lane >> 5;
    const int chunk = blockIdx.x, h = blockIdx.y, m0 = chunk * C, count = min(C, a.M - m0);
    const int v_tiles = (sh.vdim + kOuter - 1) / kOuter, d0 = blockIdx.z / v_tiles * kOuter, v0 = blockIdx.z % v_tiles * kOuter;
    const int nd = min(kOuter, sh.dim - d0), nv = min(kOuter, sh.vdim - v0);
    const int cols_k = (nd + 31) / 32 * 32, cols_v = (nv + 31) / 32 * 32;
    // the rows are requested before the gates are formed
    float k_part[kBatch][W], v_part[kBatch][W];
    auto request = [&](int first) {
#pragma unroll
        for (int u = 0; u < kBatch; u++) {
            const int i = t + (first + u) * kThreads, s = i / kPer, c = i % kPer * W;
            const float* row = a.in + (size_t)(m0 + min(s, count - 1)) * a.ld_in;
            read_part<W>(k_part[u], row + sh.at_k + h * sh.dim + d0 + c, s < count && c < nd);
            read_part<W>(v_part[u], row + sh.at_v + h * sh.vdim + v0 + c, s < count && c < nv);
        }
    };
    request(0);
    if (wave == 0) {
        const ChunkGates g = chunk_gates(a, m0, count, h);
        const double most = __shfl(g.most, 63, 64);
        weight[lane] = lane < count ? expf((float)(g.a - most)) : 0.f;
        if (lane == 63 && blockIdx.z == 0) {
            float* st = a.chunk_stats + 2 * ((size_t)chunk * sh.heads + h);
            st[0] = (float)most;
            st[1] = (float)g.b;
        }
    }
    dense_lds_barrier();
    for (int first = 0; first < kLoads; first += kBatch) {
        if (first) request(first);
#pragma unroll
        for (int u = 0; u < kBatch; u++) {
            const int i = t + (first + u) * kThreads, s = i / kPer, c = i % kPer * W, at = s * kOuter + (c ^ ((s & 1) << 5));
            const float w = weight[s];
#pragma unroll
            for (int e = 0; e < W; e++) k_part[u][e] *= w;
            write_part<W>(ks + at, k_part[u]);
            write_part<W>(vs + at, v_part[u]);
        }
    }
    __syncthreads();
    float* out = a.chunk_states + ((size_t)chunk * sh.heads + h) * sh.chunk_size();
    const int v_pieces = cols_v / 32, pieces = cols_k / 32 * v_pieces;
    for (int piece = wave; piece < pieces; piece += kThreads / 64) {
        const int pd = piece / v_pieces * 32, pv = piece % v_pieces * 32;
        f32x16 acc;
#pragma unroll
        for (int i = 0; i < 16; i++) acc[i] = 0.f;
#pragma unroll 8
        for (int s = 0; s < C; s += 2) {
            const int row = (s + half) * kOuter, turn = half << 5;
            acc = mfma32(ks[row + ((pd + l31) ^ turn)], vs[row + ((pv + l31) ^ turn)], acc);
        }
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int d = pd + 8 * (i >> 2) + 4 * half + (i & 3), v = pv + l31;
            if (d < nd && v < nv) out[(size_t)(d0 + d) * sh.vdim + v0 + v] = acc[i];
        }
    }
    if (v0 == 0 && t < nd) {
        float s = 0.f;
#pragma unroll 8
        for (int k = 0; k < C; k++) s += ks[k * kOuter + (t ^ ((k & 1) << 5))];
        out[(size_t)sh.dim * sh.vdim + d0 + t] = s;
    }
}

// The chain over chunks for W neighbouring elements of a head's S and n: chunk_states becomes the state before each chunk,
// the state itself the one after the last; chunk_m the scales.
template <int W>
__global__ __launch_bounds__(kThreads) void memory_chain_kernel(MemoryArgs a, int chunks) {
    constexpr int kAhead = 4;
    const MemoryShape sh = a.sh;
    const int h = blockIdx.y, pos = max(a.pos_dev[0], 0);
    const size_t e = ((size_t)blockIdx.x * kThreads + threadIdx.x) * W, s_size = (size_t)sh.dim * sh.vdim, size = sh.chunk_size();
    const size_t nm = (size_t)h * (sh.dim + 1);
    float m = state_nm(a, pos)[nm + sh.dim];
    const bool scale_writer = e == 0;
    if (e >= size) return;
    const bool in_s = e < s_size;  // W > 1: the parts are whole multiples of W
    const float* from = in_s ? a.state + h * s_size + e : state_nm(a, pos) + nm + (e - s_size);
    float* to = in_s ? a.state + h * s_size + e : state_nm(a, pos + a.M) + nm + (e - s_size);
    float cur[W];
#pragma unroll
    for (int w = 0; w < W; w++) cur[w] = from[w];
    const size_t step = (size_t)sh.heads * size;
    float* at = a.chunk_states + h * size + e;
    auto load = [&](float* dst, int c) {
        const float* src = at + (size_t)min(c, chunks - 1) * step;
        if constexpr (W == 4)
            *reinterpret_cast<float4*>(dst) = load4(src);
        else
            dst[0] = src[0];
    };
    alignas(16) float next[kAhead][W];
#pragma unroll
    for (int u = 0; u < kAhead; u++) load(next[u], u);
    for (int c0 = 0; c0 < chunks; c0 += kAhead) {
        alignas(16) float now[kAhead][W];
#pragma unroll
        for (int u = 0; u < kAhead; u++)
#pragma unroll
            for (int w = 0; w < W; w++) now[u][w] = next[u][w];
        if (c0 + kAhead < chunks) {
#pragma unroll
            for (int u = 0; u < kAhead; u++) load(next[u], c0 + kAhead + u);
        }
#pragma unroll
        for (int u = 0; u < kAhead; u++) {
            const int c = c0 + u;
            if (c >= chunks) break;
            const float* st = a.chunk_stats + 2 * ((size_t)c * sh.heads + h);
            const float most = fmaxf(m, st[0]), keep = expf(m - most), add = expf(st[0] - most);
            if (scale_writer) a.chunk_m[(size_t)c * sh.heads + h] = m;
            if constexpr (W == 4)
                store4(at + c * step, *reinterpret_cast<const float4*>(cur));
            else
                at[c * step] = cur[0];
#pragma unroll
            for (int w = 0; w < W; w++) cur[w] = fmaf(keep, cur[w], add * now[u][w]);
            m = st[1] + most;
        }
    }
#pragma unroll
    for (int w = 0; w < W; w++) to[w] = cur[w];
    if (scale_writer) a.chunk_m[(size_t)chunks * sh.heads + h] = m;
}

// Outputs of a chunk for one head, 64 tokens x vdim columns in the accumulators: 64 x 32 VF per wave.  q and k come through
// LDS, 64 columns at a time; rows of S and v go from memory to the matrix operands, requested ahead of the barriers.
constexpr int kStep = 64;          // columns of q and k in LDS at a time
constexpr int kLd = kStep + 4;     // floats of an LDS row: sixteen-byte reads of neighbouring rows spread over the banks
template <typename T, int W, int WAVES, int VF>
__global__ __launch_bounds__(64 * WAVES) void memory_outputs_kernel(MemoryArgs a, int chunks, T* __restrict__ out, int ld_out) {
    constexpr int kT = 64 * WAVES, kPer = kStep / W, kLoads = C * kPer / kT;
    constexpr int kTeam = kT / C;  // threads that share a token's sums
    __shared__ __attribute__((aligned(16))) float qs[C * kLd], ks[C * kLd];  // ks holds the weighted scores afterwards
    __shared__ double log_a[C], log_most[C];                                // a_s, M_t
    __shared__ float start[C], floor_t[C], den[C], inv[C], squares[C][WAVES], n_part[kStep];
    const MemoryShape sh = a.sh;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l31 = lane & 31, half = lane >> 5;
    const int chunk = blockIdx.x, h = blockIdx.y, m0 = chunk * C, count = min(C, a.M - m0);
    const float m_start = a.chunk_m[(size_t)chunk * sh.heads + h];
    const float* S = a.chunk_states + ((size_t)chunk * sh.heads + h) * sh.chunk_size();
    const float* n = S + (size_t)sh.dim * sh.vdim;
    const int col0 = wave * 32 * VF + l31;
    float q_part[kLoads][W], k_part[kLoads][W], n_own = 0.f;
    auto request = [&](int d0) {
#pragma unroll
        for (int u = 0; u < kLoads; u++) {
            const int i = t + u * kT, s = i / kPer, d = d0 + i % kPer * W;
            const float* row = a.in + (size_t)(m0 + min(s, count - 1)) * a.ld_in + h * sh.dim + d;
            const bool real = s < count && d < sh.dim;
            read_part<W>(q_part[u], row + sh.at_q, real);
            read_part<W>(k_part[u], row + sh.at_k, real);
        }
        if (t < kStep) n_own = d0 + t < sh.dim ? n[d0 + t] : 0.f;
    };
    constexpr int kHalf = kStep / 16;  // operand steps of eight columns: half of those of a pass
    float b[kHalf][VF][4];
    auto request_states = [&](int d0) {
#pragma unroll
        for (int kk = 0; kk < kHalf; kk++)
#pragma unroll
            for (int f = 0; f < VF; f++)
#pragma unroll
                for (int j = 0; j < 4; j++)
                    b[kk][f][j] = S[(size_t)min(d0 + 4 * (2 * kk + half) + j, sh.dim - 1) * sh.vdim + min(col0 + 32 * f, sh.vdim - 1)];
    };
    request(0);
    if (wave == 0) {
        const ChunkGates g = chunk_gates(a, m0, count, h);
        const double most = fmax((double)m_start, g.most);
        log_a[lane] = g.a;
        log_most[lane] = most;
        start[lane] = expf((float)((double)m_start - most));
        floor_t[lane] = expf(-(float)(g.b + most));
    }
    // the scale after the last chunk goes to the state only now: the chain's workgroups all read the old one
    if (chunk == chunks - 1 && t == 0)
        state_nm(a, max(a.pos_dev[0], 0) + a.M)[(size_t)h * (sh.dim + 1) + sh.dim] = a.chunk_m[(size_t)chunks * sh.heads + h];
    f32x16 acc[2][VF], score;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        score[i] = 0.f;
#pragma unroll
        for (int f = 0; f < VF; f++) acc[0][f][i] = acc[1][f][i] = 0.f;
    }
    // this wave's piece of the scores, tokens st.. and keys ss..; the waves from 4 on take every second operand step
    const int st = (wave & 1) * 32, ss = (wave >> 1 & 1) * 32;
    float nq = 0.f;  // of token t / kTeam, a share of the columns
    for (int d0 = 0; d0 < sh.dim; d0 += kStep) {
        request_states(d0);
        if (d0) dense_lds_barrier();  // nobody still reads the columns before
#pragma unroll
        for (int u = 0; u < kLoads; u++) {
            const int i = t + u * kT, at = i / kPer * kLd + i % kPer * W;
#pragma unroll
            for (int e = 0; e < W; e++) q_part[u][e] *= sh.q_scale;
            write_part<W>(qs + at, q_part[u]);
            write_part<W>(ks + at, k_part[u]);
        }
        if (t < kStep) n_part[t] = n_own;
        dense_lds_barrier();
        if (d0 + kStep < sh.dim) request(d0 + kStep);
#pragma unroll
        for (int part = 0; part < 2; part++) {
            if (part) request_states(d0 + kStep / 2);
            if (d0 + part * (kStep / 2) >= sh.dim) break;
#pragma unroll
            for (int kk = 0; kk < kHalf; kk++) {
                const int step = part * kHalf + kk, at = 4 * (2 * step + half);
                alignas(16) float q[2][4], k[4];
#pragma unroll
                for (int i = 0; i < 2; i++) *reinterpret_cast<float4*>(q[i]) = load4(qs + (i * 32 + l31) * kLd + at);
#pragma unroll
                for (int f = 0; f < VF; f++)
#pragma unroll
                    for (int j = 0; j < 4; j++)
#pragma unroll
                        for (int i = 0; i < 2; i++) acc[i][f] = mfma32(q[i][j], b[kk][f][j], acc[i][f]);
                // a piece whose keys all come later counts nothing
                if (ss <= st && (WAVES == 4 || (step & 1) == wave >> 2)) {
                    *reinterpret_cast<float4*>(k) = load4(ks + (ss + l31) * kLd + at);
#pragma unroll
                    for (int j = 0; j < 4; j++) score = mfma32(st ? q[1][j] : q[0][j], k[j], score);
                }
            }
        }
#pragma unroll
        for (int c = 0; c < kStep / kTeam; c++) {
            const int d = t % kTeam + kTeam * c;
            nq = fmaf(qs[t / kTeam * kLd + d], n_part[d], nq);
        }
    }
    // the first rows of v, while the scores are weighted
    constexpr int kRowsAhead = 4;
    const float* v_rows = a.in + sh.at_v + h * sh.vdim;
    float v[kRowsAhead][VF][4];
    auto request_values = [&](int kk0) {
#pragma unroll
        for (int kk = 0; kk < kRowsAhead; kk++)
#pragma unroll
            for (int f = 0; f < VF; f++)
#pragma unroll
                for (int j = 0; j < 4; j++)
                    v[kk][f][j] = v_rows[(size_t)(m0 + min(4 * (2 * (kk0 + kk) + half) + j, count - 1)) * a.ld_in + min(col0 + 32 * f, sh.vdim - 1)];
    };
    request_values(0);
    dense_lds_barrier();
    float* weighted = ks;  // [token][key]
    for (int turn = 0; turn < WAVES / 4; turn++) {
        if (wave >> 2 == turn) {
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const int token = st + 8 * (i >> 2) + 4 * half + (i & 3), key = ss + l31;
                float& w = weighted[token * kLd + key];
                const float own = key <= token ? score[i] * expf((float)(log_a[key] - log_most[token])) : 0.f;
                w = turn ? w + own : own;
            }
        }
        dense_lds_barrier();
    }
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const float w = start[i * 32 + 8 * (r >> 2) + 4 * half + (r & 3)];
#pragma unroll
            for (int f = 0; f < VF; f++) acc[i][f][r] *= w;
        }
    {
        const int token = t / kTeam;
        float sum = nq * start[token];
#pragma unroll
        for (int c = 0; c < C / kTeam; c++) sum += weighted[token * kLd + t % kTeam + kTeam * c];
        sum = dense_wave_sum(sum, kTeam);
        if (t % kTeam == 0) den[token] = 1.0f / (fmaxf(fabsf(sum), floor_t[token]) + kMemoryFloor);
    }
#pragma unroll
    for (int kk0 = 0; kk0 < C / 8; kk0 += kRowsAhead) {
        if (kk0) request_values(kk0);
#pragma unroll
        for (int kk = 0; kk < kRowsAhead; kk++) {
            const int at = 4 * (2 * (kk0 + kk) + half);
            alignas(16) float p[2][4];
#pragma unroll
            for (int i = 0; i < 2; i++) *reinterpret_cast<float4*>(p[i]) = load4(weighted + (i * 32 + l31) * kLd + at);
#pragma unroll
            for (int f = 0; f < VF; f++)
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    if (kk0 + kk < C / 16) acc[0][f] = mfma32(p[0][j], v[kk][f][j], acc[0][f]);
                    acc[1][f] = mfma32(p[1][j], v[kk][f][j], acc[1][f]);
                }
        }
    }
    dense_lds_barrier();
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int token = i * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
            const float d = den[token];
            float sum = 0.f;
#pragma unroll
            for (int f = 0; f < VF; f++) {
                acc[i][f][r] *= d;
                if (col0 + 32 * f < sh.vdim) sum = fmaf(acc[i][f][r], acc[i][f][r], sum);
            }
            sum = dense_wave_sum(sum, 32);
            if (l31 == 0) squares[token][wave] = sum;
        }
    __syncthreads();
    if (t < C) {
        float sum = 0.f;
        for (int w = 0; w < WAVES; w++) sum += squares[t][w];
        inv[t] = 1.0f / sqrtf(sum / (float)sh.vdim + sh.eps);
    }
    __syncthreads();
#pragma unroll
    for (int f = 0; f < VF; f++) {
        const int col = col0 + 32 * f;
        if (col >= sh.vdim) continue;
        const float w = a.norm[h * sh.vdim + col];
#pragma unroll
        for (int i = 0; i < 2; i++) {
            float gate[16];
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int token = min(i * 32 + 8 * (r >> 2) + 4 * half + (r & 3), count - 1);
                gate[r] = a.in[(size_t)(m0 + token) * a.ld_in + sh.at_g + h * sh.vdim + col];
            }
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int token = i * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
                if (token < count)
                    out[(size_t)(m0 + token) * ld_out + h * sh.vdim + col] = (T)(acc[i][f][r] * inv[token] * w * sigmoid(gate[r]));
            }
        }
    }
}

// whether heads, rows and what is read of them are whole float4s
bool whole_quads(const MemoryArgs& a) {
    const MemoryShape& sh = a.sh;
    return (sh.dim | sh.vdim | a.ld_in | sh.at_q | sh.at_k | sh.at_v) % 4 == 0;
}

template <typename T, int W>
hipError_t launch_chunks(const MemoryArgs& a, T* out, int ld_out, hipStream_t s) {
    const MemoryShape& sh = a.sh;
    const int chunks = (a.M + C - 1) / C, tiles = ((sh.dim + kOuter - 1) / kOuter) * ((sh.vdim + kOuter - 1) / kOuter);
    const int parts = (int)(sh.chunk_size() / W);
    hipLaunchKernelGGL(memory_outer_kernel<W>, dim3(chunks, sh.heads, tiles), dim3(kThreads), 0, s, a);
    hipLaunchKernelGGL(memory_chain_kernel<W>, dim3((parts + kThreads - 1) / kThreads, sh.heads), dim3(kThreads), 0, s, a, chunks);
    const dim3 grid(chunks, sh.heads);
    if (sh.vdim <= 128)
        hipLaunchKernelGGL((memory_outputs_kernel<T, W, 4, 1>), grid, dim3(256), 0, s, a, chunks, out, ld_out);
    else if (sh.vdim <= 256)
        hipLaunchKernelGGL((memory_outputs_kernel<T, W, 8, 1>), grid, dim3(512), 0, s, a, chunks, out, ld_out);
    else
        hipLaunchKernelGGL((memory_outputs_kernel<T, W, 8, 2>), grid, dim3(512), 0, s, a, chunks, out, ld_out);
    return hipGetLastError();
}

}  // namespace

hipError_t launch_memory_steps(const MemoryArgs& a, float* o, hipStream_t s) {
    const dim3 grid((a.sh.vdim + kSlice - 1) / kSlice, a.sh.heads);
    auto lds = [&](int w) { return (3 * (size_t)a.sh.dim + kThreads * w + kThreads / 64) * sizeof(float); };
    if (a.sh.vdim % 4 == 0)
        hipLaunchKernelGGL(memory_steps_kernel<4>, grid, dim3(kThreads), lds(4), s, a, o);
    else
        hipLaunchKernelGGL(memory_steps_kernel<1>, grid, dim3(kThreads), lds(1), s, a, o);
    return hipGetLastError();
}

template <typename T>
hipError_t launch_memory_norm(const MemoryArgs& a, const float* o, T* out, int ld_out, hipStream_t s) {
    hipLaunchKernelGGL(memory_norm_kernel<T>, dim3(a.M), dim3(kThreads), (a.sh.heads + kThreads / 64) * sizeof(float), s, a, o, out, ld_out);
    return hipGetLastError();
}

bool memory_chunks_fit(const MemoryShape& sh) { return sh.vdim <= 512; }

template <typename T>
hipError_t launch_memory_chunks(const MemoryArgs& a, T* out, int ld_out, hipStream_t s) {
    return whole_quads(a) ? launch_chunks<T, 4>(a, out, ld_out, s) : launch_chunks<T, 1>(a, out, ld_out, s);
}

#define INSTANTIATE(T)                                                                                   \
    template hipError_t launch_memory_norm<T>(const MemoryArgs&, const float*, T*, int, hipStream_t);     \
    template hipError_t launch_memory_chunks<T>(const MemoryArgs&, T*, int, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)

}  // namespace a81w41
