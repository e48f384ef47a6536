// The parity hooks of include/a81w41_dense.h: argument checks in front of the launchers.
#include "../../include/a81w41_dense.h"

#include <algorithm>
#include <cmath>

#include "decoder_session.h"
#include "dense.h"

using namespace a81w41;

namespace {
bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
template <typename T>
int gemm(const void* A, int lda, const void* W, int ldw, float* C, int ldc, int M, int N, int K, hipStream_t s) {
    constexpr int step = 128 / (int)sizeof(T);
    if (lda % step || ldw % step || lda < pad_k<T>(K) || ldw < pad_k<T>(K) || ldc < N)
        return failf(A81W41_ERR_INVALID_ARG, "row strides must be whole multiples of 128 bytes and cover K");
    GemmArgs g;
    g.A = A, g.W = W, g.C = C, g.M = M, g.N = N, g.K = pad_k<T>(K), g.lda = lda, g.ldw = ldw, g.ldc = ldc;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    return 0;
}
}  // namespace

extern "C" {

int a81w41_dense_gemm(const void* A, int lda, const void* W, int ldw, float* C, int ldc, int M, int N, int K, int is_bf16, void* stream) {
    if (!A || !W || !C || M < 1 || N < 1 || K < 1 || !aligned16(A) || !aligned16(W)) return failf(A81W41_ERR_INVALID_ARG, "bad product");
    hipStream_t s = static_cast<hipStream_t>(stream);
    return is_bf16 ? gemm<bf16>(A, lda, W, ldw, C, ldc, M, N, K, s) : gemm<float>(A, lda, W, ldw, C, ldc, M, N, K, s);
}

int a81w41_latent_attention(const void* q, const void* cache, int ld, int rank, int rot, int heads, const int* pos_dev, int max_seq, int M,
                            float scale, void* out, int is_bf16, int variant, int splits, float* part, float* stats, void* stream) {
    if (!q || !cache || !pos_dev || !out || rank < 1 || rot < 0 || heads < 1 || max_seq < 1 || M < 1 || rank + rot > 4096 ||
        ld < rank + rot || ld % (is_bf16 ? 64 : 32) || variant < 0 || variant > 1 || !aligned16(q) || !aligned16(cache))
        return failf(A81W41_ERR_INVALID_ARG, "bad attention shape");
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int width = (rank + rot + 7) / 8 * 8;
    auto set = [&](auto& a, auto type) {
        using T = decltype(type);
        a.q = static_cast<const T*>(q), a.ld_q = ld, a.q_token = heads * ld, a.rows = M * heads, a.rows_per_token = heads;
        a.k_own = static_cast<const T*>(cache), a.ld_k_own = ld, a.k_own_width = width, a.dv = rank;
        a.ld_out = rank, a.out_token = heads * rank, a.scale = scale, a.pos_dev = pos_dev, a.max_seq = max_seq;
    };
    AttendArgs<float> af;
    AttendArgs<bf16> a;
    if (!is_bf16) {
        if (variant) return failf(A81W41_ERR_INVALID_ARG, "the matrix-core attention does not take this shape");
        set(af, 0.f);
        A81W41_HIP_TRY((launch_attend_vector<float, float>(af, 1, static_cast<float*>(out), s)));
        return 0;
    }
    set(a, bf16{});
    if (variant == 0) {
        A81W41_HIP_TRY((launch_attend_vector<bf16, bf16>(a, 1, static_cast<bf16*>(out), s)));
        return 0;
    }
    if (!attend_shared_fits(rank + rot, rank) || splits < 1 || splits > kAttendMaxSplits || (splits > 1 && (!part || !stats)))
        return failf(A81W41_ERR_INVALID_ARG, "the matrix-core attention does not take this shape");
    a.out = static_cast<bf16*>(out), a.splits = splits, a.part = part, a.part_stats = stats, a.ld_part = (rank + 3) / 4 * 4;
    A81W41_HIP_TRY(launch_attend_shared(a, s));
    if (splits > 1) A81W41_HIP_TRY(launch_merge_shares(a, 1, s));
    return 0;
}

int a81w41_formed_attention(const void* q, const void* k, const void* k_rot, int ld_rot, const void* v_t, int ld_v, const float* gates,
                            int heads, int dim, int rot, int vdim, const int* pos_dev, int max_seq, int M, float scale, void* out,
                            void* stream) {
    if (!q || !k || !k_rot || !v_t || !gates || !pos_dev || !out || heads < 1 || dim < 1 || rot < 1 || vdim < 1 || max_seq < 1 || M < 1 ||
        ld_rot < rot || ld_rot % 8 || ld_v % 64 || ld_v < max_seq || !attend_expanded_fits(dim, rot, vdim) || !aligned16(q) || !aligned16(k) ||
        !aligned16(k_rot) || !aligned16(v_t))
        return failf(A81W41_ERR_INVALID_ARG, "bad attention shape");
    AttendArgs<bf16> a;
    a.q = static_cast<const bf16*>(q), a.q_head = dim + rot, a.q_token = heads * (dim + rot), a.rows = M;
    a.k_own = static_cast<const bf16*>(k), a.k_own_head = dim, a.ld_k_own = heads * dim, a.k_own_width = dim;
    a.k_shared = static_cast<const bf16*>(k_rot), a.ld_k_shared = ld_rot, a.k_shared_width = rot;
    a.v_t = static_cast<const bf16*>(v_t), a.ld_v = ld_v, a.dv = vdim, a.head_gate = gates, a.ld_gate = heads;
    a.out = static_cast<bf16*>(out), a.out_head = vdim, a.out_token = heads * vdim;
    a.scale = scale, a.pos_dev = pos_dev, a.max_seq = max_seq;
    A81W41_HIP_TRY(launch_attend_expanded(a, heads, static_cast<hipStream_t>(stream)));
    return 0;
}

int a81w41_grouped_attention(const void* q, const void* rows, int ld, int heads, int kv_heads, int key_width, int value_width, int vdim,
                             const int* pos_dev, int max_seq, int M, float scale, int chunk, int sink, void* out, int is_bf16, int variant,
                             int splits, float* part, float* stats, void* stream) {
    if (!q || !rows || !pos_dev || !out || heads < 1 || kv_heads < 1 || heads % kv_heads || key_width < 8 || key_width % 8 || value_width < 8 ||
        value_width % 8 || key_width > 4096 || value_width > 4096 || vdim < 1 || vdim > value_width || max_seq < 1 || M < 1 || chunk < 0 ||
        ld < kv_heads * (key_width + value_width) || ld % 8 || variant < 0 || variant > 1 || !aligned16(q) || !aligned16(rows))
        return failf(A81W41_ERR_INVALID_ARG, "bad attention shape");
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int R = heads / kv_heads;
    auto set = [&](auto& a, auto type) {
        using T = decltype(type);
        a.q = static_cast<const T*>(q), a.q_head = (long long)R * key_width, a.q_token = heads * key_width, a.ld_q = key_width;
        a.rows = M * R, a.rows_per_token = R, a.k_own = static_cast<const T*>(rows), a.k_own_head = key_width + value_width;
        a.ld_k_own = ld, a.k_own_width = key_width, a.v_width = value_width, a.dv = vdim;
        a.out_head = (long long)R * vdim, a.out_token = heads * vdim, a.ld_out = vdim;
        a.scale = scale, a.chunk = chunk, a.sink = sink != 0, a.pos_dev = pos_dev, a.max_seq = max_seq;
    };
    AttendArgs<float> af;
    AttendArgs<bf16> a;
    if (!is_bf16) {
        if (variant) return failf(A81W41_ERR_INVALID_ARG, "the matrix-core attention does not take this shape");
        set(af, 0.f);
        A81W41_HIP_TRY((launch_attend_vector<float, float>(af, kv_heads, static_cast<float*>(out), s)));
        return 0;
    }
    set(a, bf16{});
    if (variant == 0) {
        A81W41_HIP_TRY((launch_attend_vector<bf16, bf16>(a, kv_heads, static_cast<bf16*>(out), s)));
        return 0;
    }
    if (!attend_rows_fits(key_width, value_width) || splits < 1 || splits > kAttendMaxSplits || (splits > 1 && (!part || !stats)))
        return failf(A81W41_ERR_INVALID_ARG, "the matrix-core attention does not take this shape");
    a.out = static_cast<bf16*>(out), a.splits = splits, a.part = part, a.part_stats = stats, a.ld_part = (vdim + 3) / 4 * 4;
    A81W41_HIP_TRY(launch_attend_rows(a, kv_heads, s));
    if (splits > 1) A81W41_HIP_TRY(launch_merge_shares(a, kv_heads, s));
    return 0;
}

static MemoryShape memory_shape(int heads, int dim, int vdim) {
    MemoryShape sh;
    sh.heads = heads, sh.dim = dim, sh.vdim = vdim;
    return sh;
}

size_t a81w41_matrix_memory_state(int heads, int dim, int vdim) { return memory_shape(heads, dim, vdim).state_size(); }

size_t a81w41_matrix_memory_scratch(int heads, int dim, int vdim, int M) {
    const MemoryShape sh = memory_shape(heads, dim, vdim);
    const size_t chunks = (M + kMemoryChunk - 1) / kMemoryChunk, H = heads;
    return std::max(chunks * H * sh.chunk_size() + (3 * chunks + 1) * H, (size_t)M * H * vdim);
}

int a81w41_matrix_memory(const float* in, int ld_in, int M, int heads, int dim, int vdim, float cap, float eps, const float* bias_i,
                         const float* bias_f, const float* norm, float* state, const int* pos_dev, int variant, float* scratch, float* out,
                         void* stream) {
    MemoryArgs a;
    a.sh = memory_shape(heads, dim, vdim);
    if (!in || !bias_i || !bias_f || !norm || !state || !pos_dev || !scratch || !out || M < 1 || heads < 1 || dim < 1 || vdim < 1 ||
        dim > 4096 || vdim > 16384 || heads > 4096 || !(cap > 0.f) || variant < 0 || variant > 1 || ld_in < a.sh.place_columns() ||
        !aligned16(in) || !aligned16(state) || !aligned16(scratch) || (variant == 1 && !memory_chunks_fit(a.sh)))
        return failf(A81W41_ERR_INVALID_ARG, "bad matrix memory");
    a.sh.cap = cap, a.sh.eps = eps, a.sh.q_scale = 1.0f / std::sqrt((float)dim);
    a.in = in, a.ld_in = ld_in, a.M = M, a.bias_i = bias_i, a.bias_f = bias_f, a.norm = norm, a.state = state, a.pos_dev = pos_dev;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (variant == 0) {
        A81W41_HIP_TRY(launch_memory_steps(a, scratch, s));
        A81W41_HIP_TRY(launch_memory_norm<float>(a, scratch, out, heads * vdim, s));
        return 0;
    }
    const size_t chunks = (M + kMemoryChunk - 1) / kMemoryChunk;
    a.chunk_states = scratch;
    a.chunk_m = scratch + chunks * heads * a.sh.chunk_size();
    a.chunk_stats = a.chunk_m + (chunks + 1) * heads;
    A81W41_HIP_TRY(launch_memory_chunks<float>(a, out, heads * vdim, s));
    return 0;
}

int a81w41_router(const float* logits, int ld, const float* bias, int experts, int top, int M, int* chosen, float* weights, void* stream) {
    if (!logits || !bias || !chosen || !weights || experts < 1 || experts > kMaxRouted || top < 1 || top > kMaxTop || top > experts || M < 1 ||
        ld < experts)
        return failf(A81W41_ERR_INVALID_ARG, "bad router");
    A81W41_HIP_TRY(launch_router(logits, ld, bias, experts, top, M, chosen, weights, static_cast<hipStream_t>(stream)));
    return 0;
}

}  // extern "C"
