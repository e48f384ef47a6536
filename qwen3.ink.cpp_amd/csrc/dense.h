// Kernels of the models whose weights are kept as they are (bfloat16, or float in the 32-bit mode): matrix
// products, row norms, attention (latent, grouped), matrix memories and experts (by table, by router).  T below is the
// element type of weights, matrix operands and cache; everything else, recurrent states included, is fp32.
//
// Operand rules.  Rows of T are `ld` elements apart and 128-byte aligned; a K extent is padded to whole 128-byte
// steps (pad_k).  The padding of a weight is zero, that of an activation any finite value.
// Launchers validate nothing: the models check sizes when they are created.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace a81w41 {

using bf16 = __bf16;

template <typename T>
constexpr int pad_k(int k) {
    constexpr int step = 128 / (int)sizeof(T);
    return (k + step - 1) / step * step;
}

// ---- matrix products (dense_gemm.hip) -------------------------------------------------------
enum class Epilogue {
    kFloat,      // C is float
    kElement,    // C is T
    kGatedPair,  // columns come as 16 gates, then their 16 ups, and so on: C (T) has N / 2 columns, the unit of gate and up
    kHeadGate,   // C (T) times the sigmoid of head_gate[row][batch]
    kHeads,      // queries, keys and values: rotated and stored as HeadRows says
};
// g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(slope g) (u + shift).  As it stands: silu(gate) up.
struct GatedUnit {
    float limit = __builtin_inff(), slope = 1.f, shift = 0.f;
};
// Columns [queries: heads x dim | keys: kv_heads x dim | values: kv_heads x vdim | rest], dim and vdim stored widths (even).
// The first 2 rot_pairs columns of a query or key turn in neighbouring pairs: (u, v) -> (u cos - v sin, v cos + u sin) with
// the angle of (position, pair); a rotation that pairs column i with i + dims / 2 comes here by the order of the weight's
// rows, which a query and its keys share.  Row m is the token at position *pos_dev + m; its cache row holds
// [values vdim | key dim] for every kv head.  The rest goes to fp32 rows.
template <typename T>
struct HeadRows {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, rot_pairs = 0;
    T* q = nullptr;  // [M][heads dim]
    T* cache = nullptr;
    int ld_cache = 0;
    const float *cos_t = nullptr, *sin_t = nullptr;  // [max_seq][rot_pairs]
    const int* pos_dev = nullptr;
    int max_seq = 0;
    float* rest = nullptr;
    int ld_rest = 0;
};
// A row tile of a grouped product: rows [row0, row0 + rows) belong to one expert.
struct GroupTile {
    int expert, row0, rows;
};
constexpr int kGroupTileRows = 64;
struct GemmArgs {
    const void* A = nullptr;  // [M][lda], or gathered: row r of the product is row a_rows[r] of A
    const void* W = nullptr;  // [N][ldw]
    void* C = nullptr;        // [M][ldc]: C = A W^T
    int M = 0, N = 0, K = 0;  // K is a padded extent
    int lda = 0, ldw = 0, ldc = 0;
    const int* a_rows = nullptr;
    // batch b (of `batches`) works on A + b a_step, W + b w_step, C + b c_step (elements)
    int batches = 1;
    long long a_step = 0, w_step = 0, c_step = 0;
    const float* head_gate = nullptr;
    int ld_gate = 0;
    GatedUnit unit;
    // grouped: tile t of *n_tiles (at most max_tiles) runs its rows against expert e's weights W + e w_step
    const GroupTile* tiles = nullptr;
    const int* n_tiles = nullptr;
    int max_tiles = 0;
};
template <typename T>
hipError_t launch_dense_gemm(const GemmArgs& g, Epilogue epi, hipStream_t s);
template <typename T>
hipError_t launch_dense_gemm_heads(const GemmArgs& g, const HeadRows<T>& heads, hipStream_t s);  // g.C is not used

// ---- rows (dense_rows.hip) ------------------------------------------------------------------
// Norm in groups: the row is cut into `groups` parts, each divided by sqrt(mean of its squares + eps); times w.
struct GroupNorm {
    const float* w = nullptr;
    int groups = 1;
    float eps = 0.f;
    float scale = 1.f;  // of a sublayer's output where there is no norm (w null)
};
template <typename T>
hipError_t launch_group_norm(const float* x, int M, int width, const GroupNorm& norm, T* out, int ld_out, hipStream_t s);

// What a sublayer hands to the residual stream: y [M][width]; or, with experts, the mean of each token's `top` rows of
// y (slot k of token m is row slot_rows[m * top + k]), weighted by weights[m * top + k] if there are weights, plus, if there
// is one, the row that every token has (a shared expert's, or a mixer's beside the experts).
struct SublayerOut {
    const float* y = nullptr;
    const int* slot_rows = nullptr;
    int top = 0;
    const float* weights = nullptr;
    const float* shared = nullptr;
};
// Weighted mean over depth: states[j] [rows][width] is the stream after j layers; the new stream is
// sum_{j < n} coef[j] states[j] + coef[n] r, and r itself goes to states[n].
struct DepthAverage {
    float* states = nullptr;  // null: no averaging, the new stream is r
    long long state_step = 0;
    const float* coef = nullptr;  // null: no averaging, r still goes to states[n]
    int n = 0;
};
// r = x + norm_y(sublayer), or x + norm_y.scale * sublayer where norm_y has no weight; the new stream x_out (see above; may be
// x itself), plus the vector `add` if there is one; h = norm_h(x_out) as T.  y.y == null: r = x.
template <typename T>
hipError_t launch_residual_norm(const float* x, const SublayerOut& y, const GroupNorm& norm_y, const DepthAverage& depth, float* x_out,
                                const GroupNorm& norm_h, T* h, int ld_h, int M, int width, hipStream_t s, const float* add = nullptr);

// ---- experts (dense_rows.hip) ----------------------------------------------------------------
// Token m uses the experts table[ids[m]][0..top), or table[m][0..top) without ids (entries of one row are distinct).  Rows
// sorted by expert: src_rows[r] = token of row r, slot_rows[m * top + k] = row of slot k; tiles of at most kGroupTileRows
// rows, their number in *n_tiles.
hipError_t launch_expert_rows(const int* ids, const int* table, int vocab, int top, int experts, int M, int* src_rows,
                              int* slot_rows, GroupTile* tiles, int* n_tiles, hipStream_t s);
// The `top` largest of logits[m][0..experts) + bias (the lower number first among equals): chosen [M][top], largest first,
// and weights [M][top], the softmax over the chosen logits.
hipError_t launch_router(const float* logits, int ld, const float* bias, int experts, int top, int M, int* chosen, float* weights,
                         hipStream_t s);
constexpr int kMaxRouted = 2048, kMaxTop = 64;  // experts of a router, and of a token

// ---- latent attention (latent_attention.hip) ------------------------------------------------
// Sizes of one mixer.  A cache row is [latent (rank) | rotated shared key part (rot)], zero up to ld_cache.
struct LatentShape {
    int heads = 0, dim = 0, rot = 0, vdim = 0, rank = 0, q_rank = 0;
    int ld_cache = 0;
    float scale = 0.f;
};
// The fused down-projection row is [query latent (q_rank) | latent (rank) | rotated part (rot) | head gates (heads)],
// without the middle two where the layer reads another layer's cache.
struct LatentRows {
    const float* down = nullptr;  // [M][ld_down]
    int ld_down = 0;
    const float *q_norm = nullptr, *kv_norm = nullptr;
    float eps = 0.f;
    const float *cos_t = nullptr, *sin_t = nullptr;  // [max_seq][rot / 2]
    const int* pos_dev = nullptr;
    int max_seq = 0;
};
// Normed query latent -> q_latent [M][ld_q] (T); with a cache also the normed latent and the rotated key part into its
// rows pos .. pos + M - 1.
template <typename T>
hipError_t launch_latent_rows(const LatentRows& in, const LatentShape& sh, int M, T* q_latent, int ld_q, T* cache, hipStream_t s);
// q [M][ld_q] head by head [dim | rot]: the unrotated parts to nope (head h of token m at (m heads + h) ld_nope), the
// rotated parts to rot_out (at (m heads + h) ld_rot).
template <typename T>
hipError_t launch_rotate_queries(const float* q, int ld_q, const LatentRows& in, const LatentShape& sh, int M, T* nope, int ld_nope,
                                 T* rot_out, int ld_rot, hipStream_t s);

// ---- attention (attend_vector.hip, attend_mfma.hip) ------------------------------------------
// Query row r of head z belongs to token r / rows_per_token of the pass: q + z q_head + token q_token + (r %
// rows_per_token) ld_q; `out` is laid out likewise.  It sees the keys 0 .. pos + token, with chunk > 0 those from the first
// position of its own chunk of that many positions on.  sink: a further key of score 0 without a value.
// Results go to out, or, with splits > 1 (the keys dealt to that many workgroups), unnormalised to part
// [splits][heads][rows][ld_part] with part_stats [splits][heads][rows][2] (maximum in powers of two, sum), for
// launch_merge_shares.
constexpr int kAttendMaxSplits = 64;
constexpr int kAttendFewRows = 64;  // up to here a workgroup takes 16 query rows, above 64 or more
template <typename T>
struct AttendArgs {
    const T* q = nullptr;
    long long q_head = 0;
    int q_token = 0, ld_q = 0, rows = 0, rows_per_token = 1;
    // key rows at k_own + z k_own_head + key ld_k_own, 16-byte aligned; widths are multiples of 8.
    //   shared:   [key k_own_width], the first dv columns are also the value
    //   rows:     [value v_width | key k_own_width]
    //   expanded: [key k_own_width], and k_shared + key ld_k_shared (k_shared_width) for all heads
    const T* k_own = nullptr;
    long long k_own_head = 0;
    int ld_k_own = 0, k_own_width = 0, v_width = 0;
    const T* k_shared = nullptr;
    int ld_k_shared = 0, k_shared_width = 0;
    // expanded: value column d of head z is v_t + (z dv + d) ld_v, readable up to a multiple of 64 keys
    const T* v_t = nullptr;
    int ld_v = 0, dv = 0;
    const float* head_gate = nullptr;  // expanded: result times the sigmoid of head_gate[r ld_gate + z]
    int ld_gate = 0;
    T* out = nullptr;
    long long out_head = 0;
    int out_token = 0, ld_out = 0;
    int splits = 1;
    float *part = nullptr, *part_stats = nullptr;
    int ld_part = 0;  // a multiple of 4
    float scale = 0.f;
    int chunk = 0;
    bool sink = false;
    const int* pos_dev = nullptr;
    int max_seq = 0;
};
// Keys and values in the same rows (shared or rows form), any sizes; ignores a.out, splits and part.
template <typename T, typename O>
hipError_t launch_attend_vector(const AttendArgs<T>& a, int heads, O* out, hipStream_t s);
// The matrix cores, bfloat16.
bool attend_shared_fits(int dk, int dv);
bool attend_rows_fits(int key, int value);  // stored widths
bool attend_expanded_fits(int own, int shared, int dv);
hipError_t launch_attend_shared(const AttendArgs<bf16>& a, hipStream_t s);
hipError_t launch_attend_rows(const AttendArgs<bf16>& a, int heads, hipStream_t s);
hipError_t launch_attend_expanded(const AttendArgs<bf16>& a, int heads, hipStream_t s);
hipError_t launch_merge_shares(const AttendArgs<bf16>& a, int heads, hipStream_t s);

// ---- matrix memory (matrix_memory.hip) -------------------------------------------------------
// Per head a state S [dim][vdim], n [dim] and a scale m, with the gates' logarithms i = cap tanh(zi / cap), f = logsigmoid(cap
// tanh(zf / cap)) and k, v, q of a token:
//   m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T;  n' likewise with k;
//   o = S'^T q / (max(|n' q|, e^-m') + kMemoryFloor)
// A token's row `in` has q and k [heads][dim], v and g [heads][vdim], zi and zf [heads] at the given columns.
constexpr float kMemoryFloor = 1e-6f;
constexpr int kMemoryChunk = 64;  // tokens of a chunk of the prompt kernels
struct MemoryShape {
    int heads = 0, dim = 0, vdim = 0;
    float cap = 1.f, q_scale = 1.f, eps = 0.f;
    int at_q = 0, at_k = 0, at_v = 0, at_g = 0, at_i = 0, at_f = 0;
    // columns in this order; the first one behind them
    int place_columns() {
        at_q = 0, at_k = at_q + heads * dim, at_v = at_k + heads * dim, at_g = at_v + heads * vdim, at_i = at_g + heads * vdim;
        at_f = at_i + heads;
        return at_f + heads;
    }
    // floats of a sequence's state: S of all heads, then two copies of [n dim | m] per head: the one of parity p is valid at
    // positions of that parity, so that workgroups can read one while another is written
    __host__ __device__ size_t s_size() const { return (size_t)heads * dim * vdim; }
    size_t state_size() const { return s_size() + 2 * (size_t)heads * (dim + 1); }
    __host__ __device__ size_t chunk_size() const { return (size_t)dim * vdim + dim; }  // floats of a head's S and n
};
struct MemoryArgs {
    MemoryShape sh;
    const float* in = nullptr;  // [M][ld_in]
    int ld_in = 0, M = 0;
    const float *bias_i = nullptr, *bias_f = nullptr;  // [heads]
    const float* norm = nullptr;                       // [heads vdim]
    float* state = nullptr;
    const int* pos_dev = nullptr;
    // prompt kernels: [chunks][heads][chunk_size], [chunks + 1][heads], [chunks][heads][2]
    float *chunk_states = nullptr, *chunk_m = nullptr, *chunk_stats = nullptr;
};
// Token by token, any sizes: o [M][heads vdim] as it is.
hipError_t launch_memory_steps(const MemoryArgs& a, float* o, hipStream_t s);
// A row of o, per head divided by its root mean square, times norm, times sigmoid(g), as T.
template <typename T>
hipError_t launch_memory_norm(const MemoryArgs& a, const float* o, T* out, int ld_out, hipStream_t s);
// A prompt in chunks on the matrix cores (32-bit products), the row's norm and gate included.
bool memory_chunks_fit(const MemoryShape& sh);
template <typename T>
hipError_t launch_memory_chunks(const MemoryArgs& a, T* out, int ld_out, hipStream_t s);

// ---- one-token products with the row work fused in (dense_gemv.hip) --------------------------
// Their input rows sit in LDS as fp32: a row (or, for the experts' second product, all of a token's) may have at most
// kGemvMaxRow elements, padding and norm groups included.
constexpr int kGemvMaxRow = 15000;
// r = x + norm_y(y), or x + norm_y.scale * y where norm_y has no weight (y may be null); the stream before + *coef r (before
// null: r; coef null: 1), the row its norm_h.  Workgroup 0 writes r to state, the stream to x_out and the row to h_out (each
// may be null); none may be a buffer the step reads.
struct RowStep {
    const float *x = nullptr, *y = nullptr;
    GroupNorm norm_y;
    const float *before = nullptr, *coef = nullptr;
    float *state = nullptr, *x_out = nullptr, *h_out = nullptr;
    GroupNorm norm_h;
    int width = 0;
};
template <typename T>
hipError_t launch_gemv_step(const RowStep& p, const T* w, int ld, int N, float* C, hipStream_t s);
// The product's columns are stored as HeadRows says.
template <typename T>
hipError_t launch_gemv_step_heads(const RowStep& p, const T* w, int ld, int N, const HeadRows<T>& heads, hipStream_t s);
template <typename T>
hipError_t launch_gemv_plain(const float* x, int K, const T* w, int ld, int N, float* C, hipStream_t s);
// Queries; also the token's cache row (cache may be null) and before = sum_{j < depth.n} coef[j] states[j].
template <typename T>
hipError_t launch_gemv_query(const LatentRows& in, const LatentShape& sh, const T* w, int ld, float* q, T* cache, const DepthAverage& depth,
                             int width, float* before, hipStream_t s);
template <typename T>
hipError_t launch_gemv_absorb(const float* q, const LatentRows& in, const LatentShape& sh, const T* uk_t, int ld, T* q_lat, hipStream_t s);
// The weighted latents of the heads: o_lat [heads][ld_o], or the shares of launch_attend_shared over `heads` rows.
struct LatentShares {
    const float *part = nullptr, *stats = nullptr;
    int splits = 0, ld = 0;
};
template <typename T>
hipError_t launch_gemv_values(const float* o_lat, int ld_o, const LatentShares& shares, const LatentShape& sh, const T* uv, int ld,
                              const float* gates, float* attn, hipStream_t s);
// The feed-forwards a token uses: `top` of `experts` by table (0: none), and one every token uses (dense_ff 0: none).
struct ExpertRows {
    const int *ids = nullptr, *table = nullptr;
    int vocab = 1, top = 0, experts = 0, ff = 0, pair_rows = 0;  // pair_rows: gate/up rows of one expert
    int dense_ff = 0;
    int ld_act = 0;  // activations of slot k (the dense one after the experts) at k ld_act
    GatedUnit unit;
    // by router instead of by table: logits [experts] and bias; the gate/up product leaves the choice in chosen and weights
    const float *logits = nullptr, *bias = nullptr;
    int* chosen = nullptr;
    float* weights = nullptr;
};
// The experts' and the dense feed-forward's input: the row of p, or, if it is not null, h [p.width], already normed.
template <typename T>
hipError_t launch_gemv_gate_up(const RowStep& p, const float* h, const ExpertRows& e, const T* experts, const T* dense, int ld, float* act,
                               hipStream_t s);
template <typename T>
hipError_t launch_gemv_ff_down(const ExpertRows& e, const float* act, const T* experts, int ld, const T* dense, int ld_dense, int N,
                               float* y, hipStream_t s);
// What a mixer leaves for its output product, one row of `width`: attention's (merged from its shares if there are any, at
// most kMixerShares: `heads` rows of `vdim`; every workgroup of the product repeats the merge), or a matrix memory's before its norm and gate.
constexpr int kMixerShares = 8;
struct MixerRow {
    const float* row = nullptr;
    int width = 0;
    LatentShares shares;
    int heads = 0, vdim = 0;
    const float *norm = nullptr, *gates = nullptr;  // matrix memory: [width] each
    float eps = 0.f;
};
// y = W_o . mixer row + the weighted sum over the router's experts of W_e . act_e (e.top 0: the mixer alone).
template <typename T>
hipError_t launch_gemv_mixer_down(const MixerRow& m, const T* wo, int ld_wo, const ExpertRows& e, const float* act, const T* experts,
                                  int ld, int N, float* y, hipStream_t s);

}  // namespace a81w41
