// Kernels of the models whose weights are kept as they are (bfloat16, or float in the 32-bit mode): matrix
// products, row norms, latent attention and table-routed experts.  T below is the element type of weights,
// matrix operands and cache; everything else is fp32.
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
    kSiluPair,   // columns come as 16 gates, then their 16 ups, and so on: C (T) has N / 2 columns silu(gate) * up
    kHeadGate,   // C (T) times the sigmoid of head_gate[row][batch]
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
    // grouped: tile t of *n_tiles (at most max_tiles) runs its rows against expert e's weights W + e w_step
    const GroupTile* tiles = nullptr;
    const int* n_tiles = nullptr;
    int max_tiles = 0;
};
template <typename T>
hipError_t launch_dense_gemm(const GemmArgs& g, Epilogue epi, hipStream_t s);

// ---- rows (dense_rows.hip) ------------------------------------------------------------------
// Norm in groups: the row is cut into `groups` parts, each divided by sqrt(mean of its squares + eps); times w.
struct GroupNorm {
    const float* w = nullptr;
    int groups = 1;
    float eps = 0.f;
};
template <typename T>
hipError_t launch_group_norm(const float* x, int M, int width, const GroupNorm& norm, T* out, int ld_out, hipStream_t s);

// What a sublayer hands to the residual stream: y [M][width]; or, with experts, the mean of each token's `top` rows of
// y (slot k of token m is row slot_rows[m * top + k]) plus, if there is one, the shared expert's row.
struct SublayerOut {
    const float* y = nullptr;
    const int* slot_rows = nullptr;
    int top = 0;
    const float* shared = nullptr;
};
// Weighted mean over depth: states[j] [rows][width] is the stream after j layers; the new stream is
// sum_{j < n} coef[j] states[j] + coef[n] r, and r itself goes to states[n].
struct DepthAverage {
    float* states = nullptr;  // null: no averaging, the new stream is r
    long long state_step = 0;
    const float* coef = nullptr;
    int n = 0;
};
// r = x + norm_y(sublayer), the new stream x_out (see above; may be x itself), h = norm_h(x_out) as T.
// y.y == null: r = x.
template <typename T>
hipError_t launch_residual_norm(const float* x, const SublayerOut& y, const GroupNorm& norm_y, const DepthAverage& depth, float* x_out,
                                const GroupNorm& norm_h, T* h, int ld_h, int M, int width, hipStream_t s);

// ---- experts chosen by a table (dense_rows.hip) ---------------------------------------------
// Token m uses the experts table[ids[m]][0..top).  Rows sorted by expert: src_rows[r] = token of row r,
// slot_rows[m * top + k] = row of slot k; tiles of at most kGroupTileRows rows, their number in *n_tiles.
hipError_t launch_table_route(const int* ids, const int* table, int vocab, int top, int experts, int M, int* src_rows,
                              int* slot_rows, GroupTile* tiles, int* n_tiles, hipStream_t s);

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
// Attention in latent space: query rows [M heads][ld_cache] like cache rows (the key up-projection is in the query),
// causal over cache rows 0 .. pos + m; out [M heads][ld_out] the weighted latents (T or float).
// The vector kernel takes any sizes.
template <typename T, typename O>
hipError_t launch_latent_attention_vector(const T* q, const T* cache, const LatentShape& sh, const int* pos_dev, int max_seq, int M,
                                          O* out, int ld_out, hipStream_t s);

// ---- attention on the matrix cores, bfloat16 (attend_mfma.hip) ------------------------------
// Query row r of head z: q + z q_head + r ld_q; it belongs to token r / rows_per_token of the pass and sees the keys
// 0 .. pos + token.  The results go to out, or, with splits > 1 (the keys dealt to that many workgroups), unnormalised
// to part [splits][rows][ld_part] with part_stats [splits][rows][2] (maximum, sum), for launch_merge_shares.
constexpr int kAttendMaxSplits = 64;
constexpr int kAttendFewRows = 64;  // up to here a workgroup takes 16 query rows, above 64
struct AttendArgs {
    const bf16* q = nullptr;
    long long q_head = 0;
    int ld_q = 0, rows = 0, rows_per_token = 1;
    // key = [k_own + z k_own_head + key ld_k_own (k_own_width) | k_shared + key ld_k_shared (k_shared_width)]; widths
    // are multiples of 8, rows 16-byte aligned
    const bf16* k_own = nullptr;
    long long k_own_head = 0;
    int ld_k_own = 0, k_own_width = 0;
    const bf16* k_shared = nullptr;
    int ld_k_shared = 0, k_shared_width = 0;
    // expanded: value column d of head z is v_t + (z dv + d) ld_v, readable up to a multiple of 64 keys
    const bf16* v_t = nullptr;
    int ld_v = 0, dv = 0;
    const float* head_gate = nullptr;  // expanded: result times the sigmoid of head_gate[r ld_gate + z]
    int ld_gate = 0;
    bf16* out = nullptr;
    long long out_head = 0;
    int ld_out = 0;
    int splits = 1;
    float *part = nullptr, *part_stats = nullptr;
    int ld_part = 0;  // a multiple of 4
    float scale = 0.f;
    const int* pos_dev = nullptr;
    int max_seq = 0;
};
bool attend_shared_fits(int dk, int dv);
bool attend_expanded_fits(int own, int shared, int dv);
// Keys and values are the same rows (k_own), the values their first dv columns.
hipError_t launch_attend_shared(const AttendArgs& a, hipStream_t s);
hipError_t launch_attend_expanded(const AttendArgs& a, int heads, hipStream_t s);
hipError_t launch_merge_shares(const AttendArgs& a, hipStream_t s);

// ---- one-token products with the row work fused in (dense_gemv.hip) --------------------------
// Their input rows sit in LDS as fp32: a row (or, for the experts' second product, all of a token's) may have at most
// kGemvMaxRow elements, padding and norm groups included.
constexpr int kGemvMaxRow = 15000;
// r = x + norm_y(y) (y may be null), the stream before + *coef r (before null: r), the row its norm_h.  Workgroup 0
// writes r to state and the stream to x_out (either may be null); neither may be a buffer the step reads.
struct RowStep {
    const float *x = nullptr, *y = nullptr;
    GroupNorm norm_y;
    const float *before = nullptr, *coef = nullptr;
    float *state = nullptr, *x_out = nullptr;
    GroupNorm norm_h;
    int width = 0;
};
template <typename T>
hipError_t launch_gemv_step(const RowStep& p, const T* w, int ld, int N, float* C, hipStream_t s);
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
};
template <typename T>
hipError_t launch_gemv_gate_up(const RowStep& p, const ExpertRows& e, const T* experts, const T* dense, int ld, float* act, hipStream_t s);
template <typename T>
hipError_t launch_gemv_ff_down(const ExpertRows& e, const float* act, const T* experts, int ld, const T* dense, int ld_dense, int N,
                               float* y, hipStream_t s);

}  // namespace a81w41
