// The Takosun design on the shared decoder session: latent attention whose cache several layers may read, grouped
// norms before and after each sublayer, dense or table-routed expert feed-forwards, and a weighted mean over depth
// after every layer.  This file owns the weights and activation buffers and enqueues the kernels of a pass; the
// mechanisms are in dense_gemm.hip, dense_rows.hip and latent_attention.hip, the loop in decoder_session.cpp.
//
// With X_0 the embedding rows, x = X_0 and, for layer i,
//   a       = x + N1b(mixer(N1(x)))
//   X_{i+1} = a + N2b(feed_forward(N2(a)))            (or a, without a feed-forward)
//   x       = sum_{j <= i+1} dwa_i[j] X_j
// logits = head N(x).
#include <cstring>
#include <memory>

#include "dense_model.h"
#include "json.h"

namespace a81w41 {
namespace {

struct FeedForwardConfig {
    bool present = false, experts_by_table = false;
    int ff = 0;                         // of the dense form, or of one expert
    int experts = 0, top = 0, shared_ff = 0;
};
struct LayerConfig {
    LatentShape mix;
    int kv_from = -1;
    double rot_base = 0;
    FeedForwardConfig mlp;
};
struct Config {
    int vocab = 0, width = 0, groups = 1;
    float eps = 0.f;
    std::vector<LayerConfig> layers;
};

Config read_config(const Json& j) {
    Config c;
    c.vocab = j.size("vocab");
    c.width = j.size("width");
    c.groups = j.at("norm").size("groups");
    c.eps = (float)j.at("norm").at("eps").number();
    require(c.eps >= 0.f, "norm.eps must not be negative");
    require(c.width % c.groups == 0 && c.width + c.groups <= 16000, "width must be a multiple of norm.groups, the two together at most 16000");
    for (const Json& l : j.at("layers").array()) {
        const std::string where = "layer " + std::to_string(c.layers.size()) + ": ";
        LayerConfig out;
        require(l.at("type").string() == "latent_attention", where + "unknown type '" + l.at("type").string() + "'");
        const Json& m = l.at("mixer");
        out.mix.heads = m.size("heads");
        out.mix.dim = m.size("dim");
        out.mix.rot = m.size("rot_dim");
        out.mix.vdim = m.size("vdim");
        out.mix.rank = m.size("kv_rank");
        out.mix.q_rank = m.size("q_rank");
        out.mix.scale = (float)m.at("scale").number();
        require(m.at("rot").size("dims") == out.mix.rot && out.mix.rot % 2 == 0, where + "rot.dims must equal rot_dim and be even");
        out.rot_base = m.at("rot").at("base").number();
        require(out.rot_base > 0, where + "rot.base must be positive");
        require(out.mix.rank + out.mix.rot <= 4096 && out.mix.q_rank <= 32768, where + "latent too large");
        if (m.has("kv_from")) {
            const long long from = m.at("kv_from").integer();
            require(from >= 0 && from < (long long)c.layers.size(), where + "kv_from must name an earlier layer");
            const LayerConfig& src = c.layers[from];
            require(src.kv_from < 0 && src.mix.rank == out.mix.rank && src.mix.rot == out.mix.rot && src.rot_base == out.rot_base,
                    where + "kv_from must name a layer with a latent of its own, of the same sizes and rotation");
            out.kv_from = (int)from;
        }
        if (l.has("mlp")) {
            const Json& f = l.at("mlp");
            const std::string& kind = f.at("kind").string();
            out.mlp.present = true;
            if (kind == "dense") {
                out.mlp.ff = f.size("ff");
            } else {
                require(kind == "moe", where + "unknown feed-forward '" + kind + "'");
                out.mlp.experts_by_table = true;
                out.mlp.experts = f.at("router").size("experts");
                out.mlp.top = f.at("router").size("top");
                out.mlp.ff = f.at("expert").size("ff");
                if (f.has("shared")) out.mlp.shared_ff = f.at("shared").size("ff");
                require(out.mlp.top <= out.mlp.experts && out.mlp.experts <= 4096 && out.mlp.top <= 64, where + "router out of range");
            }
        }
        c.layers.push_back(out);
    }
    require(!c.layers.empty(), "no layers");
    return c;
}

}  // namespace

template <typename T>
class TakosunModel final : public DenseModel<T> {
    using Base = DenseModel<T>;
    using Base::cache, Base::ids, Base::logits, Base::max_seq, Base::plan_ctx, Base::pos, Base::stream, Base::want_dev;
    using Base::allocate_array, Base::finish, Base::init_session, Base::kMatrixAttention, Base::kTable, Base::load_feed_forward,
        Base::load_matrix, Base::load_rotation, Base::load_vector, Base::product, Base::put_matrix, Base::upload_array;
    using Staging = typename Base::Staging;

   public:
    explicit TakosunModel(Config c) : cfg_(std::move(c)) {}
    int create(int max_seq, TensorSource& src) {
        A81W41_TRY(load_weights(max_seq, src));
        A81W41_TRY(allocate(max_seq));
        return 0;
    }
    // unfused: one-token passes take the kernels of longer ones; attention: 0 by shape, 1 the vector kernel, 2 in latent
    // space, 3 on formed keys and values; attention_split: shares of the keys in latent space, 0 by length
    int set_option(const char* name, int value) override {
        const std::string n = name;
        if (n == "unfused" && value >= 0 && value <= 1)
            opt_unfused_ = value;
        else if (n == "attention" && value >= 0 && value <= 3)
            opt_attention_ = value;
        else if (n == "attention_split" && value >= 0 && value <= kAttendMaxSplits)
            opt_split_ = value;
        else
            return failf(A81W41_ERR_INVALID_ARG, "no option '%s' with value %d", name, value);
        return 0;
    }
    // state<i>: [tokens of the last pass][width], the stream after i layers, before the mean over depth
    int read_buffer(const char* name, float* host_out, size_t count) override {
        int i = -1;
        if (sscanf(name, "state%d", &i) != 1 || i < 0 || i > n_layers()) return DecoderSession::read_buffer(name, host_out, count);
        if (count > (size_t)rows_ * cfg_.width) return failf(A81W41_ERR_INVALID_ARG, "state holds fewer values");
        A81W41_HIP_TRY(hipStreamSynchronize(stream));
        A81W41_HIP_TRY(hipMemcpy(host_out, states_ + i * state_step(), count * sizeof(float), hipMemcpyDeviceToHost));
        return 0;
    }

   protected:
    int enqueue_pass(int M, const int* want, int n_want, hipStream_t s) override;

   private:
    using FeedForward = GatedWeights<T>;
    struct Layer {
        float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr, *dwa = nullptr;
        float *q_norm = nullptr, *kv_norm = nullptr;
        Weight<T> down;  // [dq | dkv | g]
        Weight<T> uq, uk, uk_t, uv, o;  // uk_t: per head, transposed; uk as stored, for formed keys
        FeedForward ff, shared;
        int* table = nullptr;
        T* cache = nullptr;
        float *cos_t = nullptr, *sin_t = nullptr;
    };
    // whether a layer can form its keys and values per head for many new tokens
    static bool can_expand(const LatentShape& sh) {
        return kMatrixAttention && sh.rank % 8 == 0 && attend_expanded_fits(sh.dim, sh.rot, sh.vdim);
    }
    int n_layers() const { return (int)cfg_.layers.size(); }
    long long state_step() const { return (long long)rows_ * cfg_.width; }
    GroupNorm norm(const float* w) const { return GroupNorm{w, cfg_.groups, cfg_.eps}; }

    int load_weights(int max_seq, TensorSource& src);
    int allocate(int max_seq);
    int attention(const Layer& L, const LayerConfig& lc, int M, hipStream_t s);
    int attend_latent(const Layer& L, const LatentShape& sh, int M, hipStream_t s);
    int attend_formed(const Layer& L, const LatentShape& sh, int M, const float* gates, hipStream_t s);
    AttendArgs<T> shared_attend(const Layer& L, const LatentShape& sh, int M) const;
    int enqueue_one_token(int n_want, hipStream_t s);
    int feed_forward_one_token(const Layer& L, const LayerConfig& lc, const RowStep& step, hipStream_t s);
    LatentRows latent_rows(const Layer& L) const;
    int feed_forward(const Layer& L, const LayerConfig& lc, int M, hipStream_t s, SublayerOut* out);
    int pair_product(const FeedForward& f, int ff, const T* h, const GemmArgs& base, T* act, hipStream_t s);

    Config cfg_;
    std::vector<Layer> layers_;
    Weight<T> embed_, head_;
    float* final_norm_ = nullptr;
    // activations of one pass
    int rows_ = 0, ld_h_ = 0, ld_down_ = 0, ld_q_ = 0, ld_cq_ = 0, ld_attn_ = 0;
    float *x_ = nullptr, *states_ = nullptr, *down_ = nullptr, *q_ = nullptr, *y_ = nullptr, *y2_ = nullptr, *y_shared_ = nullptr;
    T *h_ = nullptr, *c_q_ = nullptr, *nope_ = nullptr, *q_lat_ = nullptr, *o_lat_ = nullptr, *attn_ = nullptr, *act_ = nullptr;
    bf16 *k_formed_ = nullptr, *v_formed_ = nullptr;  // [max_seq][heads dim], [heads vdim][ld_v_]
    int ld_v_ = 0;
    float *part_ = nullptr, *part_stats_ = nullptr;  // shares of the attention in latent space
    size_t part_rows_ = 0;
    int ld_part_ = 0;
    // of the one-token pass
    float *row_x_[2] = {nullptr, nullptr}, *row_mid_ = nullptr, *before_ = nullptr, *y_ff_ = nullptr;
    float *o_lat_row_ = nullptr, *attn_row_ = nullptr, *act_row_ = nullptr;
    int ld_act_row_ = 0;
    bool one_token_fits_ = true;
    int opt_unfused_ = 0, opt_attention_ = 0, opt_split_ = 0;
    int *src_rows_ = nullptr, *slot_rows_ = nullptr, *n_tiles_ = nullptr;
    GroupTile* tiles_ = nullptr;
};

template <typename T>
int TakosunModel<T>::load_weights(int max_seq, TensorSource& src) {
    const int width = cfg_.width;
    A81W41_TRY(load_matrix(src, "embed", cfg_.vocab, width, &embed_));
    layers_.resize(n_layers());
    for (int i = 0; i < n_layers(); i++) {
        LayerConfig& lc = cfg_.layers[i];
        LatentShape& sh = lc.mix;
        Layer& L = layers_[i];
        const std::string p = "l" + std::to_string(i) + ".", mix = p + "mix.", mlp = p + "mlp.";
        A81W41_TRY(load_vector(src, p + "norm1", width, &L.norm1));
        A81W41_TRY(load_vector(src, p + "norm1b", width, &L.norm1b));
        A81W41_TRY(load_vector(src, p + "dwa", i + 2, &L.dwa));
        A81W41_TRY(load_vector(src, mix + "dq.norm", sh.q_rank, &L.q_norm));
        sh.ld_cache = pad_k<T>(sh.rank + sh.rot);
        const bool own = lc.kv_from < 0;
        const int kv = own ? sh.rank + sh.rot : 0;
        Staging down(sh.q_rank + kv + sh.heads, width);
        A81W41_TRY(put_matrix(src, mix + "dq", sh.q_rank, width, down, 0));
        if (own) {
            A81W41_TRY(put_matrix(src, mix + "dkv", kv, width, down, sh.q_rank));
            A81W41_TRY(load_vector(src, mix + "dkv.norm", sh.rank, &L.kv_norm));
            void* plane = nullptr;
            A81W41_TRY(cache.add((size_t)max_seq * sh.ld_cache * sizeof(T), &plane));
            L.cache = static_cast<T*>(plane);
        } else {
            L.cache = layers_[lc.kv_from].cache;
        }
        A81W41_TRY(put_matrix(src, mix + "g", sh.heads, width, down, sh.q_rank + kv));
        A81W41_TRY(finish(down, &L.down));
        A81W41_TRY(load_rotation(sh.rot, lc.rot_base, max_seq, &L.cos_t, &L.sin_t));
        A81W41_TRY(load_matrix(src, mix + "uq", sh.heads * (sh.dim + sh.rot), sh.q_rank, &L.uq));
        {   // the key up-projection of a head, transposed: it maps an unrotated query to latent space
            std::vector<float> uk, row(sh.dim);
            A81W41_TRY(src.matrix(mix + "uk", sh.heads * sh.dim, sh.rank, uk));
            if (can_expand(sh)) {
                Staging st(sh.heads * sh.dim, sh.rank);
                for (int r = 0; r < st.rows; r++) st.put(r, uk.data() + (size_t)r * sh.rank);
                A81W41_TRY(finish(st, &L.uk));
            }
            Staging t(sh.heads * sh.rank, sh.dim);
            for (int h = 0; h < sh.heads; h++)
                for (int r = 0; r < sh.rank; r++) {
                    for (int d = 0; d < sh.dim; d++) row[d] = uk[(size_t)(h * sh.dim + d) * sh.rank + r];
                    t.put(h * sh.rank + r, row.data());
                }
            A81W41_TRY(finish(t, &L.uk_t));
        }
        A81W41_TRY(load_matrix(src, mix + "uv", sh.heads * sh.vdim, sh.rank, &L.uv));
        A81W41_TRY(load_matrix(src, mix + "o", width, sh.heads * sh.vdim, &L.o));
        const FeedForwardConfig& f = lc.mlp;
        if (!f.present) continue;
        A81W41_TRY(load_vector(src, p + "norm2", width, &L.norm2));
        A81W41_TRY(load_vector(src, p + "norm2b", width, &L.norm2b));
        if (!f.experts_by_table) {
            A81W41_TRY(load_feed_forward(src, {mlp}, width, f.ff, &L.ff));
            continue;
        }
        std::vector<std::string> names;
        for (int e = 0; e < f.experts; e++) names.push_back(mlp + "e" + std::to_string(e) + ".");
        A81W41_TRY(load_feed_forward(src, names, width, f.ff, &L.ff));
        if (f.shared_ff) A81W41_TRY(load_feed_forward(src, {mlp + "shared."}, width, f.shared_ff, &L.shared));
        std::vector<int> table;
        A81W41_TRY(src.table(mlp + "table", cfg_.vocab, f.top, f.experts, table));
        A81W41_TRY(upload_array(table, &L.table));
    }
    A81W41_TRY(load_vector(src, "final.norm", width, &final_norm_));
    return load_matrix(src, "head", cfg_.vocab, width, &head_);
}

template <typename T>
int TakosunModel<T>::allocate(int max_seq) {
    rows_ = std::min(max_seq, kPassRows);
    A81W41_TRY(init_session(max_seq, cfg_.vocab, rows_));
    ld_h_ = pad_k<T>(cfg_.width);
    size_t nope = 0, q_lat = 0, o_lat = 0, act = 0, expert_rows = 0, tiles = 0, formed_k = 0, formed_v = 0;
    int slots = 1, heads = 0;
    one_token_fits_ = ld_h_ + cfg_.groups <= kGemvMaxRow;
    for (const LayerConfig& lc : cfg_.layers) {
        const LatentShape& sh = lc.mix;
        ld_down_ = std::max(ld_down_, sh.q_rank + sh.rank + sh.rot + sh.heads);
        ld_q_ = std::max(ld_q_, sh.heads * (sh.dim + sh.rot));
        ld_cq_ = std::max(ld_cq_, pad_k<T>(sh.q_rank));
        ld_attn_ = std::max(ld_attn_, pad_k<T>(sh.heads * sh.vdim));
        nope = std::max(nope, (size_t)sh.heads * pad_k<T>(sh.dim));
        q_lat = std::max(q_lat, (size_t)sh.heads * sh.ld_cache);
        o_lat = std::max(o_lat, (size_t)sh.heads * pad_k<T>(sh.rank));
        heads = std::max(heads, sh.heads);
        ld_part_ = std::max(ld_part_, (sh.rank + 3) / 4 * 4);
        one_token_fits_ = one_token_fits_ && pad_k<T>(sh.q_rank) <= kGemvMaxRow && pad_k<T>(sh.heads * sh.vdim) <= kGemvMaxRow;
        if (can_expand(sh)) {
            formed_k = std::max(formed_k, (size_t)sh.heads * sh.dim);
            formed_v = std::max(formed_v, (size_t)sh.heads * sh.vdim);
            nope = std::max(nope, (size_t)sh.heads * (sh.dim + sh.rot));
        }
        const FeedForwardConfig& f = lc.mlp;
        if (!f.present) continue;
        act = std::max(act, (size_t)std::max(f.top, 1) * pad_k<T>(f.ff));
        act = std::max(act, (size_t)pad_k<T>(f.shared_ff));
        ld_act_row_ = std::max(ld_act_row_, (std::max(f.ff, f.shared_ff) + 3) / 4 * 4);
        slots = std::max(slots, f.top + 1);
        one_token_fits_ = one_token_fits_ && std::max(f.top, 1) * pad_k<T>(f.ff) + pad_k<T>(f.shared_ff) <= kGemvMaxRow;
        if (f.experts_by_table) {
            expert_rows = std::max(expert_rows, (size_t)f.top);
            tiles = std::max(tiles, (size_t)rows_ * f.top / kGroupTileRows + f.experts);
        }
    }
    const size_t R = rows_, W = cfg_.width;
    A81W41_TRY(allocate_array(R * W, &x_));
    A81W41_TRY(allocate_array((size_t)(n_layers() + 1) * R * W, &states_));
    A81W41_TRY(allocate_array(R * ld_h_, &h_));
    A81W41_TRY(allocate_array(R * ld_down_, &down_));
    A81W41_TRY(allocate_array(R * ld_q_, &q_));
    A81W41_TRY(allocate_array(R * ld_cq_, &c_q_));
    A81W41_TRY(allocate_array(R * nope, &nope_));
    A81W41_TRY(allocate_array(R * q_lat, &q_lat_));
    A81W41_TRY(allocate_array(R * o_lat, &o_lat_));
    A81W41_TRY(allocate_array(R * ld_attn_, &attn_));
    A81W41_TRY(allocate_array(R * act, &act_));
    A81W41_TRY(allocate_array(R * W, &y_));
    if (formed_k) {
        ld_v_ = (max_seq + 63) / 64 * 64;
        A81W41_TRY(allocate_array((size_t)max_seq * formed_k, &k_formed_));
        A81W41_TRY(allocate_array(formed_v * ld_v_, &v_formed_));
    }
    part_rows_ = std::max((size_t)heads * kAttendMaxSplits, (size_t)8192);
    A81W41_TRY(allocate_array(part_rows_ * ld_part_, &part_));
    A81W41_TRY(allocate_array(part_rows_ * 2, &part_stats_));
    for (float** row : {&row_x_[0], &row_x_[1], &row_mid_, &before_, &y_ff_}) A81W41_TRY(allocate_array(W, row));
    A81W41_TRY(allocate_array(o_lat, &o_lat_row_));
    A81W41_TRY(allocate_array((size_t)ld_attn_, &attn_row_));
    A81W41_TRY(allocate_array((size_t)slots * ld_act_row_, &act_row_));
    if (expert_rows) {
        A81W41_TRY(allocate_array(R * expert_rows * W, &y2_));
        A81W41_TRY(allocate_array(R * W, &y_shared_));
        A81W41_TRY(allocate_array(R * expert_rows, &src_rows_));
        A81W41_TRY(allocate_array(R * expert_rows, &slot_rows_));
        A81W41_TRY(allocate_array(tiles, &tiles_));
        A81W41_TRY(allocate_array(1, &n_tiles_));
    }
    return 0;
}

template <typename T>
LatentRows TakosunModel<T>::latent_rows(const Layer& L) const {
    LatentRows in;
    in.down = down_, in.ld_down = ld_down_, in.q_norm = L.q_norm, in.kv_norm = L.kv_norm, in.eps = cfg_.eps;
    in.cos_t = L.cos_t, in.sin_t = L.sin_t, in.pos_dev = pos, in.max_seq = max_seq();
    return in;
}

// Query rows q_lat_ (like cache rows) against the layer's cache.
template <typename T>
AttendArgs<T> TakosunModel<T>::shared_attend(const Layer& L, const LatentShape& sh, int M) const {
    AttendArgs<T> a;
    a.q = q_lat_, a.ld_q = sh.ld_cache, a.q_token = sh.heads * sh.ld_cache, a.rows = M * sh.heads, a.rows_per_token = sh.heads;
    a.k_own = L.cache, a.ld_k_own = sh.ld_cache, a.k_own_width = (sh.rank + sh.rot + 7) / 8 * 8;
    a.dv = sh.rank, a.scale = sh.scale, a.pos_dev = pos, a.max_seq = max_seq();
    a.part = part_, a.part_stats = part_stats_, a.ld_part = (sh.rank + 3) / 4 * 4;
    // enough workgroups for the chip, at least 64 keys for each
    const int groups = a.rows <= kAttendFewRows ? (a.rows + 15) / 16 : (a.rows + 63) / 64;
    a.splits = opt_split_ ? opt_split_ : std::min({kAttendMaxSplits, (plan_ctx + 63) / 64, std::max(1, 512 / groups)});
    a.splits = std::max<int>(1, std::min<size_t>(a.splits, part_rows_ / a.rows));
    return a;
}

// Attention in latent space: the key up-projection moves into the query, the value up-projection behind the sum.
// Leaves the weighted latents in o_lat_.
template <typename T>
int TakosunModel<T>::attend_latent(const Layer& L, const LatentShape& sh, int M, hipStream_t s) {
    const LatentRows in = latent_rows(L);
    const int ld_nope = pad_k<T>(sh.dim), ld_rank = pad_k<T>(sh.rank);
    A81W41_HIP_TRY(launch_rotate_queries<T>(q_, ld_q_, in, sh, M, nope_, ld_nope, q_lat_ + sh.rank, sh.ld_cache, s));
    GemmArgs g = product(nope_, sh.heads * ld_nope, L.uk_t, q_lat_, sh.heads * sh.ld_cache, M);
    g.N = sh.rank, g.batches = sh.heads, g.a_step = ld_nope, g.w_step = (long long)sh.rank * L.uk_t.ld, g.c_step = sh.ld_cache;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kElement, s));
    bool done = false;
    if constexpr (kMatrixAttention) {
        if (opt_attention_ != 1 && attend_shared_fits(sh.rank + sh.rot, sh.rank)) {
            AttendArgs<T> a = shared_attend(L, sh, M);
            a.out = o_lat_, a.ld_out = ld_rank, a.out_token = sh.heads * ld_rank;
            A81W41_HIP_TRY(launch_attend_shared(a, s));
            if (a.splits > 1) A81W41_HIP_TRY(launch_merge_shares(a, 1, s));
            done = true;
        }
    }
    if (!done) {
        AttendArgs<T> a = shared_attend(L, sh, M);
        a.ld_out = ld_rank, a.out_token = sh.heads * ld_rank;
        A81W41_HIP_TRY((launch_attend_vector<T, T>(a, 1, o_lat_, s)));
    }
    return 0;
}

// Attention on keys and values formed per head: fewer operations per key once there are many new tokens.
template <typename T>
int TakosunModel<T>::attend_formed(const Layer& L, const LatentShape& sh, int M, const float* gates, hipStream_t s) {
    if constexpr (kMatrixAttention) {
        const int ctx = plan_ctx, dk = sh.dim + sh.rot;  // a pass of several tokens is planned for exactly its context
        GemmArgs g = product(L.cache, sh.ld_cache, L.uk, k_formed_, sh.heads * sh.dim, ctx);
        A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kElement, s));
        // values transposed: the roles of weight and cache change
        g.A = L.uv.data, g.lda = L.uv.ld, g.M = L.uv.rows, g.W = L.cache, g.ldw = sh.ld_cache, g.N = ctx, g.K = L.uv.ld;
        g.C = v_formed_, g.ldc = ld_v_;
        A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kElement, s));
        A81W41_HIP_TRY(launch_rotate_queries<T>(q_, ld_q_, latent_rows(L), sh, M, nope_, dk, nope_ + sh.dim, dk, s));
        AttendArgs<T> a;
        a.q = nope_, a.q_head = dk, a.q_token = sh.heads * dk, a.rows = M;
        a.k_own = k_formed_, a.k_own_head = sh.dim, a.ld_k_own = sh.heads * sh.dim, a.k_own_width = sh.dim;
        a.k_shared = L.cache + sh.rank, a.ld_k_shared = sh.ld_cache, a.k_shared_width = sh.rot;
        a.v_t = v_formed_, a.ld_v = ld_v_, a.dv = sh.vdim;
        a.head_gate = gates, a.ld_gate = ld_down_;
        a.out = attn_, a.out_head = sh.vdim, a.out_token = ld_attn_;
        a.scale = sh.scale, a.pos_dev = pos, a.max_seq = max_seq();
        A81W41_HIP_TRY(launch_attend_expanded(a, sh.heads, s));
    }
    return 0;
}

// The mixer on h_: leaves its output rows in y_.
template <typename T>
int TakosunModel<T>::attention(const Layer& L, const LayerConfig& lc, int M, hipStream_t s) {
    const LatentShape& sh = lc.mix;
    const bool own = lc.kv_from < 0;
    const float* gates = down_ + sh.q_rank + (own ? sh.rank + sh.rot : 0);
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(h_, ld_h_, L.down, down_, ld_down_, M), Epilogue::kFloat, s));
    A81W41_HIP_TRY(launch_latent_rows<T>(latent_rows(L), sh, M, c_q_, ld_cq_, own ? L.cache : nullptr, s));
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(c_q_, ld_cq_, L.uq, q_, ld_q_, M), Epilogue::kFloat, s));
    // per key and head, latent space costs M (2 rank + rot) against M (dim + rot + vdim) and rank (dim + vdim) once
    const bool many = (long long)M * (2 * sh.rank - sh.dim - sh.vdim) > (long long)sh.rank * (sh.dim + sh.vdim);
    if (can_expand(sh) && (opt_attention_ == 3 || (opt_attention_ == 0 && many))) {
        A81W41_TRY(attend_formed(L, sh, M, gates, s));
    } else {
        A81W41_TRY(attend_latent(L, sh, M, s));
        const int ld_rank = pad_k<T>(sh.rank);
        GemmArgs g = product(o_lat_, sh.heads * ld_rank, L.uv, attn_, ld_attn_, M);
        g.N = sh.vdim, g.batches = sh.heads, g.a_step = ld_rank, g.w_step = (long long)sh.vdim * L.uv.ld, g.c_step = sh.vdim;
        g.head_gate = gates, g.ld_gate = ld_down_;
        A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kHeadGate, s));
    }
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(attn_, ld_attn_, L.o, y_, cfg_.width, M), Epilogue::kFloat, s));
    return 0;
}

// The feed-forward on h_.
template <typename T>
int TakosunModel<T>::feed_forward(const Layer& L, const LayerConfig& lc, int M, hipStream_t s, SublayerOut* out) {
    const FeedForwardConfig& f = lc.mlp;
    const int W = cfg_.width;
    auto two_products = [&](const FeedForward& w, int ff, float* y) -> int {
        const int ld = pad_k<T>(ff);
        A81W41_HIP_TRY(launch_dense_gemm<T>(product(h_, ld_h_, w.gate_up, act_, ld, M), Epilogue::kGatedPair, s));
        A81W41_HIP_TRY(launch_dense_gemm<T>(product(act_, ld, w.down, y, W, M), Epilogue::kFloat, s));
        return 0;
    };
    *out = SublayerOut{};
    out->y = y_;
    if (!f.experts_by_table) return two_products(L.ff, f.ff, y_);
    if (f.shared_ff) {
        A81W41_TRY(two_products(L.shared, f.shared_ff, y_shared_));
        out->shared = y_shared_;
    }
    A81W41_HIP_TRY(launch_expert_rows(ids, L.table, cfg_.vocab, f.top, f.experts, M, src_rows_, slot_rows_, tiles_, n_tiles_, s));
    const int ld = pad_k<T>(f.ff), cols = pair_columns(f.ff);
    GemmArgs g = product(h_, ld_h_, L.ff.gate_up, act_, ld, M * f.top);
    g.N = cols, g.w_step = (long long)cols * L.ff.gate_up.ld, g.a_rows = src_rows_;
    g.tiles = tiles_, g.n_tiles = n_tiles_, g.max_tiles = M * f.top / kGroupTileRows + std::min(f.experts, M * f.top);
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kGatedPair, s));
    g.A = act_, g.lda = ld, g.a_rows = nullptr, g.W = L.ff.down.data, g.ldw = g.K = L.ff.down.ld;
    g.N = W, g.w_step = (long long)W * L.ff.down.ld, g.C = y2_, g.ldc = W;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    out->y = y2_, out->slot_rows = slot_rows_, out->top = f.top;
    return 0;
}

// The same feed-forward for one token behind the residual step `step`: leaves its output row in y_ff_.
template <typename T>
int TakosunModel<T>::feed_forward_one_token(const Layer& L, const LayerConfig& lc, const RowStep& step, hipStream_t s) {
    const FeedForwardConfig& f = lc.mlp;
    const FeedForward& every = f.experts_by_table ? L.shared : L.ff;  // what every token uses
    ExpertRows e;
    e.dense_ff = f.experts_by_table ? f.shared_ff : f.ff;
    e.ld_act = ld_act_row_;
    if (f.experts_by_table) {
        e.ids = ids, e.table = L.table, e.vocab = cfg_.vocab, e.top = f.top, e.experts = f.experts, e.ff = f.ff;
        e.pair_rows = pair_columns(f.ff);
    }
    A81W41_HIP_TRY(launch_gemv_gate_up<T>(step, nullptr, e, L.ff.gate_up.data, every.gate_up.data, L.ff.gate_up.ld, act_row_, s));
    A81W41_HIP_TRY(launch_gemv_ff_down<T>(e, act_row_, L.ff.down.data, L.ff.down.ld, every.down.data, every.down.ld, cfg_.width, y_ff_, s));
    return 0;
}

// The pass for one token: the row work between two products runs inside the product that consumes it, eight launches a
// layer.  The sum over the earlier states of the mean over depth is
// formed beside the query product, so that the next layer's first product adds only the newest state.
template <typename T>
int TakosunModel<T>::enqueue_one_token(int n_want, hipStream_t s) {
    const int W = cfg_.width, n = n_layers();
    A81W41_HIP_TRY(launch_embed_rows(ids, embed_.data, kTable, embed_.ld, states_, 1, W,
                                     cfg_.vocab, s));
    RowStep step;  // what the next product's prologue does
    step.x = states_, step.width = W, step.norm_h = norm(layers_[0].norm1);
    for (int i = 0; i < n; i++) {
        const Layer& L = layers_[i];
        const LayerConfig& lc = cfg_.layers[i];
        const LatentShape& sh = lc.mix;
        const bool own = lc.kv_from < 0;
        A81W41_HIP_TRY(launch_gemv_step<T>(step, L.down.data, L.down.ld, L.down.rows, down_, s));
        const float* x = i ? step.x_out : states_;
        DepthAverage depth;
        depth.states = states_, depth.state_step = state_step(), depth.coef = L.dwa, depth.n = i + 1;
        const LatentRows in = latent_rows(L);
        A81W41_HIP_TRY(launch_gemv_query<T>(in, sh, L.uq.data, L.uq.ld, q_, own ? L.cache : nullptr, depth, W, before_, s));
        A81W41_HIP_TRY(launch_gemv_absorb<T>(q_, in, sh, L.uk_t.data, L.uk_t.ld, q_lat_, s));
        const int ld_rank = pad_k<T>(sh.rank);
        LatentShares shares;
        if constexpr (kMatrixAttention) {
            if (opt_attention_ != 1 && attend_shared_fits(sh.rank + sh.rot, sh.rank)) {
                AttendArgs<T> a = shared_attend(L, sh, 1);
                a.splits = std::max(a.splits, 2);  // shares stay fp32; the product with W_uv merges them
                A81W41_HIP_TRY(launch_attend_shared(a, s));
                shares = LatentShares{a.part, a.part_stats, a.splits, a.ld_part};
            }
        }
        if (!shares.part) {
            AttendArgs<T> a = shared_attend(L, sh, 1);
            a.ld_out = ld_rank, a.out_token = sh.heads * ld_rank;
            A81W41_HIP_TRY((launch_attend_vector<T, float>(a, 1, o_lat_row_, s)));
        }
        A81W41_HIP_TRY(launch_gemv_values<T>(o_lat_row_, ld_rank, shares, sh, L.uv.data, L.uv.ld, down_ + sh.q_rank + (own ? sh.rank + sh.rot : 0),
                                             attn_row_, s));
        A81W41_HIP_TRY(launch_gemv_plain<T>(attn_row_, sh.heads * sh.vdim, L.o.data, L.o.ld, W, y_, s));
        step = RowStep{};
        step.width = W, step.x = x, step.y = y_, step.norm_y = norm(L.norm1b);
        if (lc.mlp.present) {
            step.x_out = row_mid_, step.norm_h = norm(L.norm2);
            A81W41_TRY(feed_forward_one_token(L, lc, step, s));
            step.x = row_mid_, step.y = y_ff_, step.norm_y = norm(L.norm2b);
        }
        step.before = before_, step.coef = L.dwa + i + 1, step.state = states_ + (i + 1) * state_step();
        step.x_out = row_x_[i & 1];
        step.norm_h = norm(i + 1 < n ? layers_[i + 1].norm1 : final_norm_);
    }
    if (n_want) A81W41_HIP_TRY(launch_gemv_step<T>(step, head_.data, head_.ld, head_.rows, logits, s));
    A81W41_HIP_TRY(launch_advance(pos, 1, s));
    return 0;
}

template <typename T>
int TakosunModel<T>::enqueue_pass(int M, const int* want, int n_want, hipStream_t s) {
    (void)want;  // the head product reads want_dev
    if (M == 1 && one_token_fits_ && !opt_unfused_) return enqueue_one_token(n_want, s);
    const int W = cfg_.width, n = n_layers();
    A81W41_HIP_TRY(launch_embed_rows(ids, embed_.data, kTable, embed_.ld, states_, M, W,
                                     cfg_.vocab, s));
    A81W41_HIP_TRY(launch_group_norm<T>(states_, M, W, norm(layers_[0].norm1), h_, ld_h_, s));
    const float* x = states_;
    for (int i = 0; i < n; i++) {
        const Layer& L = layers_[i];
        const LayerConfig& lc = cfg_.layers[i];
        A81W41_TRY(attention(L, lc, M, s));
        SublayerOut y;
        y.y = y_;
        const float* norm_y = L.norm1b;
        if (lc.mlp.present) {
            A81W41_HIP_TRY(launch_residual_norm<T>(x, y, norm(L.norm1b), DepthAverage{}, x_, norm(L.norm2), h_, ld_h_, M, W, s));
            x = x_;
            A81W41_TRY(feed_forward(L, lc, M, s, &y));
            norm_y = L.norm2b;
        }
        DepthAverage depth;
        depth.states = states_, depth.state_step = state_step(), depth.coef = L.dwa, depth.n = i + 1;
        const float* next = i + 1 < n ? layers_[i + 1].norm1 : final_norm_;
        A81W41_HIP_TRY(launch_residual_norm<T>(x, y, norm(norm_y), depth, x_, norm(next), h_, ld_h_, M, W, s));
        x = x_;
    }
    if (n_want) {
        GemmArgs g = product(h_, ld_h_, head_, logits, cfg_.vocab, n_want);
        if (M > 1) g.a_rows = want_dev;
        A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    }
    A81W41_HIP_TRY(launch_advance(pos, M, s));
    return 0;
}

namespace {

int load_registered(const LoadRequest& req, a81w41_model** out) {
    return create_dense_model<TakosunModel>(read_config(*req.config), req, out);
}
const RegisterModel registered("Takosun", load_registered);

}  // namespace
}  // namespace a81w41
