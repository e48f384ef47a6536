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
#include <algorithm>
#include <cmath>
#include <cstring>
#include <map>
#include <memory>
#include <new>

#include "dense.h"
#include "json.h"
#include "tensor_source.h"

namespace a81w41 {
namespace {

constexpr int kPassRows = 4096;  // tokens of one pass; longer portions are cut

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

void require(bool ok, const std::string& what) {
    if (!ok) throw std::runtime_error(what);
}

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

// Columns of a gate/up pair: 16 gates, their 16 ups, and so on.
int pair_columns(int ff) { return (ff + 15) / 16 * 32; }
int pair_row(int j, bool up) { return (j >> 4) * 32 + (up ? 16 : 0) + (j & 15); }

template <typename T>
struct Weight {  // [rows][ld], K padded with zeros
    T* data = nullptr;
    int rows = 0, k = 0, ld = 0;
};

}  // namespace

template <typename T>
class TakosunModel final : public a81w41_model {
   public:
    explicit TakosunModel(Config c) : cfg_(std::move(c)) {}
    ~TakosunModel() override {
        if (stream) (void)hipStreamSynchronize(stream);
        for (void* p : owned_) (void)hipFree(p);
    }
    int create(int max_seq, TensorSource& src) {
        A81W41_TRY(load_weights(max_seq, src));
        A81W41_TRY(allocate(max_seq));
        return 0;
    }
    size_t weight_bytes() const override { return weight_bytes_; }

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
    int ready() const override { return 0; }  // create() loads everything or fails
    int enqueue_pass(int M, const int* want, int n_want, hipStream_t s) override;

   private:
    struct FeedForward {
        Weight<T> gate_up, down;  // experts: one after the other
    };
    struct Layer {
        float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr, *dwa = nullptr;
        float *q_norm = nullptr, *kv_norm = nullptr;
        Weight<T> down;  // [dq | dkv | g]
        Weight<T> uq, uk_t, uv, o;
        FeedForward ff, shared;
        int* table = nullptr;
        T* cache = nullptr;
        float *cos_t = nullptr, *sin_t = nullptr;
    };
    int n_layers() const { return (int)cfg_.layers.size(); }
    long long state_step() const { return (long long)rows_ * cfg_.width; }
    GroupNorm norm(const float* w) const { return GroupNorm{w, cfg_.groups, cfg_.eps}; }

    template <typename E>
    int allocate_array(size_t n, E** out, bool weight = false) {
        void* p = nullptr;
        A81W41_HIP_TRY(hipMalloc(&p, std::max<size_t>(n, 1) * sizeof(E)));
        owned_.push_back(p);
        A81W41_HIP_TRY(hipMemset(p, 0, std::max<size_t>(n, 1) * sizeof(E)));
        if (weight) weight_bytes_ += n * sizeof(E);
        *out = static_cast<E*>(p);
        return 0;
    }
    template <typename E>
    int upload_array(const std::vector<E>& v, E** out) {
        A81W41_TRY(allocate_array(v.size(), out, true));
        A81W41_HIP_TRY(hipMemcpy(*out, v.data(), v.size() * sizeof(E), hipMemcpyHostToDevice));
        return 0;
    }
    // A weight under construction on the host: rows are put one tensor at a time, then it goes to the device.
    struct Staging {
        std::vector<T> data;
        int rows, k, ld;
        Staging(int rows_, int k_) : data((size_t)rows_ * pad_k<T>(k_)), rows(rows_), k(k_), ld(pad_k<T>(k_)) {}
        void put(int row, const float* src) {
            for (int i = 0; i < k; i++) data[(size_t)row * ld + i] = (T)src[i];
        }
    };
    int finish(const Staging& st, Weight<T>* w) {
        w->rows = st.rows;
        w->k = st.k;
        w->ld = st.ld;
        return upload_array(st.data, &w->data);
    }
    int load_vector(TensorSource& src, const std::string& name, int n, float** out) {
        std::vector<float> v;
        A81W41_TRY(src.matrix(name, 0, n, v));
        return upload_array(v, out);
    }
    int put_matrix(TensorSource& src, const std::string& name, int rows, int k, Staging& st, int row0) {
        std::vector<float> v;
        A81W41_TRY(src.matrix(name, rows, k, v));
        for (int r = 0; r < rows; r++) st.put(row0 + r, v.data() + (size_t)r * k);
        return 0;
    }
    int load_matrix(TensorSource& src, const std::string& name, int rows, int k, Weight<T>* w) {
        Staging st(rows, k);
        A81W41_TRY(put_matrix(src, name, rows, k, st, 0));
        return finish(st, w);
    }
    int load_feed_forward(TensorSource& src, const std::vector<std::string>& prefixes, int ff, FeedForward* out) {
        const int n = (int)prefixes.size(), width = cfg_.width, cols = pair_columns(ff);
        Staging gu(n * cols, width), down(n * width, ff);
        std::vector<float> v;
        for (int e = 0; e < n; e++) {
            for (int up = 0; up < 2; up++) {
                A81W41_TRY(src.matrix(prefixes[e] + (up ? "up" : "gate"), ff, width, v));
                for (int j = 0; j < ff; j++) gu.put(e * cols + pair_row(j, up), v.data() + (size_t)j * width);
            }
            A81W41_TRY(put_matrix(src, prefixes[e] + "down", width, ff, down, e * width));
        }
        A81W41_TRY(finish(gu, &out->gate_up));
        return finish(down, &out->down);
    }
    int load_weights(int max_seq, TensorSource& src);
    int load_rotation(const LayerConfig& lc, int max_seq, Layer* L);
    int allocate(int max_seq);
    int attention(const Layer& L, const LayerConfig& lc, int M, hipStream_t s);
    int feed_forward(const Layer& L, const LayerConfig& lc, int M, hipStream_t s, SublayerOut* out);
    int pair_product(const FeedForward& f, int ff, const T* h, const GemmArgs& base, T* act, hipStream_t s);
    GemmArgs product(const T* A, int lda, const Weight<T>& w, void* C, int ldc, int M) const {
        GemmArgs g;
        g.A = A, g.lda = lda, g.W = w.data, g.ldw = w.ld, g.K = w.ld, g.N = w.rows, g.C = C, g.ldc = ldc, g.M = M;
        return g;
    }

    Config cfg_;
    std::vector<Layer> layers_;
    Weight<T> embed_, head_;
    float* final_norm_ = nullptr;
    std::vector<void*> owned_;
    size_t weight_bytes_ = 0;
    std::map<std::pair<int, double>, std::pair<float*, float*>> rotations_;
    // activations of one pass
    int rows_ = 0, ld_h_ = 0, ld_down_ = 0, ld_q_ = 0, ld_cq_ = 0, ld_attn_ = 0;
    float *x_ = nullptr, *states_ = nullptr, *down_ = nullptr, *q_ = nullptr, *y_ = nullptr, *y2_ = nullptr, *y_shared_ = nullptr;
    T *h_ = nullptr, *c_q_ = nullptr, *nope_ = nullptr, *q_lat_ = nullptr, *o_lat_ = nullptr, *attn_ = nullptr, *act_ = nullptr;
    int *src_rows_ = nullptr, *slot_rows_ = nullptr, *n_tiles_ = nullptr;
    GroupTile* tiles_ = nullptr;
};

template <typename T>
int TakosunModel<T>::load_rotation(const LayerConfig& lc, int max_seq, Layer* L) {
    auto& slot = rotations_[{lc.mix.rot, lc.rot_base}];
    if (!slot.first) {
        const int half = lc.mix.rot / 2;
        std::vector<float> cs((size_t)max_seq * half), sn(cs.size());
        for (int i = 0; i < half; i++) {
            const double f = std::pow(lc.rot_base, -2.0 * i / lc.mix.rot);
            for (int p = 0; p < max_seq; p++) {
                cs[(size_t)p * half + i] = (float)std::cos(p * f);
                sn[(size_t)p * half + i] = (float)std::sin(p * f);
            }
        }
        A81W41_TRY(upload_array(cs, &slot.first));
        A81W41_TRY(upload_array(sn, &slot.second));
    }
    L->cos_t = slot.first;
    L->sin_t = slot.second;
    return 0;
}

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
        A81W41_TRY(load_rotation(lc, max_seq, &L));
        A81W41_TRY(load_matrix(src, mix + "uq", sh.heads * (sh.dim + sh.rot), sh.q_rank, &L.uq));
        {   // the key up-projection of a head, transposed: it maps an unrotated query to latent space
            std::vector<float> uk, row(sh.dim);
            A81W41_TRY(src.matrix(mix + "uk", sh.heads * sh.dim, sh.rank, uk));
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
            A81W41_TRY(load_feed_forward(src, {mlp}, f.ff, &L.ff));
            continue;
        }
        std::vector<std::string> names;
        for (int e = 0; e < f.experts; e++) names.push_back(mlp + "e" + std::to_string(e) + ".");
        A81W41_TRY(load_feed_forward(src, names, f.ff, &L.ff));
        if (f.shared_ff) A81W41_TRY(load_feed_forward(src, {mlp + "shared."}, f.shared_ff, &L.shared));
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
    size_t nope = 0, q_lat = 0, o_lat = 0, act = 0, expert_rows = 0, tiles = 0;
    for (const LayerConfig& lc : cfg_.layers) {
        const LatentShape& sh = lc.mix;
        ld_down_ = std::max(ld_down_, sh.q_rank + sh.rank + sh.rot + sh.heads);
        ld_q_ = std::max(ld_q_, sh.heads * (sh.dim + sh.rot));
        ld_cq_ = std::max(ld_cq_, pad_k<T>(sh.q_rank));
        ld_attn_ = std::max(ld_attn_, pad_k<T>(sh.heads * sh.vdim));
        nope = std::max(nope, (size_t)sh.heads * pad_k<T>(sh.dim));
        q_lat = std::max(q_lat, (size_t)sh.heads * sh.ld_cache);
        o_lat = std::max(o_lat, (size_t)sh.heads * pad_k<T>(sh.rank));
        const FeedForwardConfig& f = lc.mlp;
        if (!f.present) continue;
        act = std::max(act, (size_t)std::max(f.top, 1) * pad_k<T>(f.ff));
        act = std::max(act, (size_t)pad_k<T>(f.shared_ff));
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

// The mixer on h_: leaves its output rows in y_.
template <typename T>
int TakosunModel<T>::attention(const Layer& L, const LayerConfig& lc, int M, hipStream_t s) {
    const LatentShape& sh = lc.mix;
    const bool own = lc.kv_from < 0;
    const int gates_at = sh.q_rank + (own ? sh.rank + sh.rot : 0);
    LatentRows in;
    in.down = down_, in.ld_down = ld_down_, in.q_norm = L.q_norm, in.kv_norm = L.kv_norm, in.eps = cfg_.eps;
    in.cos_t = L.cos_t, in.sin_t = L.sin_t, in.pos_dev = pos, in.max_seq = max_seq();
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(h_, ld_h_, L.down, down_, ld_down_, M), Epilogue::kFloat, s));
    A81W41_HIP_TRY(launch_latent_rows<T>(in, sh, M, c_q_, ld_cq_, own ? L.cache : nullptr, s));
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(c_q_, ld_cq_, L.uq, q_, ld_q_, M), Epilogue::kFloat, s));
    const int ld_nope = pad_k<T>(sh.dim), ld_rank = pad_k<T>(sh.rank);
    // query rows like cache rows: the part in latent space comes from the product below
    A81W41_HIP_TRY(launch_rotate_queries<T>(q_, ld_q_, in, sh, M, nope_, ld_nope, q_lat_ + sh.rank, sh.ld_cache, s));
    GemmArgs g = product(nope_, sh.heads * ld_nope, L.uk_t, q_lat_, sh.heads * sh.ld_cache, M);
    g.N = sh.rank, g.batches = sh.heads, g.a_step = ld_nope, g.w_step = (long long)sh.rank * L.uk_t.ld, g.c_step = sh.ld_cache;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kElement, s));
    A81W41_HIP_TRY(launch_latent_attention_vector<T>(q_lat_, L.cache, sh, pos, max_seq(), M, o_lat_, ld_rank, s));
    g = product(o_lat_, sh.heads * ld_rank, L.uv, attn_, ld_attn_, M);
    g.N = sh.vdim, g.batches = sh.heads, g.a_step = ld_rank, g.w_step = (long long)sh.vdim * L.uv.ld, g.c_step = sh.vdim;
    g.head_gate = down_ + gates_at, g.ld_gate = ld_down_;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kHeadGate, s));
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
        A81W41_HIP_TRY(launch_dense_gemm<T>(product(h_, ld_h_, w.gate_up, act_, ld, M), Epilogue::kSiluPair, s));
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
    A81W41_HIP_TRY(launch_table_route(ids, L.table, cfg_.vocab, f.top, f.experts, M, src_rows_, slot_rows_, tiles_, n_tiles_, s));
    const int ld = pad_k<T>(f.ff), cols = pair_columns(f.ff);
    GemmArgs g = product(h_, ld_h_, L.ff.gate_up, act_, ld, M * f.top);
    g.N = cols, g.w_step = (long long)cols * L.ff.gate_up.ld, g.a_rows = src_rows_;
    g.tiles = tiles_, g.n_tiles = n_tiles_, g.max_tiles = M * f.top / kGroupTileRows + std::min(f.experts, M * f.top);
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kSiluPair, s));
    g.A = act_, g.lda = ld, g.a_rows = nullptr, g.W = L.ff.down.data, g.ldw = g.K = L.ff.down.ld;
    g.N = W, g.w_step = (long long)W * L.ff.down.ld, g.C = y2_, g.ldc = W;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    out->y = y2_, out->slot_rows = slot_rows_, out->top = f.top;
    return 0;
}

template <typename T>
int TakosunModel<T>::enqueue_pass(int M, const int* want, int n_want, hipStream_t s) {
    const int W = cfg_.width, n = n_layers();
    A81W41_HIP_TRY(launch_embed_rows(ids, embed_.data, sizeof(T) == 2 ? TableType::kBf16 : TableType::kFp32, embed_.ld, states_, M, W,
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

template <typename T>
int create_model(const Config& c, const LoadRequest& req, TensorSource& src, a81w41_model** out) {
    auto m = std::make_unique<TakosunModel<T>>(c);
    A81W41_TRY(m->create(req.max_seq, src));
    *out = m.release();
    return 0;
}

int load_registered(const LoadRequest& req, a81w41_model** out) {
    const Config c = read_config(*req.config);
    std::unique_ptr<TensorSource> src;
    if (req.random_weights)
        src = random_tensors(req.seed);
    else
        A81W41_TRY(open_safetensors(req.dir + "/model.safetensors", &src));
    return req.dtype == "float32" ? create_model<float>(c, req, *src, out) : create_model<bf16>(c, req, *src, out);
}
const RegisterModel registered("Takosun", load_registered);

}  // namespace
}  // namespace a81w41
