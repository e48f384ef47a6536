// The Dimesun design on the shared decoder session: layers whose mixer (grouped attention over chunks of positions with a
// sink, or a matrix memory) and routed experts read one norm side by side, some of them run several times in a row with a
// cache or state for every pass.  This file owns the weights and activation buffers and enqueues the kernels of a pass; the
// mechanisms are in dense_gemm.hip, dense_rows.hip, attend_mfma.hip, attend_vector.hip and matrix_memory.hip, the loop over
// tokens in decoder_session.cpp.
//
// With N the RMS norm of weight 1 + w, a layer run is
//   x <- x + m (mixer(N1 x) + experts(N1 x)),
// ahead of which the first layer of a pass t over the repeated layers adds the vector step_t to x.
// logits = embed N(x).
#include <cmath>
#include <cstring>
#include <memory>

#include "dense_model.h"
#include "json.h"

namespace a81w41 {
namespace {

struct AttentionConfig {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, rot_dims = 0, chunk = 0;
    double rot_base = 0;
    float scale = 0.f;
    // widths as stored: whole 16-byte pieces in bfloat16
    int key_width() const { return (dim + 7) / 8 * 8; }
    int value_width() const { return (vdim + 7) / 8 * 8; }
    int row_width() const { return key_width() + value_width(); }
    int group() const { return heads / kv_heads; }
    int columns() const { return heads * key_width() + kv_heads * row_width(); }
};
struct ExpertsConfig {
    int experts = 0, top = 0, ff = 0;
    float limit = 0.f;
};
struct LayerConfig {
    bool memory = false, routed = false;
    AttentionConfig att;
    MemoryShape mem;
    ExpertsConfig moe;
    int mixer_width() const { return memory ? mem.heads * mem.vdim : att.heads * att.vdim; }
    int mixer_columns() const { return memory ? mem.at_f + mem.heads : att.columns(); }
    int columns() const { return mixer_columns() + (routed ? moe.experts : 0); }
    // floats of a row that leaves the product: all columns, or those that no head takes
    int row_stride() const { return ((memory ? columns() : columns() - mixer_columns()) + 3) / 4 * 4; }
};
struct Config {
    int vocab = 0, width = 0, loop_times = 0;
    float eps = 0.f, residual_mult = 1.f;
    std::vector<LayerConfig> layers;
    struct Run {
        int layer, opens;  // opens: the pass over the repeated layers that begins here, or -1
    };
    std::vector<Run> runs;
};

AttentionConfig read_attention(const Json& m, const std::string& where) {
    AttentionConfig a;
    a.heads = m.size("heads");
    a.kv_heads = m.size("kv_heads");
    a.dim = m.size("dim");
    a.vdim = m.size("vdim");
    a.chunk = m.at("mask").size("size");
    a.rot_dims = m.at("rot").size("dims");
    a.rot_base = m.at("rot").at("base").number();
    a.scale = (float)m.at("scale").number();
    require(a.heads % a.kv_heads == 0, where + "heads must be a multiple of kv_heads");
    require(a.rot_dims % 2 == 0 && a.rot_dims <= a.dim, where + "rot.dims must be even and at most dim");
    require(a.rot_base > 0, where + "rot.base must be positive");
    require(a.dim <= 4096 && a.vdim <= 4096 && a.heads <= 4096, where + "attention too large");
    return a;
}

MemoryShape read_memory(const Json& m, float eps, const std::string& where) {
    MemoryShape s;
    s.heads = m.size("heads");
    s.dim = m.size("dim");
    s.vdim = m.size("vdim");
    s.cap = (float)m.at("gate_cap").number();
    require(s.cap > 0.f, where + "gate_cap must be positive");
    require(s.dim <= 4096 && s.vdim <= 16384 && s.heads <= 4096, where + "matrix memory too large");
    s.q_scale = 1.0f / std::sqrt((float)s.dim);
    s.eps = eps;
    s.place_columns();
    return s;
}

Config read_config(const Json& j) {
    Config c;
    c.vocab = j.size("vocab");
    c.width = j.size("width");
    c.eps = (float)j.at("norm").at("eps").number();
    c.residual_mult = (float)j.at("residual_mult").number();
    require(c.eps >= 0.f, "norm.eps must not be negative");
    require(c.width <= 15000, "width must be at most 15000");
    for (const Json& l : j.at("layers").array()) {
        const std::string where = "layer " + std::to_string(c.layers.size()) + ": ", &type = l.at("type").string();
        LayerConfig out;
        if (type == "mlstm") {
            out.memory = true;
            out.mem = read_memory(l.at("mixer"), c.eps, where);
        } else {
            require(type == "attention", where + "unknown type '" + type + "'");
            out.att = read_attention(l.at("mixer"), where);
        }
        if (l.has("mlp")) {
            const Json& f = l.at("mlp");
            require(f.at("kind").string() == "moe", where + "unknown feed-forward '" + f.at("kind").string() + "'");
            out.routed = true;
            out.moe.experts = f.at("router").size("experts");
            out.moe.top = f.at("router").size("top");
            out.moe.ff = f.at("expert").size("ff");
            out.moe.limit = (float)f.at("expert").at("limit").number();
            require(out.moe.top <= out.moe.experts && out.moe.experts <= kMaxRouted && out.moe.top <= kMaxTop, where + "router out of range");
            require(out.moe.limit >= 0.f, where + "expert.limit must not be negative");
        }
        c.layers.push_back(out);
    }
    const int n = (int)c.layers.size();
    require(n > 0, "no layers");
    int start = n, stop = n;
    if (j.has("loop")) {
        const Json& loop = j.at("loop");
        const long long from = loop.at("start").integer(), to = loop.at("stop").integer();
        require(from >= 0 && from < to && to <= n, "loop.start and loop.stop must enclose layers");
        c.loop_times = loop.size("times");
        require(c.loop_times <= 4096, "loop.times is out of range");
        start = (int)from, stop = (int)to;
    }
    for (int i = 0; i < start; i++) c.runs.push_back({i, -1});
    for (int t = 0; t < c.loop_times; t++)
        for (int i = start; i < stop; i++) c.runs.push_back({i, i == start ? t : -1});
    for (int i = stop; i < n; i++) c.runs.push_back({i, -1});
    return c;
}

}  // namespace

template <typename T>
class DimesunModel final : public DenseModel<T> {
    using Base = DenseModel<T>;
    using Base::cache, Base::ids, Base::logits, Base::max_seq, Base::plan_ctx, Base::pos, Base::stream, Base::want_dev;
    using Base::allocate_array, Base::finish, Base::init_session, Base::kMatrixAttention, Base::kTable, Base::load_feed_forward,
        Base::load_matrix, Base::load_rotation, Base::load_vector, Base::product, Base::put_matrix, Base::upload_array;
    using Staging = typename Base::Staging;

   public:
    explicit DimesunModel(Config c) : cfg_(std::move(c)) {}
    int create(int max_seq, TensorSource& src) {
        A81W41_TRY(load_weights(max_seq, src));
        A81W41_TRY(allocate(max_seq));
        return 0;
    }
    // unfused: one-token passes take the kernels of longer ones; attention: 0 by shape, 1 the vector kernel;
    // attention_split: shares of the keys, 0 by length; memory: 0 by length, 1 token by token, 2 in chunks;
    // keep_states: the stream after every layer run is kept for read_buffer
    int set_option(const char* name, int value) override {
        const std::string n = name;
        if (n == "unfused" && value >= 0 && value <= 1)
            opt_unfused_ = value;
        else if (n == "attention" && value >= 0 && value <= 1)
            opt_attention_ = value;
        else if (n == "attention_split" && value >= 0 && value <= kAttendMaxSplits)
            opt_split_ = value;
        else if (n == "memory" && value >= 0 && value <= 2)
            opt_memory_ = value;
        else if (n == "keep_states" && value >= 0 && value <= 1) {
            if (value && !states_) A81W41_TRY(allocate_array((size_t)n_runs() * state_step(), &states_));
            opt_keep_ = value;
        } else {
            return failf(A81W41_ERR_INVALID_ARG, "no option '%s' with value %d", name, value);
        }
        return 0;
    }
    // state<i>: [tokens of the last pass][width], the stream after the i-th layer run
    int read_buffer(const char* name, float* host_out, size_t count) override {
        int i = -1;
        if (sscanf(name, "state%d", &i) != 1 || i < 0 || i >= n_runs() || !states_) return DecoderSession::read_buffer(name, host_out, count);
        if (count > (size_t)state_step()) return failf(A81W41_ERR_INVALID_ARG, "state holds fewer values");
        A81W41_HIP_TRY(hipStreamSynchronize(stream));
        A81W41_HIP_TRY(hipMemcpy(host_out, states_ + i * state_step(), count * sizeof(float), hipMemcpyDeviceToHost));
        return 0;
    }

   protected:
    int enqueue_pass(int M, const int* want, int n_want, hipStream_t s) override;

   private:
    struct Layer {
        float* norm1 = nullptr;
        Weight<T> in, o;  // in: all that reads the norm except the experts, [mixer's parts | router]
        GatedWeights<T> experts;
        float* router_bias = nullptr;
        float *cos_t = nullptr, *sin_t = nullptr;                              // attention
        float *bias_i = nullptr, *bias_f = nullptr, *memory_norm = nullptr;    // matrix memory
    };
    struct RunCache {
        T* rows = nullptr;       // attention
        float* state = nullptr;  // matrix memory
    };
    int n_runs() const { return (int)cfg_.runs.size(); }
    long long state_step() const { return (long long)rows_ * cfg_.width; }
    GroupNorm norm(const float* w) const { return GroupNorm{w, 1, cfg_.eps}; }
    GroupNorm residual() const { return GroupNorm{nullptr, 1, cfg_.eps, cfg_.residual_mult}; }
    const float* next_norm(int run) const { return run + 1 < n_runs() ? layers_[cfg_.runs[run + 1].layer].norm1 : final_norm_; }
    // the vector that is added ahead of a run
    const float* step_of(int run) const {
        const int t = run < n_runs() ? cfg_.runs[run].opens : -1;
        return t < 0 ? nullptr : loop_step_ + (size_t)t * cfg_.width;
    }
    int ld_cache(const AttentionConfig& c) const { return pad_k<T>(c.kv_heads * c.row_width()); }
    bool memory_in_chunks(const MemoryShape& sh, int M) const {
        return memory_chunks_fit(sh) && (opt_memory_ == 2 || (opt_memory_ == 0 && M > 1));
    }

    int load_weights(int max_seq, TensorSource& src);
    int load_attention(TensorSource& src, const std::string& mix, const LayerConfig& lc, Staging& in);
    int load_memory(TensorSource& src, const std::string& mix, const MemoryShape& sh, Staging& in, Layer* L);
    int allocate(int max_seq);
    HeadRows<T> head_rows(const Layer& L, const AttentionConfig& c, const RunCache& kept, float* rest, int ld_rest) const;
    AttendArgs<T> attend_args(const AttentionConfig& c, const RunCache& kept, int M) const;
    MemoryArgs memory_args(const Layer& L, const MemoryShape& sh, const RunCache& kept, int ld_in, int M) const;
    int attention(const Layer& L, const LayerConfig& lc, const RunCache& kept, int M, hipStream_t s);
    int memory(const Layer& L, const LayerConfig& lc, const RunCache& kept, int M, hipStream_t s);
    int routed_experts(const Layer& L, const LayerConfig& lc, int M, hipStream_t s, SublayerOut* out);
    int mixer_one_token(const Layer& L, const LayerConfig& lc, const RunCache& kept, const RowStep& step, MixerRow* out, hipStream_t s);
    int enqueue_one_token(int n_want, hipStream_t s);

    Config cfg_;
    std::vector<Layer> layers_;
    std::vector<RunCache> kept_;
    Weight<T> embed_;
    float *final_norm_ = nullptr, *loop_step_ = nullptr;
    // activations of one pass
    int rows_ = 0, ld_h_ = 0, ld_in_ = 0, ld_attn_ = 0;
    float *x_ = nullptr, *states_ = nullptr, *in_ = nullptr, *y_ = nullptr, *y2_ = nullptr, *o_memory_ = nullptr;
    T *h_ = nullptr, *q_ = nullptr, *attn_ = nullptr, *act_ = nullptr;
    float *part_ = nullptr, *part_stats_ = nullptr;  // shares of the attention
    size_t part_rows_ = 0;
    float *chunk_states_ = nullptr, *chunk_m_ = nullptr, *chunk_stats_ = nullptr;
    int *chosen_ = nullptr, *src_rows_ = nullptr, *slot_rows_ = nullptr, *n_tiles_ = nullptr;
    float* expert_weights_ = nullptr;
    GroupTile* tiles_ = nullptr;
    // of the one-token pass
    float *row_x_[2] = {nullptr, nullptr}, *h_row_ = nullptr, *mixer_row_ = nullptr, *act_row_ = nullptr;
    int ld_act_row_ = 0;
    bool one_token_fits_ = true;
    int opt_unfused_ = 0, opt_attention_ = 0, opt_split_ = 0, opt_memory_ = 0, opt_keep_ = 0;
};

// Queries, keys and values with their stored widths.  The rotation pairs component i of a head with i + dims / 2; rows are put
// so that the two are neighbours, which no score sees: a query and its keys share the order.
template <typename T>
int DimesunModel<T>::load_attention(TensorSource& src, const std::string& mix, const LayerConfig& lc, Staging& in) {
    const AttentionConfig& c = lc.att;
    const int width = cfg_.width, half = c.rot_dims / 2;
    auto place = [&](int d) { return d >= c.rot_dims ? d : d < half ? 2 * d : 2 * (d - half) + 1; };
    std::vector<float> v;
    int row0 = 0;
    for (const char* part : {"q", "k"}) {
        const int heads = part[0] == 'q' ? c.heads : c.kv_heads;
        A81W41_TRY(src.matrix(mix + part, heads * c.dim, width, v));
        for (int h = 0; h < heads; h++)
            for (int d = 0; d < c.dim; d++) in.put(row0 + h * c.key_width() + place(d), v.data() + (size_t)(h * c.dim + d) * width);
        row0 += heads * c.key_width();
    }
    A81W41_TRY(src.matrix(mix + "v", c.kv_heads * c.vdim, width, v));
    for (int h = 0; h < c.kv_heads; h++)
        for (int d = 0; d < c.vdim; d++) in.put(row0 + h * c.value_width() + d, v.data() + (size_t)(h * c.vdim + d) * width);
    return 0;
}

template <typename T>
int DimesunModel<T>::load_memory(TensorSource& src, const std::string& mix, const MemoryShape& sh, Staging& in, Layer* L) {
    const int keys = sh.heads * sh.dim, values = sh.heads * sh.vdim;
    A81W41_TRY(put_matrix(src, mix + "q", keys, cfg_.width, in, sh.at_q));
    A81W41_TRY(put_matrix(src, mix + "k", keys, cfg_.width, in, sh.at_k));
    A81W41_TRY(put_matrix(src, mix + "v", values, cfg_.width, in, sh.at_v));
    A81W41_TRY(put_matrix(src, mix + "g", values, cfg_.width, in, sh.at_g));
    A81W41_TRY(put_matrix(src, mix + "i", sh.heads, cfg_.width, in, sh.at_i));
    A81W41_TRY(put_matrix(src, mix + "f", sh.heads, cfg_.width, in, sh.at_f));
    A81W41_TRY(load_vector(src, mix + "i.b", sh.heads, &L->bias_i));
    A81W41_TRY(load_vector(src, mix + "f.b", sh.heads, &L->bias_f));
    return load_vector(src, mix + "norm", values, &L->memory_norm);
}

template <typename T>
int DimesunModel<T>::load_weights(int max_seq, TensorSource& src) {
    const int width = cfg_.width;
    A81W41_TRY(load_matrix(src, "embed", cfg_.vocab, width, &embed_));
    if (cfg_.loop_times) {
        std::vector<float> v;
        A81W41_TRY(src.matrix("loop.step", cfg_.loop_times, width, v));
        A81W41_TRY(upload_array(v, &loop_step_));
    }
    layers_.resize(cfg_.layers.size());
    for (size_t i = 0; i < layers_.size(); i++) {
        const LayerConfig& lc = cfg_.layers[i];
        Layer& L = layers_[i];
        const std::string p = "l" + std::to_string(i) + ".", mix = p + "mix.", mlp = p + "mlp.";
        A81W41_TRY(load_vector(src, p + "norm1", width, &L.norm1, true));
        Staging in(lc.columns(), width);
        if (lc.memory) {
            A81W41_TRY(load_memory(src, mix, lc.mem, in, &L));
        } else {
            A81W41_TRY(load_attention(src, mix, lc, in));
            A81W41_TRY(load_rotation(lc.att.rot_dims, lc.att.rot_base, max_seq, &L.cos_t, &L.sin_t));
        }
        A81W41_TRY(load_matrix(src, mix + "o", width, lc.mixer_width(), &L.o));
        if (lc.routed) {
            A81W41_TRY(put_matrix(src, mlp + "router", lc.moe.experts, width, in, lc.mixer_columns()));
            A81W41_TRY(load_vector(src, mlp + "router.b", lc.moe.experts, &L.router_bias));
            std::vector<std::string> names;
            for (int e = 0; e < lc.moe.experts; e++) names.push_back(mlp + "e" + std::to_string(e) + ".");
            A81W41_TRY(load_feed_forward(src, names, width, lc.moe.ff, &L.experts));
        }
        A81W41_TRY(finish(in, &L.in));
    }
    for (const Config::Run& run : cfg_.runs) {
        const LayerConfig& lc = cfg_.layers[run.layer];
        RunCache kept;
        void* p = nullptr;
        if (lc.memory) {
            A81W41_TRY(cache.add_state(lc.mem.state_size() * sizeof(float), &p));
            kept.state = static_cast<float*>(p);
        } else {
            A81W41_TRY(cache.add((size_t)max_seq * ld_cache(lc.att) * sizeof(T), &p));
            kept.rows = static_cast<T*>(p);
        }
        kept_.push_back(kept);
    }
    return load_vector(src, "final.norm", width, &final_norm_, true);
}

template <typename T>
int DimesunModel<T>::allocate(int max_seq) {
    rows_ = std::min(max_seq, kPassRows);
    A81W41_TRY(init_session(max_seq, cfg_.vocab, rows_));
    ld_h_ = pad_k<T>(cfg_.width);
    const size_t R = rows_, W = cfg_.width, chunks = (R + kMemoryChunk - 1) / kMemoryChunk;
    size_t q = 0, act = 0, o_memory = 0, chunk_states = 0, tiles = 0;
    int top = 0, heads = 0, memory_heads = 0, vdim = 0;
    one_token_fits_ = ld_h_ + 1 <= kGemvMaxRow;
    for (const LayerConfig& lc : cfg_.layers) {
        ld_in_ = std::max(ld_in_, lc.row_stride());
        ld_attn_ = std::max(ld_attn_, pad_k<T>(lc.mixer_width()));
        int row = pad_k<T>(lc.mixer_width());
        if (lc.memory) {
            o_memory = std::max(o_memory, (size_t)lc.mixer_width());
            chunk_states = std::max(chunk_states, lc.mem.heads * lc.mem.chunk_size());
            memory_heads = std::max(memory_heads, lc.mem.heads);
            row += lc.mem.heads;
        } else {
            q = std::max(q, (size_t)lc.att.heads * lc.att.key_width());
            heads = std::max(heads, lc.att.heads);
            vdim = std::max(vdim, (lc.att.vdim + 3) / 4 * 4);
            row += lc.att.heads * kMixerShares;
        }
        if (lc.routed) {
            top = std::max(top, lc.moe.top);
            act = std::max(act, (size_t)lc.moe.top * pad_k<T>(lc.moe.ff));
            ld_act_row_ = std::max(ld_act_row_, (lc.moe.ff + 3) / 4 * 4);
            tiles = std::max(tiles, R * lc.moe.top / kGroupTileRows + lc.moe.experts);
            row += lc.moe.top * pad_k<T>(lc.moe.ff);
            one_token_fits_ = one_token_fits_ && ld_h_ + lc.moe.experts <= kGemvMaxRow;
        }
        one_token_fits_ = one_token_fits_ && row <= kGemvMaxRow;
    }
    A81W41_TRY(allocate_array(R * W, &x_));
    A81W41_TRY(allocate_array(R * ld_h_, &h_));
    A81W41_TRY(allocate_array(R * ld_in_, &in_));
    A81W41_TRY(allocate_array(R * ld_attn_, &attn_));
    A81W41_TRY(allocate_array(R * W, &y_));
    A81W41_TRY(allocate_array(R * q, &q_));
    if (heads) {
        part_rows_ = std::max((size_t)heads * kAttendMaxSplits, (size_t)8192);
        A81W41_TRY(allocate_array(part_rows_ * vdim, &part_));
        A81W41_TRY(allocate_array(part_rows_ * 2, &part_stats_));
    }
    if (memory_heads) {
        A81W41_TRY(allocate_array(R * o_memory, &o_memory_));
        A81W41_TRY(allocate_array(chunks * chunk_states, &chunk_states_));
        A81W41_TRY(allocate_array((chunks + 1) * memory_heads, &chunk_m_));
        A81W41_TRY(allocate_array(chunks * memory_heads * 2, &chunk_stats_));
    }
    if (top) {
        A81W41_TRY(allocate_array(R * act, &act_));
        A81W41_TRY(allocate_array(R * top * W, &y2_));
        A81W41_TRY(allocate_array(R * top, &chosen_));
        A81W41_TRY(allocate_array(R * top, &expert_weights_));
        A81W41_TRY(allocate_array(R * top, &src_rows_));
        A81W41_TRY(allocate_array(R * top, &slot_rows_));
        A81W41_TRY(allocate_array(tiles, &tiles_));
        A81W41_TRY(allocate_array(1, &n_tiles_));
    }
    for (float** row : {&row_x_[0], &row_x_[1], &h_row_}) A81W41_TRY(allocate_array(W, row));
    A81W41_TRY(allocate_array((size_t)ld_attn_, &mixer_row_));
    return allocate_array((size_t)std::max(top, 1) * ld_act_row_, &act_row_);
}

template <typename T>
HeadRows<T> DimesunModel<T>::head_rows(const Layer& L, const AttentionConfig& c, const RunCache& kept, float* rest, int ld_rest) const {
    HeadRows<T> r;
    r.heads = c.heads, r.kv_heads = c.kv_heads, r.dim = c.key_width(), r.vdim = c.value_width(), r.rot_pairs = c.rot_dims / 2;
    r.q = q_, r.cache = kept.rows, r.ld_cache = ld_cache(c), r.cos_t = L.cos_t, r.sin_t = L.sin_t, r.pos_dev = pos, r.max_seq = max_seq();
    r.rest = rest, r.ld_rest = ld_rest;
    return r;
}

template <typename T>
AttendArgs<T> DimesunModel<T>::attend_args(const AttentionConfig& c, const RunCache& kept, int M) const {
    AttendArgs<T> a;
    const int R = c.group(), key = c.key_width();
    a.q = q_, a.q_head = (long long)R * key, a.q_token = c.heads * key, a.ld_q = key, a.rows = M * R, a.rows_per_token = R;
    a.k_own = kept.rows, a.k_own_head = c.row_width(), a.ld_k_own = ld_cache(c), a.k_own_width = key;
    a.v_width = c.value_width(), a.dv = c.vdim;
    a.out_head = (long long)R * c.vdim, a.out_token = ld_attn_, a.ld_out = c.vdim;
    a.part = part_, a.part_stats = part_stats_, a.ld_part = (c.vdim + 3) / 4 * 4;
    a.scale = c.scale, a.chunk = c.chunk, a.sink = true, a.pos_dev = pos, a.max_seq = max_seq();
    // enough workgroups for the chip, at least 64 keys for each
    const int keys = std::min(plan_ctx, c.chunk + M - 1);
    const int groups = c.kv_heads * (a.rows <= kAttendFewRows ? (a.rows + 15) / 16 : (a.rows + 63) / 64);
    a.splits = opt_split_ ? opt_split_ : std::min({kAttendMaxSplits, (keys + 63) / 64, std::max(1, 512 / groups)});
    a.splits = std::max<int>(1, std::min<size_t>(a.splits, part_rows_ / ((size_t)c.heads * M)));
    return a;
}

template <typename T>
MemoryArgs DimesunModel<T>::memory_args(const Layer& L, const MemoryShape& sh, const RunCache& kept, int ld_in, int M) const {
    MemoryArgs a;
    a.sh = sh, a.in = in_, a.ld_in = ld_in, a.M = M, a.bias_i = L.bias_i, a.bias_f = L.bias_f, a.norm = L.memory_norm;
    a.state = kept.state, a.pos_dev = pos;
    a.chunk_states = chunk_states_, a.chunk_m = chunk_m_, a.chunk_stats = chunk_stats_;
    return a;
}

// Attention on h_: leaves the heads' rows in attn_, the router's logits in in_.
template <typename T>
int DimesunModel<T>::attention(const Layer& L, const LayerConfig& lc, const RunCache& kept, int M, hipStream_t s) {
    const AttentionConfig& c = lc.att;
    A81W41_HIP_TRY(launch_dense_gemm_heads<T>(product(h_, ld_h_, L.in, nullptr, 0, M), head_rows(L, c, kept, in_, lc.row_stride()), s));
    AttendArgs<T> a = attend_args(c, kept, M);
    a.out = attn_;
    if constexpr (kMatrixAttention) {
        if (opt_attention_ != 1 && attend_rows_fits(c.key_width(), c.value_width())) {
            A81W41_HIP_TRY(launch_attend_rows(a, c.kv_heads, s));
            if (a.splits > 1) A81W41_HIP_TRY(launch_merge_shares(a, c.kv_heads, s));
            return 0;
        }
    }
    A81W41_HIP_TRY((launch_attend_vector<T, T>(a, c.kv_heads, attn_, s)));
    return 0;
}

// The matrix memory on h_: leaves the normed and gated rows in attn_, the router's logits in in_.
template <typename T>
int DimesunModel<T>::memory(const Layer& L, const LayerConfig& lc, const RunCache& kept, int M, hipStream_t s) {
    const int ld = lc.row_stride();
    A81W41_HIP_TRY(launch_dense_gemm<T>(product(h_, ld_h_, L.in, in_, ld, M), Epilogue::kFloat, s));
    const MemoryArgs a = memory_args(L, lc.mem, kept, ld, M);
    if (memory_in_chunks(lc.mem, M)) {
        A81W41_HIP_TRY(launch_memory_chunks<T>(a, attn_, ld_attn_, s));
    } else {
        A81W41_HIP_TRY(launch_memory_steps(a, o_memory_, s));
        A81W41_HIP_TRY(launch_memory_norm<T>(a, o_memory_, attn_, ld_attn_, s));
    }
    return 0;
}

// The experts on h_, chosen by the logits in in_.
template <typename T>
int DimesunModel<T>::routed_experts(const Layer& L, const LayerConfig& lc, int M, hipStream_t s, SublayerOut* out) {
    const ExpertsConfig& f = lc.moe;
    const int W = cfg_.width, ld = pad_k<T>(f.ff), cols = pair_columns(f.ff);
    const float* logits = lc.memory ? in_ + lc.mixer_columns() : in_;
    A81W41_HIP_TRY(launch_router(logits, lc.row_stride(), L.router_bias, f.experts, f.top, M, chosen_, expert_weights_, s));
    A81W41_HIP_TRY(launch_expert_rows(nullptr, chosen_, M, f.top, f.experts, M, src_rows_, slot_rows_, tiles_, n_tiles_, s));
    GemmArgs g = product(h_, ld_h_, L.experts.gate_up, act_, ld, M * f.top);
    g.N = cols, g.w_step = (long long)cols * L.experts.gate_up.ld, g.a_rows = src_rows_;
    g.unit = GatedUnit{f.limit, 1.702f, 1.f};
    g.tiles = tiles_, g.n_tiles = n_tiles_, g.max_tiles = M * f.top / kGroupTileRows + std::min(f.experts, M * f.top);
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kGatedPair, s));
    g.A = act_, g.lda = ld, g.a_rows = nullptr, g.W = L.experts.down.data, g.ldw = g.K = L.experts.down.ld;
    g.N = W, g.w_step = (long long)W * L.experts.down.ld, g.C = y2_, g.ldc = W;
    A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    out->y = y2_, out->slot_rows = slot_rows_, out->top = f.top, out->weights = expert_weights_;
    return 0;
}

// A mixer for one token behind the residual step `step`; the router's logits go to in_.
template <typename T>
int DimesunModel<T>::mixer_one_token(const Layer& L, const LayerConfig& lc, const RunCache& kept, const RowStep& step, MixerRow* out,
                                     hipStream_t s) {
    out->width = lc.mixer_width();
    out->row = mixer_row_;
    if (lc.memory) {
        const MemoryShape& sh = lc.mem;
        A81W41_HIP_TRY(launch_gemv_step<T>(step, L.in.data, L.in.ld, L.in.rows, in_, s));
        A81W41_HIP_TRY(launch_memory_steps(memory_args(L, sh, kept, lc.row_stride(), 1), mixer_row_, s));
        out->heads = sh.heads, out->vdim = sh.vdim, out->norm = L.memory_norm, out->gates = in_ + sh.at_g, out->eps = sh.eps;
        return 0;
    }
    const AttentionConfig& c = lc.att;
    A81W41_HIP_TRY(launch_gemv_step_heads<T>(step, L.in.data, L.in.ld, L.in.rows, head_rows(L, c, kept, in_, lc.row_stride()), s));
    AttendArgs<T> a = attend_args(c, kept, 1);
    out->heads = c.heads, out->vdim = c.vdim;
    if constexpr (kMatrixAttention) {
        if (opt_attention_ != 1 && attend_rows_fits(c.key_width(), c.value_width())) {
            a.splits = std::max(2, std::min(a.splits, kMixerShares));  // shares stay fp32; the output product merges them
            A81W41_HIP_TRY(launch_attend_rows(a, c.kv_heads, s));
            out->shares = LatentShares{a.part, a.part_stats, a.splits, a.ld_part};
            return 0;
        }
    }
    A81W41_HIP_TRY((launch_attend_vector<T, float>(a, c.kv_heads, mixer_row_, s)));
    return 0;
}

// The pass for one token, four launches a run: [residual step, norm, product of all that reads the norm], the mixer, [choice
// of the experts, gate and up], [the mixer's norm and gate or the merge of its shares, output and down products].
template <typename T>
int DimesunModel<T>::enqueue_one_token(int n_want, hipStream_t s) {
    const int W = cfg_.width;
    A81W41_HIP_TRY(launch_embed_rows(ids, embed_.data, kTable, embed_.ld, x_, 1, W, cfg_.vocab, s));
    RowStep step;  // what the next product's prologue does
    step.width = W, step.x = x_, step.norm_h = norm(layers_[cfg_.runs[0].layer].norm1);
    for (int i = 0; i < n_runs(); i++) {
        const Layer& L = layers_[cfg_.runs[i].layer];
        const LayerConfig& lc = cfg_.layers[cfg_.runs[i].layer];
        step.before = step_of(i), step.x_out = row_x_[i & 1], step.h_out = h_row_;
        MixerRow mixed;
        A81W41_TRY(mixer_one_token(L, lc, kept_[i], step, &mixed, s));
        ExpertRows e;
        if (lc.routed) {
            e.top = lc.moe.top, e.experts = lc.moe.experts, e.ff = lc.moe.ff, e.pair_rows = pair_columns(lc.moe.ff), e.ld_act = ld_act_row_;
            e.unit = GatedUnit{lc.moe.limit, 1.702f, 1.f};
            e.logits = lc.memory ? in_ + lc.mixer_columns() : in_, e.bias = L.router_bias, e.chosen = chosen_, e.weights = expert_weights_;
            A81W41_HIP_TRY(launch_gemv_gate_up<T>(step, h_row_, e, L.experts.gate_up.data, nullptr, L.experts.gate_up.ld, act_row_, s));
        }
        A81W41_HIP_TRY(launch_gemv_mixer_down<T>(mixed, L.o.data, L.o.ld, e, act_row_, L.experts.down.data, L.experts.down.ld, W, y_, s));
        step = RowStep{};
        step.width = W, step.x = row_x_[i & 1], step.y = y_, step.norm_y = residual(), step.norm_h = norm(next_norm(i));
        if (opt_keep_) step.state = states_ + i * state_step();
    }
    step.x_out = row_x_[n_runs() & 1];  // the state may be asked for even where no logits are
    A81W41_HIP_TRY(launch_gemv_step<T>(step, embed_.data, embed_.ld, n_want ? embed_.rows : 1, logits, s));
    A81W41_HIP_TRY(launch_advance(pos, 1, s));
    return 0;
}

template <typename T>
int DimesunModel<T>::enqueue_pass(int M, const int* want, int n_want, hipStream_t s) {
    (void)want;  // the head product reads want_dev
    if (M == 1 && one_token_fits_ && !opt_unfused_) return enqueue_one_token(n_want, s);
    const int W = cfg_.width;
    A81W41_HIP_TRY(launch_embed_rows(ids, embed_.data, kTable, embed_.ld, x_, M, W, cfg_.vocab, s));
    A81W41_HIP_TRY(launch_residual_norm<T>(x_, SublayerOut{}, GroupNorm{}, DepthAverage{}, x_, norm(layers_[cfg_.runs[0].layer].norm1), h_,
                                           ld_h_, M, W, s, step_of(0)));
    for (int i = 0; i < n_runs(); i++) {
        const Layer& L = layers_[cfg_.runs[i].layer];
        const LayerConfig& lc = cfg_.layers[cfg_.runs[i].layer];
        A81W41_TRY(lc.memory ? memory(L, lc, kept_[i], M, s) : attention(L, lc, kept_[i], M, s));
        A81W41_HIP_TRY(launch_dense_gemm<T>(product(attn_, ld_attn_, L.o, y_, W, M), Epilogue::kFloat, s));
        SublayerOut y;
        y.y = y_;
        if (lc.routed) {
            A81W41_TRY(routed_experts(L, lc, M, s, &y));
            y.shared = y_;
        }
        DepthAverage keep;
        if (opt_keep_) keep.states = states_, keep.state_step = state_step(), keep.n = i;
        A81W41_HIP_TRY(launch_residual_norm<T>(x_, y, residual(), keep, x_, norm(next_norm(i)), h_, ld_h_, M, W, s, step_of(i + 1)));
    }
    if (n_want) {
        GemmArgs g = product(h_, ld_h_, embed_, logits, cfg_.vocab, n_want);
        if (M > 1) g.a_rows = want_dev;
        A81W41_HIP_TRY(launch_dense_gemm<T>(g, Epilogue::kFloat, s));
    }
    A81W41_HIP_TRY(launch_advance(pos, M, s));
    return 0;
}

namespace {

int load_registered(const LoadRequest& req, a81w41_model** out) {
    return create_dense_model<DimesunModel>(read_config(*req.config), req, out);
}
const RegisterModel registered("Dimesun", load_registered);

}  // namespace
}  // namespace a81w41
