// What the models with dense weights share on top of the session: weights on the device in the element type T, zero-padded
// to whole 128-byte steps, rotation tables, and the operands of a product.
#pragma once
#include <algorithm>
#include <cmath>
#include <map>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

#include "decoder_session.h"
#include "dense.h"
#include "tensor_source.h"

namespace a81w41 {

constexpr int kPassRows = 4096;  // tokens of one pass; longer portions are cut

inline void require(bool ok, const std::string& what) {
    if (!ok) throw std::runtime_error(what);
}

// Columns of a gate/up pair: 16 gates, their 16 ups, and so on.
inline int pair_columns(int ff) { return (ff + 15) / 16 * 32; }
inline int pair_row(int j, bool up) { return (j >> 4) * 32 + (up ? 16 : 0) + (j & 15); }

template <typename T>
struct Weight {  // [rows][ld], K padded with zeros
    T* data = nullptr;
    int rows = 0, k = 0, ld = 0;
};
// Gate/up pairs and the way back; experts one after the other.
template <typename T>
struct GatedWeights {
    Weight<T> gate_up, down;
};

template <typename T>
class DenseModel : public a81w41_model {
   public:
    ~DenseModel() override {
        if (stream) (void)hipStreamSynchronize(stream);
        for (void* p : owned_) (void)hipFree(p);
    }
    size_t weight_bytes() const override { return weight_bytes_; }

   protected:
    static constexpr bool kMatrixAttention = sizeof(T) == 2;
    static constexpr TableType kTable = sizeof(T) == 2 ? TableType::kBf16 : TableType::kFp32;

    int ready() const override { return 0; }  // creation loads everything or fails

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
    // around_zero: the tensor holds the distance from one
    int load_vector(TensorSource& src, const std::string& name, int n, float** out, bool around_zero = false) {
        std::vector<float> v;
        A81W41_TRY(src.matrix(name, 0, n, v));
        if (around_zero)
            for (float& x : v) x += 1.0f;
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
    int load_feed_forward(TensorSource& src, const std::vector<std::string>& prefixes, int width, int ff, GatedWeights<T>* out) {
        const int n = (int)prefixes.size(), cols = pair_columns(ff);
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
    // cos and sin of position * base^(-2 i / dims), [max_seq][dims / 2]; formed in double, one pair of tables per rotation
    int load_rotation(int dims, double base, int max_seq, float** cos_t, float** sin_t) {
        auto& slot = rotations_[{dims, base}];
        if (!slot.first) {
            const int half = dims / 2;
            std::vector<float> cs((size_t)max_seq * half), sn(cs.size());
            for (int i = 0; i < half; i++) {
                const double f = std::pow(base, -2.0 * i / dims);
                for (int p = 0; p < max_seq; p++) {
                    cs[(size_t)p * half + i] = (float)std::cos(p * f);
                    sn[(size_t)p * half + i] = (float)std::sin(p * f);
                }
            }
            A81W41_TRY(upload_array(cs, &slot.first));
            A81W41_TRY(upload_array(sn, &slot.second));
        }
        *cos_t = slot.first;
        *sin_t = slot.second;
        return 0;
    }
    GemmArgs product(const T* A, int lda, const Weight<T>& w, void* C, int ldc, int M) const {
        GemmArgs g;
        g.A = A, g.lda = lda, g.W = w.data, g.ldw = w.ld, g.K = w.ld, g.N = w.rows, g.C = C, g.ldc = ldc, g.M = M;
        return g;
    }

   private:
    std::vector<void*> owned_;
    size_t weight_bytes_ = 0;
    std::map<std::pair<int, double>, std::pair<float*, float*>> rotations_;
};

// The two instances of a model class by the request's precision, from its folder or with random weights.
template <template <typename> class Model, typename Config>
int create_dense_model(const Config& c, const LoadRequest& req, a81w41_model** out) {
    std::unique_ptr<TensorSource> src;
    if (req.random_weights)
        src = random_tensors(req.seed);
    else
        A81W41_TRY(open_safetensors(req.dir + "/model.safetensors", &src));
    auto create = [&](auto model) -> int {
        A81W41_TRY(model->create(req.max_seq, *src));
        *out = model.release();
        return 0;
    };
    return req.dtype == "float32" ? create(std::make_unique<Model<float>>(c)) : create(std::make_unique<Model<bf16>>(c));
}

}  // namespace a81w41
