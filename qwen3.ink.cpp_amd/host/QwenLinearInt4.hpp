// Host-side mirror of the reference's linear-layer interface on top of the C ABI
// (include/a81w41.h).  A caller written against the reference's
//   ModelContext                           qwen3/include/qwen/QwenOperator.h:34-43
//   Qwen_Linear_with_bias_Int4             qwen3/include/qwen/QwenOperator.h:86-231
//   Matrix3D<float>                        qwen3/include/common.h:13
// compiles against these classes unchanged for the hot path: same constructor
// arguments (ctx, path, 1, N, K), same forward(const Matrix3D<float>&) returning a
// Matrix3D<float>(batch, M, N), same M-dispatch (M == 1: fp16-parameter quantiser
// + GEMV, M > 1: fp32-parameter quantiser + GEMM).  Weights live on the GPU; the
// activations are copied in and the result out on every call, like any caller
// that keeps its tensors in host memory must.
//
// Header only; link with -la81w41 -la81w41_core.  Failures throw std::runtime_error with the
// library's message (the reference aborts on asserts / throws on file errors).
#pragma once

#include <algorithm>
#include <memory>
#include <stdexcept>
#include <string>

#include "../../include/a81w41.h"

namespace a81w41 {

inline void check(int status, const char* what) {
    if (status != A81W41_OK)
        throw std::runtime_error(std::string(what) + ": " + a81w41_status_string(status) + ": " + a81w41_last_error());
}

// Minimal owning row-major x*y*z tensor with the member names the reference's
// layers use (m_data, m_dim_x/y/z, data(), size()).
template <typename T>
class Matrix3D {
   public:
    std::unique_ptr<T[]> m_data;
    int m_dim_x = 0, m_dim_y = 0, m_dim_z = 0;

    Matrix3D() = default;
    Matrix3D(int dim_x, int dim_y, int dim_z) : m_dim_x(dim_x), m_dim_y(dim_y), m_dim_z(dim_z) {
        if (size() > 0) m_data = std::make_unique<T[]>(size());
    }
    Matrix3D(const T* src, int dim_x, int dim_y, int dim_z) : Matrix3D(dim_x, dim_y, dim_z) {
        if (src && size() > 0) std::copy(src, src + size(), m_data.get());
    }
    Matrix3D(const Matrix3D& o) : Matrix3D(o.data(), o.m_dim_x, o.m_dim_y, o.m_dim_z) {}
    Matrix3D(Matrix3D&& o) noexcept = default;
    Matrix3D& operator=(Matrix3D o) noexcept {
        std::swap(m_data, o.m_data);
        std::swap(m_dim_x, o.m_dim_x);
        std::swap(m_dim_y, o.m_dim_y);
        std::swap(m_dim_z, o.m_dim_z);
        return *this;
    }
    T* data() { return m_data.get(); }
    const T* data() const { return m_data.get(); }
    size_t size() const { return (size_t)m_dim_x * m_dim_y * m_dim_z; }
    T& operator()(int x, int y, int z) { return m_data[((size_t)x * m_dim_y + y) * m_dim_z + z]; }
    const T& operator()(int x, int y, int z) const { return m_data[((size_t)x * m_dim_y + y) * m_dim_z + z]; }
};

// The scratch every layer quantises its activations into (device memory here).
// The reference sizes it for max_sqlen x 12288 activations (QwenForCausalLM.cc:101-113).
struct ModelContext {
    a81w41_context* handle = nullptr;
    explicit ModelContext(int max_rows = 4096, int max_cols = 12288) {
        check(a81w41_context_create(max_rows, max_cols, &handle), "a81w41_context_create");
    }
    ~ModelContext() { a81w41_context_destroy(handle); }
    ModelContext(const ModelContext&) = delete;
    ModelContext& operator=(const ModelContext&) = delete;
};

class Qwen_Linear_with_bias_Int4 {
    int weight_cols = 0, weight_rows = 0;
    ModelContext* context_ = nullptr;
    std::shared_ptr<a81w41_linear> layer_;  // copies of a layer share the (read-only) device blobs

    void adopt(a81w41_linear* raw) { layer_ = std::shared_ptr<a81w41_linear>(raw, a81w41_linear_destroy); }

   public:
    Qwen_Linear_with_bias_Int4() = default;

    // Reads <path>weight_int4.bin, scaling_factor_int4.bin, offset_int4.bin and repacks
    // them into both block layouts (QwenOperator.h:112-157).
    Qwen_Linear_with_bias_Int4(ModelContext* ctx, std::string path, int weight_dim_x, int weight_dim_y,
                               int weight_dim_z)
        : weight_cols(weight_dim_y), weight_rows(weight_dim_z), context_(ctx) {
        a81w41_linear* raw = nullptr;
        check(a81w41_linear_load(ctx->handle, path.c_str(), weight_dim_x, weight_dim_y, weight_dim_z, &raw),
              "a81w41_linear_load");
        adopt(raw);
    }

    // Same layer from arrays already in memory in the file layout.
    Qwen_Linear_with_bias_Int4(ModelContext* ctx, int N, int K, const uint8_t* weight_int4, const float* scale,
                               const float* offset)
        : weight_cols(N), weight_rows(K), context_(ctx) {
        a81w41_linear* raw = nullptr;
        check(a81w41_linear_create(ctx->handle, N, K, weight_int4, scale, offset, &raw), "a81w41_linear_create");
        adopt(raw);
    }

    // activation: (batch, M, K) with batch == 1 as everywhere in the reference; returns (batch, M, N).
    Matrix3D<float> forward(const Matrix3D<float>& activation) {
        if (!layer_) throw std::runtime_error("Qwen_Linear_with_bias_Int4::forward on an empty layer");
        if (activation.m_dim_z != weight_rows)
            throw std::runtime_error("Qwen_Linear_with_bias_Int4::forward: activation has the wrong inner dimension");
        const int bs = activation.m_dim_x, m = activation.m_dim_y;
        Matrix3D<float> output(bs, m, weight_cols);
        // batch entries are independent rows for the linear layer: (bs*m) x K; the M-dispatch
        // follows m like QwenOperator.cc:96 (bs is 1 in every caller)
        for (int b = 0; b < bs; b++)
            check(a81w41_linear_forward_host(layer_.get(), activation.data() + (size_t)b * m * weight_rows, m,
                                             output.data() + (size_t)b * m * weight_cols),
                  "a81w41_linear_forward_host");
        return output;
    }

    int in_features() const { return weight_rows; }
    int out_features() const { return weight_cols; }
    a81w41_linear* handle() const { return layer_.get(); }
};

}  // namespace a81w41
