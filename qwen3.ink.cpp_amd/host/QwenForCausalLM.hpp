// Host-side mirror of the reference's model-level interface on top of the C ABI
// (include/a81w41.h, a81w41_qwen3_*).  A caller written against
//   qwen3_config                     qwen3/include/qwen/QwenConfig.h:22-62
//   Qwen3ForCausalLM_Input/_Output   qwen3/include/qwen/QwenForCausalLM.h:10-24
//   Qwen3ForCausalLM                 qwen3/include/qwen/QwenForCausalLM.h:26-45, src/qwen/QwenForCausalLM.cc:11-121
// keeps its generate loop (Pipeline.cc:402-413): construct from the weight directory,
// call forward() with the new token ids, read logits(0, 0, v) of the last token.  The
// model keeps its own position, like the reference's past_sqlen member.
//
// Header only; link with -la81w41 -la81w41_core.  Failures throw std::runtime_error.
#pragma once

#include <string>

#include "QwenLinearInt4.hpp"

namespace a81w41 {

struct qwen3_config {
    int batchsize, max_sqlen;
    int num_layers = 36, num_q_head = 32, num_kv_head = 8, num_key_value_heads = 8;
    int hidden_dim = 4096, head_dim = 128, mlp_dim = 12288, vocsize = 151936, qk = 32;
    int bos_token_id = 151643, eos_token_id = 151645, pad_token_id = 151643, im_start_id = 151644, im_end_id = 151645;
    float rope_theta = 1e6f, rms_eps = 1e-6f;
    qwen3_config() = delete;
    qwen3_config(int batch, int max_sqlen_) : batchsize(batch), max_sqlen(max_sqlen_) {}
};

struct Qwen3ForCausalLM_Input {
    Matrix3D<int>* input_ids;  // (1, 1, sqlen)
    explicit Qwen3ForCausalLM_Input(Matrix3D<int>* input_ids_) : input_ids(input_ids_) {}
};

struct Qwen3ForCausalLM_Output {
    Matrix3D<float> logits;  // (1, 1, vocsize): the last token's
    explicit Qwen3ForCausalLM_Output(Matrix3D<float>&& l) : logits(std::move(l)) {}
    Qwen3ForCausalLM_Output(const Qwen3ForCausalLM_Output&) = delete;
    Qwen3ForCausalLM_Output& operator=(const Qwen3ForCausalLM_Output&) = delete;
    Qwen3ForCausalLM_Output(Qwen3ForCausalLM_Output&&) = default;
};

class Qwen3ForCausalLM {
    std::shared_ptr<a81w41_qwen3> model_;
    int vocsize_ = 0;

   public:
    Qwen3ForCausalLM() = default;
    Qwen3ForCausalLM(std::string param_path, const qwen3_config config) : vocsize_(config.vocsize) {
        if (config.batchsize != 1 || config.head_dim != 128)
            throw std::runtime_error("Qwen3ForCausalLM: batch size 1 and head_dim 128 only");
        a81w41_qwen3_config c{config.num_layers, config.hidden_dim, config.num_q_head, config.num_kv_head, config.mlp_dim,
                              config.vocsize,    config.max_sqlen,  config.rope_theta, config.rms_eps};
        a81w41_qwen3* raw = nullptr;
        check(a81w41_qwen3_load(param_path.c_str(), &c, &raw), "a81w41_qwen3_load");
        model_ = std::shared_ptr<a81w41_qwen3>(raw, a81w41_qwen3_destroy);
    }

    Qwen3ForCausalLM_Output forward(const Qwen3ForCausalLM_Input& input) {
        if (!model_ || !input.input_ids) throw std::runtime_error("Qwen3ForCausalLM::forward on an empty model or input");
        Matrix3D<float> logits(1, 1, vocsize_);
        check(a81w41_qwen3_forward(model_.get(), input.input_ids->data(), input.input_ids->m_dim_z, logits.data()),
              "a81w41_qwen3_forward");
        return Qwen3ForCausalLM_Output(std::move(logits));
    }

    // Forget the context (the reference builds a new model per conversation).
    void reset() { check(a81w41_qwen3_reset(model_.get()), "a81w41_qwen3_reset"); }
    a81w41_qwen3* handle() const { return model_.get(); }
};

}  // namespace a81w41
