// The session shared by all decoder models (portions, wanted logits, greedy generation from a captured graph), the
// model registry, and the C interface of include/a81w41_model.h.
#include "decoder_session.h"

#include <algorithm>
#include <cstdio>
#include <cstring>
#include <fstream>
#include <map>
#include <memory>
#include <sstream>

#include "json.h"

namespace a81w41 {

CachePlanes::~CachePlanes() {
    for (void* p : planes_) (void)hipFree(p);
}

int CachePlanes::add(size_t bytes, void** plane) {
    *plane = nullptr;
    void* p = nullptr;
    A81W41_HIP_TRY(hipMalloc(&p, bytes));
    planes_.push_back(p);
    bytes_ += bytes;
    A81W41_HIP_TRY(hipMemset(p, 0, bytes));
    *plane = p;
    return 0;
}

int CachePlanes::add_state(size_t bytes, void** state) {
    A81W41_TRY(add(bytes, state));
    states_.emplace_back(*state, bytes);
    return 0;
}

int CachePlanes::clear_states() {
    for (const auto& st : states_) A81W41_HIP_TRY(hipMemset(st.first, 0, st.second));
    return 0;
}

int DecoderSession::init_session(int max_seq, int vocab, int max_rows) {
    max_seq_ = max_seq;
    vocab_ = vocab;
    max_rows_ = max_rows;
    history_len = std::max(8192, max_seq);
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&ids), (size_t)max_rows * sizeof(int)));
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&want_dev), (size_t)max_rows * sizeof(int)));
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&pos), sizeof(int)));
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&step), sizeof(int)));
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&history), (size_t)history_len * sizeof(int)));
    A81W41_HIP_TRY(hipMemset(ids, 0, (size_t)max_rows * sizeof(int)));
    A81W41_HIP_TRY(hipMemset(pos, 0, sizeof(int)));
    A81W41_HIP_TRY(hipMemset(step, 0, sizeof(int)));
    A81W41_TRY(reserve_logits(1));
    A81W41_HIP_TRY(hipStreamCreate(&stream));
    return 0;
}

DecoderSession::~DecoderSession() {
    if (stream) (void)hipStreamSynchronize(stream);
    void* bufs[] = {ids, want_dev, pos, step, history, logits};
    for (void* b : bufs) (void)hipFree(b);
    if (stream) (void)hipStreamDestroy(stream);
}

int DecoderSession::reserve_logits(int rows) {
    if (rows <= logits_rows) return 0;
    if (stream) A81W41_HIP_TRY(hipStreamSynchronize(stream));
    (void)hipFree(logits);
    logits = nullptr;
    logits_rows = 0;
    A81W41_HIP_TRY(hipMalloc(reinterpret_cast<void**>(&logits), (size_t)rows * vocab_ * sizeof(float)));
    logits_rows = rows;
    return 0;
}

int DecoderSession::reset() {
    A81W41_HIP_TRY(hipStreamSynchronize(stream));
    A81W41_HIP_TRY(hipMemset(pos, 0, sizeof(int)));
    A81W41_HIP_TRY(hipMemset(step, 0, sizeof(int)));
    A81W41_TRY(cache.clear_states());
    host_pos = 0;
    return 0;
}

// The ids and wanted rows of a pass of at most max_rows_ tokens.
int DecoderSession::upload(const int* token_ids, int n, const int* want, int n_want) {
    A81W41_HIP_TRY(hipMemcpy(ids, token_ids, (size_t)n * sizeof(int), hipMemcpyHostToDevice));
    if (n_want) A81W41_HIP_TRY(hipMemcpy(want_dev, want, (size_t)n_want * sizeof(int), hipMemcpyHostToDevice));
    return 0;
}

int DecoderSession::forward(const int* token_ids, int n, const int* want, int n_want, float* logits_host) {
    if (!token_ids || n_want < 0 || (n_want && !want)) return failf(A81W41_ERR_INVALID_ARG, "null argument");
    A81W41_TRY(ready());
    if (n < 1 || n > max_seq_ - host_pos)
        return failf(A81W41_ERR_INVALID_ARG, "%d tokens on top of %d do not fit max_seq %d", n, host_pos, max_seq_);
    for (int i = 0; i < n_want; i++)
        if (want[i] < (i ? want[i - 1] + 1 : 0) || want[i] >= n)
            return failf(A81W41_ERR_INVALID_ARG, "the wanted places must rise and lie among the tokens");
    std::vector<int> local;
    int w0 = 0;
    for (int at = 0; at < n; at += max_rows_) {
        const int m = std::min(max_rows_, n - at);
        local.clear();
        while (w0 + (int)local.size() < n_want && want[w0 + local.size()] < at + m) local.push_back(want[w0 + local.size()] - at);
        const int nw = (int)local.size();
        A81W41_TRY(reserve_logits(std::max(nw, 1)));
        plan_ctx = host_pos + m;
        A81W41_TRY(upload(token_ids + at, m, local.data(), nw));
        A81W41_TRY(enqueue_pass(m, local.data(), nw, stream));
        A81W41_HIP_TRY(hipStreamSynchronize(stream));
        host_pos += m;
        A81W41_TRY(check_passes());
        if (logits_host && nw)
            A81W41_HIP_TRY(hipMemcpy(logits_host + (size_t)w0 * vocab_, logits, (size_t)nw * vocab_ * sizeof(float), hipMemcpyDeviceToHost));
        w0 += nw;
    }
    return 0;
}

int DecoderSession::generate_greedy(const int* prompt, int n_prompt, int n_new, int* out_tokens, double* prefill_ms,
                                    double* decode_ms) {
    if (!prompt || !out_tokens) return failf(A81W41_ERR_INVALID_ARG, "null argument");
    A81W41_TRY(ready());
    if (n_prompt < 1 || n_new < 1 || n_new > history_len || (long long)host_pos + n_prompt + n_new - 1 > max_seq_)
        return failf(A81W41_ERR_INVALID_ARG, "prompt of %d and %d new tokens on top of %d do not fit max_seq %d", n_prompt, n_new,
                     host_pos, max_seq_);
    hipStream_t s = stream;
    // events and graph objects are released on every way out of this function
    struct Scoped {
        hipEvent_t ev[4] = {nullptr, nullptr, nullptr, nullptr};
        hipGraph_t graph = nullptr;
        hipGraphExec_t exec = nullptr;
        ~Scoped() {
            for (hipEvent_t e : ev)
                if (e) (void)hipEventDestroy(e);
            if (exec) (void)hipGraphExecDestroy(exec);
            if (graph) (void)hipGraphDestroy(graph);
        }
    } own;
    for (hipEvent_t& e : own.ev) A81W41_HIP_TRY(hipEventCreate(&e));
    const hipEvent_t e0 = own.ev[0], e1 = own.ev[1], e2 = own.ev[2], e3 = own.ev[3];
    const int last_row = (n_prompt - 1) % max_rows_;  // of the prompt's last portion
    A81W41_TRY(upload(prompt, std::min(n_prompt, max_rows_), &last_row, 1));
    A81W41_HIP_TRY(hipMemset(step, 0, sizeof(int)));
    A81W41_HIP_TRY(hipEventRecord(e0, s));
    const int last_ctx = host_pos + n_prompt + n_new - 1;  // also what the decode steps captured below will reach
    for (int at = 0; at < n_prompt; at += max_rows_) {
        const int m = std::min(max_rows_, n_prompt - at);
        plan_ctx = m == 1 ? last_ctx : host_pos + at + m;
        if (at) A81W41_TRY(upload(prompt + at, m, nullptr, 0));
        A81W41_TRY(enqueue_pass(m, &last_row, at + m == n_prompt ? 1 : 0, s));
    }
    // first new token: argmax of the prompt's logits; it becomes the next pass's input id
    A81W41_HIP_TRY(launch_argmax_token(logits, vocab_, ids, history, history_len, step, s));
    A81W41_HIP_TRY(hipEventRecord(e1, s));
    A81W41_HIP_TRY(hipStreamSynchronize(s));
    host_pos += n_prompt;

    const int n_steps = n_new - 1;
    if (n_steps > 0) {
        plan_ctx = last_ctx;
        const int row0 = 0;
        // one decode step = a pass over the single id in ids[0] + argmax; captured once, replayed
        bool captured = false;
        if (hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal) == hipSuccess) {
            int st = enqueue_pass(1, &row0, 1, s);
            if (st == 0 && launch_argmax_token(logits, vocab_, ids, history, history_len, step, s) != hipSuccess) st = 1;
            const hipError_t ee = hipStreamEndCapture(s, &own.graph);
            if (st == 0 && ee == hipSuccess && own.graph && hipGraphInstantiate(&own.exec, own.graph, nullptr, nullptr, 0) == hipSuccess)
                captured = true;
        }
        (void)hipGetLastError();
        A81W41_HIP_TRY(hipEventRecord(e3, s));
        for (int i = 0; i < n_steps; i++) {
            if (captured) {
                A81W41_HIP_TRY(hipGraphLaunch(own.exec, s));
            } else {
                A81W41_TRY(enqueue_pass(1, &row0, 1, s));
                A81W41_HIP_TRY(launch_argmax_token(logits, vocab_, ids, history, history_len, step, s));
            }
        }
        A81W41_HIP_TRY(hipEventRecord(e2, s));
        A81W41_HIP_TRY(hipStreamSynchronize(s));
        host_pos += n_steps;
    } else {
        A81W41_HIP_TRY(hipEventRecord(e2, s));
        A81W41_HIP_TRY(hipStreamSynchronize(s));
    }
    float ms01 = 0.f, ms12 = 0.f;
    A81W41_HIP_TRY(hipEventElapsedTime(&ms01, e0, e1));
    if (n_steps > 0) A81W41_HIP_TRY(hipEventElapsedTime(&ms12, e3, e2));
    if (prefill_ms) *prefill_ms = ms01;
    if (decode_ms) *decode_ms = ms12;
    A81W41_TRY(check_passes());
    A81W41_HIP_TRY(hipMemcpy(out_tokens, history, (size_t)n_new * sizeof(int), hipMemcpyDeviceToHost));
    return 0;
}

int DecoderSession::set_option(const char* name, int) { return failf(A81W41_ERR_INVALID_ARG, "no option '%s'", name); }
int DecoderSession::read_buffer(const char* name, float*, size_t) { return failf(A81W41_ERR_INVALID_ARG, "no buffer '%s'", name); }

// ---- registry ------------------------------------------------------------------------------
namespace {
std::map<std::string, ModelFactory>& factories() {
    static std::map<std::string, ModelFactory> table;
    return table;
}
int create(const std::string& text, LoadRequest req, a81w41_model** out) {
    try {
        const Json config = Json::parse(text);
        req.config = &config;
        const std::string name = config.at("architecture").string();
        const auto it = factories().find(name);
        if (it == factories().end()) return failf(A81W41_ERR_UNSUPPORTED, "no model class for architecture '%s' is loaded", name.c_str());
        if (req.dtype != "bfloat16" && req.dtype != "float32") return failf(A81W41_ERR_INVALID_ARG, "dtype must be bfloat16 or float32");
        if (req.max_seq < 1) return failf(A81W41_ERR_INVALID_ARG, "max_seq must be at least 1");
        return it->second(req, out);
    } catch (const std::bad_alloc&) {
        return failf(A81W41_ERR_HIP, "out of host memory");
    } catch (const std::exception& e) {
        return failf(A81W41_ERR_INVALID_ARG, "config.json: %s", e.what());
    }
}
}  // namespace

RegisterModel::RegisterModel(const char* architecture, ModelFactory factory) { factories()[architecture] = factory; }

}  // namespace a81w41

extern "C" {

int a81w41_model_load(const char* dir, const char* dtype, int max_seq, a81w41_model** out) {
    if (!dir || !dtype || !out) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null argument");
    *out = nullptr;
    std::ifstream f(std::string(dir) + "/config.json", std::ios::binary);
    if (!f) return a81w41::failf(A81W41_ERR_IO, "cannot open %s/config.json", dir);
    std::stringstream text;
    text << f.rdbuf();
    a81w41::LoadRequest req;
    req.dir = dir;
    req.dtype = dtype;
    req.max_seq = max_seq;
    return a81w41::create(text.str(), req, out);
}

int a81w41_model_create_random(const char* config_json, const char* dtype, int max_seq, uint64_t seed, a81w41_model** out) {
    if (!config_json || !dtype || !out) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null argument");
    *out = nullptr;
    a81w41::LoadRequest req;
    req.dtype = dtype;
    req.max_seq = max_seq;
    req.random_weights = true;
    req.seed = seed;
    return a81w41::create(config_json, req, out);
}

void a81w41_model_destroy(a81w41_model* model) { delete model; }
int a81w41_model_vocab(const a81w41_model* m) { return m ? m->vocab() : 0; }
int a81w41_model_max_seq(const a81w41_model* m) { return m ? m->max_seq() : 0; }
int a81w41_model_position(const a81w41_model* m) { return m ? m->position() : 0; }

int a81w41_model_reset(a81w41_model* m) { return m ? m->reset() : a81w41::failf(A81W41_ERR_INVALID_ARG, "null model"); }

int a81w41_model_forward(a81w41_model* m, const int* token_ids, int n_tokens, const int* want, int n_want, float* logits_host) {
    if (!m) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null model");
    return m->forward(token_ids, n_tokens, want, n_want, logits_host);
}

int a81w41_model_generate_greedy(a81w41_model* m, const int* prompt, int n_prompt, int n_new, int* out_tokens, double* prefill_ms,
                                 double* decode_ms) {
    if (!m) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null model");
    return m->generate_greedy(prompt, n_prompt, n_new, out_tokens, prefill_ms, decode_ms);
}

int a81w41_model_set_option(a81w41_model* m, const char* name, int value) {
    if (!m || !name) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null argument");
    return m->set_option(name, value);
}

int a81w41_model_read_buffer(a81w41_model* m, const char* name, float* host_out, size_t count) {
    if (!m || !name || !host_out) return a81w41::failf(A81W41_ERR_INVALID_ARG, "null argument");
    return m->read_buffer(name, host_out, count);
}

size_t a81w41_model_resident_bytes(const a81w41_model* m, size_t* weights, size_t* cache) {
    if (!m) return 0;
    if (weights) *weights = m->weight_bytes();
    if (cache) *cache = m->cache_bytes();
    return m->weight_bytes() + m->cache_bytes();
}

}  // extern "C"
