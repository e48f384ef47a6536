// What every decoder model of this framework shares: one sequence on one GPU.  A session owns the token ids,
// the device position, the cache planes, the logits, the stream and the generation loop; a model derives from
// it and enqueues the kernels of one pass.  The model registry creates models by the architecture name of a
// checkpoint's config.json.
#pragma once
#include <hip/hip_runtime.h>

#include <cstdarg>
#include <cstddef>
#include <cstdint>
#include <string>
#include <utility>
#include <vector>

#include "../../include/a81w41.h"
#include "../../include/a81w41_model.h"

namespace a81w41 {

// Record the calling thread's last error and return `status`.
int report_failure(int status, const char* message);
int failf(int status, const char* fmt, ...) __attribute__((format(printf, 2, 3)));

#define A81W41_HIP_TRY(expr)                                                                                          \
    do {                                                                                                              \
        hipError_t _e = (expr);                                                                                       \
        if (_e != hipSuccess) return a81w41::failf(A81W41_ERR_HIP, "%s: %s", #expr, hipGetErrorString(_e));           \
    } while (0)
#define A81W41_TRY(expr)         \
    do {                         \
        int _st = (expr);        \
        if (_st) return _st;     \
    } while (0)

// ---- kernels of the loop (decoder_ops.hip) -------------------------------------------------
enum class TableType { kFp16, kBf16, kFp32 };
// out[m][0..hidden) = table[ids[m]][0..hidden) as fp32; table rows are ld elements apart; ids are clamped into the table.
hipError_t launch_embed_rows(const int* ids, const void* table, TableType type, int ld, float* out, int M, int hidden, int vocab,
                             hipStream_t s);
hipError_t launch_argmax_token(const float* logits, int n, int* next_id, int* history, int history_len, int* step_dev,
                               hipStream_t s);
hipError_t launch_advance(int* pos_dev, int by, hipStream_t s);

// What a sequence holds on the device, zero when allocated, freed with the object: cache planes of max_seq rows, which a new
// sequence overwrites, and recurrent states, which go back to zero when the sequence is given back.
class CachePlanes {
   public:
    CachePlanes() = default;
    CachePlanes(const CachePlanes&) = delete;
    CachePlanes& operator=(const CachePlanes&) = delete;
    ~CachePlanes();
    int add(size_t bytes, void** plane);
    int add_state(size_t bytes, void** state);
    int clear_states();
    size_t bytes() const { return bytes_; }

   private:
    std::vector<void*> planes_;
    std::vector<std::pair<void*, size_t>> states_;
    size_t bytes_ = 0;
};

class DecoderSession {
   public:
    virtual ~DecoderSession();

    int reset();
    // n new tokens on top of the cached context; logits of the rows want[0..n_want) (rising places among the n tokens) go
    // to logits_host [n_want][vocab] (may be null).  Cut into passes of at most max_rows tokens.  Synchronises.
    int forward(const int* token_ids, int n, const int* want, int n_want, float* logits_host);
    // The prompt, then n_new tokens by first maximum: the decode step is captured as a graph once and replayed.
    int generate_greedy(const int* prompt, int n_prompt, int n_new, int* out_tokens, double* prefill_ms, double* decode_ms);

    int max_seq() const { return max_seq_; }
    int vocab() const { return vocab_; }
    int position() const { return host_pos; }

    // Test and measurement hooks; a model without the option or buffer reports an error.
    virtual int set_option(const char* name, int value);
    virtual int read_buffer(const char* name, float* host_out, size_t count);
    virtual size_t weight_bytes() const { return 0; }
    size_t cache_bytes() const { return cache.bytes(); }

   protected:
    int init_session(int max_seq, int vocab, int max_rows);
    // Whether every weight is there.
    virtual int ready() const = 0;
    // Enqueue one pass over the M ids in `ids`: n_want rows of logits into `logits`, then the device position
    // advances by M.  want_dev holds the wanted rows on the device (a pass over one token may not read it: it can
    // be part of a captured graph).  Enqueues only.
    virtual int enqueue_pass(int M, const int* want, int n_want, hipStream_t s) = 0;
    // After a synchronisation: whether the passes so far really worked.
    virtual int check_passes() { return 0; }

   public:  // read by the models' C entry points
    int *ids = nullptr, *pos = nullptr, *step = nullptr, *history = nullptr, *want_dev = nullptr;
    float* logits = nullptr;
    int logits_rows = 0;
    int history_len = 0;
    int host_pos = 0;
    int plan_ctx = 0;  // longest context the passes being enqueued will see (picks an attention's key split)
    hipStream_t stream = nullptr;
    CachePlanes cache;

   private:
    int reserve_logits(int rows);
    int upload(const int* token_ids, int n, const int* want, int n_want);
    int max_seq_ = 0, vocab_ = 0, max_rows_ = 0;
};

}  // namespace a81w41

// The C handle is the session itself; models derive from it.
struct a81w41_model : a81w41::DecoderSession {};

namespace a81w41 {

// ---- registry ------------------------------------------------------------------------------
class Json;
struct LoadRequest {
    std::string dir;       // folder of config.json and the weights
    const Json* config = nullptr;
    std::string dtype;     // "bfloat16": what the model is served in; "float32"
    int max_seq = 0;
    bool random_weights = false;  // seeded weights of the configuration's shapes instead of the folder's
    uint64_t seed = 0;
};
using ModelFactory = int (*)(const LoadRequest&, a81w41_model** out);
struct RegisterModel {
    RegisterModel(const char* architecture, ModelFactory factory);
};

}  // namespace a81w41
