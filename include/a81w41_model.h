/*
 * a81w41_model.h -- decoder models behind one C interface: load by config.json, feed tokens, read logits,
 * generate.  The architecture name in config.json picks the model class; liba81w41_dense.so holds the models with
 * bfloat16 weights, liba81w41.so the Qwen3 model on A81W41 layers; both register with liba81w41_core.so, which
 * exports the functions below.
 *
 * A model serves one sequence at a time.  Tokens may come in portions of any size: a call runs only the tokens it
 * brings, on top of what the cache holds.  Every function returns an a81w41_status; a81w41_last_error() has the text.
 */
#ifndef A81W41_MODEL_H
#define A81W41_MODEL_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef struct a81w41_model a81w41_model;

/* dir holds config.json and the weights.  dtype: "bfloat16" = the precision the model is served in, "float32" = all of
 * it in true 32-bit (A81W41_ERR_UNSUPPORTED if the model has no such path).  max_seq: the longest sequence. */
int a81w41_model_load(const char *dir, const char *dtype, int max_seq, a81w41_model **out);
/* The configuration alone (JSON text) with seeded random weights of its shapes: for benchmarks. */
int a81w41_model_create_random(const char *config_json, const char *dtype, int max_seq, uint64_t seed, a81w41_model **out);
void a81w41_model_destroy(a81w41_model *model);

int a81w41_model_vocab(const a81w41_model *model);
int a81w41_model_max_seq(const a81w41_model *model);
int a81w41_model_position(const a81w41_model *model); /* tokens in the cache */

/* Give back what the sequence holds in the cache: the next token is at position 0. */
int a81w41_model_reset(a81w41_model *model);
/* n_tokens new tokens (host) on top of the cached ones.  logits_host [n_want][vocab] receives the logits at the
 * places want[0..n_want) among them, which must rise; n_want may be 0.  Synchronises. */
int a81w41_model_forward(a81w41_model *model, const int *token_ids, int n_tokens, const int *want, int n_want,
                         float *logits_host);
/* Prefill the prompt, then n_new greedy tokens (first maximum), the decode step replayed from a captured HIP graph. */
int a81w41_model_generate_greedy(a81w41_model *model, const int *prompt, int n_prompt, int n_new, int *out_tokens,
                                 double *prefill_ms, double *decode_ms);

/* Test switches and parity hooks by name; which ones exist is the model's affair. */
int a81w41_model_set_option(a81w41_model *model, const char *name, int value);
int a81w41_model_read_buffer(a81w41_model *model, const char *name, float *host_out, size_t count);
/* Device bytes of the weights and of the cache. */
size_t a81w41_model_resident_bytes(const a81w41_model *model, size_t *weights, size_t *cache);

#ifdef __cplusplus
}
#endif
#endif /* A81W41_MODEL_H */
