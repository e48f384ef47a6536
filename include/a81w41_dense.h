/*
 * a81w41_dense.h -- parity hooks of liba81w41_dense.so: the mechanisms of the models with dense weights on their own.
 * Device pointers, enqueued on `stream`; element type bf16 != 0: bfloat16, else float.  For tests and measurements.
 */
#ifndef A81W41_DENSE_H
#define A81W41_DENSE_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

/* C = A W^T: A [M][lda], W [N][ldw] elements, C [M][ldc] floats.  lda, ldw: at least K rounded up to 128 bytes, whole
 * multiples of 128 bytes; the columns of W beyond K are zero, those of A finite. */
int a81w41_dense_gemm(const void *A, int lda, const void *W, int ldw, float *C, int ldc, int M, int N, int K, int bf16, void *stream);
/* Attention in latent space.  q [M heads][ld], cache [max_seq][ld] with rows [latent (rank) | rotated part (rot)] and zeros
 * up to ld (a multiple of 128 bytes); token m sees cache rows 0 .. pos + m.  out [M heads][rank] elements.
 * variant 0: the vector kernel; 1: matrix cores (bfloat16 only), the keys dealt to `splits` (1 .. 64) workgroups, with
 * part [splits M heads][rank rounded up to 4] and stats [splits M heads][2] floats as scratch. */
int a81w41_latent_attention(const void *q, const void *cache, int ld, int rank, int rot, int heads, const int *pos_dev, int max_seq, int M,
                            float scale, void *out, int bf16, int variant, int splits, float *part, float *stats, void *stream);
/* Attention on formed keys and values, bfloat16.  q [M][heads][dim + rot], k [max_seq][heads dim] and k_rot
 * [max_seq][ld_rot] (first rot columns), v_t [heads vdim][ld_v] transposed with ld_v a multiple of 64, at least max_seq;
 * gates [M][heads] floats (before the sigmoid), out [M][heads vdim].  dim, rot, ld_rot: multiples of 8. */
int a81w41_formed_attention(const void *q, const void *k, const void *k_rot, int ld_rot, const void *v_t, int ld_v, const float *gates,
                            int heads, int dim, int rot, int vdim, const int *pos_dev, int max_seq, int M, float scale, void *out,
                            void *stream);
/* Grouped attention.  q [M][heads][key_width], cache rows [max_seq][ld] with [value (value_width) | key (key_width)] for each of
 * kv_heads; query head h reads kv head h / (heads / kv_heads).  Token m sees the rows 0 .. pos + m, with chunk > 0 those from
 * the first position of its own chunk on; sink: a further key of score 0 without a value.  Widths are multiples of 8, the
 * first vdim value columns count; out [M][heads][vdim] elements.  variant, splits, part, stats: as above, with
 * splits M heads rows of scratch, vdim rounded up to 4. */
int a81w41_grouped_attention(const void *q, const void *rows, int ld, int heads, int kv_heads, int key_width, int value_width, int vdim,
                             const int *pos_dev, int max_seq, int M, float scale, int chunk, int sink, void *out, int bf16, int variant,
                             int splits, float *part, float *stats, void *stream);
/* A matrix memory over M tokens at positions *pos_dev .. of a sequence.  in [M][ld_in] floats, columns [q | k | v | output gate |
 * input gate | forget gate] of all heads; q is scaled by dim^-1/2 here.  state: a81w41_matrix_memory_state() floats, zero at
 * position 0; scratch: a81w41_matrix_memory_scratch() floats; all 16-byte aligned.  out [M][heads vdim]: per head divided by its
 * root mean square, times norm, times the sigmoid of the output gate.  variant 0: token by token; 1: in chunks. */
size_t a81w41_matrix_memory_state(int heads, int dim, int vdim);
size_t a81w41_matrix_memory_scratch(int heads, int dim, int vdim, int M);
int a81w41_matrix_memory(const float *in, int ld_in, int M, int heads, int dim, int vdim, float cap, float eps, const float *bias_i,
                         const float *bias_f, const float *norm, float *state, const int *pos_dev, int variant, float *scratch, float *out,
                         void *stream);
/* chosen [M][top]: the largest of logits [M][ld] (first `experts` columns) + bias, largest first; weights [M][top]: the softmax
 * over them. */
int a81w41_router(const float *logits, int ld, const float *bias, int experts, int top, int M, int *chosen, float *weights, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* A81W41_DENSE_H */
