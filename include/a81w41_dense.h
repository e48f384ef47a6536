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

#ifdef __cplusplus
}
#endif
#endif /* A81W41_DENSE_H */
