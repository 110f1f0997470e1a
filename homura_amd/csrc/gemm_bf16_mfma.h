// Internal launch interface of the MFMA GEMM used by the prefill path.
#pragma once

#include <cstdint>

#include "gated_act.h"
#include "grouped_tiles.h"
#include "hm_common.h"

namespace homura {

// C[M][N] f32 = (sum of the pieces of A)[M][K] x B[N][K]^T. d_a_split is [M][pieces * K] bf16: piece p
// of every f32 activation in columns [p K, (p+1) K) (what the kernels of prefill.hip write). B is the
// K-contiguous stream layout of the model weights. K % 32 == 0, pieces 1..3.
// With parts != NULL the product may be cut along K into up to max_parts slices when M x N alone
// leaves most of the chip idle: slice s lands in d_c + s * M * N, *parts says how many there are, and
// the caller adds them up in index order (d_c must hold max_parts * M * N floats).
int gemm_split_nk(hm_ctx *ctx, const uint16_t *d_a_split, int pieces, const uint16_t *d_b_nk, float *d_c, int M, int K,
                  int N, int max_parts = 1, int *parts = nullptr);

// The same sum of piece products against B in the reference's layout [K][N] (N contiguous; N % 8 == 0, K % 32 == 0).
int gemm_split_kn(hm_ctx *ctx, const uint16_t *d_a_split, int pieces, const uint16_t *d_b_kn, float *d_c, int M, int K,
                  int N);

// C = A x B^T for two f32 matrices, each given as three bf16 pieces per element: d_a_split [M][3 K],
// d_b_split [N][3 K] (piece p in columns [p K, (p+1) K)). The six products of an A piece and a B piece
// whose indices add up to at most 2 are accumulated; what is left out is below 2^-24 of the result.
// K % 64 == 0. Row r of C starts at d_c + r * ldc (ldc = 0: N); slices as in gemm_split_nk, slice s at
// d_c + s * M * ldc.
int gemm_split_split_nk(hm_ctx *ctx, const uint16_t *d_a_split, const uint16_t *d_b_split, float *d_c, int M, int K,
                        int N, int max_parts = 1, int *parts = nullptr, int ldc = 0);

// The same products with every tile loaded once (gemm_pieces_mfma.hip): a_pieces x b_pieces = 2 x 1 or 3 x 1
// (d_b_split is then the plain [N][K] bf16 matrix) or 3 x 3. K % 32 == 0. Slices and ldc as above.
int gemm_pieces_nk(hm_ctx *ctx, const uint16_t *d_a_split, int a_pieces, const uint16_t *d_b_split, int b_pieces,
                   float *d_c, int M, int K, int N, int max_parts = 1, int *parts = nullptr, int ldc = 0);

// A batch of 3 x 1 products of one shape (block-diagonal matrices): problem z reads d_a_split + z * a_batch ([M][3 K])
// and d_b_nk + z * b_batch ([N][K]), writes row r at d_c + z * c_batch + r * ldc. K % 32 == 0.
int gemm_pieces_batched(hm_ctx *ctx, const uint16_t *d_a_split, size_t a_batch, const uint16_t *d_b_nk, size_t b_batch,
                        float *d_c, size_t c_batch, int batch, int M, int K, int N, int ldc);

// Products of one B [N][K] per group (a mixture of experts) over the rows that the groups' lists name: d_list
// [groups][list_cap] entries, d_count [groups], `entries` of them in all. Entry e reads row e % a_rows of the split matrix
// and writes row e of d_c [.][N]. 1 or 3 pieces; K % 32 == 0.
// With act (gemm_gated_fits): neighbouring columns are (gate, up) pairs, and act(w gate, w up) with the entry's weight w
// leaves as bf16, d_c being [.][N / 2] of them.
// (gemm_grouped_dma: the same for one piece and K % 64 == 0, behind gemm_grouped_nk's checks.)
inline bool gemm_gated_fits(int pieces, int K, int N) { return pieces == 1 && K % 64 == 0 && N % 4 == 0; }
int gemm_grouped_dma(hm_ctx *ctx, const uint16_t *d_a, const uint16_t *d_b_nk, float *d_c, const GroupLists &lists, unsigned tiles,
                     int K, int N, const GatedAct *act, const float *d_weight);
int gemm_grouped_nk(hm_ctx *ctx, const uint16_t *d_a_split, int pieces, int a_rows, const uint16_t *d_b_nk, float *d_c,
                    const int *d_list, const int *d_count, int groups, int list_cap, int entries, int K, int N,
                    const GatedAct *act = nullptr, const float *d_weight = nullptr);

// 3 x 1 pieces against a block-scaled integer matrix: d_b_ints [N][K] bf16 holds the integers of a Q8_0 / Q4_0
// matrix (exact), d_scales [K / 32][npad] f32 the scale of every 32-wide block of every row (npad >= N rounded
// up to 128). C = sum over blocks of scale * (A x ints^T over the block). Slices and ldc as above.
int gemm_pieces_scaled_nk(hm_ctx *ctx, const uint16_t *d_a_split, const uint16_t *d_b_ints, const float *d_scales, int npad,
                          float *d_c, int M, int K, int N, int max_parts = 1, int *parts = nullptr, int ldc = 0);
int gemm_pieces_any(hm_ctx *ctx, const uint16_t *d_a_split, int a_pieces, const uint16_t *d_b_split, int b_pieces,
                    const float *d_scales, int npad, float *d_c, int M, int K, int N, int max_parts, int *parts, int ldc);

}  // namespace homura
