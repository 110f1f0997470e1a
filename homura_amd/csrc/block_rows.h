// Row kernels of decoders with a norm ahead of and behind every sublayer.
#pragma once
#include <cstdint>

#include "hm_common.h"

namespace homura {

// Per row: r = x + y, or x + RMSNorm(y) * y_w with y_w; then the row that leaves is r, or RMSNorm(r) * w with w.
// Both norms take their means over the first norm_dim of dim elements (padded rows hold zeros behind them).
struct RowNormArgs {
    const float *x = nullptr;      // [rows][dim] or NULL (r = y)
    const float *y = nullptr;      // [rows][dim] as y_parts K slices y_stride floats apart, or NULL (r = x)
    int y_parts = 1;
    size_t y_stride = 0;
    const float *y_w = nullptr;    // [dim]
    float *r_out = nullptr;        // [rows][dim]: r, may be x
    const float *w = nullptr;      // [dim]
    float *out = nullptr;          // [rows][dim] f32
    uint16_t *out_split = nullptr; // [rows][pieces * split_ld], split_ld = dim or, with cat, 2 dim
    int pieces = 3;
    const float *cat = nullptr;    // [rows][dim]: follows the row in the split matrix (columns dim .. 2 dim - 1)
    int rows = 0, dim = 0, norm_dim = 0;  // dim % 4 == 0, dim <= 8192
    float eps = 0.f;
};
int row_norm_launch(hm_ctx *ctx, const RowNormArgs &a);

// out[rows][n_out] = the first n_out columns of a projection given as K slices. With d_split its first split_cols
// columns also leave as a three-piece split matrix [rows][3 * split_cols]. n_out % 4 == 0, split_cols % 4 == 0.
int sum_parts_launch(hm_ctx *ctx, const float *d_x, int ld, int parts, size_t stride, float *d_out, int rows, int n_out,
                     uint16_t *d_split = nullptr, int split_cols = 0);

// Sinusoidal positions added to an embedding: element 2i of position p is sin(p freq[i]), element 2i + 1 the cosine, for
// the first `width` elements. Angles are f64 until they are reduced.
struct PositionWaves {
    const double *freq = nullptr;  // [(width + 1) / 2], NULL: none
    int width = 0;
};
// out[i] = scale * table[id_i] (+ waves of position past + i), ids int32 on the device (checked by the caller)
int embed_scaled_launch(hm_ctx *ctx, const int32_t *d_ids, const float *d_table, float *d_out, int n_ids, int vocab,
                        int hidden, float scale, PositionWaves waves = PositionWaves(), int past = 0);
// The decode step's row (this step's forced id or the last pick), written to d_out and, if given, d_out2.
int embed_step_scaled_launch(hm_ctx *ctx, const DecodeState *state, const int32_t *d_forced, const float *d_table,
                             float *d_out, float *d_out2, int vocab, int hidden, float scale, PositionWaves waves = PositionWaves());

}  // namespace homura
