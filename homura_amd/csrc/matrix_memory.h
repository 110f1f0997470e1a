// Matrix memory with exponential gates (the mLSTM of xLSTM): per head a memory C (dim x vdim) and a normaliser z (dim),
//
//   C <- e^f C + e^i k v^T,   z <- e^f z + e^i k,   o = C^T q / max(|z . q|, 1)
//
// with log gates i = cap tanh((. + b) / cap), f = logsigmoid(cap tanh((. + b) / cap)). Both are kept divided by e^m, m the
// running maximum of the log weights, which starts at 0: m' = max(f + m, i), and o = C^T q / (max(|z . q|, e^-m) + 1e-6).
// Every head's o is then divided by its root mean square, weighted and gated by a sigmoid.
//
// The normaliser is one more column of the memory, whose value is 1. State of a layer, f32: per head
// [tiles][dim_pad][16] (tiles of 16 columns over vdim + 1, zero behind the true sizes), then m of every head, twice: the
// one ahead of position p in half p % 2, so that no launch reads what it writes.
//
// A prompt goes through in chunks of 64 tokens. With F the running sum of f inside a chunk, a_s = i_s - F_s and
// M_t = max(m, a_0 .. a_t): the weight of token s in row t is e^(a_s - M_t), that of the memory ahead of the chunk e^(m - M_t),
// and m_t = F_t + M_t. The sums are f64, the weights f32.
#pragma once
#include <cstdint>

#include "hm_common.h"
#include "row_source.h"

namespace homura {

constexpr int MM_MAX_DIM = 1024;
constexpr int MM_CHUNK = 64;
constexpr int MM_MAX_ROWS = 2048;  // of a prompt launch

struct MatrixMemoryShape {
    int heads = 0, dim = 0, vdim = 0;
    int dim_pad = 0;                 // matrix_memory_dim_pad(dim)
    float cap = 1.f;
    __host__ __device__ int tiles() const { return (vdim + 1 + 15) / 16; }
    __host__ __device__ int cols() const { return tiles() * 16; }
    __host__ __device__ size_t memory_floats() const { return (size_t)heads * tiles() * dim_pad * 16; }
    size_t state_floats() const { return memory_floats() + 2 * (size_t)heads; }
};
int matrix_memory_dim_pad(int dim);

// Columns of the input projection: q, k, v, output gate, log gates.
struct MatrixMemoryColumns { int q = 0, k = 0, v = 0, g = 0, i = 0, f = 0; };

// ── decode step ──
struct MatrixMemoryStepArgs {
    MatrixMemoryShape s;
    MatrixMemoryColumns at;
    const float *row = nullptr;               // the projection row
    const float *i_bias = nullptr, *f_bias = nullptr;
    float *state = nullptr;
    float *raw = nullptr;                     // [heads][cols]: C^T q, and z . q in column vdim
    const float *norm = nullptr;              // [heads * vdim]
    float eps = 0.f;
    float *out = nullptr;                     // [heads * vdim]
    const DecodeState *cursor = nullptr;
};
int matrix_memory_step_launch(hm_ctx *ctx, const MatrixMemoryStepArgs &a);
int matrix_memory_step_out_launch(hm_ctx *ctx, const MatrixMemoryStepArgs &a);

// ── prompt pass, n rows at positions past .. past + n - 1 ──
struct MatrixMemoryRowsArgs {
    MatrixMemoryShape s;
    MatrixMemoryColumns at;
    const float *rows = nullptr;              // projection rows as parts K slices
    int ld = 0, parts = 1;
    size_t stride = 0;
    const float *x = nullptr;                 // [n][x_ld]: what the projection took, for the gates, which keep all its bits
    int x_ld = 0;                             // % 32 == 0
    const uint16_t *gate_w = nullptr;         // [2 * heads][x_ld] bf16: input gates, forget gates
    float *gates = nullptr;                   // [n][2 * heads]
    const float *i_bias = nullptr, *f_bias = nullptr;
    int pieces = 1;                           // of q, k and v inside a chunk: 1 or 3
    uint16_t *q = nullptr, *k = nullptr;      // [pieces][heads][n][dim_pad]
    double *log_w = nullptr;                  // [2][heads][chunks * 64]: a, M, in units of ln 2
    float *weights = nullptr;                 // [3][heads][chunks * 64]: e^(m - M), e^(a - M of the chunk's end), e^-m_t
    float *decay = nullptr;                   // [heads][chunks]: e^(m - M of the chunk's end)
    uint16_t *values = nullptr;               // matrix_memory_value_bytes: the values as operands
    uint16_t *ahead = nullptr;                // matrix_memory_ahead_bytes: the memory ahead of every chunk
    float *state = nullptr;
    float *raw = nullptr;                     // [n][heads * cols]
    const float *norm = nullptr;
    float eps = 0.f;
    uint16_t *out_split = nullptr;            // [n][out_pieces * out_cols]
    int out_pieces = 3, out_cols = 0;
    int n = 0, past = 0;
    int chunks() const { return (n + MM_CHUNK - 1) / MM_CHUNK; }
};
// whether heads of this width go through in chunks on the matrix cores (token by token otherwise)
bool matrix_memory_tiled(const MatrixMemoryShape &s, int pieces);
size_t matrix_memory_value_bytes(const MatrixMemoryShape &s, int pieces, int rows);
size_t matrix_memory_ahead_bytes(const MatrixMemoryShape &s, int pieces, int rows);
// q, k and v as the scan takes them; gates and log weights of every token; the scan; norm and output gate behind it
int matrix_memory_rows_launch(hm_ctx *ctx, const MatrixMemoryRowsArgs &a);

}  // namespace homura
