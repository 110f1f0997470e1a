// Latent attention: keys and values of all heads are linear images of one normed latent row per token, next to one
// rotated key part that all heads share. The cache keeps just these (a ring of the rows a sliding window needs).
//
// Cache row: `pieces` (1: bf16, 3: the three bf16 pieces of the f32 values) times [latent (rank_pad) | rotated key
// (rot_pad)], zero behind the true widths; row of position p in slot p % rows.
//
// A decode step attends over the latents themselves: the queries take the key matrix onto their side
// (q' = W_uk^T q per head), the result is a mix of latents per head, and the value matrix comes last. The prompt
// pass expands keys and values of the visible rows with one GEMM and hands them to the causal attention of
// prefill.h.
#pragma once
#include <cstdint>

#include "hm_common.h"
#include "row_source.h"

namespace homura {

struct LatentShape {
    int heads = 0, dim = 0, rot_dim = 0, rot_dims = 0, vdim = 0, rank = 0;
    int rank_pad = 0, rot_pad = 0;   // multiples of 32
    int pieces = 1;                  // of a cache row
    int window = 0;                  // 0: every earlier token
    int ring_rows = 0;
    __host__ __device__ int row_width() const { return rank_pad + rot_pad; }
    __host__ __device__ int row_elems() const { return pieces * row_width(); }
};

// ── decode step ──
struct LatentStepArgs {
    LatentShape s;
    const float *q = nullptr;          // [heads * (dim + rot_dim)] raw
    const float *kv = nullptr;         // [rank | rot_dim] raw
    const float *kv_norm = nullptr;    // [rank_pad]
    const uint16_t *uk = nullptr;      // [heads * dim][rank_pad] bf16
    const uint16_t *uv = nullptr;      // [heads * vdim][rank_pad] bf16
    const float *cos_tab = nullptr, *sin_tab = nullptr;  // [positions][rot_dims]
    float eps = 0.f, scale = 1.f;
    uint16_t *ring = nullptr;
    float *q_latent = nullptr;         // [heads][row_width]: scaled q' and rotated part
    float *part_o = nullptr, *part_ml = nullptr;  // [splits][heads][rank_pad], [splits][heads][2]
    const float *gate = nullptr;       // [heads * vdim] raw (output times its sigmoid) or NULL
    float *out = nullptr;              // [heads * vdim]
    const DecodeState *cursor = nullptr;
    int span = 0;                      // rows the step can see at most (the window or the cache's capacity)
};
int latent_step_splits(const LatentShape &s, int span);
// q' and rotated parts of the queries; the token's cache row
int latent_step_prep_launch(hm_ctx *ctx, const LatentStepArgs &a);
int latent_step_attn_launch(hm_ctx *ctx, const LatentStepArgs &a);
// joins the splits, value matrix, output gate
int latent_step_fold_launch(hm_ctx *ctx, const LatentStepArgs &a);

// ── prompt pass, n rows at positions past .. past + n - 1 ──
struct LatentRowsArgs {
    LatentShape s;
    RowSource down;                    // rows [q latent (q_rank_pad) | kv latent | rotated key ...]
    int q_rank = 0, q_rank_pad = 0;    // the kv part starts at column q_rank_pad
    const float *q_norm = nullptr, *kv_norm = nullptr;
    const float *cos_tab = nullptr, *sin_tab = nullptr;
    float eps = 0.f;
    uint16_t *q_split = nullptr;       // [n][q_pieces * q_rank_pad]
    int q_pieces = 3;
    uint16_t *ring = nullptr;
    int n = 0, past = 0;
};
int latent_rows_launch(hm_ctx *ctx, const LatentRowsArgs &a);
// q rows [n][heads * width] f32 with rotation, zero behind dim + rot_dim, from the raw projection
int latent_q_rows_launch(hm_ctx *ctx, const LatentShape &s, const RowSource &q, const float *cos_tab, const float *sin_tab,
                         float *d_out, int width, int n, int past);
// latents of positions first .. first + rows - 1 as a split matrix [rows][pieces * rank_pad]
int latent_gather_launch(hm_ctx *ctx, const LatentShape &s, const uint16_t *ring, uint16_t *d_out, int first, int rows);
// keys [heads][cap][kw] and values [heads][cap][vw] as planes of s.pieces pieces (heads * cap * kw / vw elements
// apart) from the expanded rows [rows][heads * dim | heads * vdim] f32 (the values start at column v_at) and the rotated keys
int latent_kv_rows_launch(hm_ctx *ctx, const LatentShape &s, const RowSource &kv, int v_at, const uint16_t *ring, uint16_t *d_k,
                          uint16_t *d_v, int kw, int vw, int cap, int first, int rows);

}  // namespace homura
