// Grouped-query attention whose keys and queries are normed per head, over a sliding window next to kept first tokens,
// without rotation. Position i sees j <= i with i - j < window or j < keep.
//
// Cache of one layer: planes of pieces (1: bf16, 3: the three bf16 pieces of the f32 values), keys then values, each
// [kv_heads][slots][width], zero behind the true head sizes. Kept tokens have slots of their own, the others take
// turns in a ring. Several layers may read one cache with queries, windows and kept tokens of their own; the ring is
// sized for the widest of them. Prompts go through the causal attention of prefill.h, straight from the slots.
#pragma once
#include <cstdint>

#include "hm_common.h"
#include "row_source.h"

namespace homura {

constexpr int WA_MAX_DIM = 256;
// padded width of keys and values: 64, 128 or 256 (0: neither fits)
int window_head_width(int dim, int vdim);

// Where positions sit: position p in slot p below keep, in slot keep + (p - keep) % ring from there on.
struct SlotMap {
    int keep = 0, ring = 1;
    __host__ __device__ int slots() const { return keep + ring; }
    __host__ __device__ int slot(int p) const { return p < keep ? p : keep + (p - keep) % ring; }
};

struct WindowAttentionShape {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    int width = 0;                   // window_head_width(dim, vdim)
    int pieces = 1;                  // of a cache row
    int window = 0, keep = 0;        // what this layer sees (window 0: every earlier token)
    SlotMap map;                     // of the cache it reads
    __host__ __device__ size_t plane() const { return (size_t)kv_heads * map.slots() * width; }
    size_t row_bytes() const { return (size_t)pieces * kv_heads * 2 * width * 2; }  // of a cached token
};

// ── decode step ──
struct WindowStepArgs {
    WindowAttentionShape s;
    const float *q = nullptr;                     // [heads * dim] raw
    const float *k = nullptr, *v = nullptr;       // [kv_heads * dim], [kv_heads * vdim] raw; NULL: the row is cached already
    const float *q_norm = nullptr, *k_norm = nullptr;  // [dim]
    float eps = 0.f, scale = 1.f;
    uint16_t *cache = nullptr;
    float *part_o = nullptr, *part_ml = nullptr;  // [splits][heads][width], [splits][heads][2]
    float *out = nullptr;                         // [heads * vdim]
    const DecodeState *cursor = nullptr;
    int span = 0;                                 // rows the step can see at most
};
int window_step_span(const WindowAttentionShape &s, int max_len);
int window_step_splits(int span);
int window_step_attn_launch(hm_ctx *ctx, const WindowStepArgs &a);
int window_step_fold_launch(hm_ctx *ctx, const WindowStepArgs &a);

// ── prompt pass, n rows at positions past .. past + n - 1 ──
// Queries normed into [n][heads * width] f32, keys (normed) and values into the cache. Parts of a projection row: the
// query heads from column 0, key heads from k_at, value heads from v_at (kv_heads 0 of them when the cache is another
// layer's: k_norm NULL).
struct WindowRowsArgs {
    WindowAttentionShape s;
    RowSource in;
    int k_at = 0, v_at = 0;
    const float *q_norm = nullptr, *k_norm = nullptr;
    float eps = 0.f;
    float *q = nullptr;
    uint16_t *cache = nullptr;
    int n = 0, past = 0;
};
int window_rows_launch(hm_ctx *ctx, const WindowRowsArgs &a);

}  // namespace homura
