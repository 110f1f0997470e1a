// Mixtures of experts, and the row kernel of gated activations. The router's logits z = W_r x rank the experts of a token;
// each of the `top` first ones takes sigmoid(z) x for its input. Its projections being linear, gate and up values are
// scaled instead.
//
// A prompt of n tokens has top * n entries, entry e = place * n + token. Experts read token rows and write entry rows, so
// the results of the places are to be added like the K slices of a product, n * width apart.
#pragma once
#include <cstdint>

#include "gated_act.h"
#include "hm_common.h"
#include "row_source.h"

namespace homura {

constexpr int EXPERTS_MAX = 1024, EXPERTS_MAX_TOP = 64;

// ── prompt pass ──
// out_split = split(act(w gate, w up)) of rows with gate and up interleaved, w the row's weight (NULL: 1)
struct GatedRowsArgs {
    RowSource in;                       // [rows][2 * width]
    const float *weight = nullptr;      // [rows]
    GatedAct act;
    uint16_t *out_split = nullptr;      // [rows][pieces * width]
    int pieces = 3, rows = 0, width = 0;
};
int gated_rows_launch(hm_ctx *ctx, const GatedRowsArgs &a);

struct RouteRowsArgs {
    RowSource logits;                   // [n][>= experts]
    int experts = 0, top = 0, n = 0;
    int *choice = nullptr;              // [top * n]: expert of an entry
    float *weight = nullptr;            // [top * n]
    int *list = nullptr;                // [experts][n]: entries of an expert, ascending
    int *count = nullptr;               // [experts]
};
int route_rows_launch(hm_ctx *ctx, const RouteRowsArgs &a);

// y[0][i] = sum over the places of y[place][i], for more places than a consumer adds up by itself
int sum_places_launch(hm_ctx *ctx, float *d_y, int places, size_t n);

// ── decode step ──
struct ExpertsStepArgs {
    const float *x = nullptr;           // [K]
    const float *logits = nullptr;      // [experts]
    const uint16_t *gate_up = nullptr;  // [experts][2 * ff][K], gate and up rows interleaved
    const uint16_t *down = nullptr;     // [experts][width][ff]
    int experts = 0, top = 0, K = 0, ff = 0, width = 0;  // K % 32 == 0, ff % 32 == 0
    GatedAct act;
    int *choice = nullptr;              // [top]
    float *hidden = nullptr;            // [top][ff]
    float *y = nullptr;                 // [width]
};
int experts_step_up_launch(hm_ctx *ctx, const ExpertsStepArgs &a);
int experts_step_down_launch(hm_ctx *ctx, const ExpertsStepArgs &a);

}  // namespace homura
