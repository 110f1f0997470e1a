// Recurrent mixers: a short causal convolution per channel, the selective scan (a diagonal state space per channel
// whose step size, input and output vectors depend on the token) and the real-gated linear recurrence. Each has a
// prompt form (a chunk of rows at once) and a decode form (one row; the convolution of a decode step is the
// epilogue of the projection in front of it, gemv_bf16.h: GemvConv). Everything recurrent is f32.
#pragma once
#include <cstdint>

#include "hm_common.h"
#include "row_source.h"

namespace homura {

// The latest inputs of a convolution: input of position p in slot p % taps of [taps][width].
struct TapRing {
    float *ring = nullptr;
    int taps = 0, width = 0;
};

// out[t][c] = act(b[c] + sum_j w[j][c] in[t - (taps - 1) + j][c]) for n rows at positions past .. past + n - 1, the
// inputs ahead of the chunk from the ring (positions below 0 count as zero). The ring is only read: the mixer's
// kernel behind it stores the chunk's last inputs. Besides the f32 rows the result leaves as three-piece (or
// `pieces`) split matrices, one per block of block_width channels: [blocks][n][pieces * block_pad].
struct ConvRowsArgs {
    RowSource in;
    TapRing ring;
    const float *w = nullptr, *b = nullptr;  // [taps][width], [width]
    bool silu = false;
    float *out = nullptr;                    // [n][width]
    uint16_t *out_split = nullptr;
    int pieces = 3, channels = 0, block_width = 0, block_pad = 0;
    // columns [width, width + side_cols) of the input rows only go through an activation: side[n][side_cols]
    enum Act { None = 0, Silu = 1, Gelu = 2 };
    float *side = nullptr;
    int side_cols = 0, side_act = None;
    int n = 0, past = 0;
};
int conv_rows_launch(hm_ctx *ctx, const ConvRowsArgs &a);

// Selective scan, for channel c with step d = softplus(projection + bias) and input u: every state n of the channel
// becomes s_n = e^(d A_cn) s_n + d u B_n; the result is (<s, C> + D_c u) * z_c.
constexpr int SSM_MAX_STATE = 128;
int ssm_state_pad(int state);  // states per channel in memory: 16, 32, 64 or 128
struct SelectiveScanArgs {
    const float *x = nullptr;          // [n][inner] convolved rows
    const float *dt = nullptr, *dt_bias = nullptr;  // [n][inner] before bias and softplus, [inner]
    const float *b = nullptr, *c = nullptr;  // [n][bc_ld] f32, state_pad columns each (zero behind the true ones)
    int bc_ld = 0;
    const float *a_log2 = nullptr;     // [inner][state_pad]: A * log2(e), 0 behind the true states
    const float *d = nullptr;          // [inner]
    const float *z = nullptr;          // [n][inner]: silu of the gate rows
    float *state = nullptr;            // [inner][state_pad]
    uint16_t *out_split = nullptr;     // [n][pieces * inner]
    int pieces = 3;
    RowSource conv_in;                 // the convolution's input rows: the last of them go into the ring
    TapRing ring;
    int n = 0, inner = 0, state_pad = 0, past = 0;  // inner % 32 == 0
};
int selective_scan_launch(hm_ctx *ctx, const SelectiveScanArgs &a);

// One token: xz = [x (convolved, silu) | z], p = [dt low rank (dt_pad) | B | C].
struct SelectiveStepArgs {
    const float *xz = nullptr, *p = nullptr;
    const uint16_t *dt_w = nullptr;    // [inner][dt_pad] bf16
    const float *dt_b = nullptr, *a_log2 = nullptr, *d = nullptr;
    float *state = nullptr, *y = nullptr;
    const DecodeState *cursor = nullptr;
    int inner = 0, dt_pad = 0, state_pad = 0;
};
int selective_step_launch(hm_ctx *ctx, const SelectiveStepArgs &a);

// Gated linear recurrence: per channel r = sigmoid(gate_r), i = sigmoid(gate_i), a = exp(decay_c * r) with
// decay_c < 0, S <- a S + sqrt(1 - a^2) i u; the result is S * y.
struct LinearRecurrenceArgs {
    const float *u = nullptr;          // [n][width]
    const float *gates = nullptr;      // [n][blocks * 2 * block_pad]: block b's r columns, then its i columns
    const float *r_bias = nullptr, *i_bias = nullptr, *decay = nullptr;  // [width]
    const float *y = nullptr;          // [n][width]: gelu_tanh of the other branch
    float *state = nullptr;            // [width]
    uint16_t *out_split = nullptr;     // [n][pieces * width]
    int pieces = 3;
    RowSource conv_in;
    TapRing ring;
    int n = 0, channels = 0, width = 0, block_width = 0, block_pad = 0, past = 0;
};
int linear_recurrence_launch(hm_ctx *ctx, const LinearRecurrenceArgs &a);

// One token: uy = [u (convolved) | gelu_tanh(y)], width apart; the gates are multiplied here.
struct LinearRecurrenceStepArgs {
    const float *uy = nullptr;
    const uint16_t *gate_w = nullptr;  // [blocks][2 * block_pad][block_pad] bf16: r rows, then i rows
    const float *r_bias = nullptr, *i_bias = nullptr, *decay = nullptr;
    float *state = nullptr, *out = nullptr;
    const DecodeState *cursor = nullptr;
    int channels = 0, width = 0, block_width = 0, block_pad = 0;
};
int linear_recurrence_step_launch(hm_ctx *ctx, const LinearRecurrenceStepArgs &a);

}  // namespace homura
