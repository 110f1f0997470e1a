// A decoder put together from a list of layers, each a mixer (latent attention, attention over a window and kept first
// tokens, selective scan, gated linear recurrence, matrix memory) and optionally a feed-forward (gated, or a mixture of
// experts), with norms behind every sublayer and, in some designs, ahead of it, and a stretch of layers that may run
// several times in a row. The Nokuvik and Ludalix models are of this kind; their config.json is what
// block_config_from_json reads, and the weight slots carry their tensor names.
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "../block_rows.h"
#include "../gated_act.h"
#include "../latent_attention.h"
#include "../matrix_memory.h"
#include "../window_attention.h"
#include "decoder.h"
#include "json.h"

namespace homura {

enum class MixerKind { LatentAttention, SelectiveScan, LinearRecurrence, WindowAttention, MatrixMemory };

struct LatentAttentionSpec {
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    int window = 0;  // 0: no limit
    int rot_dims = 0;
    double rot_base = 10000.0, scale = 1.0;
};
struct SelectiveScanSpec { int inner = 0, taps = 0, dt_rank = 0, state = 0; };
struct LinearRecurrenceSpec { int width = 0, taps = 0, blocks = 0; };
struct WindowAttentionSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    int window = 0, keep = 0;  // 0: no limit / no tokens kept
    int kv_from = -1;          // layer whose keys and values are read instead of own ones
    double scale = 1.0;
};
struct MatrixMemorySpec {
    int heads = 0, dim = 0, vdim = 0;
    double gate_cap = 1.0;
};

struct FeedForwardSpec {
    int width = 0;             // of the one, or of every expert; 0: no feed-forward
    GatedAct act;
    int experts = 0, top = 0;  // 0 experts: a dense one
};

struct BlockLayerSpec {
    MixerKind mixer = MixerKind::LatentAttention;
    LatentAttentionSpec attn;
    SelectiveScanSpec scan;
    LinearRecurrenceSpec rec;
    WindowAttentionSpec wattn;
    MatrixMemorySpec mem;
    FeedForwardSpec ff;
};

struct BlockConfig {
    int vocab = 0, width = 0;
    double eps = 1e-6, embed_scale = 1.0;
    bool pre_norms = true;        // a norm ahead of every sublayer, next to the one behind it
    double residual_mult = 1.0;   // of what a sublayer adds to the residual
    bool position_waves = false;  // sinusoidal positions are added to the embedding
    std::vector<BlockLayerSpec> layers;
    // layers [loop_start, loop_stop) run loop_times times in a row, each pass with its own cache, and ahead of each
    // pass the residual becomes loop.in [x; x0] (0 times: no loop)
    int loop_start = 0, loop_stop = 0, loop_times = 0;

    struct Run { int layer; bool begins_pass; };
    std::vector<Run> runs() const;  // layers in running order
};

bool block_config_from_json(const Json &j, BlockConfig *cfg, std::string *err);

class BlockModel : public DecoderModel {
  public:
    // compute BF16: projections of the prompt pass take activations rounded to bf16 and the attention cache is bf16;
    // F32: activations as three bf16 pieces, which hold all of an f32, and the cache as the pieces of f32 rows.
    // Weights are bf16 in both, decode steps, norms, gates, recurrences and the residual f32.
    static std::unique_ptr<BlockModel> create(hm_ctx *ctx, const BlockConfig &cfg, DType compute);
    ~BlockModel() override;

    const BlockConfig &config() const { return cfg_; }
    DType compute_dtype() const { return compute_; }
    int vocab_size() const override { return cfg_.vocab; }
    int hidden_size() const override { return cfg_.width; }
    int num_layers() const override { return (int)cfg_.layers.size(); }
    int set_weight(int slot, const void *h_data, size_t bytes) override;
    int set_weight_nk(int slot, const void *h_data, size_t bytes) override;
    int finalize(int max_seq_len) override;
    bool prefill_available() const override;
    // 1 to 3 (compute F32: 3). Gates, step sizes and the residual's way through loop.in always take three.
    int set_prefill_pieces(int n) override;
    // Rows a chunk, 16 to MAX_CHUNK (the default): larger chunks fill the chip, smaller ones need less scratch and smaller
    // rings of window rows.
    static constexpr int MAX_CHUNK = 2048;
    int set_prefill_chunk(int rows) override;
    size_t cache_bytes() const { return plan_ && plan_->state_cache() ? plan_->state_cache()->bytes() : 0; }
    // Test support: the residual rows behind every layer run of the next prompt-pass chunks, [runs][rows][width]
    // for the rows of the latest chunk (0 runs captured: nothing).
    int capture_residuals(bool on);
    int captured_residuals(float *h_out, size_t n_floats);

  private:
    BlockModel() = default;

    // A matrix in HBM, [np][kp] bf16, rows and columns behind the true ones zero (multiples of 32, so that every
    // activation row is a whole number of vectors with zeros behind it).
    struct Linear {
        Buffer w;
        int np = 0, kp = 0;
        const uint16_t *ptr(size_t row = 0) const { return w.as<uint16_t>() + row * kp; }
    };
    struct Vec { Buffer b; int n = 0; const float *ptr() const { return b.as<float>(); } };
    struct LayerWeights {
        Vec norm1, norm1b, norm2, norm2b;
        Linear gate_up, down;
        // latent attention: [q down | kv down + rotated key | output gate], q up, [key up | value up], output
        Linear la_down, la_uq, la_ukv, la_o;
        Vec q_norm, kv_norm;
        // selective scan: [x | z], [dt | B | C], dt, output
        Linear ss_in, ss_x, ss_dt, ss_o;
        Vec conv_w, conv_b, dt_b, a_log2, d;
        // linear recurrence: [x | y] with biases, per block [r rows | i rows], output
        Linear lr_in, lr_gates, lr_o;
        Vec lr_in_b, r_b, i_b, decay;
        // window attention: [q | k | v] (q alone over another layer's cache), output; its head norms
        Linear wa_in, wa_o;
        Vec head_q_norm, head_k_norm;
        // matrix memory: [q | k | v | output gate | log gates], output
        Linear mm_in, mm_o;
        Vec mm_norm, mm_i_b, mm_f_b;
        // mixture of experts: router; gate_up and down hold the experts one after the other
        Linear router;
    };
    // Where a slot goes: rows of a matrix (row r to (r / group) * group_stride + (r % group) * mult + off) or a
    // vector, through a transformation.
    struct Target {
        Linear *lin = nullptr;
        int rows = 0, cols = 0, group = 0, group_stride = 0, mult = 1, off = 0;
        Vec *vec = nullptr;
        int vec_off = 0;
        enum How { Plain, Residual, Taps, StateDecay, ChannelDecay, Rows } how = Plain;
    };
    // widths in memory of one layer
    struct Dims {
        int q_rank = 0, kv = 0, gate = 0, down_n = 0, uq_n = 0, v_at = 0, ukv_n = 0, head_k = 0, head_v = 0;  // latent attention
        int inner = 0, dt = 0, state = 0;                                                                     // selective scan
        int width = 0, block = 0, block_pad = 0;                                                              // linear recurrence
        int k_at = 0, wa_n = 0;                                                                               // window attention (v_at, gate as above)
        int mm_n = 0;                                                                                         // matrix memory (gate as above)
        MatrixMemoryColumns mm_at;
        int ff = 0, router_n = 0;
        LatentShape shape;
        WindowAttentionShape wshape;
        MatrixMemoryShape mshape;
    };

    int add_slots(std::string *err);
    int upload_matrix(const Target &t, const uint16_t *h_nk);
    int upload_vector(const Target &t, const float *h);
    int step_inputs(std::vector<Buffer *> &inputs) override;
    int prefill_chunk(const int32_t *h_ids, int n, float *h_logits) override;
    const char *prefill_needs() const override;
    int mark_position() override;
    int rewind_to_mark(int mark_len, const std::vector<int32_t> &kept) override;
    PositionWaves waves() const { return PositionWaves{wave_freq_ ? wave_freq_.as<double>() : nullptr, cfg_.width}; }
    int place_windows();
    int alloc_scratch();
    int emit_plan();
    int prepare_prefill();
    int prefill_window_attention(int run, int layer, int n, int past, int *y_parts);
    int prefill_matrix_memory(int run, int layer, const float *x, int n, int past, int *y_parts);
    int prefill_feed_forward(int layer, int n, int *y_parts);
    int prefill_mixer(int run, int layer, const float *cos_tab, const float *sin_tab, int n, int past, int *y_parts);

    BlockConfig cfg_;
    DType compute_ = DType::BF16;
    int wp_ = 0;                        // width in memory
    std::vector<BlockConfig::Run> runs_;
    std::vector<LayerWeights> layers_;
    std::vector<Dims> dims_;
    std::vector<int> cache_run_;        // by run: the run whose window rows it reads (its own, or an earlier layer's)
    Linear loop_in_, head_;
    Vec embed_, final_norm_;
    Buffer wave_freq_;                  // f64, PositionWaves
    std::vector<Target> targets_;       // by slot
    struct Rope { int dims; double base; Buffer cos, sin; };
    std::vector<std::unique_ptr<Rope>> ropes_;
    std::vector<Rope *> layer_rope_;    // by layer (NULL: no rotation)

    // decode step: activations, one f32 row each
    struct StepScratch {
        Buffer cat, xa, xb, y, d1, d2, act, qlat, part_o, part_ml, normed, cand_val, cand_idx, choice;
        int cand_cap = 0;
    };
    std::shared_ptr<StepScratch> step_;
    Buffer ids_view_;
    // prompt pass
    struct PrefillScratch {
        static constexpr int MAX_PARTS = 8;
        int rows = 0;
        Buffer ids, x, x0, y, d1, d2, d3, f1, f2, f3, split_a, split_b, lat, kvf, kws, vws, logits;
        Buffer mm_q, mm_k, mm_values, mm_ahead, mm_gates, mm_log_w, mm_weights, mm_decay;                 // matrix memory
        Buffer choice, choice_weight, expert_list, expert_count;           // mixture of experts
        Buffer captured;
        int captured_rows = 0;
        bool capture = false;
    };
    PrefillScratch pf_;
};

}  // namespace homura
