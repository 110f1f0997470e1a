// BlockModel: weights, decode plan and prompt pass (see block_model.h).
#include "block_model.h"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "../block_rows.h"
#include "../experts.h"
#include "../gemm_bf16_mfma.h"
#include "../gemv_bf16.h"
#include "../light_ops.h"
#include "../prefill.h"
#include "../recurrent.h"

namespace homura {

namespace {

int pad32(int n) { return (n + 31) / 32 * 32; }

// What a design fixes beyond its config.json.
struct Design {
    const char *name;
    bool pre_norms, position_waves;
    bool clamped_dense;  // dense feed-forwards: ClampedSigmoid with a limit of their own, otherwise SiLU
};
constexpr Design DESIGNS[] = {{"Nokuvik", true, false, false}, {"Ludalix", false, true, true}};
constexpr double CLAMPED_SLOPE = 1.702, WAVE_BASE = 10000.0;

}  // namespace

// ── configuration ────────────────────────────────────────────────────────────

std::vector<BlockConfig::Run> BlockConfig::runs() const {
    std::vector<Run> r;
    const int n = (int)layers.size();
    for (int i = 0; i < (loop_times ? loop_start : n); i++) r.push_back({i, false});
    for (int t = 0; t < loop_times; t++)
        for (int i = loop_start; i < loop_stop; i++) r.push_back({i, i == loop_start});
    if (loop_times)
        for (int i = loop_stop; i < n; i++) r.push_back({i, false});
    return r;
}

bool block_config_from_json(const Json &j, BlockConfig *cfg, std::string *err) {
    auto bad = [&](const std::string &what) {
        *err = "config.json: " + what;
        return false;
    };
    auto num = [&](const Json *o, const char *key, const std::string &where, double *out) {
        const Json *v = o ? o->get(key) : nullptr;
        if (!v || v->kind != Json::Num) return bad("missing number `" + where + key + "`");
        *out = v->num;
        return true;
    };
    auto size = [&](const Json *o, const char *key, const std::string &where, int *out) {
        double d;
        if (!num(o, key, where, &d)) return false;
        if (d < 1 || d > 1e9 || d != std::floor(d)) return bad("`" + where + key + "` is not a size");
        *out = (int)d;
        return true;
    };
    auto given = [](const Json *o, const char *key) -> const Json * {
        const Json *v = o ? o->get(key) : nullptr;
        return v && v->kind != Json::Null ? v : nullptr;
    };
    BlockConfig c;
    const Design *design = &DESIGNS[0];
    if (const Json *a = given(&j, "architecture")) {
        design = nullptr;
        for (const Design &d : DESIGNS)
            if (a->kind == Json::Str && a->str == d.name) design = &d;
        if (!design) return bad("`architecture` \"" + a->str + "\" is not known");
    }
    c.pre_norms = design->pre_norms;
    c.position_waves = design->position_waves;
    if (given(&j, "residual_mult") && !num(&j, "residual_mult", "", &c.residual_mult)) return false;
    if (!size(&j, "vocab", "", &c.vocab) || !size(&j, "width", "", &c.width) || !num(j.get("norm"), "eps", "norm.", &c.eps)) return false;
    if (const Json *e = given(&j, "embedding"))
        if (given(e, "scale") && !num(e, "scale", "embedding.", &c.embed_scale)) return false;
    const Json *layers = j.get("layers");
    if (!layers || layers->kind != Json::Arr || layers->arr.empty()) return bad("missing list `layers`");
    for (size_t i = 0; i < layers->arr.size(); i++) {
        const Json &l = layers->arr[i];
        const std::string at = "layers[" + std::to_string(i) + "].", m_at = at + "mixer.";
        const Json *type = l.get("type"), *m = l.get("mixer");
        if (!type || type->kind != Json::Str || !m || m->kind != Json::Obj) return bad("missing `" + at + "type` or `" + at + "mixer`");
        BlockLayerSpec s;
        if (type->str == "latent_attention") {
            s.mixer = MixerKind::LatentAttention;
            LatentAttentionSpec &a = s.attn;
            if (!size(m, "heads", m_at, &a.heads) || !size(m, "dim", m_at, &a.dim) || !size(m, "rot_dim", m_at, &a.rot_dim) ||
                !size(m, "vdim", m_at, &a.vdim) || !size(m, "q_rank", m_at, &a.q_rank) || !size(m, "kv_rank", m_at, &a.kv_rank) ||
                !num(m, "scale", m_at, &a.scale))
                return false;
            if (const Json *mask = given(m, "mask"))
                if (given(mask, "size") && !size(mask, "size", m_at + "mask.", &a.window)) return false;
            if (const Json *rot = given(m, "rot")) {
                if (!size(rot, "dims", m_at + "rot.", &a.rot_dims) || !num(rot, "base", m_at + "rot.", &a.rot_base)) return false;
                if (a.rot_dims % 2 || a.rot_dims > a.rot_dim) return bad("`" + m_at + "rot.dims` must be even and at most rot_dim");
            }
        } else if (type->str == "mamba1") {
            s.mixer = MixerKind::SelectiveScan;
            SelectiveScanSpec &a = s.scan;
            if (!size(m, "inner", m_at, &a.inner) || !size(m, "conv", m_at, &a.taps) || !size(m, "dt_rank", m_at, &a.dt_rank) ||
                !size(m, "state", m_at, &a.state))
                return false;
        } else if (type->str == "rglru") {
            s.mixer = MixerKind::LinearRecurrence;
            LinearRecurrenceSpec &a = s.rec;
            if (!size(m, "width", m_at, &a.width) || !size(m, "conv", m_at, &a.taps) || !size(m, "blocks", m_at, &a.blocks)) return false;
            if (a.width % a.blocks) return bad("`" + m_at + "width` is not a multiple of its blocks");
        } else if (type->str == "attention") {
            s.mixer = MixerKind::WindowAttention;
            WindowAttentionSpec &a = s.wattn;
            if (!size(m, "heads", m_at, &a.heads) || !size(m, "kv_heads", m_at, &a.kv_heads) || !size(m, "dim", m_at, &a.dim) ||
                !size(m, "vdim", m_at, &a.vdim) || !num(m, "scale", m_at, &a.scale))
                return false;
            if (a.heads % a.kv_heads) return bad("`" + m_at + "heads` is not a multiple of its kv_heads");
            if (const Json *mask = given(m, "mask")) {
                if (given(mask, "size") && !size(mask, "size", m_at + "mask.", &a.window)) return false;
                double keep = 0;
                if (given(mask, "keep_first") && !num(mask, "keep_first", m_at + "mask.", &keep)) return false;
                if (keep < 0 || keep > 1e9 || keep != std::floor(keep)) return bad("`" + m_at + "mask.keep_first` is not a count");
                a.keep = a.window ? (int)keep : 0;
            }
            if (given(m, "kv_from")) {
                double from;
                if (!num(m, "kv_from", m_at, &from)) return false;
                const BlockLayerSpec *src = from >= 0 && from < (double)i && from == std::floor(from) ? &c.layers[(size_t)from] : nullptr;
                if (!src || src->mixer != MixerKind::WindowAttention || src->wattn.kv_from >= 0 || src->wattn.kv_heads != a.kv_heads ||
                    src->wattn.dim != a.dim || src->wattn.vdim != a.vdim)
                    return bad("`" + m_at + "kv_from` must name an earlier attention layer with keys of its own and the same heads");
                a.kv_from = (int)from;
            }
        } else if (type->str == "mlstm") {
            s.mixer = MixerKind::MatrixMemory;
            MatrixMemorySpec &a = s.mem;
            if (!size(m, "heads", m_at, &a.heads) || !size(m, "dim", m_at, &a.dim) || !size(m, "vdim", m_at, &a.vdim) ||
                !num(m, "gate_cap", m_at, &a.gate_cap))
                return false;
            if (!(a.gate_cap > 0)) return bad("`" + m_at + "gate_cap` must be positive");
        } else {
            return bad("`" + at + "type` \"" + type->str + "\" is not known");
        }
        if (const Json *mlp = given(&l, "mlp")) {
            const Json *kind = mlp->get("kind");
            const bool dense = kind && kind->kind == Json::Str && kind->str == "dense";
            if (!dense && (!kind || kind->kind != Json::Str || kind->str != "moe")) return bad("`" + at + "mlp.kind` must be \"dense\" or \"moe\"");
            if (dense) {
                if (!size(mlp, "ff", at + "mlp.", &s.ff.width)) return false;
                if (design->clamped_dense) {
                    double limit;
                    if (!num(mlp, "limit", at + "mlp.", &limit)) return false;
                    if (!(limit > 0)) return bad("`" + at + "mlp.limit` must be positive");
                    s.ff.act.kind = GatedAct::ClampedSigmoid;
                    s.ff.act.limit = (float)limit;
                    s.ff.act.slope = (float)CLAMPED_SLOPE;
                }
            } else {
                if (!size(mlp->get("expert"), "ff", at + "mlp.expert.", &s.ff.width) || !size(mlp->get("router"), "experts", at + "mlp.router.", &s.ff.experts) ||
                    !size(mlp->get("router"), "top", at + "mlp.router.", &s.ff.top))
                    return false;
                if (s.ff.top > s.ff.experts) return bad("`" + at + "mlp.router.top` exceeds its experts");
            }
        }
        c.layers.push_back(s);
    }
    if (const Json *loop = given(&j, "loop")) {
        double start, stop;
        if (!num(loop, "start", "loop.", &start) || !num(loop, "stop", "loop.", &stop) || !size(loop, "times", "loop.", &c.loop_times)) return false;
        if (start < 0 || start != std::floor(start) || stop != std::floor(stop) || stop <= start || stop > (double)c.layers.size())
            return bad("`loop` does not name a stretch of the layers");
        c.loop_start = (int)start;
        c.loop_stop = (int)stop;
    }
    *cfg = c;
    return true;
}

// ── weights ──────────────────────────────────────────────────────────────────

std::unique_ptr<BlockModel> BlockModel::create(hm_ctx *ctx, const BlockConfig &cfg, DType compute) {
    auto fail = [&](const std::string &msg) -> std::unique_ptr<BlockModel> {
        hm_set_error(ctx, HM_ERR_INVALID, "BlockModel: %s", msg.c_str());
        return nullptr;
    };
    if (compute != DType::BF16 && compute != DType::F32) return fail("compute dtype must be BF16 or F32");
    if (cfg.vocab <= 0 || cfg.width <= 0 || cfg.layers.empty()) return fail("empty configuration");
    if (pad32(cfg.width) > 8192) return fail("width above 8192");
    std::unique_ptr<BlockModel> m(new BlockModel());
    m->ctx_ = ctx;
    m->cfg_ = cfg;
    m->compute_ = compute;
    m->prefill_pieces_ = compute == DType::F32 ? 3 : 1;
    m->chunk_rows_ = MAX_CHUNK;
    m->wp_ = pad32(cfg.width);
    m->runs_ = cfg.runs();
    for (size_t r = 0; r < m->runs_.size(); r++) {
        const int from = cfg.layers[m->runs_[r].layer].wattn.kv_from;
        int at = (int)r;
        if (from >= 0)  // the latest run of the layer it reads
            while (at > 0 && m->runs_[at].layer != from) at--;
        m->cache_run_.push_back(at);
    }
    m->layers_.resize(cfg.layers.size());
    m->dims_.resize(cfg.layers.size());
    for (size_t i = 0; i < cfg.layers.size(); i++) {
        const BlockLayerSpec &s = cfg.layers[i];
        Dims &d = m->dims_[i];
        d.ff = pad32(s.ff.width);
        d.router_n = pad32(s.ff.experts);
        if (d.ff > 16384) return fail("feed-forward width above 16384");
        if (s.ff.experts && cfg.pre_norms) return fail("a mixture of experts reads the residual itself: no norm ahead of it");
        if (s.ff.experts > EXPERTS_MAX || s.ff.top > EXPERTS_MAX_TOP) return fail("more than 1024 experts, or more than 64 of them a token");
        if (s.mixer == MixerKind::LatentAttention) {
            const LatentAttentionSpec &a = s.attn;
            d.q_rank = pad32(a.q_rank);
            d.kv = pad32(a.kv_rank + a.rot_dim);
            d.gate = pad32(a.heads * a.vdim);
            d.down_n = d.q_rank + d.kv + d.gate;
            d.uq_n = pad32(a.heads * (a.dim + a.rot_dim));
            d.v_at = pad32(a.heads * a.dim);
            d.ukv_n = d.v_at + d.gate;
            LatentShape &l = d.shape;
            l.heads = a.heads;
            l.dim = a.dim;
            l.rot_dim = a.rot_dim;
            l.rot_dims = a.rot_dims;
            l.vdim = a.vdim;
            l.rank = a.kv_rank;
            l.rank_pad = pad32(a.kv_rank);
            l.rot_pad = pad32(a.rot_dim);
            l.pieces = compute == DType::F32 ? 3 : 1;
            l.window = a.window;
            if (l.rank_pad > 1024) return fail("kv_rank above 1024");
            if (d.q_rank > 8192 || d.gate > 16384) return fail("q_rank above 8192 or heads * vdim above 16384");
            static const int classes[4][2] = {{64, 64}, {128, 128}, {192, 128}, {256, 256}};
            for (const auto &cl : classes)
                if (!d.head_k && a.dim + a.rot_dim <= cl[0] && a.vdim <= cl[1]) {
                    d.head_k = cl[0];
                    d.head_v = cl[1];
                }
        } else if (s.mixer == MixerKind::SelectiveScan) {
            const SelectiveScanSpec &a = s.scan;
            d.inner = pad32(a.inner);
            d.dt = pad32(a.dt_rank);
            d.state = ssm_state_pad(a.state);
            if (a.state > SSM_MAX_STATE) return fail("more than 128 states per channel");
            if (d.inner > 16384 || d.dt > 8192) return fail("inner above 16384 or dt_rank above 8192");
            if (a.taps > 32) return fail("more than 32 convolution taps");
        } else if (s.mixer == MixerKind::WindowAttention) {
            const WindowAttentionSpec &a = s.wattn;
            const bool own = a.kv_from < 0;
            d.k_at = pad32(a.heads * a.dim);
            d.v_at = d.k_at + pad32(a.kv_heads * a.dim);
            d.wa_n = own ? d.v_at + pad32(a.kv_heads * a.vdim) : d.k_at;
            d.gate = pad32(a.heads * a.vdim);
            WindowAttentionShape &l = d.wshape;
            l.heads = a.heads;
            l.kv_heads = a.kv_heads;
            l.dim = a.dim;
            l.vdim = a.vdim;
            l.width = window_head_width(a.dim, a.vdim);
            l.pieces = compute == DType::F32 ? 3 : 1;
            l.window = a.window;
            l.keep = a.keep;
            if (!l.width) return fail("attention heads above 256 elements");
            if (d.gate > 16384) return fail("heads * vdim above 16384");
        } else if (s.mixer == MixerKind::MatrixMemory) {
            const MatrixMemorySpec &a = s.mem;
            if (a.dim > MM_MAX_DIM) return fail("matrix memory with keys above 1024 elements");
            d.mm_at.k = pad32(a.heads * a.dim);
            d.mm_at.v = 2 * d.mm_at.k;
            d.gate = pad32(a.heads * a.vdim);
            d.mm_at.g = d.mm_at.v + d.gate;
            d.mm_at.i = d.mm_at.g + d.gate;
            d.mm_at.f = d.mm_at.i + a.heads;
            d.mm_n = d.mm_at.i + pad32(2 * a.heads);
            MatrixMemoryShape &l = d.mshape;
            l.heads = a.heads;
            l.dim = a.dim;
            l.vdim = a.vdim;
            l.dim_pad = matrix_memory_dim_pad(a.dim);
            l.cap = (float)a.gate_cap;
            if (d.gate > 16384) return fail("heads * vdim above 16384");
        } else {
            const LinearRecurrenceSpec &a = s.rec;
            d.width = pad32(a.width);
            d.block = a.width / a.blocks;
            d.block_pad = pad32(d.block);
            if (d.width > 16384) return fail("recurrence width above 16384");
            if (a.taps > 32) return fail("more than 32 convolution taps");
        }
    }
    std::string err;
    if (m->add_slots(&err) != HM_OK) return fail(err);
    for (size_t i = 0; i < m->infos_.size(); i++) m->slot_by_name_[m->infos_[i].name] = (int)i;
    m->weight_set_.assign(m->infos_.size(), false);
    return m;
}

BlockModel::~BlockModel() {
    if (ctx_) hm_sync(ctx_);
}

int BlockModel::add_slots(std::string *err) {
    bool ok = true;
    auto alloc = [&](Buffer &b, size_t elems, DType t) {
        b = Buffer::alloc(ctx_, {(int64_t)elems}, t);
        ok = ok && b && hm_fill_zero(ctx_, b.ptr(), b.bytes()) == HM_OK;
    };
    auto linear = [&](Linear &l, int np, int kp) {
        l.np = np;
        l.kp = kp;
        alloc(l.w, (size_t)np * kp, DType::BF16);
    };
    auto vec = [&](Vec &v, int n) {
        v.n = n;
        alloc(v.b, n, DType::F32);
    };
    auto mat_slot = [&](const std::string &name, Linear &l, int rows, int cols, int off, int mult = 1, int group = 0, int group_stride = 0) {
        Target t;
        t.lin = &l;
        t.rows = rows;
        t.cols = cols;
        t.off = off;
        t.mult = mult;
        t.group = group ? group : rows;
        t.group_stride = group_stride;
        targets_.push_back(t);
        infos_.push_back(WeightSlotInfo{name, DType::BF16, cols, rows, (size_t)rows * cols * 2});
    };
    auto vec_slot = [&](const std::string &name, Vec &v, int rows, int cols = 1, int off = 0, Target::How how = Target::Plain) {
        Target t;
        t.vec = &v;
        t.rows = rows;
        t.cols = cols;
        t.vec_off = off;
        t.how = how;
        targets_.push_back(t);
        infos_.push_back(WeightSlotInfo{name, DType::F32, rows, cols, (size_t)rows * cols * 4});
    };
    const int W = cfg_.width;
    embed_.n = 0;
    alloc(embed_.b, (size_t)cfg_.vocab * wp_, DType::F32);
    vec_slot("embed", embed_, cfg_.vocab, W, wp_, Target::Rows);
    if (cfg_.loop_times) {
        linear(loop_in_, wp_, 2 * wp_);
        // [out][x | x0]: both halves start at a padded width, so the two are cut apart on upload
        mat_slot("loop.in", loop_in_, W, 2 * W, 0);
    }
    for (size_t i = 0; i < cfg_.layers.size(); i++) {
        const BlockLayerSpec &s = cfg_.layers[i];
        const Dims &d = dims_[i];
        LayerWeights &l = layers_[i];
        const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
        // the norm behind a sublayer carries the factor of what joins the residual
        auto norms = [&](const std::string &name, Vec &ahead, Vec &behind) {
            if (cfg_.pre_norms) {
                vec(ahead, wp_);
                vec_slot(name, ahead, W);
            }
            vec(behind, wp_);
            vec_slot(cfg_.pre_norms ? name + "b" : name, behind, W, 1, 0, Target::Residual);
        };
        norms(p + "norm1", l.norm1, l.norm1b);
        if (s.mixer == MixerKind::LatentAttention) {
            const LatentAttentionSpec &a = s.attn;
            linear(l.la_down, d.down_n, wp_);
            linear(l.la_uq, d.uq_n, d.q_rank);
            linear(l.la_ukv, d.ukv_n, d.shape.rank_pad);
            linear(l.la_o, wp_, d.gate);
            vec(l.q_norm, d.q_rank);
            vec(l.kv_norm, d.shape.rank_pad);
            mat_slot(m + "dq", l.la_down, a.q_rank, W, 0);
            vec_slot(m + "dq.norm", l.q_norm, a.q_rank);
            mat_slot(m + "uq", l.la_uq, a.heads * (a.dim + a.rot_dim), a.q_rank, 0);
            mat_slot(m + "dkv", l.la_down, a.kv_rank + a.rot_dim, W, d.q_rank);
            vec_slot(m + "dkv.norm", l.kv_norm, a.kv_rank);
            mat_slot(m + "uk", l.la_ukv, a.heads * a.dim, a.kv_rank, 0);
            mat_slot(m + "uv", l.la_ukv, a.heads * a.vdim, a.kv_rank, d.v_at);
            mat_slot(m + "g", l.la_down, a.heads * a.vdim, W, d.q_rank + d.kv);
            mat_slot(m + "o", l.la_o, W, a.heads * a.vdim, 0);
        } else if (s.mixer == MixerKind::SelectiveScan) {
            const SelectiveScanSpec &a = s.scan;
            linear(l.ss_in, 2 * d.inner, wp_);
            linear(l.ss_x, d.dt + 2 * d.state, d.inner);
            linear(l.ss_dt, d.inner, d.dt);
            linear(l.ss_o, wp_, d.inner);
            vec(l.conv_w, a.taps * d.inner);
            vec(l.conv_b, d.inner);
            vec(l.dt_b, d.inner);
            vec(l.a_log2, d.inner * d.state);
            vec(l.d, d.inner);
            // both halves, and the three parts, start at a padded row
            mat_slot(m + "in", l.ss_in, 2 * a.inner, W, 0, 1, a.inner, d.inner);
            vec_slot(m + "conv", l.conv_w, a.inner, a.taps, d.inner, Target::Taps);
            vec_slot(m + "conv.b", l.conv_b, a.inner);
            mat_slot(m + "x", l.ss_x, a.dt_rank + 2 * a.state, a.inner, 0);
            mat_slot(m + "dt", l.ss_dt, a.inner, a.dt_rank, 0);
            vec_slot(m + "dt.b", l.dt_b, a.inner);
            vec_slot(m + "A_log", l.a_log2, a.inner, a.state, d.state, Target::StateDecay);
            vec_slot(m + "D", l.d, a.inner);
            mat_slot(m + "o", l.ss_o, W, a.inner, 0);
        } else if (s.mixer == MixerKind::WindowAttention) {
            const WindowAttentionSpec &a = s.wattn;
            linear(l.wa_in, d.wa_n, wp_);
            linear(l.wa_o, wp_, d.gate);
            vec(l.head_q_norm, a.dim);
            mat_slot(m + "q", l.wa_in, a.heads * a.dim, W, 0);
            vec_slot(m + "q.norm", l.head_q_norm, a.dim);
            if (a.kv_from < 0) {
                vec(l.head_k_norm, a.dim);
                mat_slot(m + "k", l.wa_in, a.kv_heads * a.dim, W, d.k_at);
                mat_slot(m + "v", l.wa_in, a.kv_heads * a.vdim, W, d.v_at);
                vec_slot(m + "k.norm", l.head_k_norm, a.dim);
            }
            mat_slot(m + "o", l.wa_o, W, a.heads * a.vdim, 0);
        } else if (s.mixer == MixerKind::MatrixMemory) {
            const MatrixMemorySpec &a = s.mem;
            linear(l.mm_in, d.mm_n, wp_);
            linear(l.mm_o, wp_, d.gate);
            vec(l.mm_norm, d.gate);
            vec(l.mm_i_b, a.heads);
            vec(l.mm_f_b, a.heads);
            mat_slot(m + "q", l.mm_in, a.heads * a.dim, W, d.mm_at.q);
            mat_slot(m + "k", l.mm_in, a.heads * a.dim, W, d.mm_at.k);
            mat_slot(m + "v", l.mm_in, a.heads * a.vdim, W, d.mm_at.v);
            mat_slot(m + "g", l.mm_in, a.heads * a.vdim, W, d.mm_at.g);
            mat_slot(m + "i", l.mm_in, a.heads, W, d.mm_at.i);
            vec_slot(m + "i.b", l.mm_i_b, a.heads);
            mat_slot(m + "f", l.mm_in, a.heads, W, d.mm_at.f);
            vec_slot(m + "f.b", l.mm_f_b, a.heads);
            vec_slot(m + "norm", l.mm_norm, a.heads * a.vdim);
            mat_slot(m + "o", l.mm_o, W, a.heads * a.vdim, 0);
        } else {
            const LinearRecurrenceSpec &a = s.rec;
            linear(l.lr_in, 2 * d.width, wp_);
            linear(l.lr_gates, a.blocks * 2 * d.block_pad, d.block_pad);
            linear(l.lr_o, wp_, d.width);
            vec(l.lr_in_b, 2 * d.width);
            vec(l.conv_w, a.taps * d.width);
            vec(l.conv_b, d.width);
            vec(l.r_b, d.width);
            vec(l.i_b, d.width);
            vec(l.decay, d.width);
            mat_slot(m + "y", l.lr_in, a.width, W, d.width);
            vec_slot(m + "y.b", l.lr_in_b, a.width, 1, d.width);
            mat_slot(m + "x", l.lr_in, a.width, W, 0);
            vec_slot(m + "x.b", l.lr_in_b, a.width);
            vec_slot(m + "conv", l.conv_w, a.width, a.taps, d.width, Target::Taps);
            vec_slot(m + "conv.b", l.conv_b, a.width);
            mat_slot(m + "ra", l.lr_gates, a.width, d.block, 0, 1, d.block, 2 * d.block_pad);
            vec_slot(m + "ra.b", l.r_b, a.width);
            mat_slot(m + "ri", l.lr_gates, a.width, d.block, d.block_pad, 1, d.block, 2 * d.block_pad);
            vec_slot(m + "ri.b", l.i_b, a.width);
            vec_slot(m + "lam", l.decay, a.width, 1, 0, Target::ChannelDecay);
            mat_slot(m + "o", l.lr_o, W, a.width, 0);
        }
        if (!s.ff.width) continue;
        norms(p + "norm2", l.norm2, l.norm2b);
        const int parts = std::max(1, s.ff.experts);
        linear(l.gate_up, parts * 2 * d.ff, wp_);
        linear(l.down, parts * wp_, d.ff);
        for (int e = 0; e < parts; e++) {
            const std::string x = p + "mlp." + (s.ff.experts ? "e" + std::to_string(e) + "." : "");
            mat_slot(x + "gate", l.gate_up, s.ff.width, W, e * 2 * d.ff, 2);
            mat_slot(x + "up", l.gate_up, s.ff.width, W, e * 2 * d.ff + 1, 2);
            mat_slot(x + "down", l.down, W, s.ff.width, e * wp_);
        }
        if (s.ff.experts) {
            linear(l.router, d.router_n, wp_);
            mat_slot(p + "mlp.router", l.router, s.ff.experts, W, 0);
        }
    }
    vec(final_norm_, wp_);
    vec_slot("final.norm", final_norm_, W);
    linear(head_, cfg_.vocab, wp_);
    mat_slot("head", head_, cfg_.vocab, W, 0);
    if (!ok) *err = "out of memory for the weights";
    return ok ? HM_OK : HM_ERR_OOM;
}

int BlockModel::upload_matrix(const Target &t, const uint16_t *h_nk) {
    const size_t kp = t.lin->kp;
    auto rows_to = [&](const uint16_t *src, size_t src_cols, size_t cols, int rows, size_t dst_row, size_t dst_col) -> int {
        if (rows <= 0 || cols == 0) return HM_OK;
        HM_REQUIRE(ctx_, dst_row + (size_t)(rows - 1) * t.mult < (size_t)t.lin->np && dst_col + cols <= kp, "BlockModel: a weight does not fit its place");
        HM_HIP(ctx_, hipMemcpy2DAsync(t.lin->w.as<uint16_t>() + dst_row * kp + dst_col, (size_t)t.mult * kp * 2, src, src_cols * 2, cols * 2, rows,
                                      hipMemcpyHostToDevice, ctx_->stream));
        return HM_OK;
    };
    int rc = HM_OK;
    if (t.lin == &loop_in_) {
        const int W = cfg_.width;
        rc = rows_to(h_nk, 2 * W, W, W, 0, 0);
        if (rc == HM_OK) rc = rows_to(h_nk + W, 2 * W, W, W, 0, wp_);
    } else {
        // [dt | B | C]: the parts after the first start at padded rows of their own
        int part[4] = {0, t.rows, t.rows, t.rows}, at[3] = {0, 0, 0}, parts = 1;
        for (size_t i = 0; i < layers_.size(); i++)
            if (t.lin == &layers_[i].ss_x) {
                const SelectiveScanSpec &a = cfg_.layers[i].scan;
                part[1] = a.dt_rank;
                part[2] = a.dt_rank + a.state;
                at[1] = dims_[i].dt;
                at[2] = dims_[i].dt + dims_[i].state;
                parts = 3;
            }
        if (parts == 3) {
            for (int k = 0; k < 3 && rc == HM_OK; k++) rc = rows_to(h_nk + (size_t)part[k] * t.cols, t.cols, t.cols, part[k + 1] - part[k], at[k], 0);
        } else {
            for (int r = 0; r < t.rows && rc == HM_OK; r += t.group)
                rc = rows_to(h_nk + (size_t)r * t.cols, t.cols, t.cols, std::min(t.group, t.rows - r), (size_t)(r / t.group) * t.group_stride + t.off, 0);
        }
    }
    return rc == HM_OK ? hm_sync(ctx_) : rc;
}

int BlockModel::upload_vector(const Target &t, const float *h) {
    if (t.how == Target::Plain) return hm_upload(ctx_, t.vec->b.as<float>() + t.vec_off, h, (size_t)t.rows * 4);
    if (t.how == Target::Rows) {  // rows of a padded width (vec_off)
        HM_HIP(ctx_, hipMemcpy2DAsync(t.vec->b.ptr(), (size_t)t.vec_off * 4, h, (size_t)t.cols * 4, (size_t)t.cols * 4, t.rows, hipMemcpyHostToDevice,
                                      ctx_->stream));
        return hm_sync(ctx_);
    }
    std::vector<float> v((size_t)t.vec->n, 0.f);
    for (int r = 0; r < t.rows; r++)
        for (int c = 0; c < t.cols; c++) {
            const double x = h[(size_t)r * t.cols + c];
            if (t.how == Target::Residual) v[r] = (float)(x * cfg_.residual_mult);
            else if (t.how == Target::Taps) v[(size_t)c * t.vec_off + r] = (float)x;
            else if (t.how == Target::StateDecay) v[(size_t)r * t.vec_off + c] = (float)(-std::exp(x) * 1.4426950408889634074);
            else v[r] = (float)(-8.0 * (std::log1p(std::exp(-std::fabs(x))) + std::max(x, 0.0)));
        }
    return hm_upload(ctx_, t.vec->b.ptr(), v.data(), v.size() * 4);
}

int BlockModel::set_weight_nk(int slot, const void *h_data, size_t bytes) {
    if (slot < 0 || slot >= (int)infos_.size())
        return hm_set_error(ctx_, HM_ERR_INVALID, "weight slot %d out of range (have %zu)", slot, infos_.size());
    const WeightSlotInfo &info = infos_[slot];
    if (bytes != info.bytes)
        return hm_set_error(ctx_, HM_ERR_INVALID, "weight %s: expected %zu bytes, got %zu", info.name.c_str(), info.bytes, bytes);
    if (finalized_) return hm_set_error(ctx_, HM_ERR_STATE, "model already finalized");
    if (!h_data) return hm_set_error(ctx_, HM_ERR_INVALID, "weight %s: NULL data", info.name.c_str());
    const Target &t = targets_[slot];
    const int rc = t.lin ? upload_matrix(t, static_cast<const uint16_t *>(h_data)) : upload_vector(t, static_cast<const float *>(h_data));
    if (rc == HM_OK) weight_set_[slot] = true;
    return rc;
}

int BlockModel::set_weight(int slot, const void *h_data, size_t bytes) {
    if (slot < 0 || slot >= (int)infos_.size() || !targets_[slot].lin || !h_data || bytes != infos_[slot].bytes) return set_weight_nk(slot, h_data, bytes);
    // [K][N] -> [N][K]
    const int K = (int)infos_[slot].dim0, N = (int)infos_[slot].dim1;
    const uint16_t *src = static_cast<const uint16_t *>(h_data);
    std::vector<uint16_t> nk((size_t)K * N);
    for (int k = 0; k < K; k++)
        for (int n = 0; n < N; n++) nk[(size_t)n * K + k] = src[(size_t)k * N + n];
    return set_weight_nk(slot, nk.data(), bytes);
}

// ── finalize ─────────────────────────────────────────────────────────────────

int BlockModel::set_prefill_pieces(int n) {
    if (n < 1 || n > 3 || (compute_ == DType::F32 && n != 3))
        return hm_set_error(ctx_, HM_ERR_INVALID, "prefill pieces must be 1 to 3, with 32-bit compute 3");
    for (const BlockLayerSpec &l : cfg_.layers)
        if (n == 2 && l.ff.experts) return hm_set_error(ctx_, HM_ERR_INVALID, "prefill pieces of a mixture of experts must be 1 or 3");
    prefill_pieces_ = n;
    return HM_OK;
}

int BlockModel::set_prefill_chunk(int rows) {
    if (finalized_) return hm_set_error(ctx_, HM_ERR_STATE, "model already finalized");
    if (rows < 16 || rows > MAX_CHUNK) return hm_set_error(ctx_, HM_ERR_INVALID, "prefill chunk of %d rows (16 to %d)", rows, MAX_CHUNK);
    chunk_rows_ = rows;
    return HM_OK;
}

bool BlockModel::prefill_available() const {
    if (!finalized_) return false;
    for (size_t i = 0; i < cfg_.layers.size(); i++)
        if (cfg_.layers[i].mixer == MixerKind::LatentAttention && !dims_[i].head_k) return false;
    return true;
}

const char *BlockModel::prefill_needs() const { return "attention heads of at most 256 query and 256 value elements"; }

int BlockModel::finalize(int max_seq_len) {
    if (finalized_) return HM_OK;
    for (size_t i = 0; i < weight_set_.size(); i++)
        if (!weight_set_[i]) return hm_set_error(ctx_, HM_ERR_STATE, "missing weight: %s", infos_[i].name.c_str());
    if (max_seq_len <= 0) return hm_set_error(ctx_, HM_ERR_INVALID, "max_seq_len %d must be positive", max_seq_len);
    max_seq_len_ = max_seq_len;
    // rotation tables, one for every (dims, base) in use
    for (size_t i = 0; i < cfg_.layers.size(); i++) {
        layer_rope_.push_back(nullptr);
        if (cfg_.layers[i].mixer != MixerKind::LatentAttention) continue;
        const LatentAttentionSpec &a = cfg_.layers[i].attn;
        for (const auto &r : ropes_)
            if (r->dims == a.rot_dims && r->base == a.rot_base) layer_rope_.back() = r.get();
        if (!layer_rope_.back()) {
            std::unique_ptr<Rope> r(new Rope{a.rot_dims, a.rot_base, Buffer(), Buffer()});
            std::vector<float> c, s;
            precompute_rope_cos_sin(a.rot_dims, max_seq_len, a.rot_base, c, s);
            c.resize(std::max<size_t>(c.size(), 1));
            s.resize(c.size());
            r->cos = Buffer::alloc(ctx_, {(int64_t)c.size()}, DType::F32);
            r->sin = Buffer::alloc(ctx_, {(int64_t)s.size()}, DType::F32);
            if (!r->cos || !r->sin) return HM_ERR_OOM;
            int rc = hm_upload(ctx_, r->cos.ptr(), c.data(), c.size() * 4);
            if (rc == HM_OK) rc = hm_upload(ctx_, r->sin.ptr(), s.data(), s.size() * 4);
            if (rc != HM_OK) return rc;
            layer_rope_.back() = r.get();
            ropes_.push_back(std::move(r));
        }
        LatentShape &l = dims_[i].shape;
        // the rows a window still needs, and a chunk of new ones
        l.ring_rows = l.window ? (int)std::min<int64_t>(max_seq_len, (int64_t)l.window - 1 + chunk_rows_) : max_seq_len;
    }
    int rc = place_windows();
    if (rc == HM_OK && cfg_.position_waves) {
        std::vector<double> f((cfg_.width + 1) / 2);
        for (size_t i = 0; i < f.size(); i++) f[i] = std::pow(WAVE_BASE, -2.0 * (double)i / cfg_.width);
        wave_freq_ = Buffer::alloc(ctx_, {(int64_t)f.size() * 2}, DType::F32);
        if (!wave_freq_) return HM_ERR_OOM;
        rc = hm_upload(ctx_, wave_freq_.ptr(), f.data(), f.size() * sizeof(double));
    }
    if (rc == HM_OK) rc = alloc_scratch();
    if (rc == HM_OK) rc = emit_plan();
    if (rc == HM_OK) rc = plan_->prepare(std::max(max_seq_len, 16));
    if (rc == HM_OK) rc = plan_->ensure_kv_cache(max_seq_len_);
    if (rc != HM_OK) return rc;
    ids_view_ = Buffer::view(plan_->forced_ids(), (size_t)plan_->out_capacity() * 4, {1, DIM_DYNAMIC}, {1, 1}, DType::I64);
    finalized_ = true;
    return hm_sync(ctx_);
}

// Where the tokens of a window attention's cache sit: in a ring of the rows the widest of its readers still needs and a
// chunk of new ones, behind the kept tokens; in a row of their own each when that saves nothing.
int BlockModel::place_windows() {
    for (size_t i = 0; i < cfg_.layers.size(); i++) {
        const WindowAttentionSpec &a = cfg_.layers[i].wattn;
        if (cfg_.layers[i].mixer != MixerKind::WindowAttention || a.kv_from >= 0) continue;
        int64_t window = 0, keep = 0;
        bool all = false;
        auto reads = [&](size_t l) {
            return cfg_.layers[l].mixer == MixerKind::WindowAttention && (l == i || cfg_.layers[l].wattn.kv_from == (int)i);
        };
        for (size_t l = i; l < cfg_.layers.size(); l++) {
            if (!reads(l)) continue;
            const WindowAttentionSpec &r = cfg_.layers[l].wattn;
            all = all || !r.window;
            window = std::max<int64_t>(window, r.window);
            keep = std::max<int64_t>(keep, r.keep);
        }
        SlotMap map;
        map.ring = max_seq_len_;
        if (!all && keep + window - 1 + chunk_rows_ < max_seq_len_) {
            map.keep = (int)keep;
            map.ring = (int)(window - 1 + chunk_rows_);
        }
        for (size_t l = i; l < cfg_.layers.size(); l++)
            if (reads(l)) dims_[l].wshape.map = map;
    }
    return HM_OK;
}

int BlockModel::alloc_scratch() {
    step_ = std::make_shared<StepScratch>();
    StepScratch &s = *step_;
    int64_t d1 = 32, d2 = 32, act = 32, qlat = 32, part_o = 32, part_ml = 32;
    for (size_t i = 0; i < cfg_.layers.size(); i++) {
        const Dims &d = dims_[i];
        d1 = std::max<int64_t>({d1, d.down_n, 2 * d.inner, 2 * d.width, d.wa_n, d.mm_n});
        d2 = std::max<int64_t>({d2, d.uq_n, d.dt + 2 * d.state, d.router_n, (int64_t)d.mshape.heads * d.mshape.cols()});
        act = std::max<int64_t>({act, (int64_t)std::max(1, cfg_.layers[i].ff.top) * d.ff, d.gate, d.inner, d.width});
        if (cfg_.layers[i].mixer == MixerKind::WindowAttention) {
            const WindowAttentionShape &l = d.wshape;
            const int64_t splits = window_step_splits(window_step_span(l, max_seq_len_));
            part_o = std::max<int64_t>(part_o, splits * l.heads * l.width);
            part_ml = std::max<int64_t>(part_ml, splits * l.heads * 2);
        }
        if (cfg_.layers[i].mixer == MixerKind::LatentAttention) {
            const LatentShape &l = d.shape;
            const int span = l.window ? std::min(l.window, max_seq_len_) : max_seq_len_;
            const int64_t splits = latent_step_splits(l, span);
            qlat = std::max<int64_t>(qlat, (int64_t)l.heads * l.row_width());
            part_o = std::max<int64_t>(part_o, splits * l.heads * l.rank_pad);
            part_ml = std::max<int64_t>(part_ml, splits * l.heads * 2);
        }
    }
    s.cand_cap = 4096;
    // rows of activations keep zeros (or, shared between layers of different widths, old values) behind their true
    // width, where the weights are zero: they only have to be finite
    auto row = [&](Buffer &b, int64_t n) {
        b = Buffer::alloc(ctx_, {n}, DType::F32);
        return b && hm_fill_zero(ctx_, b.ptr(), b.bytes()) == HM_OK;
    };
    const bool ok = row(s.cat, 2 * wp_) && row(s.xa, wp_) && row(s.xb, wp_) && row(s.y, wp_) && row(s.d1, d1) && row(s.d2, d2) && row(s.act, act) &&
                    row(s.qlat, qlat) && row(s.part_o, part_o) && row(s.part_ml, part_ml) && row(s.normed, wp_) && row(s.cand_val, s.cand_cap) &&
                    row(s.cand_idx, s.cand_cap) && row(s.choice, EXPERTS_MAX_TOP);
    return ok ? HM_OK : HM_ERR_OOM;
}

// ── decode plan ──────────────────────────────────────────────────────────────

// The residual row is never written by a launch of its own inside a layer: a sublayer leaves its raw output in `y`,
// and the projection behind it forms x + norm_b(y) and its norm in its prologue (and hands the new x on).
int BlockModel::emit_plan() {
    std::vector<SlotDesc> descs;
    auto alloc = [&](int64_t n, DType dt, const char *name) -> size_t {
        descs.push_back(SlotDesc{{n}, dt, name});
        return descs.size() - 1;
    };
    const StepScratch &sb = *step_;
    auto row_slot = [&](const Buffer &b, const char *name) { return alloc(b.shape()[0], DType::F32, name); };
    // inputs: the forced ids and the activation rows, in the order of step_inputs
    const size_t ids = alloc(DIM_DYNAMIC, DType::I64, "input_ids");
    const size_t s_cat = row_slot(sb.cat, "x|x0"), s_xa = row_slot(sb.xa, "x_a"), s_xb = row_slot(sb.xb, "x_b"), s_y = row_slot(sb.y, "y"),
                 s_d1 = row_slot(sb.d1, "proj_1"), s_d2 = row_slot(sb.d2, "proj_2"), s_act = row_slot(sb.act, "act"), s_ql = row_slot(sb.qlat, "q_latent"),
                 s_normed = row_slot(sb.normed, "normed");
    const std::vector<size_t> input_slots{ids, s_cat, s_xa, s_xb, s_y, s_d1, s_d2, s_act, s_ql, s_normed};
    const size_t s_logits = alloc(cfg_.vocab, DType::F32, "logits");

    std::vector<CompiledKernel> kernels;
    std::vector<KernelStep> steps;
    auto step = [&](const std::string &ops, const std::string &name, double bytes, double bytes_per_row, std::vector<size_t> in, std::vector<size_t> out,
                    std::function<int(const StepContext &)> fn, bool moves_cursor = false) {
        CompiledKernel k;
        k.ops_label = ops;
        DeviceLaunch l;
        l.name = name;
        l.bytes_fixed = bytes;
        l.bytes_per_kv_row = bytes_per_row;
        l.moves_cursor = moves_cursor;
        l.fn = std::move(fn);
        k.launches.push_back(std::move(l));
        kernels.push_back(std::move(k));
        steps.push_back(KernelStep::kernel(kernels.size() - 1, std::move(in), std::move(out)));
    };
    const float eps = (float)cfg_.eps, escale = (float)cfg_.embed_scale;
    const int W = cfg_.width, wp = wp_, vocab = cfg_.vocab;

    const float *table = embed_.ptr();
    const PositionWaves wave = waves();
    step("Embed", "embed", wp * 12.0, 0, {ids}, {s_cat}, [=](const StepContext &sc) -> int {
        float *cat = sc.pool[s_cat]->as<float>();
        return embed_step_scaled_launch(sc.ctx, sc.plan->state(), sc.plan->forced_ids(), table, cat, cat + wp, vocab, wp, escale, wave);
    });

    size_t cur = s_cat;             // slot of the residual (its first wp elements)
    const Vec *pending = nullptr;   // y waits to be added behind this norm
    // One projection of the row in `in`; of the residual with what is pending, and through norm_w if there is one.
    auto gemv = [&](const std::string &name, const Linear &lin, size_t in, size_t out, const float *norm_w, int epi, const float *bias = nullptr,
                    std::function<void(const StepContext &, GemvArgs &)> more = nullptr) {
        const size_t src = in;
        size_t next = in;
        const float *post = nullptr;
        if (in == cur && pending) {
            post = pending->ptr();
            next = cur == s_xa ? s_xb : s_xa;
        }
        const Linear *lp = &lin;
        const bool to_act = epi == GEMV_EPI_SILU_MUL_PAIRS;
        std::vector<size_t> ins{src};
        std::vector<size_t> outs{out};
        if (post) {
            ins.push_back(s_y);
            outs.push_back(next);
        }
        const double bytes = 2.0 * lin.np * lin.kp + 4.0 * lin.kp * (post ? 5 : norm_w ? 2 : 1) + 4.0 * lin.np / (to_act ? 2 : 1);
        step("Project", name, bytes, 0, ins, outs, [=](const StepContext &sc) -> int {
            GemvArgs g;
            g.x = sc.pool[src]->as<float>();
            g.w = lp->ptr();
            g.K = lp->kp;
            g.N = lp->np;
            g.out = sc.pool[out]->as<float>();
            g.bias = bias;
            if (norm_w || post) {
                g.norm_w = norm_w;
                g.norm_dim = W;
                g.eps = eps;
            }
            if (post) {
                g.prologue_residual = sc.pool[s_y]->as<float>();
                g.post_norm_w = post;
                g.resid_out = sc.pool[next]->as<float>();
            }
            if (more) more(sc, g);
            return gemv_bf16_nk_launch(sc.ctx, g, 1, epi);
        });
        if (post) {
            cur = next;
            pending = nullptr;
        }
    };
    // x + norm_b(y) as a row of its own, or straight through a norm
    auto settle = [&](const std::string &name, size_t out, const float *norm_w) {
        const size_t src = cur;
        const Vec *post = pending;
        step("Norm", name, wp * 16.0, 0, post ? std::vector<size_t>{src, s_y} : std::vector<size_t>{src}, {out}, [=](const StepContext &sc) -> int {
            RowNormArgs r;
            r.x = sc.pool[src]->as<float>();
            if (post) {
                r.y = sc.pool[s_y]->as<float>();
                r.y_w = post->ptr();
            }
            r.w = norm_w;
            r.out = sc.pool[out]->as<float>();
            r.rows = 1;
            r.dim = wp;
            r.norm_dim = W;
            r.eps = eps;
            return row_norm_launch(sc.ctx, r);
        });
        pending = nullptr;
        cur = out;
    };

    std::vector<StateSpec> specs;
    for (size_t run = 0; run < runs_.size(); run++) {
        const int li = runs_[run].layer;
        const BlockLayerSpec &s = cfg_.layers[li];
        const Dims &d = dims_[li];
        const LayerWeights &l = layers_[li];
        const LayerWeights *lw = &l;
        const float *norm1 = cfg_.pre_norms ? l.norm1.ptr() : nullptr;
        StateSpec st;
        if (runs_[run].begins_pass) {
            if (cur != s_cat || pending) settle("row_norm[pass]", s_cat, nullptr);
            gemv("gemv[loop_in]", loop_in_, s_cat, s_xa, nullptr, GEMV_EPI_NONE);
            cur = s_xa;
        }
        const Linear *out_w = nullptr;
        if (s.mixer == MixerKind::LatentAttention) {
            const LatentAttentionSpec &a = s.attn;
            gemv("gemv[latent_down]", l.la_down, cur, s_d1, norm1, GEMV_EPI_NONE);
            const int q_rank = a.q_rank;
            const float *qn = l.q_norm.ptr();
            // (its own norm, of the query latent: nothing pending is involved)
            {
                const Linear *lp = &l.la_uq;
                step("Project", "gemv[latent_uq]", 2.0 * lp->np * lp->kp + 8.0 * lp->kp + 4.0 * lp->np, 0, {s_d1}, {s_d2}, [=](const StepContext &sc) -> int {
                    GemvArgs g;
                    g.x = sc.pool[s_d1]->as<float>();
                    g.w = lp->ptr();
                    g.K = lp->kp;
                    g.N = lp->np;
                    g.out = sc.pool[s_d2]->as<float>();
                    g.norm_w = qn;
                    g.norm_dim = q_rank;
                    g.eps = eps;
                    return gemv_bf16_nk_launch(sc.ctx, g, 1, GEMV_EPI_NONE);
                });
            }
            st.window_rows = d.shape.ring_rows;
            st.window_row_bytes = (int64_t)d.shape.row_elems() * 2;
            const float *cos_tab = layer_rope_[li]->cos.as<float>(), *sin_tab = layer_rope_[li]->sin.as<float>();
            const LatentShape shape = d.shape;
            const int q_at = d.q_rank, g_at = d.q_rank + d.kv, v_at = d.v_at;
            const int span = shape.window ? std::min(shape.window, max_seq_len_) : max_seq_len_;
            const float scale = (float)a.scale;
            std::shared_ptr<StepScratch> scr = step_;
            auto args = [=](const StepContext &sc) {
                LatentStepArgs x;
                x.s = shape;
                const float *d1 = sc.pool[s_d1]->as<float>();
                x.q = sc.pool[s_d2]->as<float>();
                x.kv = d1 + q_at;
                x.gate = d1 + g_at;
                x.kv_norm = lw->kv_norm.ptr();
                x.uk = lw->la_ukv.ptr();
                x.uv = lw->la_ukv.ptr(v_at);
                x.cos_tab = cos_tab;
                x.sin_tab = sin_tab;
                x.eps = eps;
                x.scale = scale;
                x.ring = sc.plan->state_cache()->window((int)run);
                x.q_latent = sc.pool[s_ql]->as<float>();
                x.part_o = scr->part_o.as<float>();
                x.part_ml = scr->part_ml.as<float>();
                x.out = sc.pool[s_act]->as<float>();
                x.cursor = sc.plan->state();
                x.span = span;
                return x;
            };
            const double row_b = shape.row_elems() * 2.0;
            step("LatentAttn", "latent_prep", 2.0 * a.heads * a.dim * shape.rank_pad + 4.0 * (d.uq_n + a.heads * shape.row_width()) + row_b, 0, {s_d1, s_d2}, {s_ql},
                 [=](const StepContext &sc) -> int { return latent_step_prep_launch(sc.ctx, args(sc)); });
            step("LatentAttn", "latent_attn", 4.0 * a.heads * shape.row_width() + row_b * span, 0, {s_ql}, {s_act},
                 [=](const StepContext &sc) -> int { return latent_step_attn_launch(sc.ctx, args(sc)); });
            step("LatentAttn", "latent_fold", 2.0 * a.heads * a.vdim * shape.rank_pad + 4.0 * latent_step_splits(shape, span) * a.heads * shape.rank_pad, 0, {s_d1}, {s_act},
                 [=](const StepContext &sc) -> int { return latent_step_fold_launch(sc.ctx, args(sc)); });
            out_w = &l.la_o;
        } else if (s.mixer == MixerKind::SelectiveScan) {
            st.tap_rows = s.scan.taps;
            st.tap_width = d.inner;
            st.state_floats = (int64_t)d.inner * d.state;
            const int taps = s.scan.taps, inner = d.inner, dt = d.dt, state = d.state;
            gemv("gemv[scan_in+conv]", l.ss_in, cur, s_d1, norm1, GEMV_EPI_CONV, nullptr, [=](const StepContext &sc, GemvArgs &g) {
                g.conv.rows = inner;
                g.conv.taps = taps;
                g.conv.w = lw->conv_w.ptr();
                g.conv.b = lw->conv_b.ptr();
                g.conv.ring = sc.plan->state_cache()->taps((int)run);
                g.conv.state = sc.plan->state();
                g.conv.silu = true;
            });
            gemv("gemv[scan_x]", l.ss_x, s_d1, s_d2, nullptr, GEMV_EPI_NONE);
            step("Scan", "selective_step", 2.0 * inner * dt + 4.0 * inner * (3.0 * state + 5) + 4.0 * (dt + 2 * state), 0, {s_d1, s_d2}, {s_act},
                 [=](const StepContext &sc) -> int {
                     SelectiveStepArgs x;
                     x.xz = sc.pool[s_d1]->as<float>();
                     x.p = sc.pool[s_d2]->as<float>();
                     x.dt_w = lw->ss_dt.ptr();
                     x.dt_b = lw->dt_b.ptr();
                     x.a_log2 = lw->a_log2.ptr();
                     x.d = lw->d.ptr();
                     x.state = sc.plan->state_cache()->state((int)run);
                     x.y = sc.pool[s_act]->as<float>();
                     x.cursor = sc.plan->state();
                     x.inner = inner;
                     x.dt_pad = dt;
                     x.state_pad = state;
                     return selective_step_launch(sc.ctx, x);
                 });
            out_w = &l.ss_o;
        } else if (s.mixer == MixerKind::WindowAttention) {
            const WindowAttentionSpec &a = s.wattn;
            const WindowAttentionShape shape = d.wshape;
            const bool own = a.kv_from < 0;
            if (own) {
                st.window_rows = shape.map.slots();
                st.window_row_bytes = (int64_t)shape.row_bytes();
            }
            gemv(own ? "gemv[qkv]" : "gemv[q]", l.wa_in, cur, s_d1, norm1, GEMV_EPI_NONE);
            const int k_at = d.k_at, v_at = d.v_at, span = window_step_span(shape, max_seq_len_), cache_run = cache_run_[run];
            const float scale = (float)a.scale;
            std::shared_ptr<StepScratch> scr = step_;
            auto args = [=](const StepContext &sc) {
                WindowStepArgs x;
                x.s = shape;
                x.q = sc.pool[s_d1]->as<float>();
                x.k = own ? x.q + k_at : nullptr;
                x.v = own ? x.q + v_at : nullptr;
                x.q_norm = lw->head_q_norm.ptr();
                x.k_norm = own ? lw->head_k_norm.ptr() : nullptr;
                x.eps = eps;
                x.scale = scale;
                x.cache = sc.plan->state_cache()->window(cache_run);
                x.part_o = scr->part_o.as<float>();
                x.part_ml = scr->part_ml.as<float>();
                x.out = sc.pool[s_act]->as<float>();
                x.cursor = sc.plan->state();
                x.span = span;
                return x;
            };
            step("WindowAttn", "window_attn", 4.0 * d.wa_n + (double)shape.row_bytes() * span, 0, {s_d1}, {s_act},
                 [=](const StepContext &sc) -> int { return window_step_attn_launch(sc.ctx, args(sc)); });
            step("WindowAttn", "window_fold", 4.0 * window_step_splits(span) * a.heads * (shape.width + 2) + 4.0 * a.heads * a.vdim, 0, {s_d1}, {s_act},
                 [=](const StepContext &sc) -> int { return window_step_fold_launch(sc.ctx, args(sc)); });
            out_w = &l.wa_o;
        } else if (s.mixer == MixerKind::MatrixMemory) {
            const MatrixMemoryShape shape = d.mshape;
            const MatrixMemoryColumns at = d.mm_at;
            st.state_floats = (int64_t)shape.state_floats();
            gemv("gemv[memory_in]", l.mm_in, cur, s_d1, norm1, GEMV_EPI_NONE);
            auto args = [=](const StepContext &sc) {
                MatrixMemoryStepArgs x;
                x.s = shape;
                x.at = at;
                x.row = sc.pool[s_d1]->as<float>();
                x.i_bias = lw->mm_i_b.ptr();
                x.f_bias = lw->mm_f_b.ptr();
                x.state = sc.plan->state_cache()->state((int)run);
                x.raw = sc.pool[s_d2]->as<float>();
                x.norm = lw->mm_norm.ptr();
                x.eps = eps;
                x.out = sc.pool[s_act]->as<float>();
                x.cursor = sc.plan->state();
                return x;
            };
            step("Memory", "memory_step", 8.0 * shape.memory_floats() + 4.0 * d.mm_n, 0, {s_d1}, {s_d2},
                 [=](const StepContext &sc) -> int { return matrix_memory_step_launch(sc.ctx, args(sc)); });
            step("Memory", "memory_out", 16.0 * shape.heads * shape.vdim, 0, {s_d1, s_d2}, {s_act},
                 [=](const StepContext &sc) -> int { return matrix_memory_step_out_launch(sc.ctx, args(sc)); });
            out_w = &l.mm_o;
        } else {
            st.tap_rows = s.rec.taps;
            st.tap_width = d.width;
            st.state_floats = d.width;
            const int taps = s.rec.taps, width = d.width, channels = s.rec.width, block = d.block, block_pad = d.block_pad;
            gemv("gemv[recurrence_in+conv]", l.lr_in, cur, s_d1, norm1, GEMV_EPI_CONV, l.lr_in_b.ptr(), [=](const StepContext &sc, GemvArgs &g) {
                g.conv.rows = width;
                g.conv.taps = taps;
                g.conv.w = lw->conv_w.ptr();
                g.conv.b = lw->conv_b.ptr();
                g.conv.ring = sc.plan->state_cache()->taps((int)run);
                g.conv.state = sc.plan->state();
                g.conv.gelu_from = width;
            });
            step("Recurrence", "recurrence_step", 4.0 * width * block_pad + 4.0 * width * 8, 0, {s_d1}, {s_act}, [=](const StepContext &sc) -> int {
                LinearRecurrenceStepArgs x;
                x.uy = sc.pool[s_d1]->as<float>();
                x.gate_w = lw->lr_gates.ptr();
                x.r_bias = lw->r_b.ptr();
                x.i_bias = lw->i_b.ptr();
                x.decay = lw->decay.ptr();
                x.state = sc.plan->state_cache()->state((int)run);
                x.out = sc.pool[s_act]->as<float>();
                x.cursor = sc.plan->state();
                x.channels = channels;
                x.width = width;
                x.block_width = block;
                x.block_pad = block_pad;
                return linear_recurrence_step_launch(sc.ctx, x);
            });
            out_w = &l.lr_o;
        }
        specs.push_back(st);
        gemv("gemv[mixer_out]", *out_w, s_act, s_y, nullptr, GEMV_EPI_NONE);
        pending = &l.norm1b;
        if (!s.ff.width) continue;
        const float *norm2 = cfg_.pre_norms ? l.norm2.ptr() : nullptr;
        const GatedAct gated = s.ff.act;
        if (!s.ff.experts) {
            gemv(gated.kind == GatedAct::Silu ? "gemv[gate_up+silu]" : "gemv[gate_up+clamped]", l.gate_up, cur, s_act, norm2, GEMV_EPI_SILU_MUL_PAIRS, nullptr,
                 [=](const StepContext &, GemvArgs &g) { g.act = gated; });
            gemv("gemv[down]", l.down, s_act, s_y, nullptr, GEMV_EPI_NONE);
        } else {
            gemv("gemv[router]", l.router, cur, s_d2, nullptr, GEMV_EPI_NONE);
            const size_t x_slot = cur;
            const int experts = s.ff.experts, top = s.ff.top, ff = d.ff;
            std::shared_ptr<StepScratch> scr = step_;
            auto args = [=](const StepContext &sc) {
                ExpertsStepArgs x;
                x.x = sc.pool[x_slot]->as<float>();
                x.logits = sc.pool[s_d2]->as<float>();
                x.gate_up = lw->gate_up.ptr();
                x.down = lw->down.ptr();
                x.experts = experts;
                x.top = top;
                x.K = wp;
                x.ff = ff;
                x.width = wp;
                x.act = gated;
                x.choice = scr->choice.as<int>();
                x.hidden = sc.pool[s_act]->as<float>();
                x.y = sc.pool[s_y]->as<float>();
                return x;
            };
            step("Experts", "experts_up", top * (4.0 * ff * wp + 4.0 * ff) + 4.0 * (wp + experts), 0, {x_slot, s_d2}, {s_act},
                 [=](const StepContext &sc) -> int { return experts_step_up_launch(sc.ctx, args(sc)); });
            step("Experts", "experts_down", top * (2.0 * ff * wp + 4.0 * ff) + 4.0 * wp, 0, {s_act}, {s_y},
                 [=](const StepContext &sc) -> int { return experts_step_down_launch(sc.ctx, args(sc)); });
        }
        pending = &l.norm2b;
    }
    settle("row_norm[final]", s_normed, final_norm_.ptr());
    std::shared_ptr<StepScratch> scr = step_;
    const Linear *head = &head_;
    step("LMHead", "gemv[head+argmax]", 2.0 * vocab * wp + 4.0 * wp + 4.0 * vocab, 0, {s_normed}, {s_logits}, [=](const StepContext &sc) -> int {
        GemvArgs g;
        g.x = sc.pool[s_normed]->as<float>();
        g.w = head->ptr();
        g.out = sc.pool[s_logits]->as<float>();
        g.K = head->kp;
        g.N = vocab;
        g.argmax_val = scr->cand_val.as<float>();
        g.argmax_idx = scr->cand_idx.as<int>();
        g.argmax_cap = scr->cand_cap;
        return gemv_bf16_nk_launch(sc.ctx, g, 1, GEMV_EPI_ARGMAX);
    });
    step("LMHead", "finish_step", 64, 0, {s_logits}, {s_logits}, [=](const StepContext &sc) -> int {
        const int ncand = std::min(gemv_bf16_nk_grid(sc.ctx, vocab, 4), scr->cand_cap);
        return finish_step_launch(sc.ctx, sc.plan->state(), scr->cand_val.as<float>(), scr->cand_idx.as<int>(), ncand, sc.plan->out_tokens(),
                                  sc.plan->out_capacity());
    }, true);
    const size_t num_slots = descs.size();
    plan_.reset(new ExecutionPlan(ctx_, std::move(kernels), std::move(steps), num_slots, input_slots, {}, {s_logits}, std::move(descs)));
    plan_->set_state_specs(specs);
    return HM_OK;
}

int BlockModel::step_inputs(std::vector<Buffer *> &inputs) {
    StepScratch &s = *step_;
    inputs = {&ids_view_, &s.cat, &s.xa, &s.xb, &s.y, &s.d1, &s.d2, &s.act, &s.qlat, &s.normed};
    return HM_OK;
}

// ── positions that can be returned to ────────────────────────────────────────

int BlockModel::mark_position() { return plan_->state_cache()->mark(); }

int BlockModel::rewind_to_mark(int mark_len, const std::vector<int32_t> &kept) {
    // recurrent state does not run backwards: back to the mark, and the steps that stay once more
    int rc = plan_->state_cache()->restore_mark();
    if (rc != HM_OK) return rc;
    plan_->cache()->reset(mark_len);
    if ((rc = plan_->arm(kept.data(), (int)kept.size())) != HM_OK) return rc;
    std::vector<Buffer *> inputs;
    step_inputs(inputs);
    for (size_t i = 0; i < kept.size() && rc == HM_OK; i++) rc = plan_->run_kv(inputs, weight_bufs_, max_seq_len_);
    return rc;
}

// ── prompt pass ──────────────────────────────────────────────────────────────

int BlockModel::prepare_prefill() {
    PrefillScratch &p = pf_;
    if (p.rows) return HM_OK;
    const int64_t rows = std::min(chunk_rows_, max_seq_len_);
    // A product is cut into K slices only while its 128 x 128 tiles times the slices stay within the CUs, so this
    // holds the slices of a product of any width up to n.
    auto sliced = [&](int64_t n) { return std::max<int64_t>(rows * n, (int64_t)ctx_->num_cus * 128 * 128); };
    int64_t d1 = wp_, d2 = 32, d3 = 32, f1 = 32, f2 = 32, f3 = 32, split = 2 * wp_, lat = 32, kvf = 32, kws = 32, vws = 32;
    int64_t mm_qk = 32, mm_heads = 1, mm_ahead = 32, mm_values = 32, experts = 1, top = 1;
    for (size_t i = 0; i < cfg_.layers.size(); i++) {
        const BlockLayerSpec &s = cfg_.layers[i];
        const Dims &d = dims_[i];
        const int64_t blocks = s.mixer == MixerKind::LinearRecurrence ? s.rec.blocks : 0;
        const int64_t l_top = std::max(1, s.ff.top);
        d1 = std::max<int64_t>({d1, d.down_n, 2 * d.inner, 2 * d.width, 2 * d.ff * l_top, d.wa_n, d.mm_n});
        d2 = std::max<int64_t>({d2, d.uq_n, d.dt + 2 * d.state, d.router_n});
        d3 = std::max<int64_t>({d3, d.inner, blocks * 2 * d.block_pad, (int64_t)d.mshape.heads * d.mshape.cols()});
        f1 = std::max<int64_t>({f1, d.inner, d.width, (int64_t)d.shape.heads * d.head_k, (int64_t)d.wshape.heads * d.wshape.width});
        f2 = std::max<int64_t>(f2, d.dt + 2 * d.state);
        f3 = std::max<int64_t>({f3, d.inner, d.width});
        split = std::max<int64_t>({split, d.q_rank, d.gate, d.inner, d.width, d.ff * l_top, blocks * d.block_pad, d.dt});
        if (s.mixer == MixerKind::MatrixMemory) {
            mm_qk = std::max<int64_t>(mm_qk, (int64_t)d.mshape.heads * d.mshape.dim_pad);
            mm_heads = std::max<int64_t>(mm_heads, d.mshape.heads);
            const int mp = compute_ == DType::F32 ? 3 : 1;
            mm_ahead = std::max<int64_t>(mm_ahead, matrix_memory_ahead_bytes(d.mshape, mp, (int)rows) / 2);
            mm_values = std::max<int64_t>(mm_values, matrix_memory_value_bytes(d.mshape, mp, (int)rows) / 2);
            f1 = std::max<int64_t>(f1, wp_);
        }
        experts = std::max<int64_t>(experts, s.ff.experts);
        top = std::max(top, l_top);
        if (s.mixer == MixerKind::LatentAttention) {
            const int64_t cap = d.shape.ring_rows;
            lat = std::max<int64_t>(lat, cap * d.shape.pieces * d.shape.rank_pad);
            kvf = std::max<int64_t>(kvf, cap * d.ukv_n);
            kws = std::max<int64_t>(kws, cap * d.shape.pieces * d.shape.heads * d.head_k);
            vws = std::max<int64_t>(vws, cap * d.shape.pieces * d.shape.heads * d.head_v);
        }
    }
    const int64_t mm_line = (rows + MM_CHUNK - 1) / MM_CHUNK * MM_CHUNK;
    // zeroed once: columns behind the true widths only have to be finite (their weights are zero)
    auto make = [&](Buffer &b, int64_t n, DType t) {
        b = Buffer::alloc(ctx_, {(n + 1) / 2 * 2}, t);
        return b && hm_fill_zero(ctx_, b.ptr(), b.bytes()) == HM_OK;
    };
    const bool ok = make(p.ids, rows, DType::F32) && make(p.x, rows * wp_, DType::F32) && make(p.x0, rows * wp_, DType::F32) &&
                    make(p.y, std::max(sliced(wp_), rows * top * wp_), DType::F32) && make(p.d1, sliced(d1), DType::F32) && make(p.d2, sliced(d2), DType::F32) &&
                    make(p.d3, sliced(d3), DType::F32) && make(p.f1, rows * f1, DType::F32) && make(p.f2, rows * f2, DType::F32) && make(p.f3, rows * f3, DType::F32) &&
                    make(p.split_a, rows * 3 * split, DType::BF16) && make(p.split_b, rows * 3 * split, DType::BF16) && make(p.lat, lat, DType::BF16) &&
                    make(p.kvf, kvf, DType::F32) && make(p.kws, kws, DType::BF16) && make(p.vws, vws, DType::BF16) && make(p.mm_q, rows * 3 * mm_qk, DType::BF16) &&
                    make(p.mm_k, rows * 3 * mm_qk, DType::BF16) && make(p.mm_log_w, 2 * mm_heads * mm_line * 2, DType::F32) &&
                    make(p.mm_weights, 3 * mm_heads * mm_line, DType::F32) && make(p.mm_ahead, mm_ahead, DType::BF16) && make(p.mm_values, mm_values, DType::BF16) && make(p.mm_gates, rows * 2 * mm_heads, DType::F32) && make(p.mm_decay, mm_heads * mm_line / MM_CHUNK, DType::F32) &&
                    make(p.choice, rows * top, DType::F32) && make(p.choice_weight, rows * top, DType::F32) && make(p.expert_list, rows * experts, DType::F32) &&
                    make(p.expert_count, experts, DType::F32);
    if (!ok) return HM_ERR_OOM;
    p.rows = (int)rows;
    return HM_OK;
}

// The mixer of one layer run on the normed rows in split_a; its raw output lands in y (as *y_parts K slices).
int BlockModel::prefill_mixer(int run, int layer, const float *cos_tab, const float *sin_tab, int n, int past, int *y_parts) {
    PrefillScratch &p = pf_;
    const BlockLayerSpec &s = cfg_.layers[layer];
    const Dims &d = dims_[layer];
    const LayerWeights &l = layers_[layer];
    StateCache *cache = plan_->state_cache();
    const int np = prefill_pieces_, MP = PrefillScratch::MAX_PARTS;
    const float eps = (float)cfg_.eps;
    uint16_t *sa = p.split_a.as<uint16_t>(), *sb = p.split_b.as<uint16_t>();
    float *d1 = p.d1.as<float>(), *d2 = p.d2.as<float>(), *d3 = p.d3.as<float>(), *f1 = p.f1.as<float>(), *f2 = p.f2.as<float>();
    // out (as K slices) = split x W^T
    auto gemm = [&](const Linear &w, const uint16_t *split, int pieces, float *out, RowSource *src) -> int {
        int parts = 1;
        const int rc = gemm_split_nk(ctx_, split, pieces, w.ptr(), out, n, w.kp, w.np, MP, &parts);
        *src = RowSource{out, w.np, parts, (size_t)n * w.np, nullptr};
        return rc;
    };
    int rc;
    RowSource in, second;
    if (s.mixer == MixerKind::WindowAttention) return prefill_window_attention(run, layer, n, past, y_parts);
    if (s.mixer == MixerKind::MatrixMemory) return prefill_matrix_memory(run, layer, cfg_.pre_norms ? p.f1.as<float>() : p.x.as<float>(), n, past, y_parts);
    if (s.mixer == MixerKind::LatentAttention) {
        const LatentAttentionSpec &a = s.attn;
        const LatentShape &sh = d.shape;
        uint16_t *ring = cache->window(run);
        if ((rc = gemm(l.la_down, sa, np, d1, &in)) != HM_OK) return rc;
        LatentRowsArgs r;
        r.s = sh;
        r.down = in;
        r.q_rank = a.q_rank;
        r.q_rank_pad = d.q_rank;
        r.q_norm = l.q_norm.ptr();
        r.kv_norm = l.kv_norm.ptr();
        r.cos_tab = cos_tab;
        r.sin_tab = sin_tab;
        r.eps = eps;
        r.q_split = sb;
        r.q_pieces = np;
        r.ring = ring;
        r.n = n;
        r.past = past;
        if ((rc = latent_rows_launch(ctx_, r)) != HM_OK) return rc;
        if ((rc = gemm(l.la_uq, sb, np, d2, &second)) != HM_OK) return rc;
        if ((rc = latent_q_rows_launch(ctx_, sh, second, cos_tab, sin_tab, f1, d.head_k, n, past)) != HM_OK) return rc;
        // keys and values of every visible row
        const int first = sh.window ? std::max(0, past - (sh.window - 1)) : 0, rows = past + n - first;
        if ((rc = latent_gather_launch(ctx_, sh, ring, p.lat.as<uint16_t>(), first, rows)) != HM_OK) return rc;
        if ((rc = gemm_split_nk(ctx_, p.lat.as<uint16_t>(), sh.pieces, l.la_ukv.ptr(), p.kvf.as<float>(), rows, sh.rank_pad, d.ukv_n)) != HM_OK) return rc;
        const RowSource kv{p.kvf.as<float>(), d.ukv_n, 1, 0, nullptr};
        rc = latent_kv_rows_launch(ctx_, sh, kv, d.v_at, ring, p.kws.as<uint16_t>(), p.vws.as<uint16_t>(), d.head_k, d.head_v, rows, first, rows);
        if (rc != HM_OK) return rc;
        PrefillAttnArgs at;
        at.q = f1;
        at.ldq = a.heads * d.head_k;
        at.kcache = p.kws.as<uint16_t>();
        at.vcache = p.vws.as<uint16_t>();
        at.out_split = sa;
        at.S = n;
        at.H = at.kvh = a.heads;
        at.hd = d.head_k;
        at.hdv = d.head_v;
        at.kv_pieces = sh.pieces;
        at.k_plane = (size_t)a.heads * rows * d.head_k;
        at.v_plane = (size_t)a.heads * rows * d.head_v;
        at.max_len = rows;
        at.past = past - first;
        at.scale = (float)a.scale;
        at.window = sh.window;
        at.vdim = a.vdim;
        at.out_cols = d.gate;
        at.out_pieces = np;
        at.gate = d1 + d.q_rank + d.kv;
        at.gate_ld = in.ld;
        at.gate_parts = in.parts;
        at.gate_stride = in.stride;
        if ((rc = prefill_attn_launch(ctx_, at)) != HM_OK) return rc;
        return gemm_split_nk(ctx_, sa, np, l.la_o.ptr(), p.y.as<float>(), n, l.la_o.kp, wp_, MP, y_parts);
    }
    if (s.mixer == MixerKind::SelectiveScan) {
        if ((rc = gemm(l.ss_in, sa, np, d1, &in)) != HM_OK) return rc;
        ConvRowsArgs c;
        c.in = in;
        c.ring = TapRing{cache->taps(run), s.scan.taps, d.inner};
        c.w = l.conv_w.ptr();
        c.b = l.conv_b.ptr();
        c.silu = true;
        c.out = f1;
        c.out_split = sb;
        c.pieces = np;
        c.channels = c.block_width = c.block_pad = d.inner;
        c.side = p.f3.as<float>();
        c.side_cols = d.inner;
        c.side_act = ConvRowsArgs::Silu;
        c.n = n;
        c.past = past;
        if ((rc = conv_rows_launch(ctx_, c)) != HM_OK) return rc;
        if ((rc = gemm(l.ss_x, sb, np, d2, &second)) != HM_OK) return rc;
        // [dt | B | C] as one f32 row; the step sizes keep all their bits on the way through their matrix
        const int pw = d.dt + 2 * d.state;
        if ((rc = sum_parts_launch(ctx_, d2, second.ld, second.parts, second.stride, f2, n, pw, sb, d.dt)) != HM_OK) return rc;
        if ((rc = gemm_split_nk(ctx_, sb, 3, l.ss_dt.ptr(), d3, n, l.ss_dt.kp, l.ss_dt.np)) != HM_OK) return rc;
        SelectiveScanArgs x;
        x.x = f1;
        x.dt = d3;
        x.dt_bias = l.dt_b.ptr();
        x.b = f2 + d.dt;
        x.c = f2 + d.dt + d.state;
        x.bc_ld = pw;
        x.a_log2 = l.a_log2.ptr();
        x.d = l.d.ptr();
        x.z = c.side;
        x.state = cache->state(run);
        x.out_split = sa;
        x.pieces = np;
        x.conv_in = in;
        x.ring = c.ring;
        x.n = n;
        x.inner = d.inner;
        x.state_pad = d.state;
        x.past = past;
        if ((rc = selective_scan_launch(ctx_, x)) != HM_OK) return rc;
        return gemm_split_nk(ctx_, sa, np, l.ss_o.ptr(), p.y.as<float>(), n, l.ss_o.kp, wp_, MP, y_parts);
    }
    if ((rc = gemm(l.lr_in, sa, np, d1, &in)) != HM_OK) return rc;
    RowSource xin = in;
    xin.bias = l.lr_in_b.ptr();
    ConvRowsArgs c;
    c.in = xin;
    c.ring = TapRing{cache->taps(run), s.rec.taps, d.width};
    c.w = l.conv_w.ptr();
    c.b = l.conv_b.ptr();
    c.out = f1;
    c.out_split = sb;
    c.pieces = 3;  // gates keep all the bits of their inputs
    c.channels = s.rec.width;
    c.block_width = d.block;
    c.block_pad = d.block_pad;
    c.side = p.f3.as<float>();
    c.side_cols = d.width;
    c.side_act = ConvRowsArgs::Gelu;
    c.n = n;
    c.past = past;
    if ((rc = conv_rows_launch(ctx_, c)) != HM_OK) return rc;
    const int bn = 2 * d.block_pad;
    rc = gemm_pieces_batched(ctx_, sb, (size_t)n * 3 * d.block_pad, l.lr_gates.ptr(), (size_t)bn * d.block_pad, d3, bn, s.rec.blocks, n, d.block_pad, bn,
                             s.rec.blocks * bn);
    if (rc != HM_OK) return rc;
    LinearRecurrenceArgs x;
    x.u = f1;
    x.gates = d3;
    x.r_bias = l.r_b.ptr();
    x.i_bias = l.i_b.ptr();
    x.decay = l.decay.ptr();
    x.y = c.side;
    x.state = cache->state(run);
    x.out_split = sa;
    x.pieces = np;
    x.conv_in = xin;
    x.ring = c.ring;
    x.n = n;
    x.channels = s.rec.width;
    x.width = d.width;
    x.block_width = d.block;
    x.block_pad = d.block_pad;
    x.past = past;
    if ((rc = linear_recurrence_launch(ctx_, x)) != HM_OK) return rc;
    return gemm_split_nk(ctx_, sa, np, l.lr_o.ptr(), p.y.as<float>(), n, l.lr_o.kp, wp_, MP, y_parts);
}

int BlockModel::prefill_window_attention(int run, int layer, int n, int past, int *y_parts) {
    PrefillScratch &p = pf_;
    const WindowAttentionSpec &a = cfg_.layers[layer].wattn;
    const Dims &d = dims_[layer];
    const LayerWeights &l = layers_[layer];
    const WindowAttentionShape &sh = d.wshape;
    const int np = prefill_pieces_, MP = PrefillScratch::MAX_PARTS;
    uint16_t *sa = p.split_a.as<uint16_t>(), *cache = plan_->state_cache()->window(cache_run_[run]);
    float *d1 = p.d1.as<float>();
    int parts = 1, rc;
    if ((rc = gemm_split_nk(ctx_, sa, np, l.wa_in.ptr(), d1, n, l.wa_in.kp, l.wa_in.np, MP, &parts)) != HM_OK) return rc;
    WindowRowsArgs r;
    r.s = sh;
    r.in = RowSource{d1, l.wa_in.np, parts, (size_t)n * l.wa_in.np, nullptr};
    r.k_at = d.k_at;
    r.v_at = d.v_at;
    r.q_norm = l.head_q_norm.ptr();
    r.k_norm = a.kv_from < 0 ? l.head_k_norm.ptr() : nullptr;
    r.eps = (float)cfg_.eps;
    r.q = p.f1.as<float>();
    r.cache = cache;
    r.n = n;
    r.past = past;
    if ((rc = window_rows_launch(ctx_, r)) != HM_OK) return rc;
    PrefillAttnArgs at;
    at.q = r.q;
    at.ldq = a.heads * sh.width;
    at.kcache = cache;
    at.vcache = cache + sh.pieces * sh.plane();
    at.out_split = sa;
    at.S = n;
    at.H = a.heads;
    at.kvh = a.kv_heads;
    at.hd = at.hdv = sh.width;
    at.kv_pieces = sh.pieces;
    at.k_plane = at.v_plane = sh.plane();
    at.max_len = sh.map.slots();
    at.past = past;
    at.scale = (float)a.scale;
    at.window = sh.window;
    at.keep = sh.keep;
    at.slot_keep = sh.map.keep;
    at.slot_ring = sh.keep || sh.map.slots() < max_seq_len_ ? sh.map.ring : 0;
    at.vdim = a.vdim;
    at.out_cols = d.gate;
    at.out_pieces = np;
    if ((rc = prefill_attn_launch(ctx_, at)) != HM_OK) return rc;
    return gemm_split_nk(ctx_, sa, np, l.wa_o.ptr(), p.y.as<float>(), n, l.wa_o.kp, wp_, MP, y_parts);
}

int BlockModel::prefill_matrix_memory(int run, int layer, const float *x, int n, int past, int *y_parts) {
    PrefillScratch &p = pf_;
    const Dims &d = dims_[layer];
    const LayerWeights &l = layers_[layer];
    const int np = prefill_pieces_, MP = PrefillScratch::MAX_PARTS;
    uint16_t *sa = p.split_a.as<uint16_t>();
    float *d1 = p.d1.as<float>();
    int parts = 1, rc;
    const int cols = d.mm_at.i;  // the log gates take the rows themselves
    if ((rc = gemm_split_nk(ctx_, sa, np, l.mm_in.ptr(), d1, n, l.mm_in.kp, cols, MP, &parts)) != HM_OK) return rc;
    MatrixMemoryRowsArgs r;
    r.s = d.mshape;
    r.at = d.mm_at;
    r.rows = d1;
    r.ld = cols;
    r.parts = parts;
    r.stride = (size_t)n * cols;
    r.x = x;
    r.x_ld = wp_;
    r.gate_w = l.mm_in.ptr(d.mm_at.i);
    r.gates = p.mm_gates.as<float>();
    r.i_bias = l.mm_i_b.ptr();
    r.f_bias = l.mm_f_b.ptr();
    r.pieces = compute_ == DType::F32 ? 3 : 1;
    r.q = p.mm_q.as<uint16_t>();
    r.k = p.mm_k.as<uint16_t>();
    r.log_w = p.mm_log_w.as<double>();
    r.weights = p.mm_weights.as<float>();
    r.decay = p.mm_decay.as<float>();
    r.values = p.mm_values.as<uint16_t>();
    r.ahead = p.mm_ahead.as<uint16_t>();
    r.state = plan_->state_cache()->state(run);
    r.raw = p.d3.as<float>();
    r.norm = l.mm_norm.ptr();
    r.eps = (float)cfg_.eps;
    r.out_split = sa;
    r.out_pieces = np;
    r.out_cols = d.gate;
    r.n = n;
    r.past = past;
    if ((rc = matrix_memory_rows_launch(ctx_, r)) != HM_OK) return rc;
    return gemm_split_nk(ctx_, sa, np, l.mm_o.ptr(), p.y.as<float>(), n, l.mm_o.kp, wp_, MP, y_parts);
}

// The feed-forward of one layer on the rows in split_a; its raw output lands in y (as *y_parts K slices).
int BlockModel::prefill_feed_forward(int layer, int n, int *y_parts) {
    PrefillScratch &p = pf_;
    const FeedForwardSpec &s = cfg_.layers[layer].ff;
    const LayerWeights &l = layers_[layer];
    const int np = prefill_pieces_, MP = PrefillScratch::MAX_PARTS, ff = dims_[layer].ff, wp = wp_;
    uint16_t *sa = p.split_a.as<uint16_t>(), *sb = p.split_b.as<uint16_t>();
    float *d1 = p.d1.as<float>(), *y = p.y.as<float>();
    int parts = 1, rc;
    GatedRowsArgs g;
    g.act = s.act;
    g.pieces = np;
    g.width = ff;
    g.out_split = sb;
    if (!s.experts) {
        if ((rc = gemm_split_nk(ctx_, sa, np, l.gate_up.ptr(), d1, n, wp, 2 * ff, MP, &parts)) != HM_OK) return rc;
        if (s.act.kind == GatedAct::Silu) {
            rc = silu_mul_split_launch(ctx_, d1, parts, sb, np, n, ff);
        } else {
            g.in = RowSource{d1, 2 * ff, parts, (size_t)n * 2 * ff, nullptr};
            g.rows = n;
            rc = gated_rows_launch(ctx_, g);
        }
        if (rc != HM_OK) return rc;
        return gemm_split_nk(ctx_, sb, np, l.down.ptr(), y, n, ff, wp, MP, y_parts);
    }
    if ((rc = gemm_split_nk(ctx_, sa, np, l.router.ptr(), p.d2.as<float>(), n, wp, l.router.np, MP, &parts)) != HM_OK) return rc;
    RouteRowsArgs r;
    r.logits = RowSource{p.d2.as<float>(), l.router.np, parts, (size_t)n * l.router.np, nullptr};
    r.experts = s.experts;
    r.top = s.top;
    r.n = n;
    r.choice = p.choice.as<int>();
    r.weight = p.choice_weight.as<float>();
    r.list = p.expert_list.as<int>();
    r.count = p.expert_count.as<int>();
    if ((rc = route_rows_launch(ctx_, r)) != HM_OK) return rc;
    const int entries = s.top * n;
    if (gemm_gated_fits(np, wp, 2 * ff)) {
        rc = gemm_grouped_nk(ctx_, sa, np, n, l.gate_up.ptr(), p.split_b.as<float>(), r.list, r.count, s.experts, n, entries, wp, 2 * ff, &s.act, r.weight);
    } else {
        rc = gemm_grouped_nk(ctx_, sa, np, n, l.gate_up.ptr(), d1, r.list, r.count, s.experts, n, entries, wp, 2 * ff);
        if (rc != HM_OK) return rc;
        g.in = RowSource{d1, 2 * ff, 1, 0, nullptr};
        g.weight = r.weight;
        g.rows = entries;
        rc = gated_rows_launch(ctx_, g);
    }
    if (rc != HM_OK) return rc;
    if ((rc = gemm_grouped_nk(ctx_, sb, np, entries, l.down.ptr(), y, r.list, r.count, s.experts, n, entries, ff, wp)) != HM_OK) return rc;
    *y_parts = s.top;
    if (s.top > MP) {
        rc = sum_places_launch(ctx_, y, s.top, (size_t)n * wp);
        *y_parts = 1;
    }
    return rc;
}

int BlockModel::prefill_chunk(const int32_t *h_ids, int n, float *h_logits) {
    int rc = prepare_prefill();
    if (rc != HM_OK) return rc;
    PrefillScratch &p = pf_;
    SequenceCache *cache = plan_->cache();
    const int past = cache->current_len(), np = prefill_pieces_, MP = PrefillScratch::MAX_PARTS, wp = wp_;
    const size_t row_floats = (size_t)n * wp;
    float *x = p.x.as<float>(), *x0 = p.x0.as<float>(), *y = p.y.as<float>(), *d1 = p.d1.as<float>();
    uint16_t *sa = p.split_a.as<uint16_t>();
    if ((rc = hm_upload(ctx_, p.ids.ptr(), h_ids, (size_t)n * 4)) != HM_OK) return rc;
    if ((rc = embed_scaled_launch(ctx_, p.ids.as<int32_t>(), embed_.ptr(), x, n, cfg_.vocab, wp, (float)cfg_.embed_scale, waves(), past)) != HM_OK) return rc;
    if (cfg_.loop_times && (rc = hm_copy(ctx_, x0, x, row_floats * 4)) != HM_OK) return rc;
    // x [+ norm_b(y)] -> x, and through norm_w (or as it is, with x0 behind it) into split_a
    const Vec *pending = nullptr;
    int y_parts = 1;
    auto rows = [&](const float *norm_w, int pieces, const float *cat, bool split = true, float *f32 = nullptr) -> int {
        RowNormArgs r;
        r.x = x;
        if (pending) {
            r.y = y;
            r.y_parts = y_parts;
            r.y_stride = row_floats;
            r.y_w = pending->ptr();
            r.r_out = x;
        }
        r.w = norm_w;
        r.out_split = split ? sa : nullptr;
        r.out = f32;
        r.pieces = pieces;
        r.cat = cat;
        r.rows = n;
        r.dim = wp;
        r.norm_dim = cfg_.width;
        r.eps = (float)cfg_.eps;
        pending = nullptr;
        return row_norm_launch(ctx_, r);
    };
    if (p.capture && p.captured_rows != n) {
        p.captured = Buffer::alloc(ctx_, {(int64_t)(runs_.size() * row_floats)}, DType::F32);
        if (!p.captured) return HM_ERR_OOM;
        p.captured_rows = n;
    }
    for (size_t run = 0; run < runs_.size(); run++) {
        const int li = runs_[run].layer;
        const BlockLayerSpec &s = cfg_.layers[li];
        const LayerWeights &l = layers_[li];
        if (runs_[run].begins_pass) {
            // the residual keeps all its bits on the way through the matrix of the pass
            if ((rc = rows(nullptr, 3, x0)) != HM_OK) return rc;
            int parts = 1;
            if ((rc = gemm_split_nk(ctx_, sa, 3, loop_in_.ptr(), d1, n, loop_in_.kp, wp, MP, &parts)) != HM_OK) return rc;
            if ((rc = sum_parts_launch(ctx_, d1, wp, parts, row_floats, x, n, wp)) != HM_OK) return rc;
        }
        // (matrix memories want their input in f32, too: without a norm ahead it is x)
        float *f32 = cfg_.pre_norms && s.mixer == MixerKind::MatrixMemory ? p.f1.as<float>() : nullptr;
        if ((rc = rows(cfg_.pre_norms ? l.norm1.ptr() : nullptr, np, nullptr, true, f32)) != HM_OK) return rc;
        const Rope *rope = layer_rope_[li];
        rc = prefill_mixer((int)run, li, rope ? rope->cos.as<float>() : nullptr, rope ? rope->sin.as<float>() : nullptr, n, past, &y_parts);
        if (rc != HM_OK) return rc;
        pending = &l.norm1b;
        if (s.ff.width) {
            if ((rc = rows(cfg_.pre_norms ? l.norm2.ptr() : nullptr, np, nullptr)) != HM_OK) return rc;
            if ((rc = prefill_feed_forward(li, n, &y_parts)) != HM_OK) return rc;
            pending = &l.norm2b;
        }
        if (p.capture) {
            if ((rc = rows(nullptr, 1, nullptr, false)) != HM_OK) return rc;
            if ((rc = hm_copy(ctx_, p.captured.as<float>() + run * row_floats, x, row_floats * 4)) != HM_OK) return rc;
        }
    }
    if (h_logits) {
        const size_t vocab = cfg_.vocab;
        if (!p.logits) p.logits = Buffer::alloc(ctx_, {p.rows, (int64_t)vocab}, DType::F32);
        if (!p.logits) return HM_ERR_OOM;
        rc = rows(final_norm_.ptr(), np, nullptr);
        if (rc == HM_OK) rc = gemm_split_nk(ctx_, sa, np, head_.ptr(), p.logits.as<float>(), n, wp, (int)vocab);
        if (rc == HM_OK) rc = hm_download(ctx_, h_logits, p.logits.ptr(), (size_t)n * vocab * 4);
        if (rc != HM_OK) return rc;
    }
    cache->advance_by(n);
    return HM_OK;
}

int BlockModel::capture_residuals(bool on) {
    pf_.capture = on;
    pf_.captured_rows = 0;
    pf_.captured = Buffer();
    return HM_OK;
}

int BlockModel::captured_residuals(float *h_out, size_t n_floats) {
    if (!pf_.captured || !pf_.captured_rows) return hm_set_error(ctx_, HM_ERR_STATE, "no residual rows were captured");
    const size_t lines = runs_.size() * pf_.captured_rows;
    if (n_floats != lines * cfg_.width)
        return hm_set_error(ctx_, HM_ERR_INVALID, "captured residuals: %zu floats kept, %zu asked for", lines * cfg_.width, n_floats);
    HM_HIP(ctx_, hipMemcpy2DAsync(h_out, (size_t)cfg_.width * 4, pf_.captured.ptr(), (size_t)wp_ * 4, (size_t)cfg_.width * 4, lines, hipMemcpyDeviceToHost,
                                  ctx_->stream));
    return hm_sync(ctx_);
}

}  // namespace homura
