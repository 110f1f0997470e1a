// Attention over a window and kept first tokens (see window_attention.h).
#include "window_attention.h"

#include <algorithm>

namespace {

using namespace homura;

__device__ __forceinline__ void store_pieces(uint16_t *at, size_t plane, float v, int pieces) {
    uint32_t p[3];
    split_pieces<3>(v, p);
    at[0] = (uint16_t)p[0];
    if (pieces == 3) {
        at[plane] = (uint16_t)p[1];
        at[2 * plane] = (uint16_t)p[2];
    }
}

// ── decode step ──────────────────────────────────────────────────────────────

// Workgroup (WS_ROWS visible rows, up to GB query heads of one KV head). W / 8 lanes cover a row with 16-byte loads;
// all rows of the workgroup are requested before anything waits, then the queries are normed. The workgroup with the
// newest row takes it from the projection (rounded like the cache) and the first group of its KV head stores it.
constexpr int WS_ROWS = 64;

template <int W, int KP, int GB>
__global__ __launch_bounds__(256) void window_step_attn_kernel(WindowStepArgs a) {
    constexpr int LPR = W / 8, RPI = 64 / LPR, NRG = WS_ROWS / (4 * RPI), EPT = W / 64;
    __shared__ float qs[GB][W], knew[W], vnew[W];
    __shared__ float sc[GB][WS_ROWS], s_ml[GB][2];
    __shared__ __attribute__((aligned(16))) float red[4 * RPI][GB][W];
    const WindowAttentionShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane / LPR, dl = lane % LPR;
    const int per_kv = s.heads / s.kv_heads, groups = (per_kv + GB - 1) / GB;
    const int kvh = blockIdx.y / groups, grp = blockIdx.y % groups, g_here = min(GB, per_kv - grp * GB);
    const int h0 = kvh * per_kv + grp * GB;
    const int pos = a.cursor->pos;
    const int lo = s.window ? max(0, pos - s.window + 1) : 0, kept = min(s.keep, lo);
    const int total = kept + pos - lo + 1, r0 = blockIdx.x * WS_ROWS;
    if (r0 >= total) return;
    const int cnt = min(WS_ROWS, total - r0);
    const size_t plane = s.plane();
    uint16_t *kc = a.cache + (size_t)kvh * s.map.slots() * W, *vc = kc + KP * plane;

    const bool owner = a.k && r0 + cnt == total;  // this workgroup's last row is the new one
    u32x4 kr[NRG][KP], vr[NRG][KP];
#pragma unroll
    for (int i = 0; i < NRG; i++) {
        const int row = (i * 4 + wave) * RPI + sub;
        const bool ok = row < cnt && !(owner && row == cnt - 1);
        const int r = r0 + min(row, cnt - 1);
        const size_t at = (size_t)s.map.slot(r < kept ? r : lo + r - kept) * W + dl * 8;
#pragma unroll
        for (int p = 0; p < KP; p++) {
            kr[i][p] = ok ? ld128(kc + p * plane + at) : u32x4{0u, 0u, 0u, 0u};
            vr[i][p] = ok ? ld128(vc + p * plane + at) : u32x4{0u, 0u, 0u, 0u};
        }
    }
    // rows 0 .. GB - 1: queries; GB: the new key; GB + 1: the new value. A wavefront takes every fourth.
    constexpr int TMAX = (GB + 2 + 3) / 4;
    float raw[TMAX][EPT], nw[TMAX][EPT];
#pragma unroll
    for (int j = 0; j < TMAX; j++) {
        const int t = wave + 4 * j;
        const float *src = nullptr, *w = nullptr;
        int n = s.dim;
        if (t < g_here) src = a.q + (size_t)(h0 + t) * s.dim, w = a.q_norm;
        else if (owner && t == GB) src = a.k + (size_t)kvh * s.dim, w = a.k_norm;
        else if (owner && t == GB + 1) src = a.v + (size_t)kvh * s.vdim, n = s.vdim;
#pragma unroll
        for (int e = 0; e < EPT; e++) {
            const int d = lane + 64 * e;
            raw[j][e] = src && d < n ? src[d] : 0.f;
            nw[j][e] = w && d < n ? w[d] : 1.f;
        }
    }
#pragma unroll
    for (int j = 0; j < TMAX; j++) {
        const int t = wave + 4 * j;  // wavefront-uniform
        if (t >= GB + 2 || (t >= GB && !owner)) continue;
        float inv = 1.f;
        if (t <= GB) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < EPT; e++) ss += raw[j][e] * raw[j][e];
            inv = 1.0f / sqrtf(wave_sum(ss) / (float)s.dim + a.eps);
        }
        if (t < GB) {
#pragma unroll
            for (int e = 0; e < EPT; e++) qs[t][lane + 64 * e] = (raw[j][e] * inv) * nw[j][e];
            continue;
        }
        uint16_t *row = (t == GB ? kc : vc) + (size_t)s.map.slot(pos) * W;
        float *mine = t == GB ? knew : vnew;
#pragma unroll
        for (int e = 0; e < EPT; e++) {
            const int d = lane + 64 * e;
            const float v = (raw[j][e] * inv) * nw[j][e];
            if (grp == 0) store_pieces(row + d, plane, v, KP);
            mine[d] = KP == 3 ? v : __uint_as_float((uint32_t)f32_to_bf16_rne_dev(v) << 16);
        }
    }
    __syncthreads();

    // row i of this lane's rows as f32: its pieces added up, smallest first
    auto unpack = [&](const u32x4 (&w)[KP], float (&f)[8]) {
#pragma unroll
        for (int e = 0; e < 4; e++) {
            f[2 * e] = bf16_lo(w[KP - 1][e]);
            f[2 * e + 1] = bf16_hi(w[KP - 1][e]);
#pragma unroll
            for (int p = KP - 2; p >= 0; p--) {
                f[2 * e] += bf16_lo(w[p][e]);
                f[2 * e + 1] += bf16_hi(w[p][e]);
            }
        }
    };
    float qv[GB][8];
#pragma unroll
    for (int g = 0; g < GB; g++)
#pragma unroll
        for (int e = 0; e < 8; e++) qv[g][e] = qs[g][dl * 8 + e];
#pragma unroll
    for (int i = 0; i < NRG; i++) {
        const int row = (i * 4 + wave) * RPI + sub;
        float kf[8];
        unpack(kr[i], kf);
        if (owner && row == cnt - 1) {
#pragma unroll
            for (int e = 0; e < 8; e++) kf[e] = knew[dl * 8 + e];
        }
#pragma unroll
        for (int g = 0; g < GB; g++) {
            float p = 0.f;
#pragma unroll
            for (int e = 0; e < 8; e++) p = fmaf(kf[e], qv[g][e], p);
#pragma unroll
            for (int m = 1; m < LPR; m *= 2) p += __shfl_xor(p, m);
            if (dl == 0) sc[g][row] = row < cnt ? p * a.scale : -INFINITY;
        }
    }
    __syncthreads();
    static_assert(WS_ROWS == 64, "one score a lane");
    for (int g = wave; g < GB; g += 4) {
        const float x = sc[g][lane], m = wave_max(x), p = expf(x - m);
        sc[g][lane] = p;
        const float l = wave_sum(p);
        if (lane == 0) {
            s_ml[g][0] = m;
            s_ml[g][1] = l;
        }
    }
    __syncthreads();
    float acc[GB][8];
#pragma unroll
    for (int g = 0; g < GB; g++)
#pragma unroll
        for (int e = 0; e < 8; e++) acc[g][e] = 0.f;
#pragma unroll
    for (int i = 0; i < NRG; i++) {
        const int row = (i * 4 + wave) * RPI + sub;
        float vf[8];
        unpack(vr[i], vf);
        if (owner && row == cnt - 1) {
#pragma unroll
            for (int e = 0; e < 8; e++) vf[e] = vnew[dl * 8 + e];
        }
#pragma unroll
        for (int g = 0; g < GB; g++) {
            const float p = sc[g][row];
#pragma unroll
            for (int e = 0; e < 8; e++) acc[g][e] = fmaf(p, vf[e], acc[g][e]);
        }
    }
#pragma unroll
    for (int g = 0; g < GB; g++) {
        float *dst = &red[wave * RPI + sub][g][dl * 8];
        *reinterpret_cast<f32x4 *>(dst) = f32x4{acc[g][0], acc[g][1], acc[g][2], acc[g][3]};
        *reinterpret_cast<f32x4 *>(dst + 4) = f32x4{acc[g][4], acc[g][5], acc[g][6], acc[g][7]};
    }
    __syncthreads();
    for (int i = tid; i < g_here * W; i += 256) {
        const int g = i / W, d = i % W;
        float v = 0.f;
#pragma unroll
        for (int r = 0; r < 4 * RPI; r++) v += red[r][g][d];
        a.part_o[((size_t)blockIdx.x * s.heads + h0 + g) * W + d] = v;
    }
    if (tid < g_here * 2) a.part_ml[((size_t)blockIdx.x * s.heads + h0 + (tid >> 1)) * 2 + (tid & 1)] = s_ml[tid >> 1][tid & 1];
}

// Joins the splits of a head: W columns, 256 / W groups of threads over the splits. The cursor decides how many there
// are, but the first FOLD_AHEAD of a group are asked for ahead of it (what lies behind is not used).
constexpr int FOLD_AHEAD = 8;
template <int W>
__global__ __launch_bounds__(256) void window_step_fold_kernel(WindowStepArgs a, int max_splits) {
    constexpr int GR = 256 / W;
    __shared__ float red[GR][W], red_l[GR];
    const WindowAttentionShape &s = a.s;
    const int h = blockIdx.x, d = threadIdx.x % W, gr = threadIdx.x / W;
    const size_t step = (size_t)s.heads;
    float o[FOLD_AHEAD], m[FOLD_AHEAD], l[FOLD_AHEAD];
#pragma unroll
    for (int j = 0; j < FOLD_AHEAD; j++) {
        const int sp = min(gr + j * GR, max_splits - 1);
        o[j] = a.part_o[(sp * step + h) * W + d];
        m[j] = a.part_ml[(sp * step + h) * 2];
        l[j] = a.part_ml[(sp * step + h) * 2 + 1];
    }
    const int pos = a.cursor->pos;
    const int lo = s.window ? max(0, pos - s.window + 1) : 0;
    const int splits = (min(s.keep, lo) + pos - lo + 1 + WS_ROWS - 1) / WS_ROWS;
    float top = -INFINITY;
#pragma unroll
    for (int j = 0; j < FOLD_AHEAD; j++) top = fmaxf(top, gr + j * GR < splits ? m[j] : -INFINITY);
    for (int sp = gr + FOLD_AHEAD * GR; sp < splits; sp += GR) top = fmaxf(top, a.part_ml[(sp * step + h) * 2]);
    if (d == 0) red_l[gr] = top;
    __syncthreads();
#pragma unroll
    for (int g = 0; g < GR; g++) top = fmaxf(top, red_l[g]);
    __syncthreads();
    float acc = 0.f, sum = 0.f;
#pragma unroll
    for (int j = 0; j < FOLD_AHEAD; j++)
        if (gr + j * GR < splits) {
            const float w = expf(m[j] - top);
            acc = fmaf(w, o[j], acc);
            sum = fmaf(w, l[j], sum);
        }
    for (int sp = gr + FOLD_AHEAD * GR; sp < splits; sp += GR) {
        const float *ml = a.part_ml + (sp * step + h) * 2;
        const float w = expf(ml[0] - top);
        acc = fmaf(w, a.part_o[(sp * step + h) * W + d], acc);
        sum = fmaf(w, ml[1], sum);
    }
    red[gr][d] = acc;
    if (d == 0) red_l[gr] = sum;
    __syncthreads();
    if (gr == 0 && d < s.vdim) {
        float v = 0.f, t = 0.f;
#pragma unroll
        for (int g = 0; g < GR; g++) {
            v += red[g][d];
            t += red_l[g];
        }
        a.out[(size_t)h * s.vdim + d] = v / t;
    }
}

// ── prompt pass ──────────────────────────────────────────────────────────────

// a wavefront per head of a row: query heads, key heads, value heads
template <int W>
__global__ __launch_bounds__(256) void window_rows_kernel(WindowRowsArgs a) {
    constexpr int EPT = W / 64;
    const WindowAttentionShape &s = a.s;
    const int lane = threadIdx.x & 63, kinds = s.heads + (a.k_norm ? 2 * s.kv_heads : 0);
    const size_t job = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (job >= (size_t)a.n * kinds) return;
    const int t = (int)(job / kinds), at = (int)(job % kinds);
    const bool is_q = at < s.heads, is_v = at >= s.heads + s.kv_heads;
    const int head = is_q ? at : is_v ? at - s.heads - s.kv_heads : at - s.heads;
    const int n = is_v ? s.vdim : s.dim, col = (is_q ? 0 : is_v ? a.v_at : a.k_at) + head * n;
    const float *w = is_q ? a.q_norm : a.k_norm;
    float x[EPT], nw[EPT], ss = 0.f;
#pragma unroll
    for (int e = 0; e < EPT; e++) {
        const int d = lane * EPT + e;
        x[e] = d < n ? source_at(a.in, t, col + d) : 0.f;
        nw[e] = d < n && !is_v ? w[d] : 1.f;
        ss += x[e] * x[e];
    }
    if (!is_v) {
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps);
#pragma unroll
        for (int e = 0; e < EPT; e++) x[e] = (x[e] * inv) * nw[e];
    }
    if (is_q) {
        float *out = a.q + (size_t)t * s.heads * W + (size_t)head * W + lane * EPT;
#pragma unroll
        for (int e = 0; e < EPT; e++) out[e] = x[e];
        return;
    }
    uint16_t *row = a.cache + (is_v ? (size_t)s.pieces * s.plane() : 0) + ((size_t)head * s.map.slots() + s.map.slot(a.past + t)) * W + lane * EPT;
#pragma unroll
    for (int e = 0; e < EPT; e++) store_pieces(row + e, s.plane(), x[e], s.pieces);
}

bool bad_shape(const WindowAttentionShape &s) {
    return s.heads <= 0 || s.kv_heads <= 0 || s.heads % s.kv_heads || s.dim <= 0 || s.vdim <= 0 || s.width != window_head_width(s.dim, s.vdim) ||
           s.width == 0 || (s.pieces != 1 && s.pieces != 3) || s.window < 0 || s.keep < 0 || s.map.keep < 0 || s.map.ring < 1;
}

}  // namespace

namespace homura {

int window_head_width(int dim, int vdim) {
    const int d = std::max(dim, vdim);
    return d <= 64 ? 64 : d <= 128 ? 128 : d <= WA_MAX_DIM ? 256 : 0;
}

int window_step_span(const WindowAttentionShape &s, int max_len) {
    return s.window ? (int)std::min<int64_t>(max_len, (int64_t)s.window + s.keep) : max_len;
}
int window_step_splits(int span) { return (span + WS_ROWS - 1) / WS_ROWS; }

int window_step_attn_launch(hm_ctx *ctx, const WindowStepArgs &a) {
    HM_REQUIRE(ctx, !bad_shape(a.s) && a.span > 0, "window_step_attn: bad shape");
    HM_REQUIRE(ctx, a.q && a.q_norm && a.cache && a.part_o && a.part_ml && a.cursor && (!a.k || (a.v && a.k_norm)), "window_step_attn: NULL pointer");
    const int per_kv = a.s.heads / a.s.kv_heads, splits = window_step_splits(a.span);
    // two heads a workgroup when one would leave rows to be read too often, more only when there are plenty of workgroups
    const int gb = per_kv == 1 ? 1 : per_kv == 2 || (long long)splits * a.s.kv_heads * ((per_kv + 1) / 2) <= ctx->num_cus ? 2 : 4;
    const dim3 g(splits, a.s.kv_heads * ((per_kv + gb - 1) / gb)), b(256);
#define HM_WS(WV, PV, GV)                                                                                          \
    if (a.s.width == WV && a.s.pieces == PV && gb == GV) hipLaunchKernelGGL((window_step_attn_kernel<WV, PV, GV>), g, b, 0, ctx->stream, a);
    HM_WS(64, 1, 1) HM_WS(64, 1, 2) HM_WS(64, 1, 4) HM_WS(64, 3, 1) HM_WS(64, 3, 2) HM_WS(64, 3, 4)
    HM_WS(128, 1, 1) HM_WS(128, 1, 2) HM_WS(128, 1, 4) HM_WS(128, 3, 1) HM_WS(128, 3, 2) HM_WS(128, 3, 4)
    HM_WS(256, 1, 1) HM_WS(256, 1, 2) HM_WS(256, 1, 4) HM_WS(256, 3, 1) HM_WS(256, 3, 2) HM_WS(256, 3, 4)
#undef HM_WS
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int window_step_fold_launch(hm_ctx *ctx, const WindowStepArgs &a) {
    HM_REQUIRE(ctx, !bad_shape(a.s) && a.span > 0 && a.part_o && a.part_ml && a.out && a.cursor, "window_step_fold: bad arguments");
    const dim3 g(a.s.heads), b(256);
    const int splits = window_step_splits(a.span);
    if (a.s.width == 64) hipLaunchKernelGGL(window_step_fold_kernel<64>, g, b, 0, ctx->stream, a, splits);
    else if (a.s.width == 128) hipLaunchKernelGGL(window_step_fold_kernel<128>, g, b, 0, ctx->stream, a, splits);
    else hipLaunchKernelGGL(window_step_fold_kernel<256>, g, b, 0, ctx->stream, a, splits);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int window_rows_launch(hm_ctx *ctx, const WindowRowsArgs &a) {
    HM_REQUIRE(ctx, !bad_shape(a.s) && a.q && a.q_norm && a.n > 0 && a.past >= 0 && (!a.k_norm || a.cache), "window_rows: bad arguments");
    HM_REQUIRE(ctx, !bad_source(a.in, a.k_norm ? a.v_at + a.s.kv_heads * a.s.vdim : a.s.heads * a.s.dim) &&
                        (!a.k_norm || (a.k_at >= a.s.heads * a.s.dim && a.v_at >= a.k_at + a.s.kv_heads * a.s.dim)), "window_rows: bad projection rows");
    HM_REQUIRE(ctx, !a.k_norm || a.n <= a.s.map.ring || a.past + a.n <= a.s.map.slots(), "window_rows: %d rows do not fit a ring of %d", a.n, a.s.map.ring);
    const size_t jobs = (size_t)a.n * (a.s.heads + (a.k_norm ? 2 * a.s.kv_heads : 0));
    const dim3 g((unsigned)((jobs + 3) / 4)), b(256);
    if (a.s.width == 64) hipLaunchKernelGGL(window_rows_kernel<64>, g, b, 0, ctx->stream, a);
    else if (a.s.width == 128) hipLaunchKernelGGL(window_rows_kernel<128>, g, b, 0, ctx->stream, a);
    else hipLaunchKernelGGL(window_rows_kernel<256>, g, b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
