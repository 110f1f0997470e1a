// Gated feed-forwards and mixtures of experts (see experts.h).
#include "experts.h"

#include <algorithm>

namespace {

using namespace homura;

// ── choice ───────────────────────────────────────────────────────────────────

// The `top` largest of E logits by one wavefront (scores grow with logits; of equals the lower index), emit(place, index,
// logit) in every lane. PER: E <= 64 PER.
template <int PER, class F>
__device__ __forceinline__ void choose_top(float (&z)[PER], int E, int top, F emit) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int j = 0; j < PER; j++)
        if (lane + 64 * j >= E || !(z[j] == z[j])) z[j] = -INFINITY;  // (whatever the logits are, the chosen are different experts)
    uint32_t gone = 0;
    for (int place = 0; place < top; place++) {
        float best = -INFINITY;
        int at = 0x7fffffff;
#pragma unroll
        for (int j = 0; j < PER; j++)
            if (!(gone >> j & 1) && lane + 64 * j < E && (z[j] > best || at == 0x7fffffff)) {
                best = z[j];
                at = lane + 64 * j;
            }
        const float m = wave_max(at == 0x7fffffff ? -INFINITY : best);
        int idx = best == m ? at : 0x7fffffff;
#pragma unroll
        for (int d = 1; d < 64; d *= 2) idx = min(idx, __shfl_xor(idx, d));
        if ((idx & 63) == lane) gone |= 1u << (idx >> 6);
        emit(place, idx, m);
    }
}

__device__ __forceinline__ float score(float z) { return 1.0f / (1.0f + expf(-z)); }

template <int PER>
__global__ __launch_bounds__(256) void route_rows_kernel(RouteRowsArgs a) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (t >= a.n) return;
    float z[PER];
#pragma unroll
    for (int j = 0; j < PER; j++) z[j] = lane + 64 * j < a.experts ? source_at(a.logits, t, lane + 64 * j) : 0.f;
    choose_top<PER>(z, a.experts, a.top, [&](int place, int idx, float m) {
        if (lane == 0) {
            a.choice[(size_t)place * a.n + t] = idx;
            a.weight[(size_t)place * a.n + t] = score(m);
        }
    });
}

// Workgroup: one expert. Every thread counts its stretch of the entries, then writes it at the sum of those before it.
constexpr int LIST_THREADS = 1024;
__global__ __launch_bounds__(LIST_THREADS) void expert_list_kernel(RouteRowsArgs a) {
    __shared__ int wave_total[LIST_THREADS / 64];
    const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, entries = a.top * a.n;
    const int per = (entries + 4 * LIST_THREADS - 1) / (4 * LIST_THREADS) * 4, begin = tid * per;
    typedef int i32x4 __attribute__((ext_vector_type(4)));
    auto four = [&](int i) -> uint32_t {  // which of entries i .. i + 3 are this expert's
        if (i + 4 <= entries) {
            const i32x4 v = *reinterpret_cast<const i32x4 *>(a.choice + i);
            return (v[0] == e) | (v[1] == e) << 1 | (v[2] == e) << 2 | (v[3] == e) << 3;
        }
        uint32_t m = 0;
        for (int j = 0; j < 4; j++)
            if (i + j < entries && a.choice[i + j] == e) m |= 1u << j;
        return m;
    };
    int mine = 0;
    const uint32_t first = four(begin);
    for (int i = begin; i < begin + per; i += 4) mine += __popc(i == begin ? first : four(i));
    int upto = mine;
#pragma unroll
    for (int d = 1; d < 64; d *= 2) {
        const int o = __shfl_up(upto, d);
        if (lane >= d) upto += o;
    }
    if (lane == 63) wave_total[wave] = upto;
    __syncthreads();
    int at = upto - mine;
    for (int w = 0; w < wave; w++) at += wave_total[w];
    // (a token chooses an expert once: a list holds at most n entries)
    int *list = a.list + (size_t)e * a.n;
    for (int i = begin; i < begin + per; i += 4) {
        const uint32_t m = i == begin ? first : four(i);
        for (int j = 0; j < 4; j++)
            if (m >> j & 1) list[at++] = i + j;
    }
    if (tid == LIST_THREADS - 1) a.count[e] = at;
}

// ── rows ─────────────────────────────────────────────────────────────────────

// two neighbouring outputs (four columns of the source) a thread
__global__ __launch_bounds__(256) void gated_rows_kernel(GatedRowsArgs a, size_t n2) {
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= n2) return;
    const int half = a.width / 2, c = (int)(e % half) * 2;
    const size_t row = e / half;
    f32x4 v = sum_parts4(a.in.p, row * a.in.ld + 2 * c, a.in.parts, a.in.stride);
    if (a.weight) v = v * a.weight[row];
    uint32_t w[3];
    split_pair<3>(gated_act(a.act, v[0], v[1]), gated_act(a.act, v[2], v[3]), w);
    uint16_t *out = a.out_split + row * a.pieces * a.width + c;
    for (int p = 0; p < a.pieces; p++) *reinterpret_cast<uint32_t *>(out + (size_t)p * a.width) = w[p];
}

__global__ __launch_bounds__(256) void sum_places_kernel(float *y, int places, size_t n, size_t n4) {
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= n4) return;
    f32x4 v = *reinterpret_cast<const f32x4 *>(y + e * 4);
    for (int p = 1; p < places; p++) v += *reinterpret_cast<const f32x4 *>(y + p * n + e * 4);
    *reinterpret_cast<f32x4 *>(y + e * 4) = v;
}

// ── decode step ──────────────────────────────────────────────────────────────

__device__ __forceinline__ float dot8(u32x4 w, f32x4 x0, f32x4 x1, float acc) {
    acc = fmaf(bf16_lo(w.x), x0.x, acc);
    acc = fmaf(bf16_hi(w.x), x0.y, acc);
    acc = fmaf(bf16_lo(w.y), x0.z, acc);
    acc = fmaf(bf16_hi(w.y), x0.w, acc);
    acc = fmaf(bf16_lo(w.z), x1.x, acc);
    acc = fmaf(bf16_hi(w.z), x1.y, acc);
    acc = fmaf(bf16_lo(w.w), x1.z, acc);
    return fmaf(bf16_hi(w.w), x1.w, acc);
}

// Workgroup (R rows of gate|up, place): every wavefront makes the whole choice itself, then the rows are cut across the
// four wavefronts. The first workgroup of a place writes down whom it chose.
template <int R, int PER>
__global__ __launch_bounds__(256) void experts_step_up_kernel(ExpertsStepArgs a) {
    __shared__ float part[4][R];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, row0 = blockIdx.x * R, rows = 2 * a.ff;
    float z[PER];
#pragma unroll
    for (int j = 0; j < PER; j++) z[j] = a.logits[min(lane + 64 * j, a.experts - 1)];
    constexpr int AHEAD = 2;  // chunks of 2048 whose activations are asked for before the choice is made
    f32x4 x0[AHEAD], x1[AHEAD];
#pragma unroll
    for (int c = 0; c < AHEAD; c++) {
        const int k = ((c * 4 + wave) * 64 + lane) * 8;
        x0[c] = x1[c] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (k < a.K) {
            x0[c] = *reinterpret_cast<const f32x4 *>(a.x + k);
            x1[c] = *reinterpret_cast<const f32x4 *>(a.x + k + 4);
        }
    }
    int e = 0;
    float m = 0.f;
    choose_top<PER>(z, a.experts, (int)blockIdx.y + 1, [&](int place, int idx, float logit) {
        e = idx;
        m = logit;
    });
    e = __builtin_amdgcn_readfirstlane(e);
    const uint16_t *w = a.gate_up + (size_t)e * rows * a.K;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.f;
    auto chunk = [&](int k, f32x4 v0, f32x4 v1) {
        u32x4 wv[R];
#pragma unroll
        for (int r = 0; r < R; r++) wv[r] = ld128_stream(w + (size_t)min(row0 + r, rows - 1) * a.K + k);
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = dot8(wv[r], v0, v1, acc[r]);
    };
#pragma unroll
    for (int c = 0; c < AHEAD; c++) {
        const int k = ((c * 4 + wave) * 64 + lane) * 8;
        if (k < a.K) chunk(k, x0[c], x1[c]);
    }
    for (int c = AHEAD; c * 2048 < a.K; c++) {
        const int k = ((c * 4 + wave) * 64 + lane) * 8;
        if (k < a.K) chunk(k, *reinterpret_cast<const f32x4 *>(a.x + k), *reinterpret_cast<const f32x4 *>(a.x + k + 4));
    }
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = wave_sum(acc[r]);
    if (lane == 0) {
#pragma unroll
        for (int r = 0; r < R; r++) part[wave][r] = acc[r];
    }
    __syncthreads();
    if (tid < R / 2 && row0 + 2 * tid < rows) {
        auto sum = [&](int r) { return (part[0][r] + part[1][r]) + (part[2][r] + part[3][r]); };
        const float weight = score(m);
        a.hidden[(size_t)blockIdx.y * a.ff + row0 / 2 + tid] = gated_act(a.act, weight * sum(2 * tid), weight * sum(2 * tid + 1));
    }
    if (blockIdx.x == 0 && tid == 0) a.choice[blockIdx.y] = e;
}

// Workgroup: R output rows; the hidden rows of all places are one long row, cut across the four wavefronts in pieces of
// eight elements, which never straddle two places.
template <int R, int NC>
__global__ __launch_bounds__(256) void experts_step_down_kernel(ExpertsStepArgs a) {
    __shared__ float part[4][R];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, row0 = blockIdx.x * R, K = a.top * a.ff;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.f;
    for (int base = 0; base < K; base += NC * 2048) {
        f32x4 x0[NC], x1[NC];
        const uint16_t *w[NC];
#pragma unroll
        for (int c = 0; c < NC; c++) {
            const int k = base + ((c * 4 + wave) * 64 + lane) * 8, kc = min(k, K - 8), place = kc / a.ff;
            x0[c] = *reinterpret_cast<const f32x4 *>(a.hidden + kc);
            x1[c] = *reinterpret_cast<const f32x4 *>(a.hidden + kc + 4);
            if (k >= K) x0[c] = x1[c] = f32x4{0.f, 0.f, 0.f, 0.f};
            w[c] = a.down + (size_t)a.choice[place] * a.width * a.ff + (kc - place * a.ff);
        }
        u32x4 wv[NC][R];
#pragma unroll
        for (int c = 0; c < NC; c++)
#pragma unroll
            for (int r = 0; r < R; r++) wv[c][r] = ld128_stream(w[c] + (size_t)min(row0 + r, a.width - 1) * a.ff);
#pragma unroll
        for (int c = 0; c < NC; c++)
#pragma unroll
            for (int r = 0; r < R; r++) acc[r] = dot8(wv[c][r], x0[c], x1[c], acc[r]);
    }
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = wave_sum(acc[r]);
    if (lane == 0) {
#pragma unroll
        for (int r = 0; r < R; r++) part[wave][r] = acc[r];
    }
    __syncthreads();
    if (tid < R && row0 + tid < a.width) a.y[row0 + tid] = (part[0][tid] + part[1][tid]) + (part[2][tid] + part[3][tid]);
}

bool al16(const void *p) { return ((uintptr_t)p % 16) == 0; }
bool bad_choice(int experts, int top) { return experts < 1 || experts > EXPERTS_MAX || top < 1 || top > experts || top > EXPERTS_MAX_TOP; }

}  // namespace

namespace homura {

int gated_rows_launch(hm_ctx *ctx, const GatedRowsArgs &a) {
    HM_REQUIRE(ctx, a.rows > 0 && a.width > 0 && a.width % 2 == 0 && !bad_source(a.in, 2 * a.width) && !a.in.bias && a.out_split && a.pieces >= 1 && a.pieces <= 3,
               "gated_rows: bad arguments");
    HM_REQUIRE(ctx, al16(a.in.p) && a.in.ld % 4 == 0 && a.in.stride % 4 == 0 && ((uintptr_t)a.out_split % 4) == 0, "gated_rows: misaligned rows");
    const size_t n2 = (size_t)a.rows * a.width / 2;
    hipLaunchKernelGGL(gated_rows_kernel, dim3((unsigned)((n2 + 255) / 256)), dim3(256), 0, ctx->stream, a, n2);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int route_rows_launch(hm_ctx *ctx, const RouteRowsArgs &a) {
    HM_REQUIRE(ctx, a.n > 0 && !bad_choice(a.experts, a.top) && !bad_source(a.logits, a.experts) && a.choice && a.weight && a.list && a.count && al16(a.choice) &&
                        (size_t)a.top * a.n < ((size_t)1 << 30), "route_rows: bad arguments");
    const dim3 g((a.n + 3) / 4), b(256);
    if (a.experts <= 64) hipLaunchKernelGGL(route_rows_kernel<1>, g, b, 0, ctx->stream, a);
    else if (a.experts <= 256) hipLaunchKernelGGL(route_rows_kernel<4>, g, b, 0, ctx->stream, a);
    else hipLaunchKernelGGL(route_rows_kernel<16>, g, b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    hipLaunchKernelGGL(expert_list_kernel, dim3(a.experts), dim3(LIST_THREADS), 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int sum_places_launch(hm_ctx *ctx, float *d_y, int places, size_t n) {
    HM_REQUIRE(ctx, d_y && al16(d_y) && places >= 1 && n > 0 && n % 4 == 0, "sum_places: bad arguments");
    hipLaunchKernelGGL(sum_places_kernel, dim3((unsigned)((n / 4 + 255) / 256)), dim3(256), 0, ctx->stream, d_y, places, n, n / 4);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int experts_step_up_launch(hm_ctx *ctx, const ExpertsStepArgs &a) {
    HM_REQUIRE(ctx, !bad_choice(a.experts, a.top) && a.x && a.logits && a.gate_up && a.choice && a.hidden, "experts_step_up: bad arguments");
    HM_REQUIRE(ctx, a.K > 0 && a.K % 32 == 0 && a.ff > 0 && a.ff % 32 == 0 && al16(a.x) && al16(a.gate_up), "experts_step_up: bad shape");
    constexpr int R = 4;
    const dim3 g((2 * a.ff + R - 1) / R, a.top), b(256);
    if (a.experts <= 64) hipLaunchKernelGGL((experts_step_up_kernel<R, 1>), g, b, 0, ctx->stream, a);
    else if (a.experts <= 256) hipLaunchKernelGGL((experts_step_up_kernel<R, 4>), g, b, 0, ctx->stream, a);
    else hipLaunchKernelGGL((experts_step_up_kernel<R, 16>), g, b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int experts_step_down_launch(hm_ctx *ctx, const ExpertsStepArgs &a) {
    HM_REQUIRE(ctx, !bad_choice(a.experts, a.top) && a.down && a.choice && a.hidden && a.y, "experts_step_down: bad arguments");
    HM_REQUIRE(ctx, a.width > 0 && a.ff > 0 && a.ff % 32 == 0 && al16(a.hidden) && al16(a.down), "experts_step_down: bad shape");
    const int nc = (a.top * a.ff + 2047) / 2048;
    const dim3 b(256);
    if (nc == 1) hipLaunchKernelGGL((experts_step_down_kernel<2, 1>), dim3((a.width + 1) / 2), b, 0, ctx->stream, a);
    else if (nc == 2) hipLaunchKernelGGL((experts_step_down_kernel<2, 2>), dim3((a.width + 1) / 2), b, 0, ctx->stream, a);
    else hipLaunchKernelGGL((experts_step_down_kernel<2, 4>), dim3((a.width + 1) / 2), b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
