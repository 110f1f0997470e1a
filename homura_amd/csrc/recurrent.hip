// Recurrent mixers (see recurrent.h): convolution rows, selective scan, gated linear recurrence.
#include "recurrent.h"

#include "row_pieces.h"

namespace {

using namespace homura;

// The hardware's exponential, reciprocal and square root are good to about an ulp: f32 results, without the
// instruction sequences of the exactly rounded ones.
__device__ __forceinline__ float exp_dev(float x) { return __builtin_amdgcn_exp2f(x * 1.44269504088896340736f); }
__device__ __forceinline__ float sigmoid_dev(float x) { return __builtin_amdgcn_rcpf(1.0f + exp_dev(-x)); }
// max(x, 0) + log(1 + e) with e = exp(-|x|); with u the rounded 1 + e, log(u) e / (u - 1) is log(1 + e) without the
// rounding of u, and small e take the series
__device__ __forceinline__ float softplus_dev(float x) {
    const float e = exp_dev(-fabsf(x)), u = 1.0f + e;
    const float big = __builtin_amdgcn_logf(u) * 0.69314718055994530942f * e * __builtin_amdgcn_rcpf(u - 1.0f);
    const float small = e * (1.0f - e * (0.5f - e * (1.0f / 3 - e * 0.25f)));
    return fmaxf(x, 0.f) + (e < 1.0f / 64 ? small : big);
}
// sqrt(1 - exp(t)) for t <= 0; close to 0 the difference comes from the series of exp(t) - 1, which loses nothing
__device__ __forceinline__ float input_gain(float t, float exp_t) {
    const float series = -t * (1.0f + t * (1.0f / 2) * (1.0f + t * (1.0f / 3) * (1.0f + t * (1.0f / 4) * (1.0f + t * (1.0f / 5) * (1.0f + t * (1.0f / 6))))));
    return __builtin_amdgcn_sqrtf(t > -0.25f ? series : 1.0f - exp_t);
}
__device__ __forceinline__ float gelu_tanh_row(float z) {
    const float u = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    return 0.5f * z * (1.0f + tanhf(u));
}
// sum over the 16 lanes of a DPP row, in every lane
__device__ __forceinline__ float row16_sum(float v) {
    v += dpp_move<0xB1, 0xF>(v, 0.f);
    v += dpp_move<0x4E, 0xF>(v, 0.f);
    v += dpp_move<0x141, 0xF>(v, 0.f);
    v += dpp_move<0x140, 0xF>(v, 0.f);
    return v;
}

// ── convolution rows ─────────────────────────────────────────────────────────

__device__ __forceinline__ float side_act(float v, int act) {
    return act == ConvRowsArgs::Silu ? v * sigmoid_dev(v) : act == ConvRowsArgs::Gelu ? gelu_tanh_row(v) : v;
}

// Four neighbouring channels a lane, CONV_ROWS rows a wavefront: everything a wavefront needs is requested at once.
// Columns from ring.width on are side columns, which only go through an activation. PARTS: most K slices.
constexpr int CONV_ROWS = 4;
template <int TAPS, int PARTS>
__global__ __launch_bounds__(256) void conv_rows_kernel(ConvRowsArgs a) {
    const int c = (blockIdx.x * 64 + (threadIdx.x & 63)) * 4, t0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * CONV_ROWS;
    const int width = a.ring.width;
    if (c >= width + a.side_cols || t0 >= a.n) return;
    constexpr int HIST = TAPS - 1, ROWS = HIST + CONV_ROWS;
    f32x4 v[ROWS];
    const int hist = c < width ? HIST : 0;
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const int t = t0 + r - HIST, pos = a.past + t;
        v[r] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (r < HIST - hist) continue;
        if (t >= 0)
            v[r] = sum_parts_upto<PARTS, f32x4>(a.in.p, (size_t)min(t, a.n - 1) * a.in.ld + c, a.in.parts, a.in.stride);
        else if (pos >= 0)
            v[r] = *reinterpret_cast<const f32x4 *>(a.ring.ring + (size_t)(pos % TAPS) * width + c);
    }
    if (a.in.bias) {
        const f32x4 b = *reinterpret_cast<const f32x4 *>(a.in.bias + c);
#pragma unroll
        for (int r = 0; r < ROWS; r++)
            if (t0 + r - HIST >= 0) v[r] += b;  // (the ring holds inputs with their bias)
    }
    if (c >= width) {
#pragma unroll
        for (int r = HIST; r < ROWS; r++) {
            const int t = t0 + r - HIST;
            if (t >= a.n) break;
#pragma unroll
            for (int k = 0; k < 4; k++) v[r][k] = side_act(v[r][k], a.side_act);
            *reinterpret_cast<f32x4 *>(a.side + (size_t)t * a.side_cols + c - width) = v[r];
        }
        return;
    }
    f32x4 w[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; j++) w[j] = *reinterpret_cast<const f32x4 *>(a.w + (size_t)j * width + c);
    const f32x4 bias = *reinterpret_cast<const f32x4 *>(a.b + c);
    const bool split = a.out_split && c < a.channels;
    const bool whole = a.block_width % 4 == 0;  // the four channels share a block, and their places are vectors
#pragma unroll
    for (int r = 0; r < CONV_ROWS; r++) {
        const int t = t0 + r;
        if (t >= a.n) break;
        f32x4 u = bias;
#pragma unroll
        for (int j = 0; j < TAPS; j++)
#pragma unroll
            for (int k = 0; k < 4; k++) u[k] = fmaf(w[j][k], v[r + j][k], u[k]);
        if (a.silu) {
#pragma unroll
            for (int k = 0; k < 4; k++) u[k] = u[k] * sigmoid_dev(u[k]);
        }
        *reinterpret_cast<f32x4 *>(a.out + (size_t)t * width + c) = u;
        if (!split) continue;
        if (whole) {
            const int blk = c / a.block_width;
            split_store4(a.out_split + ((size_t)blk * a.n + t) * a.pieces * a.block_pad, a.block_pad, c - blk * a.block_width, u, a.pieces);
        } else {
#pragma unroll
            for (int k = 0; k < 4; k++)
                if (c + k < a.channels) {
                    const int blk = (c + k) / a.block_width;
                    split_store(a.out_split + ((size_t)blk * a.n + t) * a.pieces * a.block_pad, a.block_pad, c + k - blk * a.block_width, u[k], a.pieces);
                }
        }
    }
}

// Any number of taps: a thread walks one channel over CONV_ANY_ROWS rows, its inputs in LDS.
constexpr int CONV_ANY_ROWS = 16;
extern __shared__ float conv_lds[];
__global__ __launch_bounds__(256) void conv_rows_any_kernel(ConvRowsArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * CONV_ANY_ROWS;
    const int width = a.ring.width, taps = a.ring.taps, hist = taps - 1;
    if (c >= width + a.side_cols) return;  // (no barrier below: a thread reads only its own column)
    const int rows = min(CONV_ANY_ROWS, a.n - t0);
    if (c >= width) {
        for (int r = 0; r < rows; r++) a.side[(size_t)(t0 + r) * a.side_cols + c - width] = side_act(source_at(a.in, t0 + r, c), a.side_act);
        return;
    }
    float *col = conv_lds + threadIdx.x;
    for (int r = -hist; r < rows; r++) {
        const int t = t0 + r, pos = a.past + t;
        float v = 0.f;
        if (t >= 0) v = source_at(a.in, t, c);
        else if (pos >= 0) v = a.ring.ring[(size_t)(pos % taps) * width + c];
        col[(r + hist) * 256] = v;
    }
    const float bias = a.b[c];
    const int blk = a.out_split && c < a.channels ? c / a.block_width : -1;
    for (int r = 0; r < rows; r++) {
        float u = bias;
        for (int j = 0; j < taps; j++) u = fmaf(a.w[(size_t)j * width + c], col[(r + j) * 256], u);
        if (a.silu) u = u * sigmoid_dev(u);
        const int t = t0 + r;
        a.out[(size_t)t * width + c] = u;
        if (blk >= 0)
            split_store(a.out_split + ((size_t)blk * a.n + t) * a.pieces * a.block_pad, a.block_pad, c - blk * a.block_width, u, a.pieces);
    }
}

// the chunk's last inputs of channels c0 .. c0 + 15 go into the ring (all threads of the workgroup)
__device__ __forceinline__ void store_taps(const RowSource &in, const TapRing &ring, int c0, int n, int past) {
    const int c = c0 + (threadIdx.x & 15);
    for (int t = max(0, n - ring.taps) + (threadIdx.x >> 4); t < n; t += blockDim.x >> 4)
        if (c < ring.width) ring.ring[(size_t)((past + t) % ring.taps) * ring.width + c] = source_at(in, t, c);
}

// ── selective scan ───────────────────────────────────────────────────────────

// 16 channels a workgroup, 16 lanes a channel, SPL states a lane. Tiles of SCAN_T tokens: the next tile is on its
// way into registers while this one is scanned out of LDS, four tokens a read (token-minor rows of SCAN_T + 4
// floats: the 16-byte reads of 16 neighbouring rows touch every bank once). Rows behind the chunk's end scan as dt = 0, which
// leaves the state as it is.
template <int SPL>
__global__ __launch_bounds__(256) void selective_scan_kernel(SelectiveScanArgs a) {
    constexpr int SCAN_T = SPL <= 2 ? 64 : 32, SCAN_LD = SCAN_T + 4;  // (longer tiles hide the loads of the next one)
    constexpr int SP = 16 * SPL;
    constexpr int E = SCAN_T * 16 / 256, EB = SCAN_T * SP / 256;
    __shared__ __attribute__((aligned(16))) float s_dt[16][SCAN_LD], s_dx[16][SCAN_LD], s_y[16][SCAN_LD];
    __shared__ __attribute__((aligned(16))) float s_b[SP][SCAN_LD], s_c[SP][SCAN_LD];
    const int tid = threadIdx.x, ch = tid >> 4, l = tid & 15, c0 = blockIdx.x * 16, n = a.n;
    float A[SPL], S[SPL];
#pragma unroll
    for (int k = 0; k < SPL; k++) {
        const size_t at = (size_t)(c0 + ch) * SP + l + 16 * k;
        A[k] = a.a_log2[at];
        S[k] = a.past ? a.state[at] : 0.f;
    }
    const int ec = c0 + l, er = tid >> 4;  // this thread's channel and first row in loads and stores
    const bool odd = l & 1, upper = l & 2;
    const float d_c = a.d[ec], dt_bias = a.dt_bias[ec];
    float r_dt[E], r_x[E], r_z[E], r_b[EB], r_c[EB];
    auto load_tile = [&](int t0) {
#pragma unroll
        for (int e = 0; e < E; e++) {
            const size_t at = (size_t)min(t0 + er + e * 16, n - 1) * a.inner + ec;
            r_dt[e] = a.dt[at];
            r_x[e] = a.x[at];
            r_z[e] = a.z[at];
        }
#pragma unroll
        for (int e = 0; e < EB; e++) {
            const int i = tid + e * 256;
            const size_t at = (size_t)min(t0 + i / SP, n - 1) * a.bc_ld + i % SP;
            r_b[e] = a.b[at];
            r_c[e] = a.c[at];
        }
    };
    load_tile(0);
    for (int t0 = 0; t0 < n; t0 += SCAN_T) {
        float x[E], z[E];
#pragma unroll
        for (int e = 0; e < E; e++) {
            float dt = softplus_dev(r_dt[e] + dt_bias);
            if (t0 + er + e * 16 >= n) dt = 0.f;
            x[e] = r_x[e];
            z[e] = r_z[e];
            s_dt[l][er + e * 16] = dt;
            s_dx[l][er + e * 16] = dt * x[e];
        }
#pragma unroll
        for (int e = 0; e < EB; e++) {
            const int i = tid + e * 256;
            s_b[i % SP][i / SP] = r_b[e];
            s_c[i % SP][i / SP] = r_c[e];
        }
        __syncthreads();
        if (t0 + SCAN_T < n) load_tile(t0 + SCAN_T);
        // straight-line code: the reads of the next four tokens are issued before this four's arithmetic, and a
        // lane keeps the result of the token it will store (token l of every sixteen)
        f32x4 dt[2], dx[2], b[2][SPL], c[2][SPL];
        auto read = [&](int set, int t) {
            dt[set] = *reinterpret_cast<const f32x4 *>(&s_dt[ch][t]);
            dx[set] = *reinterpret_cast<const f32x4 *>(&s_dx[ch][t]);
#pragma unroll
            for (int k = 0; k < SPL; k++) {
                b[set][k] = *reinterpret_cast<const f32x4 *>(&s_b[l + 16 * k][t]);
                c[set][k] = *reinterpret_cast<const f32x4 *>(&s_c[l + 16 * k][t]);
            }
        };
        read(0, 0);
        float y = 0.f;
#pragma unroll
        for (int t = 0; t < SCAN_T; t += 4) {
            const int set = (t >> 2) & 1;
            if (t + 4 < SCAN_T) read(set ^ 1, t + 4);
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < SPL; k++) {
                float g[4], h[4];
#pragma unroll
                for (int u = 0; u < 4; u++) {
                    g[u] = __builtin_amdgcn_exp2f(dt[set][u] * A[k]);
                    h[u] = dx[set][u] * b[set][k][u];
                }
#pragma unroll
                for (int u = 0; u < 4; u++) {
                    S[k] = fmaf(g[u], S[k], h[u]);
                    acc[u] = fmaf(S[k], c[set][k][u], acc[u]);
                }
            }
            // lane l receives the sum over the 16 lanes for token l % 4
            const float p0 = (odd ? acc[1] : acc[0]) + dpp_move<0xB1, 0xF>(odd ? acc[0] : acc[1], 0.f);
            const float p1 = (odd ? acc[3] : acc[2]) + dpp_move<0xB1, 0xF>(odd ? acc[2] : acc[3], 0.f);
            float v = (upper ? p1 : p0) + dpp_move<0x4E, 0xF>(upper ? p0 : p1, 0.f);
            v += dpp_move<0x124, 0xF>(v, 0.f);  // row_ror:4
            v += dpp_move<0x128, 0xF>(v, 0.f);  // row_ror:8
            y = (l >> 2) == ((t >> 2) & 3) ? v : y;
            if ((t & 15) == 12) s_y[ch][t - 12 + l] = y;
        }
        __syncthreads();
#pragma unroll
        for (int e = 0; e < E; e++) {
            const int r = er + e * 16;
            if (t0 + r < n)
                split_store(a.out_split + (size_t)(t0 + r) * a.pieces * a.inner, a.inner, ec, fmaf(d_c, x[e], s_y[l][r]) * z[e], a.pieces);
        }
        // (the next tile's staging writes none of what is read here: s_y is written behind its barrier)
    }
#pragma unroll
    for (int k = 0; k < SPL; k++) a.state[(size_t)(c0 + ch) * SP + l + 16 * k] = S[k];
    store_taps(a.conv_in, a.ring, c0, n, a.past);
}

template <int SPL>
__global__ __launch_bounds__(256) void selective_step_kernel(SelectiveStepArgs a) {
    constexpr int SP = 16 * SPL;
    const int tid = threadIdx.x, l = tid & 15, c = blockIdx.x * 16 + (tid >> 4);
    const bool fresh = a.cursor->pos == 0;
    float A[SPL], S[SPL], B[SPL], C[SPL];
#pragma unroll
    for (int k = 0; k < SPL; k++) {
        const size_t at = (size_t)c * SP + l + 16 * k;
        A[k] = a.a_log2[at];
        S[k] = a.state[at];
        B[k] = a.p[a.dt_pad + l + 16 * k];
        C[k] = a.p[a.dt_pad + SP + l + 16 * k];
    }
    const float x = a.xz[c], z = a.xz[a.inner + c];
    float low = 0.f;
    for (int k = l * 8; k < a.dt_pad; k += 128) {
        const u32x4 w = ld128(a.dt_w + (size_t)c * a.dt_pad + k);
        const f32x4 p0 = *reinterpret_cast<const f32x4 *>(a.p + k), p1 = *reinterpret_cast<const f32x4 *>(a.p + k + 4);
        low = fmaf(bf16_lo(w.x), p0[0], low);
        low = fmaf(bf16_hi(w.x), p0[1], low);
        low = fmaf(bf16_lo(w.y), p0[2], low);
        low = fmaf(bf16_hi(w.y), p0[3], low);
        low = fmaf(bf16_lo(w.z), p1[0], low);
        low = fmaf(bf16_hi(w.z), p1[1], low);
        low = fmaf(bf16_lo(w.w), p1[2], low);
        low = fmaf(bf16_hi(w.w), p1[3], low);
    }
    const float dt = softplus_dev(row16_sum(low) + a.dt_b[c]), dx = dt * x;
    float acc = 0.f;
#pragma unroll
    for (int k = 0; k < SPL; k++) {
        const float s = fmaf(__builtin_amdgcn_exp2f(dt * A[k]), fresh ? 0.f : S[k], dx * B[k]);
        a.state[(size_t)c * SP + l + 16 * k] = s;
        acc = fmaf(s, C[k], acc);
    }
    acc = row16_sum(acc);
    if (l == 0) a.y[c] = fmaf(a.d[c], x, acc) * (z / (1.0f + expf(-z)));
}

// ── gated linear recurrence ──────────────────────────────────────────────────

// 16 channels a workgroup; the chunk is cut into LR_SEGS segments of at most LR_LEN rows. A thread forms (decay,
// input) of its channel and segment in registers, with the segment's total (product of decays, what a zero state
// becomes); the state each segment starts from follows from the totals of those before it, and a second walk gives
// the states.
constexpr int LR_SEGS = 64, LR_LEN = 8, LR_MAX_ROWS = LR_SEGS * LR_LEN;
__global__ __launch_bounds__(16 * LR_SEGS) void linear_recurrence_kernel(LinearRecurrenceArgs a) {
    __shared__ float s_p[LR_SEGS][16], s_q[LR_SEGS][16];
    const int ch = threadIdx.x & 15, seg = threadIdx.x >> 4, c0 = blockIdx.x * 16, c = c0 + ch, n = a.n;
    const bool live = c < a.channels;
    const int cc = live ? c : 0;
    const int len = (n + LR_SEGS - 1) / LR_SEGS, t_begin = min(n, seg * len), rows = min(n, t_begin + len) - t_begin;
    const int blk = cc / a.block_width, gate_ld = (a.channels / a.block_width) * 2 * a.block_pad;
    const float *gr = a.gates + blk * 2 * a.block_pad + (cc - blk * a.block_width), *gi = gr + a.block_pad;
    const float rb = a.r_bias[cc], ib = a.i_bias[cc], decay = a.decay[cc];
    float av[LR_LEN], bv[LR_LEN], yv[LR_LEN];
    float S = a.past && live ? a.state[c] : 0.f;  // (read ahead of the barrier: one segment writes it at the end)
    {
        float r_[LR_LEN], i_[LR_LEN], u_[LR_LEN];
#pragma unroll
        for (int k = 0; k < LR_LEN; k++) {
            const size_t t = min(t_begin + k, n - 1);
            r_[k] = gr[t * gate_ld];
            i_[k] = gi[t * gate_ld];
            u_[k] = a.u[t * a.width + cc];
            yv[k] = a.y[t * a.width + cc];
        }
#pragma unroll
        for (int k = 0; k < LR_LEN; k++) {
            const float la = decay * sigmoid_dev(r_[k] + rb);
            av[k] = exp_dev(la);
            bv[k] = input_gain(2.0f * la, av[k] * av[k]) * (sigmoid_dev(i_[k] + ib) * u_[k]);
        }
    }
    float P = 1.f, Q = 0.f;
#pragma unroll
    for (int k = 0; k < LR_LEN; k++)
        if (k < rows) {
            P *= av[k];
            Q = fmaf(av[k], Q, bv[k]);
        }
    s_p[seg][ch] = P;
    s_q[seg][ch] = Q;
    __syncthreads();
#pragma unroll 8
    for (int s = 0; s < seg; s++) S = fmaf(s_p[s][ch], S, s_q[s][ch]);
    if (live) {
#pragma unroll
        for (int k = 0; k < LR_LEN; k++)
            if (k < rows) {
                S = fmaf(av[k], S, bv[k]);
                split_store(a.out_split + (size_t)(t_begin + k) * a.pieces * a.width, a.width, c, S * yv[k], a.pieces);
            }
        // the thread that walked the last row holds the state (trailing segments of a short chunk are empty)
        if (rows > 0 && t_begin + rows == n) a.state[c] = S;
    }
    store_taps(a.conv_in, a.ring, c0, n, a.past);
}

// A wavefront takes one channel: its halves multiply the r and the i row of the gates. VEC: blocks of whole vectors.
template <bool VEC>
__global__ __launch_bounds__(256) void linear_recurrence_step_kernel(LinearRecurrenceStepArgs a) {
    const int lane = threadIdx.x & 63, half = lane >> 5, l = lane & 31;
    const int c = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (c >= a.channels) return;
    const int blk = c / a.block_width, j = c - blk * a.block_width;
    const uint16_t *w = a.gate_w + ((size_t)(2 * blk + half) * a.block_pad + j) * a.block_pad;
    const float *u = a.uy + (size_t)blk * a.block_width;
    const bool fresh = a.cursor->pos == 0;
    const float rb = a.r_bias[c], ib = a.i_bias[c], decay = a.decay[c], s0 = a.state[c], uc = a.uy[c], yc = a.uy[a.width + c];
    float acc = 0.f;
    for (int k = l * 8; k < a.block_pad; k += 256) {  // weights behind block_width are zero
        const u32x4 v = ld128(w + k);
        float x[8];
        if (VEC) {
            const f32x4 x0 = *reinterpret_cast<const f32x4 *>(u + k), x1 = *reinterpret_cast<const f32x4 *>(u + k + 4);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                x[i] = x0[i];
                x[4 + i] = x1[i];
            }
        } else {
#pragma unroll
            for (int i = 0; i < 8; i++) x[i] = u[k + i];
        }
        acc = fmaf(bf16_lo(v.x), x[0], acc);
        acc = fmaf(bf16_hi(v.x), x[1], acc);
        acc = fmaf(bf16_lo(v.y), x[2], acc);
        acc = fmaf(bf16_hi(v.y), x[3], acc);
        acc = fmaf(bf16_lo(v.z), x[4], acc);
        acc = fmaf(bf16_hi(v.z), x[5], acc);
        acc = fmaf(bf16_lo(v.w), x[6], acc);
        acc = fmaf(bf16_hi(v.w), x[7], acc);
    }
    acc = row16_sum(acc);
    acc += __shfl_xor(acc, 16);
    const float r_dot = __shfl(acc, 0), i_dot = __shfl(acc, 32);
    if (lane == 0) {
        const float la = decay * sigmoid_dev(r_dot + rb), av = exp_dev(la);
        const float S = fmaf(av, fresh ? 0.f : s0, input_gain(2.0f * la, av * av) * (sigmoid_dev(i_dot + ib) * uc));
        a.state[c] = S;
        a.out[c] = S * yc;
    }
}

}  // namespace

namespace homura {

int ssm_state_pad(int state) { return state <= 16 ? 16 : state <= 32 ? 32 : state <= 64 ? 64 : 128; }

int conv_rows_launch(hm_ctx *ctx, const ConvRowsArgs &a) {
    const int width = a.ring.width, taps = a.ring.taps;
    HM_REQUIRE(ctx, a.ring.ring && a.w && a.b && a.out && a.n > 0 && a.past >= 0 && width > 0 && taps >= 1 && !bad_source(a.in, width),
               "conv_rows: bad arguments");
    HM_REQUIRE(ctx, !a.out_split || (a.block_width > 0 && a.block_pad >= a.block_width && a.channels <= width && a.channels > 0 && a.pieces >= 1 && a.pieces <= 3),
               "conv_rows: bad split shape");
    HM_REQUIRE(ctx, a.side_cols == 0 || (a.side && a.in.ld >= width + a.side_cols), "conv_rows: bad side columns");
    const int cols = width + a.side_cols;
    if (taps <= 4 && width % 4 == 0 && a.side_cols % 4 == 0) {
        HM_REQUIRE(ctx, a.in.ld % 4 == 0 && a.in.stride % 4 == 0 && ((uintptr_t)a.in.p % 16) == 0 && ((uintptr_t)a.in.bias % 16) == 0 &&
                            ((uintptr_t)a.out % 16) == 0 && ((uintptr_t)a.side % 16) == 0 && ((uintptr_t)a.ring.ring % 16) == 0 &&
                            ((uintptr_t)a.w % 16) == 0 && ((uintptr_t)a.b % 16) == 0 && ((uintptr_t)a.out_split % 8) == 0 && a.block_pad % 4 == 0,
                   "conv_rows: misaligned rows");
        const dim3 g((cols + 255) / 256, (a.n + 4 * CONV_ROWS - 1) / (4 * CONV_ROWS)), b(256);
#define HM_CONV(T)                                                                                                       \
    if (taps == T) {                                                                                                     \
        if (a.in.parts == 1) hipLaunchKernelGGL((conv_rows_kernel<T, 1>), g, b, 0, ctx->stream, a);                      \
        else if (a.in.parts == 2) hipLaunchKernelGGL((conv_rows_kernel<T, 2>), g, b, 0, ctx->stream, a);                 \
        else hipLaunchKernelGGL((conv_rows_kernel<T, MAX_SUM_PARTS>), g, b, 0, ctx->stream, a);                          \
    }
        HM_CONV(1) HM_CONV(2) HM_CONV(3) HM_CONV(4)
#undef HM_CONV
    } else {
        const size_t lds = (size_t)(CONV_ANY_ROWS + taps - 1) * 256 * 4;
        HM_REQUIRE(ctx, lds <= 64 * 1024, "conv_rows: %d taps need %zu bytes of LDS", taps, lds);
        hipLaunchKernelGGL(conv_rows_any_kernel, dim3((cols + 255) / 256, (a.n + CONV_ANY_ROWS - 1) / CONV_ANY_ROWS), dim3(256), lds, ctx->stream, a);
    }
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int selective_scan_launch(hm_ctx *ctx, const SelectiveScanArgs &a) {
    HM_REQUIRE(ctx, a.x && a.dt && a.dt_bias && a.z && a.b && a.c && a.a_log2 && a.d && a.state && a.out_split && a.ring.ring && a.n > 0 && a.past >= 0, "selective_scan: bad arguments");
    HM_REQUIRE(ctx, a.inner > 0 && a.inner % 16 == 0 && a.ring.width == a.inner && a.bc_ld >= a.state_pad && a.pieces >= 1 && a.pieces <= 3 &&
                        !bad_source(a.conv_in, a.inner), "selective_scan: bad shape");
    const dim3 g(a.inner / 16), b(256);
    switch (a.state_pad) {
    case 16: hipLaunchKernelGGL(selective_scan_kernel<1>, g, b, 0, ctx->stream, a); break;
    case 32: hipLaunchKernelGGL(selective_scan_kernel<2>, g, b, 0, ctx->stream, a); break;
    case 64: hipLaunchKernelGGL(selective_scan_kernel<4>, g, b, 0, ctx->stream, a); break;
    case 128: hipLaunchKernelGGL(selective_scan_kernel<8>, g, b, 0, ctx->stream, a); break;
    default: return hm_set_error(ctx, HM_ERR_INVALID, "selective_scan: %d padded states", a.state_pad);
    }
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int selective_step_launch(hm_ctx *ctx, const SelectiveStepArgs &a) {
    HM_REQUIRE(ctx, a.xz && a.p && a.dt_w && a.dt_b && a.a_log2 && a.d && a.state && a.y && a.cursor, "selective_step: NULL pointer");
    HM_REQUIRE(ctx, a.inner > 0 && a.inner % 16 == 0 && a.dt_pad % 8 == 0 && ((uintptr_t)a.p % 16) == 0 && ((uintptr_t)a.dt_w % 16) == 0, "selective_step: bad shape");
    const dim3 g(a.inner / 16), b(256);
    switch (a.state_pad) {
    case 16: hipLaunchKernelGGL(selective_step_kernel<1>, g, b, 0, ctx->stream, a); break;
    case 32: hipLaunchKernelGGL(selective_step_kernel<2>, g, b, 0, ctx->stream, a); break;
    case 64: hipLaunchKernelGGL(selective_step_kernel<4>, g, b, 0, ctx->stream, a); break;
    case 128: hipLaunchKernelGGL(selective_step_kernel<8>, g, b, 0, ctx->stream, a); break;
    default: return hm_set_error(ctx, HM_ERR_INVALID, "selective_step: %d padded states", a.state_pad);
    }
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int linear_recurrence_launch(hm_ctx *ctx, const LinearRecurrenceArgs &a) {
    HM_REQUIRE(ctx, a.u && a.gates && a.y && a.r_bias && a.i_bias && a.decay && a.state && a.out_split && a.ring.ring, "linear_recurrence: NULL pointer");
    HM_REQUIRE(ctx, a.n > 0 && a.past >= 0 && a.channels > 0 && a.channels <= a.width && a.ring.width == a.width &&
                        a.block_width > 0 && a.block_pad >= a.block_width && a.channels % a.block_width == 0 && a.pieces >= 1 && a.pieces <= 3 &&
                        !bad_source(a.conv_in, a.width), "linear_recurrence: bad shape");
    const size_t gate_ld = (size_t)(a.channels / a.block_width) * 2 * a.block_pad;
    for (int at = 0; at < a.n; at += LR_MAX_ROWS) {  // what a workgroup holds in registers at a time
        LinearRecurrenceArgs b = a;
        b.n = a.n - at < LR_MAX_ROWS ? a.n - at : LR_MAX_ROWS;
        b.past = a.past + at;
        b.u = a.u + (size_t)at * a.width;
        b.y = a.y + (size_t)at * a.width;
        b.gates = a.gates + at * gate_ld;
        b.out_split = a.out_split + (size_t)at * a.pieces * a.width;
        b.conv_in.p = a.conv_in.p + (size_t)at * a.conv_in.ld;
        hipLaunchKernelGGL(linear_recurrence_kernel, dim3((a.width + 15) / 16), dim3(16 * LR_SEGS), 0, ctx->stream, b);
        HM_LAUNCH_CHECK(ctx);
    }
    return HM_OK;
}

int linear_recurrence_step_launch(hm_ctx *ctx, const LinearRecurrenceStepArgs &a) {
    HM_REQUIRE(ctx, a.uy && a.gate_w && a.r_bias && a.i_bias && a.decay && a.state && a.out && a.cursor, "linear_recurrence_step: NULL pointer");
    HM_REQUIRE(ctx, a.channels > 0 && a.channels <= a.width && a.block_width > 0 && a.channels % a.block_width == 0 && a.block_pad >= a.block_width &&
                        a.block_pad % 8 == 0 && (a.block_pad - a.block_width) <= a.width && ((uintptr_t)a.gate_w % 16) == 0, "linear_recurrence_step: bad shape");
    const dim3 g((a.channels + 3) / 4), b(256);
    if (a.block_width % 4 == 0 && ((uintptr_t)a.uy % 16) == 0) hipLaunchKernelGGL(linear_recurrence_step_kernel<true>, g, b, 0, ctx->stream, a);
    else hipLaunchKernelGGL(linear_recurrence_step_kernel<false>, g, b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
