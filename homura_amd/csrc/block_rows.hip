// Row kernels of decoders with a norm ahead of and behind every sublayer (see block_rows.h).
#include "block_rows.h"

#include "row_pieces.h"

namespace {

using homura::RowNormArgs;

constexpr int RN_THREADS = 256;
constexpr int RN_KEEP = 8;  // vectors of four a thread keeps: rows up to 8192 wide stay in registers

__device__ __forceinline__ float wg_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();  // red may still be read from the sum before
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

__device__ __forceinline__ float dot4v(f32x4 v) { return (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }

template <int KEEP>
__global__ __launch_bounds__(RN_THREADS) void row_norm_kernel(RowNormArgs a) {
    __shared__ float red[4];
    const size_t base = (size_t)blockIdx.x * a.dim;
    const int dim = a.dim;
    f32x4 v[KEEP];
    if (a.y) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int i = (threadIdx.x + j * RN_THREADS) * 4;
            v[j] = i < dim ? sum_parts4(a.y, base + i, a.y_parts, a.y_stride) : f32x4{0.f, 0.f, 0.f, 0.f};
            ss += dot4v(v[j]);
        }
        if (a.y_w) {
            const float inv = 1.0f / sqrtf(wg_sum(ss, red) / (float)a.norm_dim + a.eps);
#pragma unroll
            for (int j = 0; j < KEEP; j++) {
                const int i = (threadIdx.x + j * RN_THREADS) * 4;
                if (i < dim) v[j] = (v[j] * inv) * *reinterpret_cast<const f32x4 *>(a.y_w + i);
            }
        }
    } else {
#pragma unroll
        for (int j = 0; j < KEEP; j++) v[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; j++) {
        const int i = (threadIdx.x + j * RN_THREADS) * 4;
        if (i < dim) {
            if (a.x) v[j] = *reinterpret_cast<const f32x4 *>(a.x + base + i) + v[j];
            if (a.r_out) *reinterpret_cast<f32x4 *>(a.r_out + base + i) = v[j];
            ss += dot4v(v[j]);
        }
    }
    float inv = 1.f;
    if (a.w) inv = 1.0f / sqrtf(wg_sum(ss, red) / (float)a.norm_dim + a.eps);
    if (!a.out && !a.out_split) return;
    const int ld = a.cat ? 2 * dim : dim;
    uint16_t *o = a.out_split ? a.out_split + (size_t)blockIdx.x * a.pieces * ld : nullptr;
#pragma unroll
    for (int j = 0; j < KEEP; j++) {
        const int i = (threadIdx.x + j * RN_THREADS) * 4;
        if (i < dim) {
            const f32x4 y = a.w ? (v[j] * inv) * *reinterpret_cast<const f32x4 *>(a.w + i) : v[j];
            if (a.out) *reinterpret_cast<f32x4 *>(a.out + base + i) = y;
            if (o) split_store4(o, ld, i, y, a.pieces);
            if (o && a.cat) split_store4(o, ld, dim + i, *reinterpret_cast<const f32x4 *>(a.cat + base + i), a.pieces);
        }
    }
}

__global__ __launch_bounds__(256) void sum_parts_kernel(const float *__restrict__ x, int ld, int parts, size_t stride,
                                                        float *__restrict__ out, int n_out, uint16_t *__restrict__ split,
                                                        int split_cols, size_t n4) {
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= n4) return;
    const size_t row = e * 4 / n_out;
    const int c = (int)(e * 4 % n_out);
    const f32x4 v = sum_parts4(x, row * ld + c, parts, stride);
    *reinterpret_cast<f32x4 *>(out + row * n_out + c) = v;
    if (split && c < split_cols) split_store4(split + row * 3 * split_cols, split_cols, c, v, 3);
}

// sine and cosine of an f64 angle: reduced to [-pi, pi] in f64, the rest in f32
__device__ __forceinline__ void wave_pair(double angle, float &sn, float &cs) {
    const double turns = rint(angle * 0.15915494309189533577);
    const float r = (float)fma(turns, -6.28318530717958647693, angle);
    sn = sinf(r);
    cs = cosf(r);
}

// one workgroup per id; ids outside the table read row 0 (the host checks them)
__global__ __launch_bounds__(256) void embed_scaled_kernel(const int32_t *__restrict__ ids, const DecodeState *__restrict__ state,
                                                           const int32_t *__restrict__ forced, const float *__restrict__ table,
                                                           float *__restrict__ out, float *__restrict__ out2, int vocab, int hidden,
                                                           float scale, homura::PositionWaves waves, int past) {
    int id, pos = past + blockIdx.x;
    if (state) {
        pos = state->pos;
        const int step = state->step, n_forced = state->n_forced, token = state->token;
        id = step < n_forced ? forced[step] : token;
    } else {
        id = ids[blockIdx.x];
    }
    if (id < 0 || id >= vocab) id = 0;
    const float *src = table + (size_t)id * hidden;
    for (int k = threadIdx.x * 4; k < hidden; k += 1024) {
        f32x4 v = *reinterpret_cast<const f32x4 *>(src + k) * scale;
        if (waves.freq) {
#pragma unroll
            for (int j = 0; j < 4; j += 2)
                if (k + j < waves.width) {
                    float sn, cs;
                    wave_pair((double)pos * waves.freq[(k + j) / 2], sn, cs);
                    v[j] += sn;
                    if (k + j + 1 < waves.width) v[j + 1] += cs;
                }
        }
        *reinterpret_cast<f32x4 *>(out + (size_t)blockIdx.x * hidden + k) = v;
        if (out2) *reinterpret_cast<f32x4 *>(out2 + (size_t)blockIdx.x * hidden + k) = v;
    }
}

bool al16(const void *p) { return ((uintptr_t)p % 16) == 0; }

}  // namespace

namespace homura {

int row_norm_launch(hm_ctx *ctx, const RowNormArgs &a) {
    HM_REQUIRE(ctx, (a.x || a.y) && (a.r_out || a.out || a.out_split), "row_norm: NULL pointer");
    HM_REQUIRE(ctx, a.rows > 0 && a.dim > 0 && a.dim % 4 == 0 && a.dim <= RN_KEEP * 1024 && a.norm_dim > 0 && a.norm_dim <= a.dim,
               "row_norm: bad shape (dim=%d, norm over %d)", a.dim, a.norm_dim);
    HM_REQUIRE(ctx, a.y_parts >= 1 && a.y_parts <= MAX_SUM_PARTS && a.y_stride % 4 == 0 && a.pieces >= 1 && a.pieces <= 3, "row_norm: bad slices or pieces");
    HM_REQUIRE(ctx, al16(a.x) && al16(a.y) && al16(a.y_w) && al16(a.r_out) && al16(a.w) && al16(a.out) && al16(a.cat) &&
                        ((uintptr_t)a.out_split % 8) == 0, "row_norm: misaligned buffer");
    const dim3 g(a.rows), b(RN_THREADS);
    if (a.dim <= 1024) hipLaunchKernelGGL(row_norm_kernel<1>, g, b, 0, ctx->stream, a);
    else if (a.dim <= 2048) hipLaunchKernelGGL(row_norm_kernel<2>, g, b, 0, ctx->stream, a);
    else if (a.dim <= 4096) hipLaunchKernelGGL(row_norm_kernel<4>, g, b, 0, ctx->stream, a);
    else hipLaunchKernelGGL(row_norm_kernel<8>, g, b, 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int sum_parts_launch(hm_ctx *ctx, const float *d_x, int ld, int parts, size_t stride, float *d_out, int rows, int n_out,
                     uint16_t *d_split, int split_cols) {
    HM_REQUIRE(ctx, d_x && d_out && al16(d_x) && al16(d_out), "sum_parts: NULL or misaligned pointer");
    HM_REQUIRE(ctx, rows > 0 && n_out > 0 && n_out % 4 == 0 && ld % 4 == 0 && ld >= n_out && parts >= 1 && parts <= MAX_SUM_PARTS && stride % 4 == 0,
               "sum_parts: bad shape");
    HM_REQUIRE(ctx, !d_split || (split_cols > 0 && split_cols % 4 == 0 && split_cols <= n_out && ((uintptr_t)d_split % 8) == 0), "sum_parts: bad split");
    const size_t n4 = (size_t)rows * n_out / 4;
    hipLaunchKernelGGL(sum_parts_kernel, dim3((unsigned)((n4 + 255) / 256)), dim3(256), 0, ctx->stream, d_x, ld, parts, stride, d_out, n_out, d_split,
                       split_cols, n4);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int embed_scaled_launch(hm_ctx *ctx, const int32_t *d_ids, const float *d_table, float *d_out, int n_ids, int vocab,
                        int hidden, float scale, PositionWaves waves, int past) {
    HM_REQUIRE(ctx, d_ids && d_table && d_out && n_ids > 0 && hidden > 0 && hidden % 4 == 0 && al16(d_table) && al16(d_out), "embed_scaled: bad arguments");
    hipLaunchKernelGGL(embed_scaled_kernel, dim3(n_ids), dim3(256), 0, ctx->stream, d_ids, nullptr, nullptr, d_table, d_out, nullptr,
                       vocab, hidden, scale, waves, past);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int embed_step_scaled_launch(hm_ctx *ctx, const DecodeState *state, const int32_t *d_forced, const float *d_table,
                             float *d_out, float *d_out2, int vocab, int hidden, float scale, PositionWaves waves) {
    HM_REQUIRE(ctx, state && d_forced && d_table && d_out && hidden > 0 && hidden % 4 == 0 && al16(d_table) && al16(d_out) && al16(d_out2),
               "embed_step_scaled: bad arguments");
    hipLaunchKernelGGL(embed_scaled_kernel, dim3(1), dim3(256), 0, ctx->stream, nullptr, state, d_forced, d_table, d_out, d_out2, vocab,
                       hidden, scale, waves, 0);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
