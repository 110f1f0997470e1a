// Matrix memory with exponential gates (see matrix_memory.h).
#include "matrix_memory.h"

#include <algorithm>

#include "lds_tiles.h"

namespace {

using namespace homura;

__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float soft_cap(float z, float cap) { return cap * tanhf(z / cap); }

// Sum over the lanes of a wavefront that share lane % 4 (every lane receives its group's).
__device__ __forceinline__ float stride4_sum(float v) {
    v += dpp_move<0x124, 0xF>(v, 0.f);  // row_ror:4
    v += dpp_move<0x128, 0xF>(v, 0.f);  // row_ror:8
    return quad_rows_sum(v);
}

// ── one token ────────────────────────────────────────────────────────────────

// A tile of 16 columns of a head's memory in the registers of 256 threads: thread (dg, c4) holds rows dg + 64 j, columns
// 4 c4 .. 4 c4 + 3.
template <int NJ>
struct TileRows {
    f32x4 S[NJ];
    // takes a token in and returns the tile's share of C^T q for columns 4 c4 .. (in the first 4 threads of the workgroup)
    __device__ __forceinline__ f32x4 token(const float (&q)[NJ], const float (&k)[NJ], f32x4 v, float keep, float take, f32x4 (&red)[4][4]) {
        const int tid = threadIdx.x, lane = tid & 63;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        const f32x4 tv = v * take;
#pragma unroll
        for (int j = 0; j < NJ; j++)
#pragma unroll
            for (int c = 0; c < 4; c++) {
                S[j][c] = fmaf(keep, S[j][c], k[j] * tv[c]);
                acc[c] = fmaf(q[j], S[j][c], acc[c]);
            }
#pragma unroll
        for (int c = 0; c < 4; c++) acc[c] = stride4_sum(acc[c]);
        if (lane < 4) red[tid >> 6][lane] = acc;
        __syncthreads();
        return (red[0][tid & 3] + red[1][tid & 3]) + (red[2][tid & 3] + red[3][tid & 3]);
    }
};

// value columns 4 c .. 4 c + 3 of a tile: v, the normaliser's 1, zeros
__device__ __forceinline__ f32x4 value_columns(const float *v, int col, int vdim) {
    f32x4 x;
#pragma unroll
    for (int c = 0; c < 4; c++) x[c] = col + c < vdim ? v[col + c] : col + c == vdim ? 1.f : 0.f;
    return x;
}

template <int NJ>
__global__ __launch_bounds__(256) void matrix_memory_step_kernel(MatrixMemoryStepArgs a) {
    __shared__ f32x4 red[4][4];
    const MatrixMemoryShape &s = a.s;
    const int tid = threadIdx.x, c4 = tid & 3, dg = tid >> 2, tiles = s.tiles();
    const int h = blockIdx.x / tiles, tile = blockIdx.x % tiles;
    f32x4 *mem = reinterpret_cast<f32x4 *>(a.state + (size_t)blockIdx.x * s.dim_pad * 16) + tid;  // (dg, c4) is thread order
    TileRows<NJ> m;
    float q[NJ], k[NJ];
#pragma unroll
    for (int j = 0; j < NJ; j++) m.S[j] = mem[j * 256];
#pragma unroll
    for (int j = 0; j < NJ; j++) {
        const int d = dg + 64 * j;
        q[j] = d < s.dim ? a.row[a.at.q + h * s.dim + d] : 0.f;
        k[j] = d < s.dim ? a.row[a.at.k + h * s.dim + d] : 0.f;
    }
    const f32x4 v = value_columns(a.row + a.at.v + (size_t)h * s.vdim, tile * 16 + c4 * 4, s.vdim);
    const float gi = a.row[a.at.i + h] + a.i_bias[h], gf = a.row[a.at.f + h] + a.f_bias[h];
    float *tops = a.state + s.memory_floats();
    const int pos = a.cursor->pos;
    const bool fresh = pos == 0;
    const float top0 = fresh ? 0.f : tops[(pos & 1) * s.heads + h];
    const float in = soft_cap(gi, s.cap), forget = log_sigmoid(soft_cap(gf, s.cap));
    const float top = fmaxf(forget + top0, in), keep = expf(forget + top0 - top), take = expf(in - top);
    const float scale = 1.0f / sqrtf((float)s.dim);
#pragma unroll
    for (int j = 0; j < NJ; j++) {
        if (fresh) m.S[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        q[j] *= scale;
    }
    const f32x4 o = m.token(q, k, v, keep, take, red);
#pragma unroll
    for (int j = 0; j < NJ; j++) mem[j * 256] = m.S[j];
    if (tid < 4) *reinterpret_cast<f32x4 *>(a.raw + (size_t)h * s.cols() + tile * 16 + c4 * 4) = o;
    if (tid == 0 && tile == 0) tops[((pos + 1) & 1) * s.heads + h] = top;
}

// norm and gates of one head: o(c) the raw columns, g(c) the output gate's logits
__device__ __forceinline__ float head_scale(float ss, int vdim, float den, float floor_, float eps, float &inv_den) {
    inv_den = 1.0f / (fmaxf(fabsf(den), floor_) + 1e-6f);
    return 1.0f / sqrtf(ss * inv_den * inv_den / (float)vdim + eps);
}

__global__ __launch_bounds__(256) void matrix_memory_step_out_kernel(MatrixMemoryStepArgs a) {
    __shared__ float red[4];
    const MatrixMemoryShape &s = a.s;
    const int h = blockIdx.x, tid = threadIdx.x;
    const float *o = a.raw + (size_t)h * s.cols();
    const float den = o[s.vdim];
    const float *g = a.row + a.at.g + (size_t)h * s.vdim, *nw = a.norm + (size_t)h * s.vdim;
    // (the first columns of a thread are asked for ahead of the cursor)
    constexpr int KEEP = 4;
    float x[KEEP], gate[KEEP], w[KEEP], ss = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; j++) {
        const int c = tid + j * 256;
        x[j] = c < s.vdim ? o[c] : 0.f;
        gate[j] = c < s.vdim ? g[c] : 0.f;
        w[j] = c < s.vdim ? nw[c] : 0.f;
    }
    const float top = a.state[s.memory_floats() + ((a.cursor->pos + 1) & 1) * s.heads + h];
#pragma unroll
    for (int j = 0; j < KEEP; j++) ss += x[j] * x[j];
    for (int c = tid + KEEP * 256; c < s.vdim; c += 256) ss += o[c] * o[c];
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    float inv_den;
    const float inv = head_scale((red[0] + red[1]) + (red[2] + red[3]), s.vdim, den, expf(-top), a.eps, inv_den);
#pragma unroll
    for (int j = 0; j < KEEP; j++) {
        const int c = tid + j * 256;
        if (c < s.vdim) a.out[(size_t)h * s.vdim + c] = x[j] * inv_den * inv * w[j] / (1.0f + expf(-gate[j]));
    }
    for (int c = tid + KEEP * 256; c < s.vdim; c += 256) a.out[(size_t)h * s.vdim + c] = o[c] * inv_den * inv * nw[c] / (1.0f + expf(-g[c]));
}

// ── prompt rows ──────────────────────────────────────────────────────────────

// q (scaled) and k as pieces, four columns a thread (dim_pad / 4 threads a head and row).
__global__ __launch_bounds__(256) void matrix_memory_split_kernel(MatrixMemoryRowsArgs a, size_t jobs) {
    const MatrixMemoryShape &s = a.s;
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= jobs) return;
    const RowSource in{a.rows, a.ld, a.parts, a.stride, nullptr};
    const int per = s.dim_pad / 4, d = (int)(e % per) * 4;
    const size_t r = e / per;
    const int hh = (int)(r % (2 * s.heads)), h = hh % s.heads, t = (int)(r / (2 * s.heads));
    const bool is_q = hh < s.heads;
    const int col = (is_q ? a.at.q : a.at.k) + h * s.dim + d;
    const float scale = is_q ? 1.0f / sqrtf((float)s.dim) : 1.0f;
    f32x4 x = {0.f, 0.f, 0.f, 0.f};
    if (s.dim % 4 == 0 && d < s.dim) {  // (columns start at multiples of 32: whole vectors)
        x = sum_parts4(a.rows, (size_t)t * a.ld + col, a.parts, a.stride);
    } else {
#pragma unroll
        for (int c = 0; c < 4; c++)
            if (d + c < s.dim) x[c] = source_at(in, t, col + c);
    }
    x = x * scale;
    uint16_t *out = (is_q ? a.q : a.k) + ((size_t)h * a.n + t) * s.dim_pad + d;
    const size_t plane = (size_t)s.heads * a.n * s.dim_pad;
    uint32_t lo[3], hi[3];
    split_pair<3>(x[0], x[1], lo);
    split_pair<3>(x[2], x[3], hi);
    for (int p = 0; p < a.pieces; p++) *reinterpret_cast<u32x2 *>(out + p * plane) = u32x2{lo[p], hi[p]};
}

// Gate logits: workgroup (16 tokens, 16 gates), the rows cut across its wavefronts in steps of 32. A = gates' weights, B =
// tokens as three pieces: lane t + 16 c receives gates 4 c .. 4 c + 3 of token t.
__global__ __launch_bounds__(256) void matrix_memory_gate_rows_kernel(MatrixMemoryRowsArgs a) {
    __shared__ f32x4 part[3][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, c4 = lane >> 4, gates = 2 * a.s.heads;
    const int t = blockIdx.x * 16 + l16, g0 = blockIdx.y * 16;
    const uint16_t *w = a.gate_w + (size_t)min(g0 + l16, gates - 1) * a.x_ld + 8 * c4;
    const float *x = a.x + (size_t)min(t, a.n - 1) * a.x_ld + 8 * c4;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    constexpr int AHEAD = 4;  // steps requested together
    for (int base = wave * 32; base < a.x_ld; base += AHEAD * 128) {
        u32x4 wv[AHEAD];
        f32x4 x0[AHEAD], x1[AHEAD];
#pragma unroll
        for (int j = 0; j < AHEAD; j++) {
            const int k = base + j * 128, kc = min(k, a.x_ld - 32);
            wv[j] = ld128(w + kc);
            if (k >= a.x_ld) wv[j] = u32x4{0u, 0u, 0u, 0u};
            x0[j] = *reinterpret_cast<const f32x4 *>(x + kc);
            x1[j] = *reinterpret_cast<const f32x4 *>(x + kc + 4);
        }
#pragma unroll
        for (int j = 0; j < AHEAD; j++) {
            const float f[8] = {x0[j][0], x0[j][1], x0[j][2], x0[j][3], x1[j][0], x1[j][1], x1[j][2], x1[j][3]};
            const bf16x8 wf = __builtin_bit_cast(bf16x8, wv[j]);
            bf16x8 xf[3];
            split8<3>(f, xf);
#pragma unroll
            for (int p = 2; p >= 0; p--) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, xf[p], acc, 0, 0, 0);
        }
    }
    if (wave) part[wave - 1][lane] = acc;
    __syncthreads();
    if (wave || t >= a.n) return;
    acc = (acc + part[0][lane]) + (part[1][lane] + part[2][lane]);
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (g0 + 4 * c4 + i < gates) a.gates[(size_t)t * gates + g0 + 4 * c4 + i] = acc[i];
}

// Log weights of a head's tokens: a wavefront a chunk, a lane a token; the chunks' running maxima follow one another
// once their totals are known.
constexpr double LOG2E = 1.4426950408889634074;
constexpr int GATE_WAVES = 16, GATE_MAX_CHUNKS = MM_MAX_ROWS / MM_CHUNK, GATE_ROUNDS = GATE_MAX_CHUNKS / GATE_WAVES;
__global__ __launch_bounds__(64 * GATE_WAVES) void matrix_memory_gates_kernel(MatrixMemoryRowsArgs a, int chunks) {
    __shared__ double s_sum[GATE_MAX_CHUNKS], s_max[GATE_MAX_CHUNKS], s_top[GATE_MAX_CHUNKS + 1];
    const MatrixMemoryShape &s = a.s;
    const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    float *tops = a.state + s.memory_floats();
    double F[GATE_ROUNDS], A[GATE_ROUNDS], M[GATE_ROUNDS];
#pragma unroll
    for (int r = 0; r < GATE_ROUNDS; r++) {
        const int c = wave + r * GATE_WAVES, t = c * MM_CHUNK + lane;
        float gi = 0.f, gf = 0.f;
        if (t < a.n) {
            gi = a.gates[(size_t)t * 2 * s.heads + h] + a.i_bias[h];
            gf = a.gates[(size_t)t * 2 * s.heads + s.heads + h] + a.f_bias[h];
        }
        const double i = t < a.n ? (double)soft_cap(gi, s.cap) : -INFINITY;
        F[r] = t < a.n ? (double)log_sigmoid(soft_cap(gf, s.cap)) : 0.0;
#pragma unroll
        for (int by = 1; by < 64; by *= 2) {
            const double o = __shfl_up(F[r], by);
            if (lane >= by) F[r] += o;
        }
        A[r] = i - F[r];
        M[r] = A[r];
#pragma unroll
        for (int by = 1; by < 64; by *= 2) {
            const double o = __shfl_up(M[r], by);
            if (lane >= by) M[r] = fmax(M[r], o);
        }
        if (lane == 63 && c < chunks) {
            s_sum[c] = F[r];
            s_max[c] = M[r];
        }
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        double m = a.past ? (double)tops[(a.past & 1) * s.heads + h] : 0.0;
        for (int c = 0; c < chunks; c++) {
            s_top[c] = m;
            m = s_sum[c] + fmax(m, s_max[c]);
        }
        s_top[chunks] = m;
        tops[((a.past + a.n) & 1) * s.heads + h] = (float)m;
    }
    __syncthreads();
    const size_t line = (size_t)chunks * MM_CHUNK, plane = line * s.heads;
#pragma unroll
    for (int r = 0; r < GATE_ROUNDS; r++) {
        const int c = wave + r * GATE_WAVES;
        if (c >= chunks) break;
        const size_t e = h * line + c * MM_CHUNK + lane;
        const double m = s_top[c], end = fmax(m, s_max[c]), top = fmax(m, M[r]);
        a.log_w[e] = A[r] * LOG2E;
        a.log_w[plane + e] = top * LOG2E;
        a.weights[e] = expf((float)(m - top));
        a.weights[plane + e] = expf((float)(A[r] - end));
        a.weights[2 * plane + e] = expf((float)-(F[r] + top));
        if (lane == 0) a.decay[h * chunks + c] = expf((float)(m - end));
    }
}

// Two kernels on the matrix cores. The first walks the chunks in order and leaves the memory ahead of every chunk, as
// pieces in the operand order of the second, which takes all chunks side by side. KP: pieces of q, k and v (3: f32).
// Contraction slot 8 c + i of tokens stands for token 4 c + i (i < 4) or 16 + 4 c + i - 4 of its 32, as in the causal
// attention, in both.
extern __shared__ __attribute__((aligned(16))) char mm_lds[];

// Operands of a tile's values over a chunk, a lane's 16 bytes each: [half of the chunk][pieces][64 lanes], plain ones (KP
// pieces) and ones times their weight at the chunk's end (three).
template <int KP>
struct ValueTile {
    static constexpr int PLAIN = 2 * KP * 1024, WEIGHTED = 2 * 3 * 1024, BYTES = PLAIN + WEIGHTED;
};

// Writes them: workgroup (chunk and head, four tiles). The values go through LDS, token rows of 64 columns; column vdim is
// the normaliser's, those behind it are zero.
template <int KP>
__global__ __launch_bounds__(256) void matrix_memory_values_kernel(MatrixMemoryRowsArgs a, int chunks) {
    __shared__ float tile_v[MM_CHUNK][65];
    const MatrixMemoryShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, c4 = lane >> 4;
    const int h = blockIdx.x % s.heads, c = blockIdx.x / s.heads, tiles = s.tiles(), col0 = blockIdx.y * 64;
    const RowSource in{a.rows, a.ld, a.parts, a.stride, nullptr};
    const int col = col0 + lane, at = a.at.v + h * s.vdim + min(col, s.vdim - 1);
    float x[MM_CHUNK / 4];
    if (a.parts == 1) {
#pragma unroll
        for (int j = 0; j < MM_CHUNK / 4; j++) x[j] = a.rows[(size_t)min(c * MM_CHUNK + wave + 4 * j, a.n - 1) * a.ld + at];
    } else {
#pragma unroll 2
        for (int j = 0; j < MM_CHUNK / 4; j++) x[j] = source_at(in, min(c * MM_CHUNK + wave + 4 * j, a.n - 1), at);
    }
#pragma unroll
    for (int j = 0; j < MM_CHUNK / 4; j++) tile_v[wave + 4 * j][lane] = col < s.vdim ? x[j] : col == s.vdim ? 1.f : 0.f;
    __syncthreads();
    const int tile = blockIdx.y * 4 + wave;
    if (tile >= tiles) return;
    const size_t line = (size_t)chunks * MM_CHUNK;
    const float *w_end = a.weights + line * s.heads + h * line + c * MM_CHUNK;
    bf16x8 *out = reinterpret_cast<bf16x8 *>(reinterpret_cast<char *>(a.values) + ((size_t)blockIdx.x * tiles + tile) * ValueTile<KP>::BYTES) + lane;
#pragma unroll
    for (int half = 0; half < 2; half++) {
        float x[8], w[8];
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const int t = 32 * half + 4 * c4 + (i < 4 ? i : 12 + i);
            x[i] = tile_v[t][wave * 16 + l16];
            w[i] = x[i] * w_end[t];
        }
        bf16x8 xf[KP], wf[3];
        split8<KP>(x, xf);
        split8<3>(w, wf);
#pragma unroll
        for (int p = 0; p < KP; p++) out[(half * KP + p) * 64] = xf[p];
#pragma unroll
        for (int p = 0; p < 3; p++) out[ValueTile<KP>::PLAIN / 16 + (half * 3 + p) * 64] = wf[p];
    }
}

// Orders LDS traffic only: loads stay in flight across it (a __syncthreads() drains them).
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// LDS reads (the first one transposes); whoever uses the result waits for it.
__device__ __forceinline__ s16x4 lds_read_tr(uint32_t addr) {
    s16x4 v;
    asm volatile("ds_read_b64_tr_b16 %0, %1" : "=v"(v) : "v"(addr) : "memory");
    return v;
}

__device__ __forceinline__ bf16x8 lds_read16(uint32_t addr) {
    bf16x8 v;
    asm volatile("ds_read_b128 %0, %1" : "=v"(v) : "v"(addr) : "memory");
    return v;
}

// K tile of a chunk into LDS by 256 threads, row-major and swizzled
template <int DIM, int KP>
struct KeyTile {
    static constexpr int PIECE = MM_CHUNK * DIM * 2, BYTES = KP * PIECE, LOADS = MM_CHUNK * DIM / 8 / 256;
    int row[LOADS], col[LOADS];
    __device__ __forceinline__ KeyTile() {
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int g = i * 256 + threadIdx.x;
            row[i] = g / (DIM / 8);
            col[i] = (k_off<DIM>(row[i], g % (DIM / 8)) - row[i] * DIM * 2) >> 1;
        }
    }
    __device__ __forceinline__ void request(const uint16_t *k, size_t plane, int chunk, int n, char *lds) const {
        char *base = lds + __builtin_amdgcn_readfirstlane((threadIdx.x >> 6) * 1024);
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const uint16_t *src = k + (size_t)min(chunk * MM_CHUNK + row[i], n - 1) * DIM + col[i];
#pragma unroll
            for (int p = 0; p < KP; p++) dma16_lds(src + p * plane, base + p * PIECE + i * 4096);
        }
    }
};

// A tile of the memory ahead of a chunk, as operands of the read-out: [piece][dim / 8][16 columns][8 dims]. The queries it
// meets have 8 bits (KP 1: two pieces, 16 bits) or all of them.
template <int DIM, int KP>
struct MemoryTile {
    static constexpr int PIECES = KP == 1 ? 2 : 3, PIECE = DIM * 32, BYTES = PIECES * PIECE;
};

// The walk: workgroup (head, tile of 16 columns), wavefront w a quarter of the memory's rows in accumulators: A = keys^T
// through the transposing LDS read, B = weighted values. Keys and values go global -> LDS directly, KB sets of them: KB - 1
// chunks are on their way while one is multiplied. Every LDS read is written out with its wait, because ahead of one of its
// own the compiler would wait for all that is on its way.
template <int DIM, int KP, int KB>
__global__ __launch_bounds__(256) void matrix_memory_walk_kernel(MatrixMemoryRowsArgs a, int chunks) {
    constexpr int DT = DIM / 64;
    using Memory = MemoryTile<DIM, KP>;
    using Keys = KeyTile<DIM, KP>;
    using Values = ValueTile<KP>;
    constexpr int SET = Keys::BYTES + Values::BYTES, VLOADS = Values::BYTES / 4096;
    static_assert(Values::BYTES % 4096 == 0, "every wavefront requests as much");
    constexpr int GROUP = KP * Keys::LOADS + VLOADS;  // requests of a chunk
    const MatrixMemoryShape &s = a.s;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, c4 = lane >> 4;
    const int h = blockIdx.x / s.tiles(), n = a.n, last = chunks - 1;
    const size_t plane = (size_t)s.heads * n * DIM;
    const uint16_t *kg = a.k + (size_t)h * n * DIM;
    float *mem = a.state + (size_t)blockIdx.x * DIM * 16;
    char *ahead = reinterpret_cast<char *>(a.ahead) + (size_t)blockIdx.x * Memory::BYTES;
    const size_t chunk_bytes = (size_t)gridDim.x * Memory::BYTES, value_bytes = (size_t)gridDim.x * Values::BYTES;
    const char *values = reinterpret_cast<const char *>(a.values) + (size_t)blockIdx.x * Values::BYTES + threadIdx.x * 16;
    const Keys keys;
    const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) char *)mm_lds;
    static_assert(MM_MAX_ROWS / MM_CHUNK <= 64, "a lane a chunk");
    const float decays = a.decay[h * chunks + min(lane, last)];
    auto request = [&](int c, int set) {
        char *base = mm_lds + set * SET;
        keys.request(kg, plane, c, n, base);
        base += Keys::BYTES + __builtin_amdgcn_readfirstlane(wave * 1024);
#pragma unroll
        for (int i = 0; i < VLOADS; i++) dma16_lds(reinterpret_cast<const uint16_t *>(values + c * value_bytes + i * 4096), base + i * 4096);
    };
    f32x4 S[DT];  // block b, value i: row wave * DIM / 4 + 16 b + 4 c4 + i, column l16
#pragma unroll
    for (int b = 0; b < DT; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) S[b][i] = a.past ? mem[(wave * (DIM / 4) + 16 * b + 4 * c4 + i) * 16 + l16] : 0.f;
    auto publish = [&](int c) {
#pragma unroll
        for (int b = 0; b < DT; b++) {
            uint32_t lo[Memory::PIECES], hi[Memory::PIECES];
            split_pair<Memory::PIECES>(S[b][0], S[b][1], lo);
            split_pair<Memory::PIECES>(S[b][2], S[b][3], hi);
            const int d = wave * (DIM / 4) + 16 * b + 4 * c4;
            char *at = ahead + c * chunk_bytes + ((d >> 3) * 16 + l16) * 16 + (d & 4) * 2;
#pragma unroll
            for (int p = 0; p < Memory::PIECES; p++) *reinterpret_cast<u32x2 *>(at + p * Memory::PIECE) = u32x2{lo[p], hi[p]};
        }
    };
    publish(0);
#pragma unroll
    for (int i = 0; i < (KB > 1 ? KB - 1 : 1); i++) request(min(i, last), i);
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(KB > 2 ? (KB - 2) * GROUP : 0) : "memory");
    auto chunk = [&](int c, int set) {
        lds_barrier();  // this chunk is in LDS, and everybody is done with the one before it
        // (behind the end the last chunk once more: the counts stay exact)
        if (KB > 1) request(min(c + KB - 1, last), (set + KB - 1) % KB);
        const float decay = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(decays), c));
        const uint32_t k0 = lds0 + set * SET, v0 = k0 + Keys::BYTES + Values::PLAIN + lane * 16;
        s16x4 lo[2][DT][KP], hi[2][DT][KP];
        bf16x8 v[2][3];
        auto read = [&](int ks) {
            const int key = 32 * ks + 4 * c4 + (l16 >> 2), within = (l16 & 1) * 8;
#pragma unroll
            for (int p = 0; p < 3; p++) v[ks][p] = lds_read16(v0 + (ks * 3 + p) * 1024);
#pragma unroll
            for (int b = 0; b < DT; b++) {
                const int at = 2 * (wave * DT + b) + ((l16 & 3) >> 1);
#pragma unroll
                for (int p = 0; p < KP; p++) {
                    lo[ks][b][p] = lds_read_tr(k0 + p * Keys::PIECE + within + k_off<DIM>(key, at));
                    hi[ks][b][p] = lds_read_tr(k0 + p * Keys::PIECE + within + k_off<DIM>(16 + key, at));
                }
            }
        };
        auto arrived = [&](int ks) {  // (the statements name the registers, so that nothing touches them earlier)
            asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(v[ks][0]), "+v"(v[ks][1]), "+v"(v[ks][2]));
#pragma unroll
            for (int b = 0; b < DT; b++)
#pragma unroll
                for (int p = 0; p < KP; p++) asm volatile("" : "+v"(lo[ks][b][p]), "+v"(hi[ks][b][p]));
        };
        read(0);
#pragma unroll
        for (int b = 0; b < DT; b++) S[b] = S[b] * decay;
        arrived(0);
        read(1);
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            if (ks == 1) arrived(1);
            piece_products<3, KP>([&](int pv, int pk) {
#pragma unroll
                for (int b = 0; b < DT; b++) {
                    struct Pair { s16x4 lo, hi; } pr{lo[ks][b][pk], hi[ks][b][pk]};
                    S[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, pr), v[ks][pv], S[b], 0, 0, 0);
                }
            });
        }
        if (KB == 1) {
            lds_barrier();  // everybody is done with the only set
            request(min(c + 1, last), 0);
        }
        // the next chunk has landed (ahead of the stores, which may take their time)
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"(KB > 2 ? (KB - 2) * GROUP : 0) : "memory");
        if (c < last) publish(c + 1);
    };
    for (int c = 0; c < chunks; c += KB)
#pragma unroll
        for (int u = 0; u < KB; u++)
            if (c + u < chunks) chunk(c + u, u);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // (a load into LDS must not outlive the workgroup)
#pragma unroll
    for (int b = 0; b < DT; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) mem[(wave * (DIM / 4) + 16 * b + 4 * c4 + i) * 16 + l16] = S[b][i];
}

// The rows of a chunk: workgroup (chunk and head, share of the column tiles).
//   scores^T   wavefront w, rows 16 w .. 16 w + 15: A = 16 keys x 32 dims from the K tile, B = queries: lane t + 16 c receives
//              keys 4 c .. 4 c + 3 of the block for row t; times their weights they are the B operand of the last product
//   o^T        A = memory^T (16 columns x 32 dims, straight from memory), B = queries; times the memory's weight of the row;
//              then A = values^T (16 columns x 32 tokens), B = weighted scores
// RB 4: the weighted scores of all rows go round through LDS and a wavefront takes every fourth tile for all rows, so that
// the memory is read once; RB 1 (queries too wide for that): every tile for its own rows.
template <int DIM, int KP, int RB>
__global__ __launch_bounds__(256) void matrix_memory_chunk_kernel(MatrixMemoryRowsArgs a, int chunks, int tiles_per) {
    constexpr int KSTEPS = DIM / 32;
    using Memory = MemoryTile<DIM, KP>;
    constexpr int MP = Memory::PIECES;
    __shared__ __attribute__((aligned(16))) double s_a[MM_CHUNK];
    const MatrixMemoryShape &s = a.s;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, c4 = lane >> 4;
    const int h = blockIdx.x % s.heads, c = blockIdx.x / s.heads, tiles = s.tiles(), n = a.n;
    const int t_begin = blockIdx.y * tiles_per, t_end = min(tiles, t_begin + tiles_per);
    const size_t plane = (size_t)s.heads * n * DIM, line = (size_t)chunks * MM_CHUNK, wplane = line * s.heads;
    const uint16_t *qg = a.q + (size_t)h * n * DIM, *kg = a.k + (size_t)h * n * DIM;
    const double *wa = a.log_w + h * line + c * MM_CHUNK, *wm = wa + wplane;
    const float *w_mem = a.weights + h * line + c * MM_CHUNK;
    const char *ahead = reinterpret_cast<const char *>(a.ahead) + ((size_t)c * s.heads + h) * tiles * Memory::BYTES;
    const char *values = reinterpret_cast<const char *>(a.values) + (size_t)blockIdx.x * tiles * ValueTile<KP>::BYTES + lane * 16;
    const KeyTile<DIM, KP> keys;
    keys.request(kg, plane, c, n, mm_lds);
    auto load_queries = [&](int rb, bf16x8(&q)[KSTEPS][KP]) {
        const uint16_t *src = qg + (size_t)min(c * MM_CHUNK + rb * 16 + l16, n - 1) * DIM + c4 * 8;
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ks++)
#pragma unroll
            for (int p = 0; p < KP; p++) q[ks][p] = *reinterpret_cast<const bf16x8 *>(src + p * plane + 32 * ks);
    };
    bf16x8 q[RB][KSTEPS][KP];
    bf16x8 pf[RB][2][3];
    float tw[RB];
    if (wave == 0) s_a[lane] = wa[lane];
    {
        bf16x8 own[KSTEPS][KP];
        load_queries(wave, own);
        const int row = wave * 16 + l16;
        const double tm = wm[row];
        if (RB == 1) tw[0] = w_mem[row];
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (RB == 1) {
#pragma unroll
            for (int ks = 0; ks < KSTEPS; ks++)
#pragma unroll
                for (int p = 0; p < KP; p++) q[0][ks][p] = own[ks][p];
        } else {
#pragma unroll
            for (int rb = 0; rb < RB; rb++) {
                load_queries(rb, q[rb]);
                tw[rb] = w_mem[rb * 16 + l16];
            }
        }
#pragma unroll
        for (int half = 0; half < 2; half++) {
            f32x4 sc[2];
            sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (2 * half <= wave) {  // wavefront-uniform: else all of these tokens lie behind the rows
#pragma unroll
                for (int ks = 0; ks < KSTEPS; ks++) {
                    bf16x8 kf[KP][2];
#pragma unroll
                    for (int p = 0; p < KP; p++)
#pragma unroll
                        for (int b = 0; b < 2; b++)
                            kf[p][b] = *reinterpret_cast<const bf16x8 *>(mm_lds + p * keys.PIECE + k_off<DIM>(32 * half + 16 * b + l16, 4 * ks + c4));
                    piece_products<KP, KP>([&](int pq, int pk) {
#pragma unroll
                        for (int b = 0; b < 2; b++) sc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[pk][b], own[ks][pq], sc[b], 0, 0, 0);
                    });
                }
            }
            float f[8];
#pragma unroll
            for (int i = 0; i < 8; i++) {
                const int key = 32 * half + 16 * (i >> 2) + 4 * c4 + (i & 3);
                const float w = __builtin_amdgcn_exp2f((float)(s_a[key] - tm));
                f[i] = key <= row ? sc[i >> 2][i & 3] * w : 0.f;
            }
            split8<3>(f, pf[0][half]);
        }
    }
    if (RB > 1) {
        bf16x8 *share = reinterpret_cast<bf16x8 *>(mm_lds + keys.BYTES);  // [row block][half][piece][lane]
#pragma unroll
        for (int half = 0; half < 2; half++)
#pragma unroll
            for (int p = 0; p < 3; p++) share[((wave * 2 + half) * 3 + p) * 64 + lane] = pf[0][half][p];
        __syncthreads();
#pragma unroll
        for (int rb = 0; rb < RB; rb++)
#pragma unroll
            for (int half = 0; half < 2; half++)
#pragma unroll
                for (int p = 0; p < 3; p++) pf[rb][half][p] = share[((rb * 2 + half) * 3 + p) * 64 + lane];
    }
    struct Tile { bf16x8 m[KSTEPS][MP]; };
    auto load = [&](int tile, Tile &t) {
        const char *at = ahead + (size_t)tile * Memory::BYTES + lane * 16;
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ks++)
#pragma unroll
            for (int p = 0; p < MP; p++) t.m[ks][p] = *reinterpret_cast<const bf16x8 *>(at + p * Memory::PIECE + ks * 1024);
    };
    auto product = [&](int tile, const Tile &t) {
        bf16x8 vf[2][KP];  // (arrive under the products with the memory)
#pragma unroll
        for (int half = 0; half < 2; half++)
#pragma unroll
            for (int p = 0; p < KP; p++) vf[half][p] = *reinterpret_cast<const bf16x8 *>(values + (size_t)tile * ValueTile<KP>::BYTES + (half * KP + p) * 1024);
        f32x4 o[RB];
#pragma unroll
        for (int rb = 0; rb < RB; rb++) o[rb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ks++)
            piece_products<MP, KP>([&](int pm, int pq) {
#pragma unroll
                for (int rb = 0; rb < RB; rb++) o[rb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(t.m[ks][pm], q[rb][ks][pq], o[rb], 0, 0, 0);
            });
#pragma unroll
        for (int rb = 0; rb < RB; rb++) o[rb] = o[rb] * tw[rb];
#pragma unroll
        for (int half = 0; half < 2; half++)
            piece_products<3, KP>([&](int pp, int pv) {
#pragma unroll
                for (int rb = 0; rb < RB; rb++)
                    if (RB == 1 || 2 * half <= rb) o[rb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[half][pv], pf[rb][half][pp], o[rb], 0, 0, 0);
            });
#pragma unroll
        for (int rb = 0; rb < RB; rb++) {
            const int row = c * MM_CHUNK + (RB > 1 ? rb : wave) * 16 + l16;
            if (row < n) __builtin_nontemporal_store(o[rb], reinterpret_cast<f32x4 *>(a.raw + ((size_t)row * s.heads + h) * s.cols() + tile * 16 + 4 * c4));
        }
    };
    constexpr int STEP = RB > 1 ? 4 : 1, SETS = RB * KP * DIM > 1024 || DIM > 256 ? 1 : 2;
    const int t0 = t_begin + (RB > 1 ? wave : 0);
    if (SETS == 1) {
        for (int tile = t0; tile < t_end; tile += STEP) {
            Tile t;
            load(tile, t);
            product(tile, t);
        }
    } else if (t0 < t_end) {  // the next tile is on its way while this one is multiplied
        Tile x, y;
        load(t0, x);
        for (int tile = t0; tile < t_end; tile += 2 * STEP) {
            load(min(tile + STEP, tiles - 1), y);
            product(tile, x);
            if (tile + STEP >= t_end) break;
            load(min(tile + 2 * STEP, tiles - 1), x);
            product(tile + STEP, y);
        }
    }
}

// Heads wider than the scan's tiles: token by token on the vector units.
template <int NJ>
__global__ __launch_bounds__(256) void matrix_memory_scan_any_kernel(MatrixMemoryRowsArgs a, int chunks) {
    __shared__ f32x4 red[2][4][4];
    const MatrixMemoryShape &s = a.s;
    const int tid = threadIdx.x, c4 = tid & 3, dg = tid >> 2, tiles = s.tiles();
    const int h = blockIdx.x / tiles, tile = blockIdx.x % tiles;
    f32x4 *mem = reinterpret_cast<f32x4 *>(a.state + (size_t)blockIdx.x * s.dim_pad * 16) + tid;
    const RowSource in{a.rows, a.ld, a.parts, a.stride, nullptr};
    const float scale = 1.0f / sqrtf((float)s.dim);
    TileRows<NJ> m;
#pragma unroll
    for (int j = 0; j < NJ; j++) m.S[j] = a.past ? mem[j * 256] : f32x4{0.f, 0.f, 0.f, 0.f};
    // from the log weights: memory held relative to M of its chunk plus what earlier chunks left behind
    const size_t line = (size_t)chunks * MM_CHUNK, plane = line * s.heads;
    const double *wa = a.log_w + h * line, *wm = wa + plane;
    const float *w_mem = a.weights + h * line;
    for (int t = 0; t < a.n; t++) {
        float q[NJ], k[NJ];
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            const int d = dg + 64 * j;
            q[j] = d < s.dim ? source_at(in, t, a.at.q + h * s.dim + d) * scale : 0.f;
            k[j] = d < s.dim ? source_at(in, t, a.at.k + h * s.dim + d) : 0.f;
        }
        f32x4 v;
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int col = tile * 16 + c4 * 4 + c;
            v[c] = col < s.vdim ? source_at(in, t, a.at.v + h * s.vdim + col) : col == s.vdim ? 1.f : 0.f;
        }
        const float keep = t % MM_CHUNK ? exp2f((float)(wm[t - 1] - wm[t])) : w_mem[t], take = exp2f((float)(wa[t] - wm[t]));
        const f32x4 o = m.token(q, k, v, keep, take, red[t & 1]);
        if (tid < 4) *reinterpret_cast<f32x4 *>(a.raw + ((size_t)t * s.heads + h) * s.cols() + tile * 16 + c4 * 4) = o;
    }
#pragma unroll
    for (int j = 0; j < NJ; j++) mem[j * 256] = m.S[j];
}

// norm, weight and gate behind the scan: a wavefront per head of a row, KEEP columns a lane in registers
__global__ __launch_bounds__(256) void matrix_memory_out_kernel(MatrixMemoryRowsArgs a, int chunks) {
    const MatrixMemoryShape &s = a.s;
    const int lane = threadIdx.x & 63;
    const size_t job = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (job >= (size_t)a.n * s.heads) return;
    const int t = (int)(job / s.heads), h = (int)(job % s.heads);
    const float *o = a.raw + job * s.cols();
    const RowSource in{a.rows, a.ld, a.parts, a.stride, nullptr};
    const size_t line = (size_t)chunks * MM_CHUNK;
    const float low = a.weights[2 * line * s.heads + h * line + t], den = o[s.vdim];
    uint16_t *out = a.out_split + (size_t)t * a.out_pieces * a.out_cols;
    float ss = 0.f, inv_den;
    if (s.vdim % 4 == 0 && s.vdim <= 1024) {
        constexpr int KEEP = 4;
        f32x4 x[KEEP], g[KEEP];
#pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int c = (lane + 64 * j) * 4;
            x[j] = g[j] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (c < s.vdim) {
                x[j] = *reinterpret_cast<const f32x4 *>(o + c);
                g[j] = sum_parts4(a.rows, (size_t)t * a.ld + a.at.g + h * s.vdim + c, a.parts, a.stride);
            }
            ss += (x[j][0] * x[j][0] + x[j][1] * x[j][1]) + (x[j][2] * x[j][2] + x[j][3] * x[j][3]);
        }
        const float inv = head_scale(wave_sum(ss), s.vdim, den, low, a.eps, inv_den);
#pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int c = (lane + 64 * j) * 4;
            if (c >= s.vdim) break;
            f32x4 y = (x[j] * inv_den * inv) * *reinterpret_cast<const f32x4 *>(a.norm + (size_t)h * s.vdim + c);
#pragma unroll
            for (int i = 0; i < 4; i++) y[i] = y[i] / (1.0f + expf(-g[j][i]));
            split_store4(out, a.out_cols, h * s.vdim + c, y, a.out_pieces);
        }
        return;
    }
    for (int c = lane; c < s.vdim; c += 64) ss += o[c] * o[c];
    const float inv = head_scale(wave_sum(ss), s.vdim, den, low, a.eps, inv_den);
    for (int c = lane; c < s.vdim; c += 64) {
        const float y = o[c] * inv_den * inv * a.norm[(size_t)h * s.vdim + c] / (1.0f + expf(-source_at(in, t, a.at.g + h * s.vdim + c)));
        split_store(out, a.out_cols, h * s.vdim + c, y, a.out_pieces);
    }
}

template <int DIM, int KP, int KB, int RB>
int launch_scan(hm_ctx *ctx, const MatrixMemoryRowsArgs &a) {
    constexpr int KEYS = KeyTile<DIM, KP>::BYTES, WALK = KB * (KEYS + ValueTile<KP>::BYTES), CHUNK = KEYS + (RB > 1 ? RB * 2 * 3 * 1024 : 0);
    static const hipError_t attr_w = hipFuncSetAttribute(reinterpret_cast<const void *>(matrix_memory_walk_kernel<DIM, KP, KB>),
                                                         hipFuncAttributeMaxDynamicSharedMemorySize, WALK);
    static const hipError_t attr_c = hipFuncSetAttribute(reinterpret_cast<const void *>(matrix_memory_chunk_kernel<DIM, KP, RB>),
                                                         hipFuncAttributeMaxDynamicSharedMemorySize, CHUNK);
    HM_REQUIRE(ctx, attr_w == hipSuccess && attr_c == hipSuccess, "matrix_memory: cannot reserve %d or %d bytes of LDS", WALK, CHUNK);
    const int chunks = a.chunks(), tiles = a.s.tiles();
    hipLaunchKernelGGL((matrix_memory_walk_kernel<DIM, KP, KB>), dim3(a.s.heads * tiles), dim3(256), WALK, ctx->stream, a, chunks);
    HM_LAUNCH_CHECK(ctx);
    // shares of the tiles: as many as give the chip its workgroups, four tiles each at least where wavefronts share them out
    const int least = RB > 1 ? 4 : 1;
    int shares = std::max(1, std::min((tiles + least - 1) / least, ctx->num_cus / (chunks * a.s.heads)));
    const int per = (tiles + shares - 1) / shares;
    shares = (tiles + per - 1) / per;
    hipLaunchKernelGGL((matrix_memory_chunk_kernel<DIM, KP, RB>), dim3(chunks * a.s.heads, shares), dim3(256), CHUNK, ctx->stream, a, chunks, per);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

bool bad_shape(const MatrixMemoryShape &s) {
    return s.heads <= 0 || s.dim <= 0 || s.vdim <= 0 || s.dim > MM_MAX_DIM || s.dim_pad != matrix_memory_dim_pad(s.dim) || !(s.cap > 0.f);
}

}  // namespace

namespace homura {

int matrix_memory_dim_pad(int dim) {
    for (int p = 64; p < MM_MAX_DIM; p *= 2)
        if (dim <= p) return p;
    return MM_MAX_DIM;
}

bool matrix_memory_tiled(const MatrixMemoryShape &s, int pieces) { return s.dim_pad <= (pieces == 1 ? 512 : 256); }
size_t matrix_memory_value_bytes(const MatrixMemoryShape &s, int pieces, int rows) {
    const size_t tile = pieces == 1 ? ValueTile<1>::BYTES : ValueTile<3>::BYTES;
    return matrix_memory_tiled(s, pieces) ? (size_t)((rows + MM_CHUNK - 1) / MM_CHUNK) * s.heads * s.tiles() * tile : 0;
}
size_t matrix_memory_ahead_bytes(const MatrixMemoryShape &s, int pieces, int rows) {
    return matrix_memory_tiled(s, pieces) ? (size_t)((rows + MM_CHUNK - 1) / MM_CHUNK) * s.heads * s.tiles() * (pieces == 1 ? 2 : 3) * s.dim_pad * 32 : 0;
}

int matrix_memory_step_launch(hm_ctx *ctx, const MatrixMemoryStepArgs &a) {
    HM_REQUIRE(ctx, !bad_shape(a.s) && a.row && a.i_bias && a.f_bias && a.state && a.raw && a.cursor, "matrix_memory_step: bad arguments");
    HM_REQUIRE(ctx, ((uintptr_t)a.state % 16) == 0 && ((uintptr_t)a.raw % 16) == 0, "matrix_memory_step: misaligned buffer");
    const dim3 g(a.s.heads * a.s.tiles()), b(256);
    switch (a.s.dim_pad) {
    case 64: hipLaunchKernelGGL(matrix_memory_step_kernel<1>, g, b, 0, ctx->stream, a); break;
    case 128: hipLaunchKernelGGL(matrix_memory_step_kernel<2>, g, b, 0, ctx->stream, a); break;
    case 256: hipLaunchKernelGGL(matrix_memory_step_kernel<4>, g, b, 0, ctx->stream, a); break;
    case 512: hipLaunchKernelGGL(matrix_memory_step_kernel<8>, g, b, 0, ctx->stream, a); break;
    default: hipLaunchKernelGGL(matrix_memory_step_kernel<16>, g, b, 0, ctx->stream, a); break;
    }
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int matrix_memory_step_out_launch(hm_ctx *ctx, const MatrixMemoryStepArgs &a) {
    HM_REQUIRE(ctx, !bad_shape(a.s) && a.row && a.state && a.raw && a.norm && a.out && a.cursor, "matrix_memory_step_out: bad arguments");
    hipLaunchKernelGGL(matrix_memory_step_out_kernel, dim3(a.s.heads), dim3(256), 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int matrix_memory_rows_launch(hm_ctx *ctx, const MatrixMemoryRowsArgs &a) {
    const MatrixMemoryShape &s = a.s;
    HM_REQUIRE(ctx, !bad_shape(s) && a.rows && a.x && a.gate_w && a.gates && a.i_bias && a.f_bias && a.q && a.k && a.log_w && a.weights && a.decay && a.state && a.raw && a.norm &&
                        a.out_split, "matrix_memory_rows: bad arguments");
    HM_REQUIRE(ctx, a.n > 0 && a.n <= MM_MAX_ROWS && a.past >= 0 && (a.pieces == 1 || a.pieces == 3) && a.out_pieces >= 1 && a.out_pieces <= 3 &&
                        a.parts >= 1 && a.parts <= MAX_SUM_PARTS && a.out_cols >= s.heads * s.vdim && a.out_cols % 4 == 0, "matrix_memory_rows: bad shape");
    const MatrixMemoryColumns &at = a.at;
    HM_REQUIRE(ctx, at.q % 4 == 0 && at.k % 4 == 0 && at.v % 4 == 0 && at.g % 4 == 0 && a.ld % 4 == 0 && a.stride % 4 == 0 &&
                        ((uintptr_t)a.rows % 16) == 0 && ((uintptr_t)a.q % 16) == 0 && ((uintptr_t)a.k % 16) == 0 && ((uintptr_t)a.raw % 16) == 0 &&
                        ((uintptr_t)a.norm % 16) == 0 && ((uintptr_t)a.state % 16) == 0 && ((uintptr_t)a.out_split % 8) == 0,
               "matrix_memory_rows: misaligned rows");
    const int qk = s.heads * s.dim, vw = (s.heads * s.vdim + 3) / 4 * 4;
    HM_REQUIRE(ctx, at.q >= 0 && at.q + qk <= at.k && at.k + qk <= at.v && at.v + vw <= at.g && at.g + vw <= a.ld && a.x_ld > 0 && a.x_ld % 32 == 0 &&
                        ((uintptr_t)a.x % 16) == 0 && ((uintptr_t)a.gate_w % 16) == 0, "matrix_memory_rows: the projection's parts overlap");
    const int chunks = a.chunks();
    const bool tiled = matrix_memory_tiled(s, a.pieces);
    HM_REQUIRE(ctx, !tiled || (a.ahead && a.values && ((uintptr_t)a.ahead % 16) == 0 && ((uintptr_t)a.values % 16) == 0), "matrix_memory_rows: no room for the memories");
    hipLaunchKernelGGL(matrix_memory_gate_rows_kernel, dim3((a.n + 15) / 16, (2 * s.heads + 15) / 16), dim3(256), 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    hipLaunchKernelGGL(matrix_memory_gates_kernel, dim3(s.heads), dim3(64 * GATE_WAVES), 0, ctx->stream, a, chunks);
    HM_LAUNCH_CHECK(ctx);
    int rc = HM_OK;
    const dim3 g(s.heads * s.tiles()), b(256);
    if (tiled) {
        const size_t jobs = (size_t)a.n * 2 * s.heads * (s.dim_pad / 4);
        hipLaunchKernelGGL(matrix_memory_split_kernel, dim3((unsigned)((jobs + 255) / 256)), b, 0, ctx->stream, a, jobs);
        HM_LAUNCH_CHECK(ctx);
        const dim3 vgrid(chunks * s.heads, (s.tiles() + 3) / 4);
        if (a.pieces == 1) hipLaunchKernelGGL(matrix_memory_values_kernel<1>, vgrid, b, 0, ctx->stream, a, chunks);
        else hipLaunchKernelGGL(matrix_memory_values_kernel<3>, vgrid, b, 0, ctx->stream, a, chunks);
        HM_LAUNCH_CHECK(ctx);
    }
    if (!tiled) {
        if (s.dim_pad == 512) hipLaunchKernelGGL(matrix_memory_scan_any_kernel<8>, g, b, 0, ctx->stream, a, chunks);
        else hipLaunchKernelGGL(matrix_memory_scan_any_kernel<16>, g, b, 0, ctx->stream, a, chunks);
        HM_LAUNCH_CHECK(ctx);
    } else if (a.pieces == 1) {
        if (s.dim_pad == 64) rc = launch_scan<64, 1, 3, 4>(ctx, a);
        else if (s.dim_pad == 128) rc = launch_scan<128, 1, 3, 4>(ctx, a);
        else if (s.dim_pad == 256) rc = launch_scan<256, 1, 3, 4>(ctx, a);
        else rc = launch_scan<512, 1, 2, 1>(ctx, a);
    } else {
        if (s.dim_pad == 64) rc = launch_scan<64, 3, 3, 4>(ctx, a);
        else if (s.dim_pad == 128) rc = launch_scan<128, 3, 2, 1>(ctx, a);
        else rc = launch_scan<256, 3, 1, 1>(ctx, a);
    }
    if (rc != HM_OK) return rc;
    hipLaunchKernelGGL(matrix_memory_out_kernel, dim3((unsigned)(((size_t)a.n * s.heads + 3) / 4)), dim3(256), 0, ctx->stream, a, chunks);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
