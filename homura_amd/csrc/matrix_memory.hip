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

// q (scaled) and k as pieces, four columns a thread (dim_pad / 4 threads a head and row); with K slices the v columns
// are added up in place.
__global__ __launch_bounds__(256) void matrix_memory_split_kernel(MatrixMemoryRowsArgs a, size_t qk_jobs, size_t v_jobs) {
    const MatrixMemoryShape &s = a.s;
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    const RowSource in{a.rows, a.ld, a.parts, a.stride, nullptr};
    if (e < qk_jobs) {
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
        return;
    }
    const size_t i = e - qk_jobs;
    if (i >= v_jobs) return;
    const int width = (s.heads * s.vdim + 3) / 4;
    const size_t at = (i / width) * a.ld + a.at.v + (i % width) * 4;  // (up to three columns of the padding behind)
    *reinterpret_cast<f32x4 *>(a.rows + at) = sum_parts4(a.rows, at, a.parts, a.stride);
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

// The scan: workgroup (head, tile of 16 columns) walks the chunks with eight wavefronts in two roles, one of each on a
// SIMD. Both read the chunk's K tile from LDS; the memory goes from the second role to the first through LDS, as three
// pieces, so the two work on the same chunk side by side.
//   rows     wavefront w, rows 16 w .. 16 w + 15 of the chunk
//     scores^T   A = 16 keys x 32 dims, B = 16 queries: lane t + 16 c receives keys 4 c .. 4 c + 3 of the block for row t;
//                times their weights they are the B operand of the last product in place
//     o^T        A = memory^T (16 columns x 32 dims), B = queries; times the memory's weight of the row; then
//                A = values^T (16 columns x 32 tokens), B = weighted scores
//   memory   wavefront w, a quarter of the memory's rows (DIM / 64 blocks of 16) in accumulators of the matrix cores
//                A = keys^T through the transposing LDS read, B = weighted values; it also requests the next K tile
// Contraction slot 8 c + i of tokens stands for token 4 c + i (i < 4) or 16 + 4 c + i - 4 of its 32, as in the causal
// attention. Values are the same registers as A operand (plain) and B operand (weighted): column lane % 16.
// KP: pieces of q, k and v (3: f32). KB: K tiles in LDS (2: the next chunk's arrives meanwhile).
extern __shared__ __attribute__((aligned(16))) char mm_lds[];

// 16 values of a lane's column as they meet the matrix cores: tokens 32 ks + 4 c4 + i and 32 ks + 16 + 4 c4 + i - 4
__device__ __forceinline__ int slot_token(int ks, int c4, int i) { return 32 * ks + 4 * c4 + (i < 4 ? i : 12 + i); }

template <int DIM, int KP, int KB>
__global__ __launch_bounds__(512) void matrix_memory_scan_kernel(MatrixMemoryRowsArgs a, int chunks) {
    constexpr int KSTEPS = DIM / 32, DT = DIM / 64;
    constexpr int KTILE = MM_CHUNK * DIM * 2, MPIECE = DIM * 32, MEM = 3 * MPIECE;  // bytes
    constexpr int KLOADS = MM_CHUNK * DIM / 8 / 256;
    __shared__ __attribute__((aligned(16))) double s_a[2][MM_CHUNK];
    const MatrixMemoryShape &s = a.s;
    const int tid = threadIdx.x & 255, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, c4 = lane >> 4;
    const bool rows_role = __builtin_amdgcn_readfirstlane(threadIdx.x >> 8) == 0;  // (a scalar branch: both sides hold barriers)
    const int tiles = s.tiles(), h = blockIdx.x / tiles, tile = blockIdx.x % tiles, n = a.n;
    const int col = tile * 16 + l16;  // this lane's column as an operand
    const bool own_v = col < s.vdim;
    const float fixed_v = col == s.vdim ? 1.f : 0.f;
    char *k_lds = mm_lds, *m_lds = mm_lds + KB * KP * KTILE;
    const size_t plane = (size_t)s.heads * n * DIM;
    const float *vg = a.rows + a.at.v + (size_t)h * s.vdim + min(col, s.vdim - 1);
    const size_t line = (size_t)chunks * MM_CHUNK, wplane = line * s.heads;
    auto load_values = [&](int c, float (&v)[2][8]) {
#pragma unroll
        for (int ks = 0; ks < 2; ks++)
#pragma unroll
            for (int i = 0; i < 8; i++) v[ks][i] = vg[(size_t)min(c * MM_CHUNK + slot_token(ks, c4, i), n - 1) * a.ld];
    };

    if (rows_role) {
        const uint16_t *qg = a.q + (size_t)h * n * DIM;
        const double *wa = a.log_w + h * line, *wm = wa + wplane;
        const float *w_mem = a.weights + h * line;
        const int row = wave * 16 + l16;
        // what a chunk brings; two sets take turns, so that the next chunk's is on its way meanwhile (one set where two
        // would not fit the registers)
        struct Rows {
            bf16x8 qf[KSTEPS][KP];
            float v[2][8];
            double tm;
            float tw;
        };
        auto load = [&](int c, Rows &r) {
            const uint16_t *src = qg + (size_t)min(c * MM_CHUNK + row, n - 1) * DIM + c4 * 8;
#pragma unroll
            for (int ks = 0; ks < KSTEPS; ks++)
#pragma unroll
                for (int p = 0; p < KP; p++) r.qf[ks][p] = *reinterpret_cast<const bf16x8 *>(src + p * plane + 32 * ks);
            load_values(c, r.v);
            r.tm = wm[c * MM_CHUNK + row];
            r.tw = w_mem[c * MM_CHUNK + row];
        };
        constexpr int SETS = KP * DIM > 256 ? 1 : 2;
        Rows set[SETS];
        load(0, set[0]);
        double ta = wa[lane];
        auto chunk = [&](int c, const Rows &r, Rows &next) {
            const bf16x8(&qf)[KSTEPS][KP] = r.qf;
            const float(&v)[2][8] = r.v;
            const double tm = r.tm;
            const float tw = r.tw;
            const int cb = c & 1;
            if (wave == 0) s_a[cb][lane] = ta;
            __syncthreads();  // keys, memory and log weights of the chunk are in LDS
            ta = wa[min(c + 1, chunks - 1) * MM_CHUNK + lane];
            if (SETS == 2) load(min(c + 1, chunks - 1), next);
            const char *kt = k_lds + (KB == 2 ? cb * KP * KTILE : 0), *mt = m_lds + cb * MEM;
            // memory ahead of the chunk, one sum for each of its pieces
            f32x4 om[3];
#pragma unroll
            for (int p = 0; p < 3; p++) om[p] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KSTEPS; ks++) {
                bf16x8 mf[3];
#pragma unroll
                for (int p = 0; p < 3; p++) mf[p] = *reinterpret_cast<const bf16x8 *>(mt + p * MPIECE + ((ks * 4 + c4) * 16 + l16) * 16);
                piece_products<3, KP>([&](int pm, int pq) { om[pm] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(mf[pm], qf[ks][pq], om[pm], 0, 0, 0); });
            }
            // tokens of the chunk up to the row's own
            f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int half = 0; half < 2; half++) {
                if (2 * half > wave) break;  // wavefront-uniform: all of them lie behind these rows
                f32x4 sc[2];
                sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < KSTEPS; ks++) {
                    bf16x8 kf[KP][2];
#pragma unroll
                    for (int p = 0; p < KP; p++)
#pragma unroll
                        for (int b = 0; b < 2; b++)
                            kf[p][b] = *reinterpret_cast<const bf16x8 *>(kt + p * KTILE + k_off<DIM>(32 * half + 16 * b + l16, 4 * ks + c4));
                    piece_products<KP, KP>([&](int pq, int pk) {
#pragma unroll
                        for (int b = 0; b < 2; b++) sc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[pk][b], qf[ks][pq], sc[b], 0, 0, 0);
                    });
                }
                float f[8], x[8];
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const int key = 32 * half + 16 * (i >> 2) + 4 * c4 + (i & 3);
                    const float w = __builtin_amdgcn_exp2f((float)(s_a[cb][key] - tm));
                    f[i] = key <= row ? sc[i >> 2][i & 3] * w : 0.f;
                    x[i] = own_v ? v[half][i] : fixed_v;
                }
                bf16x8 pf[3], vf[KP];
                split8<3>(f, pf);
                split8<KP>(x, vf);
                piece_products<3, KP>([&](int pp, int pv) { o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[pv], pf[pp], o, 0, 0, 0); });
            }
            o = o + ((om[2] + om[1]) + om[0]) * tw;
            const int t = c * MM_CHUNK + row;
            if (t < n) __builtin_nontemporal_store(o, reinterpret_cast<f32x4 *>(a.raw + ((size_t)t * s.heads + h) * s.cols() + tile * 16 + 4 * c4));
            if (KB == 1) __syncthreads();
            if (SETS == 1) load(min(c + 1, chunks - 1), next);
        };
        int c = 0;
        for (; c + 2 <= chunks; c += 2) {
            chunk(c, set[0], set[SETS - 1]);
            chunk(c + 1, set[SETS - 1], set[0]);
        }
        if (c < chunks) chunk(c, set[0], set[SETS - 1]);
        return;
    }

    const uint16_t *kg = a.k + (size_t)h * n * DIM;
    const float *w_end = a.weights + wplane + h * line;
    float *mem = a.state + (size_t)blockIdx.x * DIM * 16;
    int k_row[KLOADS], k_col[KLOADS];
#pragma unroll
    for (int i = 0; i < KLOADS; i++) {
        const int g = i * 256 + tid;
        k_row[i] = g / (DIM / 8);
        k_col[i] = (k_off<DIM>(k_row[i], g % (DIM / 8)) - k_row[i] * DIM * 2) >> 1;
    }
    const int wave_dst = __builtin_amdgcn_readfirstlane(wave * 1024);
    auto request_keys = [&](int c) {
        char *base = k_lds + (KB == 2 ? (c & 1) * KP * KTILE : 0) + wave_dst;
#pragma unroll
        for (int i = 0; i < KLOADS; i++) {
            const uint16_t *src = kg + (size_t)min(c * MM_CHUNK + k_row[i], n - 1) * DIM + k_col[i];
#pragma unroll
            for (int p = 0; p < KP; p++) dma16_lds(src + p * plane, base + p * KTILE + i * 4096);
        }
    };
    f32x4 S[DT];  // block b, value i: row wave * DIM / 4 + 16 b + 4 c4 + i, column l16
#pragma unroll
    for (int b = 0; b < DT; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) S[b][i] = a.past ? mem[(wave * (DIM / 4) + 16 * b + 4 * c4 + i) * 16 + l16] : 0.f;
    // as pieces: [piece][dim / 8][column][8 dims]
    auto publish = [&](int buf) {
#pragma unroll
        for (int b = 0; b < DT; b++) {
            uint32_t lo[3], hi[3];
            split_pair<3>(S[b][0], S[b][1], lo);
            split_pair<3>(S[b][2], S[b][3], hi);
            const int d = wave * (DIM / 4) + 16 * b + 4 * c4;
            char *at = m_lds + buf * MEM + ((d >> 3) * 16 + l16) * 16 + (d & 4) * 2;
#pragma unroll
            for (int p = 0; p < 3; p++) *reinterpret_cast<u32x2 *>(at + p * MPIECE) = u32x2{lo[p], hi[p]};
        }
    };
    float v[2][8];
    f32x4 we[2][2];
    auto load = [&](int c) {
        load_values(c, v);
#pragma unroll
        for (int ks = 0; ks < 2; ks++)
#pragma unroll
            for (int b = 0; b < 2; b++) we[ks][b] = *reinterpret_cast<const f32x4 *>(w_end + c * MM_CHUNK + 32 * ks + 16 * b + 4 * c4);
    };
    request_keys(0);
    load(0);
    publish(0);
    for (int c = 0; c < chunks; c++) {
        const float decay = a.decay[h * chunks + c];
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this chunk's keys and values have landed
        __syncthreads();  // (KB 2: everybody is done with the other K tile and the other copy of the memory)
        if (KB == 2 && c + 1 < chunks) request_keys(c + 1);
        bf16x8 vf[2][3];
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            float x[8];
#pragma unroll
            for (int i = 0; i < 8; i++) x[i] = (own_v ? v[ks][i] : fixed_v) * we[ks][i >> 2][i & 3];
            split8<3>(x, vf[ks]);
        }
        if (c + 1 < chunks) load(c + 1);
        const char *kt = k_lds + (KB == 2 ? (c & 1) * KP * KTILE : 0);
#pragma unroll
        for (int b = 0; b < DT; b++) S[b] = S[b] * decay;
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            const int key = 32 * ks + 4 * c4 + (l16 >> 2), within = (l16 & 1) * 8;
            bf16x8 kf[DT][KP];
#pragma unroll
            for (int b = 0; b < DT; b++) {
                const int chunk = 2 * (wave * DT + b) + ((l16 & 3) >> 1);
#pragma unroll
                for (int p = 0; p < KP; p++) {
                    const char *tile0 = kt + p * KTILE;
                    const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                        (s16x4 __attribute__((address_space(3))) *)(tile0 + k_off<DIM>(key, chunk) + within));
                    const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                        (s16x4 __attribute__((address_space(3))) *)(tile0 + k_off<DIM>(16 + key, chunk) + within));
                    struct Pair { s16x4 lo, hi; } pr{lo, hi};
                    kf[b][p] = __builtin_bit_cast(bf16x8, pr);
                }
            }
            piece_products<3, KP>([&](int pv, int pk) {
#pragma unroll
                for (int b = 0; b < DT; b++) S[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[b][pk], vf[ks][pv], S[b], 0, 0, 0);
            });
        }
        publish((c & 1) ^ 1);
        if (KB == 1) {
            __syncthreads();  // everybody is done with the K tile
            if (c + 1 < chunks) request_keys(c + 1);
        }
    }
#pragma unroll
    for (int b = 0; b < DT; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) mem[(wave * (DIM / 4) + 16 * b + 4 * c4 + i) * 16 + l16] = S[b][i];
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
        const f32x4 v = value_columns(a.rows + (size_t)t * a.ld + a.at.v + (size_t)h * s.vdim, tile * 16 + c4 * 4, s.vdim);
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

template <int DIM, int KP, int KB>
int launch_scan(hm_ctx *ctx, const MatrixMemoryRowsArgs &a) {
    constexpr int LDS = KB * KP * MM_CHUNK * DIM * 2 + 2 * 3 * DIM * 32;
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void *>(matrix_memory_scan_kernel<DIM, KP, KB>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    HM_REQUIRE(ctx, attr == hipSuccess, "matrix_memory: cannot reserve %d bytes of LDS: %s", LDS, hipGetErrorString(attr));
    hipLaunchKernelGGL((matrix_memory_scan_kernel<DIM, KP, KB>), dim3(a.s.heads * a.s.tiles()), dim3(512), LDS, ctx->stream, a, a.chunks());
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
    const bool tiled = s.dim_pad <= 256;
    const size_t qk_jobs = tiled ? (size_t)a.n * 2 * s.heads * (s.dim_pad / 4) : 0, v_jobs = a.parts > 1 ? (size_t)a.n * (vw / 4) : 0;
    if (qk_jobs + v_jobs > 0) {
        hipLaunchKernelGGL(matrix_memory_split_kernel, dim3((unsigned)((qk_jobs + v_jobs + 255) / 256)), dim3(256), 0, ctx->stream, a, qk_jobs, v_jobs);
        HM_LAUNCH_CHECK(ctx);
    }
    hipLaunchKernelGGL(matrix_memory_gate_rows_kernel, dim3((a.n + 15) / 16, (2 * s.heads + 15) / 16), dim3(256), 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    hipLaunchKernelGGL(matrix_memory_gates_kernel, dim3(s.heads), dim3(64 * GATE_WAVES), 0, ctx->stream, a, chunks);
    HM_LAUNCH_CHECK(ctx);
    int rc = HM_OK;
    const dim3 g(s.heads * s.tiles()), b(256);
    if (!tiled) {
        if (s.dim_pad == 512) hipLaunchKernelGGL(matrix_memory_scan_any_kernel<8>, g, b, 0, ctx->stream, a, chunks);
        else hipLaunchKernelGGL(matrix_memory_scan_any_kernel<16>, g, b, 0, ctx->stream, a, chunks);
        HM_LAUNCH_CHECK(ctx);
    } else if (a.pieces == 1) {
        rc = s.dim_pad == 64 ? launch_scan<64, 1, 2>(ctx, a) : s.dim_pad == 128 ? launch_scan<128, 1, 2>(ctx, a) : launch_scan<256, 1, 2>(ctx, a);
    } else {
        rc = s.dim_pad == 64 ? launch_scan<64, 3, 2>(ctx, a) : s.dim_pad == 128 ? launch_scan<128, 3, 2>(ctx, a) : launch_scan<256, 3, 1>(ctx, a);
    }
    if (rc != HM_OK) return rc;
    hipLaunchKernelGGL(matrix_memory_out_kernel, dim3((unsigned)(((size_t)a.n * s.heads + 3) / 4)), dim3(256), 0, ctx->stream, a, chunks);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
