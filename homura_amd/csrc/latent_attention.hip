// Latent attention (see latent_attention.h).
#include "latent_attention.h"

#include <algorithm>

#include "row_pieces.h"

namespace {

using namespace homura;

// element i of a vector whose first `dims` elements turn by the angles of one position (pairs i, i + dims / 2)
template <class At>
__device__ __forceinline__ float rotated(At at, int i, int dims, const float *__restrict__ c, const float *__restrict__ sn) {
    if (i >= dims) return at(i);
    const int half = dims / 2;
    return i < half ? at(i) * c[i] - at(i + half) * sn[i] : at(i) * c[i] + at(i - half) * sn[i];
}

__device__ __forceinline__ float wg_sum256(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

__device__ __forceinline__ void store_row_pieces(uint16_t *row, int width, int i, float v, int pieces) {
    uint32_t p[3];
    split_pieces<3>(v, p);
    row[i] = (uint16_t)p[0];
    if (pieces == 3) {
        row[width + i] = (uint16_t)p[1];
        row[2 * width + i] = (uint16_t)p[2];
    }
}

// the cache row of one token, 256 threads: latent(i) and key(i) give the raw projections
template <class Lat, class Key>
__device__ __forceinline__ void cache_row(const LatentShape &s, Lat latent, Key key, const float *__restrict__ norm_w, float eps,
                                          const float *__restrict__ c, const float *__restrict__ sn, uint16_t *row, float *red) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < s.rank; i += 256) {
        const float v = latent(i);
        ss += v * v;
    }
    const float inv = 1.0f / sqrtf(wg_sum256(ss, red) / (float)s.rank + eps);
    const int width = s.row_width();
    for (int i = threadIdx.x; i < s.rank_pad; i += 256)
        store_row_pieces(row, width, i, i < s.rank ? (latent(i) * inv) * norm_w[i] : 0.f, s.pieces);
    for (int i = threadIdx.x; i < s.rot_pad; i += 256)
        store_row_pieces(row, width, s.rank_pad + i, i < s.rot_dim ? rotated(key, i, s.rot_dims, c, sn) : 0.f, s.pieces);
}

// ── decode step ──────────────────────────────────────────────────────────────

// Workgroup (head, 64 latent columns): q'[r] = scale * sum_d uk[d][r] q[d], eight groups of threads over d, two
// columns a thread; the first slice of a head also turns its rotated part. The last workgroup writes the cache row.
__global__ __launch_bounds__(256) void latent_step_prep_kernel(LatentStepArgs a, int slices) {
    __shared__ float red[8][66];
    const LatentShape &s = a.s;
    const int tid = threadIdx.x, pos = a.cursor->pos;
    const float *c = a.cos_tab + (size_t)pos * s.rot_dims, *sn = a.sin_tab + (size_t)pos * s.rot_dims;
    if ((int)blockIdx.x == s.heads * slices) {
        cache_row(s, [&](int i) { return a.kv[i]; }, [&](int i) { return a.kv[s.rank + i]; }, a.kv_norm, a.eps, c, sn,
                  a.ring + (size_t)(pos % s.ring_rows) * s.row_elems(), &red[0][0]);
        return;
    }
    const int h = blockIdx.x / slices, slice = blockIdx.x % slices;
    const float *q = a.q + (size_t)h * (s.dim + s.rot_dim);
    const int r = slice * 64 + 2 * (tid & 31), dg = tid >> 5;
    float a0 = 0.f, a1 = 0.f;
    if (r < s.rank_pad) {
        const uint16_t *w = a.uk + (size_t)h * s.dim * s.rank_pad + r;
#pragma unroll 8
        for (int d = dg; d < s.dim; d += 8) {
            const uint32_t v = *reinterpret_cast<const uint32_t *>(w + (size_t)d * s.rank_pad);
            a0 = fmaf(bf16_lo(v), q[d], a0);
            a1 = fmaf(bf16_hi(v), q[d], a1);
        }
    }
    red[dg][2 * (tid & 31)] = a0;
    red[dg][2 * (tid & 31) + 1] = a1;
    __syncthreads();
    float *out = a.q_latent + (size_t)h * s.row_width();
    if (tid < 64 && slice * 64 + tid < s.rank_pad) {
        float v = 0.f;
#pragma unroll
        for (int g = 0; g < 8; g++) v += red[g][tid];
        out[slice * 64 + tid] = v * a.scale;
    }
    if (slice == 0)
        for (int i = tid; i < s.rot_pad; i += 256)
            out[s.rank_pad + i] = i < s.rot_dim ? rotated([&](int k) { return q[s.dim + k]; }, i, s.rot_dims, c, sn) * a.scale : 0.f;
}

// Workgroup (split of the visible rows, 16 heads): all heads share the key rows, so both products run on the matrix
// cores, 16 heads x 32 keys x row width and latent columns x 32 keys x 16 heads. A tile of 32 rows goes into LDS (rows
// 16 bytes apart from whole banks); the four wavefronts take the 32-wide steps of the row width in turn and their
// scores meet in LDS; the softmax runs on 16 lanes a head; then every wavefront mixes its share of the latent columns.
// Queries and probabilities are f32 as three bf16 pieces. Further tiles of a split rescale what is there.
//   scores: A = 16 keys x 32 of the row, B = queries: lane q + 16 c receives keys 4 c .. 4 c + 3 of the block
//   mix^T:  A = 16 columns x 32 keys through the transposing LDS read, B = probabilities, contraction slot 8 c + i
//           (i < 4) standing for key 4 c + i and slot 8 c + 4 + i for key 16 + 4 c + i
constexpr int LS_KEYS = 32;
constexpr int LS_STEPS = 5;  // 32-wide steps of the row width a wavefront asks for at once
typedef short s16x4 __attribute__((ext_vector_type(4)));

// head sh (tid / 16), keys sk and sk + 16 of a tile (tid % 16): running softmax over the scores x, probabilities to p
__device__ __forceinline__ float tile_softmax(float x0, float x1, float &m_run, float &l_run, float &p0, float &p1) {
    float mx = fmaxf(x0, x1);
    mx = fmaxf(mx, dpp_move<0xB1, 0xF>(mx, mx));
    mx = fmaxf(mx, dpp_move<0x4E, 0xF>(mx, mx));
    mx = fmaxf(mx, dpp_move<0x141, 0xF>(mx, mx));
    mx = fmaxf(mx, dpp_move<0x140, 0xF>(mx, mx));
    const float m_new = fmaxf(m_run, mx);  // finite: a tile's first key is visible
    const float alpha = expf(m_run - m_new);
    p0 = expf(x0 - m_new);
    p1 = expf(x1 - m_new);
    float sum = p0 + p1;
    sum += dpp_move<0xB1, 0xF>(sum, 0.f);
    sum += dpp_move<0x4E, 0xF>(sum, 0.f);
    sum += dpp_move<0x141, 0xF>(sum, 0.f);
    sum += dpp_move<0x140, 0xF>(sum, 0.f);
    l_run = l_run * alpha + sum;
    m_run = m_new;
    return alpha;
}

__host__ __device__ inline int ls_row_bytes(int width) { return width * 2 + 16; }

template <int KP, int NB>  // NB: 16-wide blocks of latent columns a wavefront mixes, rank_pad <= 64 * NB
__global__ __launch_bounds__(256) void latent_step_attn_lds_kernel(LatentStepArgs a, int tiles) {
    extern __shared__ __attribute__((aligned(16))) char tile[];  // [KP][32 rows]
    __shared__ f32x4 s_part[4][2][64];
    __shared__ __attribute__((aligned(16))) float s_p[16][LS_KEYS];
    __shared__ float s_alpha[16];
    const LatentShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, c4 = lane >> 4;
    const int h0 = blockIdx.y * 16;
    const int width = s.row_width(), ksteps = width / 32, row_b = ls_row_bytes(width), plane_b = LS_KEYS * row_b;
    const float *q = a.q_latent + (size_t)min(h0 + l16, s.heads - 1) * width + c4 * 8;
    // the queries of a wavefront's first steps stay in registers
    f32x4 qa[LS_STEPS], qb[LS_STEPS];
#pragma unroll
    for (int u = 0; u < LS_STEPS; u++) {
        const int ks = min(wave + 4 * u, ksteps - 1);
        qa[u] = *reinterpret_cast<const f32x4 *>(q + 32 * ks);
        qb[u] = *reinterpret_cast<const f32x4 *>(q + 32 * ks + 4);
    }
    const int pos = a.cursor->pos, lo = s.window ? max(0, pos - s.window + 1) : 0;
    const int first = lo + (int)blockIdx.x * tiles * LS_KEYS;
    if (first > pos) return;  // (the fold counts the live splits the same way)
    f32x4 acc[NB];
#pragma unroll
    for (int i = 0; i < NB; i++) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int sh = tid >> 4, sk = tid & 15;
    float m_run = -INFINITY, l_run = 0.f;
    const int blocks = s.rank_pad / 16;
    const int v_key = 4 * c4 + (l16 >> 2), v_col = (l16 & 3) * 8;  // this lane's part of a transposing read
    for (int t = 0; t < tiles; t++) {
        const int key0 = first + t * LS_KEYS;
        if (key0 > pos) break;  // workgroup-uniform
        // the tile: eight threads a row, 16 bytes each in turn
        {
            const int r = tid >> 3, sub = tid & 7, chunks = width / 8;
            const uint16_t *src = a.ring + (size_t)(min(key0 + r, pos) % s.ring_rows) * s.row_elems();
            char *dst = tile + r * row_b;
#pragma unroll
            for (int p = 0; p < KP; p++) {
                for (int base = sub; base < chunks; base += 8 * 9) {
                    u32x4 v[9];
#pragma unroll
                    for (int u = 0; u < 9; u++) v[u] = ld128(src + p * width + 8 * min(base + 8 * u, chunks - 1));
#pragma unroll
                    for (int u = 0; u < 9; u++)
                        if (base + 8 * u < chunks) *reinterpret_cast<u32x4 *>(dst + p * plane_b + 16 * (base + 8 * u)) = v[u];
                }
            }
        }
        __syncthreads();
        f32x4 sc[2];
        sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int base = wave; base < ksteps; base += 4 * LS_STEPS) {
            f32x4 q0[LS_STEPS], q1[LS_STEPS];
#pragma unroll
            for (int u = 0; u < LS_STEPS; u++) {
                q0[u] = qa[u];
                q1[u] = qb[u];
                if (base != wave) {
                    const int ks = min(base + 4 * u, ksteps - 1);
                    q0[u] = *reinterpret_cast<const f32x4 *>(q + 32 * ks);
                    q1[u] = *reinterpret_cast<const f32x4 *>(q + 32 * ks + 4);
                }
            }
#pragma unroll
            for (int u = 0; u < LS_STEPS; u++) {
                const int ks = base + 4 * u;
                if (ks >= ksteps) break;
                float f[8];
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    f[i] = q0[u][i];
                    f[4 + i] = q1[u][i];
                }
                bf16x8 qf[3], kf[KP][2];
                split8<3>(f, qf);
#pragma unroll
                for (int p = 0; p < KP; p++)
#pragma unroll
                    for (int kb = 0; kb < 2; kb++)
                        kf[p][kb] = *reinterpret_cast<const bf16x8 *>(tile + p * plane_b + (16 * kb + l16) * row_b + 64 * ks + 16 * c4);
#pragma unroll
                for (int order = KP + 1; order >= 0; order--)
#pragma unroll
                    for (int pq = 2; pq >= 0; pq--) {
                        const int pk = order - pq;
                        if (pk < 0 || pk >= KP || (KP > 1 && order > 2)) continue;
#pragma unroll
                        for (int kb = 0; kb < 2; kb++) sc[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[pk][kb], qf[pq], sc[kb], 0, 0, 0);
                    }
            }
        }
        s_part[wave][0][lane] = sc[0];
        s_part[wave][1][lane] = sc[1];
        __syncthreads();
        float x[2], p0, p1;
#pragma unroll
        for (int kb = 0; kb < 2; kb++) {
            const int from = sh + 16 * (sk >> 2);
            float v = 0.f;
#pragma unroll
            for (int w = 0; w < 4; w++) v += reinterpret_cast<const float *>(&s_part[w][kb][from])[sk & 3];
            x[kb] = key0 + 16 * kb + sk <= pos ? v : -INFINITY;
        }
        const float alpha = tile_softmax(x[0], x[1], m_run, l_run, p0, p1);
        s_p[sh][sk] = p0;
        s_p[sh][16 + sk] = p1;
        if (sk == 0) s_alpha[sh] = alpha;
        __syncthreads();
        if (t > 0) {
            const float al = s_alpha[l16];
#pragma unroll
            for (int i = 0; i < NB; i++) acc[i] *= al;
        }
        float f[8];
        {
            const f32x4 a0 = *reinterpret_cast<const f32x4 *>(&s_p[l16][4 * c4]), a1 = *reinterpret_cast<const f32x4 *>(&s_p[l16][16 + 4 * c4]);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                f[i] = a0[i];
                f[4 + i] = a1[i];
            }
        }
        bf16x8 pp[3];
        split8<3>(f, pp);
#pragma unroll
        for (int i = 0; i < NB; i++) {
            const int db = wave + 4 * i;
            if (db >= blocks) break;
            bf16x8 vf[KP];
#pragma unroll
            for (int p = 0; p < KP; p++) {
                const char *at = tile + p * plane_b + v_key * row_b + 32 * db + v_col;
                const s16x4 lo16 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3))) *)at);
                const s16x4 hi16 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3))) *)(at + 16 * row_b));
                struct Pair { s16x4 lo, hi; } pr{lo16, hi16};
                vf[p] = __builtin_bit_cast(bf16x8, pr);
            }
#pragma unroll
            for (int order = KP + 1; order >= 0; order--)
#pragma unroll
                for (int pq = 2; pq >= 0; pq--) {
                    const int pk = order - pq;
                    if (pk < 0 || pk >= KP || (KP > 1 && order > 2)) continue;
                    acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[pk], pp[pq], acc[i], 0, 0, 0);
                }
        }
        if (t + 1 < tiles) __syncthreads();  // the tile, s_part and s_p are written again
    }
    if (sk == 0 && h0 + sh < s.heads) {
        float *ml = a.part_ml + ((size_t)blockIdx.x * s.heads + h0 + sh) * 2;
        ml[0] = m_run;
        ml[1] = l_run;
    }
    if (h0 + l16 < s.heads) {
        float *o = a.part_o + ((size_t)blockIdx.x * s.heads + h0 + l16) * s.rank_pad + 4 * c4;
#pragma unroll
        for (int i = 0; i < NB; i++)
            if (wave + 4 * i < blocks) *reinterpret_cast<f32x4 *>(o + 16 * (wave + 4 * i)) = acc[i];
    }
}

// The same for rows too wide for LDS (f32 latents above 768 columns): the tile's rows are read where they are, and
// the latents mixed with f32 weights on the vector units, two columns a thread.
__global__ __launch_bounds__(256) void latent_step_attn_wide_kernel(LatentStepArgs a, int tiles) {
    constexpr int KP = 3, LS_COLS = 2;  // pieces, column pairs per thread (rank_pad <= 1024)
    __shared__ f32x4 s_part[4][2][64];
    __shared__ __attribute__((aligned(16))) float s_p[16][LS_KEYS];
    __shared__ float s_alpha[16];
    const LatentShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, c4 = lane >> 4;
    const int pos = a.cursor->pos, lo = s.window ? max(0, pos - s.window + 1) : 0;
    const int first = lo + (int)blockIdx.x * tiles * LS_KEYS, h0 = blockIdx.y * 16;
    if (first > pos) return;
    const int width = s.row_width(), ksteps = width / 32;
    const float *q = a.q_latent + (size_t)min(h0 + l16, s.heads - 1) * width + c4 * 8;
    float acc[LS_COLS][16][2];
#pragma unroll
    for (int j = 0; j < LS_COLS; j++)
#pragma unroll
        for (int h = 0; h < 16; h++) acc[j][h][0] = acc[j][h][1] = 0.f;
    const int sh = tid >> 4, sk = tid & 15;  // softmax role: head, keys sk and sk + 16
    float m_run = -INFINITY, l_run = 0.f;
    const int cols = s.rank_pad / 2;  // column pairs
    for (int t = 0; t < tiles; t++) {
        const int key0 = first + t * LS_KEYS;
        if (key0 > pos) break;  // workgroup-uniform
        // scores
        const uint16_t *row[2];
#pragma unroll
        for (int kb = 0; kb < 2; kb++)
            row[kb] = a.ring + (size_t)(min(key0 + 16 * kb + l16, pos) % s.ring_rows) * s.row_elems() + c4 * 8;
        f32x4 sc[2];
        sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int ks = wave; ks < ksteps; ks += 4) {
            float f[8];
            const f32x4 q0 = *reinterpret_cast<const f32x4 *>(q + 32 * ks), q1 = *reinterpret_cast<const f32x4 *>(q + 32 * ks + 4);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                f[i] = q0[i];
                f[4 + i] = q1[i];
            }
            bf16x8 kf[KP][2], qf[3];
#pragma unroll
            for (int p = 0; p < KP; p++)
#pragma unroll
                for (int kb = 0; kb < 2; kb++) kf[p][kb] = *reinterpret_cast<const bf16x8 *>(row[kb] + p * width + 32 * ks);
            split8<3>(f, qf);
#pragma unroll
            for (int order = 2; order >= 0; order--)
#pragma unroll
                for (int pq = order; pq >= 0; pq--)
#pragma unroll
                    for (int kb = 0; kb < 2; kb++) sc[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[order - pq][kb], qf[pq], sc[kb], 0, 0, 0);
        }
        s_part[wave][0][lane] = sc[0];
        s_part[wave][1][lane] = sc[1];
        __syncthreads();
        // head sh, key 16 kb + 4 c + i sits in lane sh + 16 c, element i of block kb
        float x[2];
#pragma unroll
        for (int kb = 0; kb < 2; kb++) {
            const int from = sh + 16 * (sk >> 2);
            float v = 0.f;
#pragma unroll
            for (int w = 0; w < 4; w++) v += reinterpret_cast<const float *>(&s_part[w][kb][from])[sk & 3];
            x[kb] = key0 + 16 * kb + sk <= pos ? v : -INFINITY;
        }
        float p0, p1;
        const float alpha = tile_softmax(x[0], x[1], m_run, l_run, p0, p1);
        s_p[sh][sk] = p0;
        s_p[sh][16 + sk] = p1;
        if (sk == 0) s_alpha[sh] = alpha;
        __syncthreads();
        // latents
#pragma unroll
        for (int j = 0; j < LS_COLS; j++) {
            const int cp = tid + j * 256;
            if (cp >= cols) break;
            if (t > 0) {
#pragma unroll
                for (int h = 0; h < 16; h++) {
                    acc[j][h][0] *= s_alpha[h];
                    acc[j][h][1] *= s_alpha[h];
                }
            }
            const int live = min(LS_KEYS, pos - key0 + 1);  // (rows behind it weigh nothing: p = 0)
            for (int k4 = 0; k4 < live; k4 += 4) {
                float v0[4], v1[4];
#pragma unroll
                for (int k = 0; k < 4; k++) {
                    const uint16_t *src = a.ring + (size_t)(min(key0 + k4 + k, pos) % s.ring_rows) * s.row_elems() + 2 * cp;
                    const uint32_t w0 = *reinterpret_cast<const uint32_t *>(src), w1 = *reinterpret_cast<const uint32_t *>(src + width),
                                   w2 = *reinterpret_cast<const uint32_t *>(src + 2 * width);
                    v0[k] = bf16_lo(w0) + (bf16_lo(w1) + bf16_lo(w2));
                    v1[k] = bf16_hi(w0) + (bf16_hi(w1) + bf16_hi(w2));
                }
#pragma unroll
                for (int h = 0; h < 16; h++) {
                    const f32x4 p = *reinterpret_cast<const f32x4 *>(&s_p[h][k4]);
#pragma unroll
                    for (int k = 0; k < 4; k++) {
                        acc[j][h][0] = fmaf(p[k], v0[k], acc[j][h][0]);
                        acc[j][h][1] = fmaf(p[k], v1[k], acc[j][h][1]);
                    }
                }
            }
        }
        __syncthreads();  // s_part and s_p are written again
    }
    if (sk == 0 && h0 + sh < s.heads) {
        float *ml = a.part_ml + ((size_t)blockIdx.x * s.heads + h0 + sh) * 2;
        ml[0] = m_run;
        ml[1] = l_run;
    }
#pragma unroll
    for (int j = 0; j < LS_COLS; j++) {
        const int cp = tid + j * 256;
        if (cp >= cols) break;
#pragma unroll
        for (int h = 0; h < 16; h++)
            if (h0 + h < s.heads) {
                float *o = a.part_o + ((size_t)blockIdx.x * s.heads + h0 + h) * s.rank_pad + 2 * cp;
                o[0] = acc[j][h][0];
                o[1] = acc[j][h][1];
            }
    }
}

// Workgroup (head, LF_ROWS value rows): the splits' mixes against the largest maximum, in split order, then the
// value rows from LDS and the gate.
constexpr int LF_ROWS = 32, LF_MAX_SPLITS = 64;  // a split a lane
constexpr int LF_THREADS = 512;
__host__ __device__ inline int fold_groups(int rank_pad) { return LF_THREADS / (rank_pad / 4); }
__global__ __launch_bounds__(LF_THREADS) void latent_step_fold_kernel(LatentStepArgs a, int tiles, int splits) {
    extern __shared__ __attribute__((aligned(16))) float o_part[];  // [groups][rank_pad]; the sum ends up in group 0
    const LatentShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x;
    // the value rows of this workgroup go out first: they are needed last, and depend on nothing
    constexpr int WAVES = LF_THREADS / 64, RW = LF_ROWS / WAVES;
    u32x4 uv[RW];
    const bool in_row = lane * 8 < s.rank_pad;
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const int j = min((int)blockIdx.y * LF_ROWS + wave + WAVES * i, s.vdim - 1);
        uv[i] = in_row ? ld128(a.uv + ((size_t)h * s.vdim + j) * s.rank_pad + lane * 8) : u32x4{0u, 0u, 0u, 0u};
    }
    // four columns a thread; the splits are dealt to as many groups as the columns leave threads for. The first
    // FOLD_AHEAD of a thread's splits are asked for at once, before it is known how many ran (what the others hold is
    // old, finite, and weighs nothing).
    const int n4 = s.rank_pad / 4, groups = fold_groups(s.rank_pad);
    const int g = tid / n4, c = (tid - g * n4) * 4;
    const float *po = a.part_o + (size_t)h * s.rank_pad + c;
    const size_t per_split = (size_t)s.heads * s.rank_pad;
    constexpr int FOLD_AHEAD = 16;
    f32x4 o[FOLD_AHEAD];
    if (g < groups) {
#pragma unroll
        for (int u = 0; u < FOLD_AHEAD; u++) o[u] = *reinterpret_cast<const f32x4 *>(po + (size_t)min(g + u * groups, splits - 1) * per_split);
    }
    // every wavefront forms the splits' weights itself, a split a lane
    float m = -INFINITY, l = 0.f;
    const int pos = a.cursor->pos, lo = s.window ? max(0, pos - s.window + 1) : 0;
    const int live = (pos - lo) / (tiles * LS_KEYS) + 1;  // splits that ran
    if (lane < splits) {
        m = a.part_ml[((size_t)lane * s.heads + h) * 2];
        l = a.part_ml[((size_t)lane * s.heads + h) * 2 + 1];
    }
    if (lane >= live) {
        m = -INFINITY;
        l = 0.f;
    }
    const float w = expf(m - wave_max(m));
    const float inv = 1.0f / wave_sum(w * l);
    {
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int u = 0; u < FOLD_AHEAD; u++) {
            const int t = g + u * groups;
            const float wt = __shfl(w, t & 63);
            if (t < live)
#pragma unroll
                for (int k = 0; k < 4; k++) v[k] = fmaf(wt, o[u][k], v[k]);
        }
        for (int t = g + FOLD_AHEAD * groups; __any(t < live); t += groups) {
            const float wt = __shfl(w, t & 63);
            if (t < live && g < groups) {
                const f32x4 x = *reinterpret_cast<const f32x4 *>(po + (size_t)t * per_split);
#pragma unroll
                for (int k = 0; k < 4; k++) v[k] = fmaf(wt, x[k], v[k]);
            }
        }
        if (g < groups) *reinterpret_cast<f32x4 *>(o_part + g * s.rank_pad + c) = v;
    }
    __syncthreads();
    if (g == 0) {
        f32x4 v = *reinterpret_cast<const f32x4 *>(o_part + c);
        for (int q = 1; q < groups; q++) v += *reinterpret_cast<const f32x4 *>(o_part + q * s.rank_pad + c);
        *reinterpret_cast<f32x4 *>(o_part + c) = v * inv;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const int j = blockIdx.y * LF_ROWS + wave + WAVES * i;
        if (j >= s.vdim) break;
        const uint16_t *wr = a.uv + ((size_t)h * s.vdim + j) * s.rank_pad;
        float acc = 0.f;
        for (int k = lane * 8; k < s.rank_pad; k += 512) {
            const u32x4 v = k < 512 ? uv[i] : ld128(wr + k);
            const f32x4 x0 = *reinterpret_cast<const f32x4 *>(o_part + k), x1 = *reinterpret_cast<const f32x4 *>(o_part + k + 4);
            acc = fmaf(bf16_lo(v.x), x0[0], acc);
            acc = fmaf(bf16_hi(v.x), x0[1], acc);
            acc = fmaf(bf16_lo(v.y), x0[2], acc);
            acc = fmaf(bf16_hi(v.y), x0[3], acc);
            acc = fmaf(bf16_lo(v.z), x1[0], acc);
            acc = fmaf(bf16_hi(v.z), x1[1], acc);
            acc = fmaf(bf16_lo(v.w), x1[2], acc);
            acc = fmaf(bf16_hi(v.w), x1[3], acc);
        }
        acc = wave_sum(acc);
        if (lane == 0) {
            const int out_c = h * s.vdim + j;
            if (a.gate) acc = acc / (1.0f + expf(-a.gate[out_c]));
            a.out[out_c] = acc;
        }
    }
}

// tiles a split, so that there are at most LF_MAX_SPLITS splits
int step_tiles(int span) {
    const int all = (span + LS_KEYS - 1) / LS_KEYS;
    return std::max(1, (all + LF_MAX_SPLITS - 1) / LF_MAX_SPLITS);
}

// ── prompt pass ──────────────────────────────────────────────────────────────

__global__ __launch_bounds__(256) void latent_rows_kernel(LatentRowsArgs a) {
    __shared__ float red[4];
    const LatentShape &s = a.s;
    const int t = blockIdx.x, pos = a.past + t;
    if (blockIdx.y == 1) {  // the cache row
        cache_row(s, [&](int i) { return source_at(a.down, t, a.q_rank_pad + i); },
                  [&](int i) { return source_at(a.down, t, a.q_rank_pad + s.rank + i); }, a.kv_norm, a.eps,
                  a.cos_tab + (size_t)pos * s.rot_dims, a.sin_tab + (size_t)pos * s.rot_dims,
                  a.ring + (size_t)(pos % s.ring_rows) * s.row_elems(), red);
        return;
    }
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.q_rank; i += 256) {
        const float v = source_at(a.down, t, i);
        ss += v * v;
    }
    const float inv = 1.0f / sqrtf(wg_sum256(ss, red) / (float)a.q_rank + a.eps);
    uint16_t *row = a.q_split + (size_t)t * a.q_pieces * a.q_rank_pad;
    for (int i = threadIdx.x; i < a.q_rank_pad; i += 256)
        split_store(row, a.q_rank_pad, i, i < a.q_rank ? (source_at(a.down, t, i) * inv) * a.q_norm[i] : 0.f, a.q_pieces);
}

// V elements of a query row a thread; V = 4 wants every part of a row to be whole vectors
template <int V>
__global__ __launch_bounds__(256) void latent_q_rows_kernel(LatentShape s, RowSource q, const float *__restrict__ cos_tab,
                                                            const float *__restrict__ sin_tab, float *__restrict__ out, int width,
                                                            int past, size_t total) {
    const size_t e = ((size_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (e >= total) return;
    const int i = (int)(e % width), h = (int)(e / width % s.heads), t = (int)(e / width / s.heads);
    const int base = h * (s.dim + s.rot_dim), half = s.rot_dims / 2, r = i - s.dim;
    if constexpr (V == 4) {
        const size_t at = (size_t)t * q.ld + base;
        auto get = [&](int k) { return sum_parts4(q.p, at + k, q.parts, q.stride); };
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < 0 || (r >= s.rot_dims && r < s.rot_dim)) {
            v = get(i);
        } else if (r < s.rot_dim) {
            const size_t tab = (size_t)(past + t) * s.rot_dims + r;
            const f32x4 c = *reinterpret_cast<const f32x4 *>(cos_tab + tab), sn = *reinterpret_cast<const f32x4 *>(sin_tab + tab);
            const f32x4 x = get(i), o = get(r < half ? i + half : i - half);
#pragma unroll
            for (int k = 0; k < 4; k++) v[k] = r < half ? x[k] * c[k] - o[k] * sn[k] : x[k] * c[k] + o[k] * sn[k];
        }
        *reinterpret_cast<f32x4 *>(out + e) = v;
    } else {
        float v = 0.f;
        if (r < 0) {
            v = source_at(q, t, base + i);
        } else if (r < s.rot_dim) {
            const int pos = past + t;
            v = rotated([&](int k) { return source_at(q, t, base + s.dim + k); }, r, s.rot_dims, cos_tab + (size_t)pos * s.rot_dims,
                        sin_tab + (size_t)pos * s.rot_dims);
        }
        out[e] = v;
    }
}

// 16 bytes a thread
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentShape s, const uint16_t *__restrict__ ring, uint16_t *__restrict__ out,
                                                            int first, size_t total) {
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= total) return;
    const int per_row = s.pieces * s.rank_pad / 8, c = (int)(e % per_row) * 8;
    const size_t r = e / per_row;
    const int p = c / s.rank_pad, i = c % s.rank_pad;
    *reinterpret_cast<u32x4 *>(out + e * 8) =
        ld128(ring + (size_t)((first + (int)r) % s.ring_rows) * s.row_elems() + p * s.row_width() + i);
}

// 8 elements of a key or value row a thread
__global__ __launch_bounds__(256) void latent_kv_rows_kernel(LatentShape s, RowSource kv, int v_at, const uint16_t *__restrict__ ring,
                                                             uint16_t *__restrict__ k_out, uint16_t *__restrict__ v_out, int kw, int vw,
                                                             int cap, int first, bool vec, size_t total) {
    const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= total) return;
    const int per = (kw + vw) / 8;  // pieces of 8 of one (row, head)
    const int i8 = (int)(e % per) * 8;
    const int h = (int)(e / per % s.heads);
    const int r = (int)(e / per / s.heads);
    const bool is_v = i8 >= kw;
    const int i0 = is_v ? i8 - kw : i8, w = is_v ? vw : kw;
    const size_t plane = (size_t)s.heads * cap * w;
    uint16_t *dst = (is_v ? v_out : k_out) + ((size_t)h * cap + r) * w + i0;
    const uint16_t *row = ring + (size_t)((first + r) % s.ring_rows) * s.row_elems() + s.rank_pad;
    uint32_t word[3][4];
    if (vec) {  // dim, rot_dim and vdim are multiples of 8: the eight elements are of one kind
        const int at = is_v ? (i0 < s.vdim ? v_at + h * s.vdim + i0 : -1) : i0 < s.dim ? h * s.dim + i0 : -1;
        if (at >= 0) {
            const f32x4 a0 = sum_parts4(kv.p, (size_t)r * kv.ld + at, kv.parts, kv.stride), a1 = sum_parts4(kv.p, (size_t)r * kv.ld + at + 4, kv.parts, kv.stride);
#pragma unroll
            for (int k = 0; k < 4; k++) {
                uint32_t p[3];
                split_pair<3>(k < 2 ? a0[2 * k] : a1[2 * k - 4], k < 2 ? a0[2 * k + 1] : a1[2 * k - 3], p);
#pragma unroll
                for (int q = 0; q < 3; q++) word[q][k] = p[q];
            }
        } else {
            const bool rot = !is_v && i0 >= s.dim && i0 < s.dim + s.rot_dim;
#pragma unroll
            for (int q = 0; q < 3; q++) {
                u32x4 v = {0u, 0u, 0u, 0u};
                if (rot && q < s.pieces) v = ld128(row + q * s.row_width() + i0 - s.dim);
                word[q][0] = v.x;
                word[q][1] = v.y;
                word[q][2] = v.z;
                word[q][3] = v.w;
            }
        }
    } else
#pragma unroll
    for (int k = 0; k < 8; k++) {
        const int i = i0 + k;
        uint32_t p[3] = {0u, 0u, 0u};
        if (is_v) {
            if (i < s.vdim) split_pieces<3>(source_at(kv, r, v_at + h * s.vdim + i), p);
        } else if (i < s.dim) {
            split_pieces<3>(source_at(kv, r, h * s.dim + i), p);
        } else if (i < s.dim + s.rot_dim) {
            for (int q = 0; q < s.pieces; q++) p[q] = row[q * s.row_width() + i - s.dim];
        }
#pragma unroll
        for (int q = 0; q < 3; q++) word[q][k / 2] = k & 1 ? word[q][k / 2] | (p[q] << 16) : p[q];
    }
#pragma unroll
    for (int q = 0; q < 3; q++)
        if (q < s.pieces) {
            u32x4 v;
            v.x = word[q][0];
            v.y = word[q][1];
            v.z = word[q][2];
            v.w = word[q][3];
            *reinterpret_cast<u32x4 *>(dst + q * plane) = v;
        }
}

int check_shape(hm_ctx *ctx, const LatentShape &s) {
    HM_REQUIRE(ctx, s.heads > 0 && s.dim > 0 && s.rot_dim >= 0 && s.rot_dims >= 0 && s.rot_dims <= s.rot_dim && s.rot_dims % 2 == 0 && s.vdim > 0 && s.rank > 0,
               "latent attention: bad shape");
    HM_REQUIRE(ctx, s.rank_pad >= s.rank && s.rank_pad % 32 == 0 && s.rot_pad >= s.rot_dim && s.rot_pad % 32 == 0 && (s.pieces == 1 || s.pieces == 3) &&
                        s.window >= 0 && s.ring_rows > 0, "latent attention: bad cache row");
    return HM_OK;
}

}  // namespace

namespace homura {

int latent_step_splits(const LatentShape &, int span) {
    const int per = step_tiles(span) * LS_KEYS;
    return (span + per - 1) / per;
}

int latent_step_prep_launch(hm_ctx *ctx, const LatentStepArgs &a) {
    int rc = check_shape(ctx, a.s);
    if (rc != HM_OK) return rc;
    HM_REQUIRE(ctx, a.q && a.kv && a.kv_norm && a.uk && a.cos_tab && a.sin_tab && a.ring && a.q_latent && a.cursor, "latent_step_prep: NULL pointer");
    const int slices = (a.s.rank_pad + 63) / 64;
    hipLaunchKernelGGL(latent_step_prep_kernel, dim3(a.s.heads * slices + 1), dim3(256), 0, ctx->stream, a, slices);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_step_attn_launch(hm_ctx *ctx, const LatentStepArgs &a) {
    int rc = check_shape(ctx, a.s);
    if (rc != HM_OK) return rc;
    HM_REQUIRE(ctx, a.q_latent && a.ring && a.part_o && a.part_ml && a.cursor && a.span > 0, "latent_step_attn: bad arguments");
    HM_REQUIRE(ctx, a.s.rank_pad <= 1024, "latent_step_attn: latent rank %d above 1024", a.s.rank);
    HM_REQUIRE(ctx, (a.s.window ? std::min(a.s.window, a.span) : a.span) <= a.s.ring_rows, "latent_step_attn: the ring is smaller than what a step sees");
    const dim3 g(latent_step_splits(a.s, a.span), (a.s.heads + 15) / 16);
    const int tiles = step_tiles(a.span);
    const size_t lds = (size_t)a.s.pieces * LS_KEYS * ls_row_bytes(a.s.row_width());
    auto launch = [&](auto kernel, size_t bytes) -> int {
        if (bytes > 48 * 1024) {
            const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
            HM_REQUIRE(ctx, e == hipSuccess, "latent_step_attn: cannot reserve %zu bytes of LDS: %s", bytes, hipGetErrorString(e));
        }
        hipLaunchKernelGGL(kernel, g, dim3(256), bytes, ctx->stream, a, tiles);
        return HM_OK;
    };
    const bool narrow = a.s.rank_pad <= 512;
    if (lds + 12 * 1024 > 160 * 1024) rc = launch(latent_step_attn_wide_kernel, 0);
    else if (a.s.pieces == 1) rc = narrow ? launch(latent_step_attn_lds_kernel<1, 8>, lds) : launch(latent_step_attn_lds_kernel<1, 16>, lds);
    else rc = narrow ? launch(latent_step_attn_lds_kernel<3, 8>, lds) : launch(latent_step_attn_lds_kernel<3, 16>, lds);
    if (rc != HM_OK) return rc;
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_step_fold_launch(hm_ctx *ctx, const LatentStepArgs &a) {
    int rc = check_shape(ctx, a.s);
    if (rc != HM_OK) return rc;
    HM_REQUIRE(ctx, a.part_o && a.part_ml && a.uv && a.out && a.cursor && a.span > 0, "latent_step_fold: bad arguments");
    HM_REQUIRE(ctx, latent_step_splits(a.s, a.span) <= LF_MAX_SPLITS, "latent_step_fold: too many splits");
    hipLaunchKernelGGL(latent_step_fold_kernel, dim3(a.s.heads, (a.s.vdim + LF_ROWS - 1) / LF_ROWS), dim3(LF_THREADS),
                       (size_t)fold_groups(a.s.rank_pad) * a.s.rank_pad * 4, ctx->stream, a, step_tiles(a.span), latent_step_splits(a.s, a.span));
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_rows_launch(hm_ctx *ctx, const LatentRowsArgs &a) {
    int rc = check_shape(ctx, a.s);
    if (rc != HM_OK) return rc;
    HM_REQUIRE(ctx, a.down.p && a.q_norm && a.kv_norm && a.cos_tab && a.sin_tab && a.q_split && a.ring && a.n > 0 && a.n <= a.s.ring_rows && a.past >= 0,
               "latent_rows: bad arguments");
    HM_REQUIRE(ctx, a.q_rank > 0 && a.q_rank_pad >= a.q_rank && a.q_pieces >= 1 && a.q_pieces <= 3 && a.down.ld >= a.q_rank_pad + a.s.rank + a.s.rot_dim &&
                        a.down.parts >= 1 && a.down.parts <= MAX_SUM_PARTS, "latent_rows: bad shape");
    hipLaunchKernelGGL(latent_rows_kernel, dim3(a.n, 2), dim3(256), 0, ctx->stream, a);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_q_rows_launch(hm_ctx *ctx, const LatentShape &s, const RowSource &q, const float *cos_tab, const float *sin_tab,
                         float *d_out, int width, int n, int past) {
    HM_REQUIRE(ctx, q.p && cos_tab && sin_tab && d_out && width >= s.dim + s.rot_dim && q.ld >= s.heads * (s.dim + s.rot_dim) && n > 0 &&
                        q.parts >= 1 && q.parts <= MAX_SUM_PARTS, "latent_q_rows: bad arguments");
    const size_t total = (size_t)n * s.heads * width;
    const bool vec = s.dim % 4 == 0 && s.rot_dim % 4 == 0 && s.rot_dims % 8 == 0 && width % 4 == 0 && q.ld % 4 == 0 && q.stride % 4 == 0 &&
                     ((uintptr_t)q.p % 16) == 0 && ((uintptr_t)d_out % 16) == 0;
    if (vec)
        hipLaunchKernelGGL(latent_q_rows_kernel<4>, dim3((unsigned)((total / 4 + 255) / 256)), dim3(256), 0, ctx->stream, s, q, cos_tab, sin_tab, d_out, width,
                           past, total);
    else
        hipLaunchKernelGGL(latent_q_rows_kernel<1>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, ctx->stream, s, q, cos_tab, sin_tab, d_out, width,
                           past, total);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_gather_launch(hm_ctx *ctx, const LatentShape &s, const uint16_t *ring, uint16_t *d_out, int first, int rows) {
    HM_REQUIRE(ctx, ring && d_out && first >= 0 && rows > 0 && rows <= s.ring_rows && ((uintptr_t)d_out % 16) == 0, "latent_gather: bad arguments");
    const size_t total = (size_t)rows * s.pieces * s.rank_pad / 8;
    hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, ctx->stream, s, ring, d_out, first, total);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

int latent_kv_rows_launch(hm_ctx *ctx, const LatentShape &s, const RowSource &kv, int v_at, const uint16_t *ring, uint16_t *d_k,
                          uint16_t *d_v, int kw, int vw, int cap, int first, int rows) {
    HM_REQUIRE(ctx, kv.p && ring && d_k && d_v && kw % 8 == 0 && vw % 8 == 0 && kw >= s.dim + s.rot_dim && vw >= s.vdim && rows > 0 && rows <= cap &&
                        rows <= s.ring_rows && v_at >= s.heads * s.dim && kv.ld >= v_at + s.heads * s.vdim && kv.parts >= 1 && kv.parts <= MAX_SUM_PARTS,
               "latent_kv_rows: bad arguments");
    const size_t total = (size_t)rows * s.heads * ((kw + vw) / 8);
    const bool vec = s.dim % 8 == 0 && s.rot_dim % 8 == 0 && s.vdim % 8 == 0 && kv.ld % 4 == 0 && kv.stride % 4 == 0 && v_at % 4 == 0 && ((uintptr_t)kv.p % 16) == 0;
    hipLaunchKernelGGL(latent_kv_rows_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, ctx->stream, s, kv, v_at, ring, d_k, d_v, kw, vw, cap,
                       first, vec, total);
    HM_LAUNCH_CHECK(ctx);
    return HM_OK;
}

}  // namespace homura
