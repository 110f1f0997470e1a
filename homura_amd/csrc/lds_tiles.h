// Device helpers of kernels that multiply row-major tiles out of LDS on the matrix cores: tile swizzles, direct
// global -> LDS loads, products of operands in bf16 pieces.
#pragma once
#include "hm_common.h"

// K / V tile in LDS: row = key, HD * 2 bytes, 16-byte chunk c of row r at slot c ^ (swizzle of r): conflict-free
// for the operand reads (16 consecutive rows, one chunk)
template <int HD>
__device__ __forceinline__ int k_off(int key, int chunk) {
    if (HD == 128 || HD == 256 || HD == 512) return key * (HD * 2) + ((chunk ^ (key & 15)) << 4);
    if (HD == 192) return key * 384 + ((chunk ^ (key & 7)) << 4);  // 24 chunks: the swizzle stays inside groups of 8
    return key * 128 + ((chunk ^ (key & 7) ^ ((key >> 3) & 7)) << 4);
}

// V tile: the transposing reads of a group of 16 lanes take 32 contiguous bytes (two chunks) from each of four
// neighbouring rows, and a pass of the LDS serves two such groups: the swizzle moves chunk PAIRS, by the row's
// low three bits, so that eight neighbouring rows land on eight different bank groups.
template <int HD>
__device__ __forceinline__ int v_off(int key, int chunk) {
    if (HD == 128 || HD == 256) return key * (HD * 2) + (((((chunk >> 1) ^ (key & 7)) << 1) | (chunk & 1)) << 4);
    return k_off<HD>(key, chunk);
}

typedef short s16x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ void dma16_lds(const uint16_t *src, char *dst) {
    __builtin_amdgcn_global_load_lds((const void __attribute__((address_space(1))) *)src,
                                     (void __attribute__((address_space(3))) *)dst, 16, 0, 0);
}

// max / sum over the four lanes l16 + 16 c of a wavefront, every lane receives it: the row swaps of gfx950
// (odd rows of one operand against even rows of the other, then the upper half against the lower) instead of
// two trips through the LDS crossbar
__device__ __forceinline__ float quad_rows_max(float x) {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    const float m = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
    const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(m), __float_as_uint(m), false, false);
    return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float quad_rows_sum(float x) {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    const float m = __uint_as_float(a[0]) + __uint_as_float(a[1]);
    const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(m), __float_as_uint(m), false, false);
    return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// products of NA and NB pieces, smallest first: f(piece of A, piece of B)
template <int NA, int NB, class F>
__device__ __forceinline__ void piece_products(F f) {
#pragma unroll
    for (int order = NA + NB - 2; order >= 0; order--)
#pragma unroll
        for (int pa = NA - 1; pa >= 0; pa--) {
            const int pb = order - pa;
            if (pb < 0 || pb >= NB || (NA > 1 && NB > 1 && order > 2)) continue;
            f(pa, pb);
        }
}
