// Rows of a projection as the kernels behind it read them.
#pragma once
#include "row_pieces.h"

namespace homura {

// Rows of a projection, possibly as K slices: element (row, c) = sum over slices of p[slice * stride + row * ld + c]
// (+ bias[c]).
struct RowSource {
    const float *p = nullptr;
    int ld = 0, parts = 1;
    size_t stride = 0;
    const float *bias = nullptr;
};

__device__ __forceinline__ float source_at(const RowSource &s, int row, int c) {
    const float v = sum_parts(s.p, (size_t)row * s.ld + c, s.parts, s.stride);
    return s.bias ? v + s.bias[c] : v;
}

inline bool bad_source(const RowSource &s, int width) { return !s.p || s.ld < width || s.parts < 1 || s.parts > MAX_SUM_PARTS; }

}  // namespace homura
