// Row tiles of grouped matrix products: every group multiplies the rows its list names, the tiles of all groups share a grid.
#pragma once
#include "hm_common.h"

namespace homura {

struct GroupLists {
    const int *list = nullptr, *count = nullptr;  // [groups][list_cap] entries, how many each group has
    int groups = 0, list_cap = 0;
    int a_rows = 1;                               // entry e reads row e % a_rows of A
    int m_tiles = 0;                              // row tiles in the grid, at least what any distribution of the entries needs
};

struct GroupTile {
    int group = -1;  // -1: nothing for this workgroup
    int rows = 0;    // entries of the group
    int m0 = 0, n0 = 0;
};

// The tile of workgroup `id` of grid, n_tiles column tiles: the tiles are ordered group by group, within a group column by
// column, so that neighbours share a matrix panel and a group's rows stay close; every die gets a stretch of that order
// (workgroups are dealt to the eight dies round-robin). Groups are looked through 64 at a time, by every wavefront for
// itself; the result is uniform. The grid holds group_grid() workgroups.
__device__ __forceinline__ GroupTile group_tile(const GroupLists &g, int id, int n_tiles, int tile_rows, int tile_cols) {
    const int lane = threadIdx.x & 63;
    GroupTile r;
    auto counts = [&](int g0, int &cnt, int &own, int &upto) {
        cnt = g0 + lane < g.groups ? g.count[g0 + lane] : 0;
        own = upto = (cnt + tile_rows - 1) / tile_rows;
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const int o = __shfl_up(upto, d);
            if (lane >= d) upto += o;
        }
    };
    int cnt, own, upto, total = 0;
    for (int g0 = 0; g0 < g.groups; g0 += 64) {
        counts(g0, cnt, own, upto);
        total += __builtin_amdgcn_readlane(upto, 63);
    }
    const int live = total * n_tiles, per = (live + 7) / 8, at = (id & 7) * per + (id >> 3);
    if ((id >> 3) >= per || at >= live) return r;
    int row_tile = at / n_tiles, before = 0;
    for (int g0 = 0; g0 < g.groups; g0 += 64) {
        if (g.groups > 64) counts(g0, cnt, own, upto);
        const uint64_t beyond = __ballot(before + upto > row_tile);
        if (beyond) {
            const int l = __ffsll((unsigned long long)beyond) - 1, mine = __builtin_amdgcn_readlane(own, l);
            const int in = at - (before + __builtin_amdgcn_readlane(upto, l) - mine) * n_tiles;  // place among the group's tiles
            r.group = g0 + l;
            r.rows = __builtin_amdgcn_readlane(cnt, l);
            r.m0 = in % mine * tile_rows;
            r.n0 = in / mine * tile_cols;
            return r;
        }
        before += __builtin_amdgcn_readlane(upto, 63);
    }
    return r;
}

// workgroups for m_tiles row tiles and n_tiles column tiles, a whole number a die
inline long long group_grid(int m_tiles, int n_tiles) { return ((long long)m_tiles * n_tiles + 7) / 8 * 8; }

}  // namespace homura
