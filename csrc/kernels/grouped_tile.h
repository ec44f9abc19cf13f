// Tiles of rows that are sorted by expert: expert e owns the places
// offs[e] .. offs[e + 1] - 1; a tile never crosses a border.  Without offs every
// expert has `per` rows, at A + e * sa and C + e * sc.
#pragma once
#include "common.h"
#include "glu_clamp.h"

namespace dnn {

constexpr int EXPERTS_MAX = 256;

struct GroupedRows {
  const int* offs;   // [E + 1]
  const int* order;  // source of a place: order[place] / div (nullptr: the place itself)
  int* counts;       // zeroed by the first workgroup (nullptr: not)
  int E, div, arows;
  int per = 0;
  long long sa = 0, sc = 0;
  GluClamp clamp = {};
  // Row r of the expert with places from `first`, among the rows from a_off on.
  __device__ __forceinline__ int row(int first, int r) const {
    if (offs == nullptr) return r;
    const int x = order != nullptr ? order[first + r] / div : first + r;
    return min(max(x, 0), arows - 1);
  }
  __device__ __forceinline__ size_t a_off(int expert) const { return offs == nullptr ? (size_t)(expert * sa) : 0; }
  __device__ __forceinline__ size_t c_off(int expert, int first, int ldc) const {
    return offs == nullptr ? (size_t)(expert * sc) : (size_t)first * ldc;
  }
};

struct GroupTile {
  int expert, first, rows, tm, tn;  // first place and rows of the expert; expert < 0: past the last tile
};

// Tile order of a matrix of ntm x ntn tiles: groups of 8 row tiles, row tile
// fastest, so that tiles running at the same time share panels of both operands.
__device__ __forceinline__ void tile_coords(int logical, int ntm, int ntn, int& tm, int& tn) {
  constexpr int GROUP_M = 8;
  const int per_group = GROUP_M * ntn;
  const int grp = logical / per_group;
  const int first = grp * GROUP_M;
  const int gm = min(ntm - first, GROUP_M);
  const int r = logical - grp * per_group;
  tm = first + r % gm;
  tn = r / gm;
}

// Tile `bid` of tiles of `bm` rows x ntn columns: expert by expert, neighbours
// on one XCD.  Every lane of every wave calls it.
__device__ __forceinline__ GroupTile group_tile(const GroupedRows& g, int bm, int ntn, int bid, int lane) {
  if (g.counts != nullptr && bid == 0)
    for (int e = threadIdx.x; e < g.E; e += blockDim.x) g.counts[e] = 0;
  int first[4], rows[4], nt[4], sum = 0;  // lane l: experts 4 l .. 4 l + 3
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = min(lane * 4 + i, g.E);
    if (g.offs != nullptr) {
      first[i] = g.offs[e];
      rows[i] = g.offs[min(e + 1, g.E)] - first[i];
    } else {
      first[i] = e * g.per;
      rows[i] = e < g.E ? g.per : 0;
    }
    nt[i] = (rows[i] + bm - 1) / bm;
    sum += nt[i];
  }
  int incl = sum;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const int u = __shfl_up(incl, o, 64);
    if (lane >= o) incl += u;
  }
  const int total = __shfl(incl, 63, 64) * ntn;
  GroupTile t{-1, 0, 0, 0, 0};
  if (bid >= total) return t;
  const int logical = xcd_remap(bid, total), mt = logical / ntn;
  const int src = __ffsll((unsigned long long)__ballot(incl > mt)) - 1;  // the lane whose experts hold the tile
  int base = incl - sum, e = lane * 4, f = first[0], r = rows[0], n = nt[0];
#pragma unroll
  for (int i = 0; i < 3; ++i)
    if (mt >= base + nt[i] && e == lane * 4 + i) 
      base += nt[i], e = lane * 4 + i + 1, f = first[i + 1], r = rows[i + 1], n = nt[i + 1];
  t.expert = __builtin_amdgcn_readfirstlane(__shfl(e, src, 64));
  t.first = __builtin_amdgcn_readfirstlane(__shfl(f, src, 64));
  t.rows = __builtin_amdgcn_readfirstlane(__shfl(r, src, 64));
  tile_coords(logical - __builtin_amdgcn_readfirstlane(__shfl(base, src, 64)) * ntn,
              __builtin_amdgcn_readfirstlane(__shfl(n, src, 64)), ntn, t.tm, t.tn);
  return t;
}

// Upper bound of the row tiles of `rows` places over E experts.
inline int group_tiles_max(int rows, int bm, int E) { return rows / bm + (rows < E ? rows : E); }

}  // namespace dnn
