// Mixture of experts (gfx950): router selection, placement of rows by expert,
// and products of the placed rows with their experts' weights.
//
//   route        softmax or sigmoid of the router logits, the best experts
//                within the best groups, their weights, and a place for every
//                (row, choice) so that an expert's rows are neighbours; one
//                workgroup for up to 64 rows, two launches beyond
//   grouped GEMM many rows per expert: the 256x256 tile kernel (gemm_tile.h)
//                with gathered rows; few: weights streamed in fragment order,
//                four waves splitting K over 16 to 64 rows
//
// A place's result depends on its row and expert only, so the order of places
// within an expert (it comes from atomics) leaves no trace in the output.
#include "common.h"
#include "gemm_tile.h"
#include "mixer_api.h"

namespace dnn {

// One row by half a wave: lane l of 32 holds the logits of experts l, l + 32,
// ...; both halves call it together, a half past the rows with live = false.
// f(t, expert) for every choice.  NR: experts a lane holds at most.
template <int NR, typename F>
__device__ __forceinline__ void route_row(const RouteArgs& a, int m, bool live, int l, int half, F f) {
  const int nr = (a.E + 31) / 32;  // registers that hold experts
  float s[NR], w[NR];  // choice scores, scores
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int e = i * 32 + l;
    s[i] = live && i < nr && e < a.E ? a.logits[(size_t)m * a.ldl + e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  if (a.sigmoid) {
#pragma unroll
    for (int i = 0; i < NR; ++i) w[i] = 1.0f / (1.0f + expf(-s[i]));
  } else {
    mx = group_max<32>(mx);
    if (!live) mx = 0.f;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      s[i] = expf(s[i] - mx);  // 0 past the experts
      sum += s[i];
    }
    sum = live ? group_sum<32>(sum) : 1.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) w[i] = s[i] / sum;
  }
  const int per = a.E / a.groups;
  int grp[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    s[i] = a.correction != nullptr && i < nr && i * 32 + l < a.E ? w[i] + a.correction[i * 32 + l] : w[i];
    grp[i] = i < nr ? (i * 32 + l) / per : 0;
  }
  // the best expert among ok: the largest score, the lower index first
  auto best = [&](unsigned ok, float& v) __attribute__((always_inline)) {
    float m1 = -INFINITY;
#pragma unroll
    for (int i = 0; i < NR; ++i)
      if (i < nr && (ok >> i & 1) != 0 && i * 32 + l < a.E) m1 = fmaxf(m1, s[i]);
    v = m1 = group_max<32>(m1);
    int e = a.E - 1;
#pragma unroll
    for (int i = NR - 1; i >= 0; --i) {
      if (i >= nr) continue;
      const unsigned at = (unsigned)(__ballot((ok >> i & 1) != 0 && i * 32 + l < a.E && s[i] == m1) >> (32 * half));
      if (at != 0) e = i * 32 + __ffs(at) - 1;
    }
    return e;
  };
  unsigned open = ~0u, in = a.keep >= a.groups ? ~0u : 0u;
  if (a.keep < a.groups && a.group_top > 1 && per > 1) {
    // every expert takes its group's score, the sum of its two best, and groups
    // are chosen by it: the lower group first where two are equal
    float gs[NR];
    for (int g = 0; g < a.groups; ++g) {
      unsigned ok = 0u;
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (i < nr && grp[i] == g) ok |= 1u << i;
      float v1, v2;
      const int e = best(ok, v1);
      if ((e & 31) == l) ok &= ~(1u << (e >> 5));
      best(ok, v2);
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (grp[i] == g) gs[i] = v1 + v2;
    }
    for (int k = 0; k < a.keep; ++k) {
      float m1 = -INFINITY;
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (i < nr && (open >> i & 1) != 0 && i * 32 + l < a.E) m1 = fmaxf(m1, gs[i]);
      m1 = group_max<32>(m1);
      int g = a.groups;
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (i < nr && (open >> i & 1) != 0 && i * 32 + l < a.E && gs[i] == m1) g = min(g, grp[i]);
      g = (int)-group_max<32>(-(float)g);
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (grp[i] == g) open &= ~(1u << i), in |= 1u << i;
    }
  } else {
    // the best groups: the group of the best expert outside those already taken
    for (int k = 0; k < a.keep && a.keep < a.groups; ++k) {
      float v;
      const int g = best(open, v) / per;
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (grp[i] == g) open &= ~(1u << i), in |= 1u << i;
    }
  }
  float total = 0.f;
  float mine[2] = {0.f, 0.f};
  int me[2] = {0, 0};
  for (int t = 0; t < a.top; ++t) {
    float v;
    const int e = best(in, v);
    if (a.correction != nullptr) {
      v = 0.f;
#pragma unroll
      for (int i = 0; i < NR; ++i)
        if (i == e >> 5) v = w[i];
      v = __shfl(v, half * 32 + (e & 31), 64);
    }
    total += v;
    if ((t & 31) == l) {
      if (t < 32) mine[0] = v, me[0] = e;
      else mine[1] = v, me[1] = e;
    }
    if ((e & 31) == l) in &= ~(1u << (e >> 5));
    if (live) f(t, e);
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (live && i * 32 + l < a.top) {
      a.idx[(size_t)m * a.top + i * 32 + l] = me[i];
      a.w[(size_t)m * a.top + i * 32 + l] = a.normalise ? mine[i] / (total + 1e-20f) : mine[i];
    }
}

constexpr int RT_ROWS = 16;  // rows of a workgroup of 4 waves

template <int NR>
__global__ __launch_bounds__(256) void route_kernel(RouteArgs a) {
  __shared__ int hist[EXPERTS_MAX], base[EXPERTS_MAX];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, m0 = blockIdx.x * RT_ROWS;
  hist[tid] = 0;
  __syncthreads();
  for (int r = wave * 2; r < RT_ROWS; r += 8) {
    const int half = lane >> 5, l = lane & 31, m = m0 + r + half;
    route_row<NR>(a, m, m < a.M, l, half, [&](int t, int e) __attribute__((always_inline)) {
      if (l == 0) a.rank[(size_t)m * a.top + t] = atomicAdd(&hist[e], 1);
    });
  }
  __syncthreads();
  if (tid < a.E && hist[tid] > 0) base[tid] = atomicAdd(&a.counts[tid], hist[tid]);
  __syncthreads();  // also makes this workgroup's idx / rank stores visible to it
  const int n = min(RT_ROWS, a.M - m0) * a.top;
  for (int i = tid; i < n; i += 256) {
    const size_t x = (size_t)m0 * a.top + i;
    a.rank[x] += base[min(max(a.idx[x], 0), a.E - 1)];
  }
}

// Exclusive prefix sums of counts[E] by the first wave into offs[E + 1].
__device__ __forceinline__ void expert_offsets(const int* counts, int E, int* offs, int tid) {
  if (tid < 64) {
    int c[4], sum = 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      c[i] = tid * 4 + i < E ? counts[tid * 4 + i] : 0;
      sum += c[i];
    }
    int incl = sum;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int u = __shfl_up(incl, o, 64);
      if (tid >= o) incl += u;
    }
    int b = incl - sum;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (tid * 4 + i <= E) offs[tid * 4 + i] = b;
      b += c[i];
    }
    if (tid == 63 && E == 256) offs[256] = b;
  }
}

__global__ __launch_bounds__(256) void place_kernel(RouteArgs a) {
  __shared__ int offs[EXPERTS_MAX + 1];
  const int tid = threadIdx.x;
  expert_offsets(a.counts, a.E, offs, tid);
  __syncthreads();
  if (blockIdx.x == 0)
    for (int e = tid; e <= a.E; e += 256) a.offs[e] = offs[e];
  const int i = blockIdx.x * 256 + tid;
  if (i >= a.M * a.top) return;
  const int p = offs[min(max(a.idx[i], 0), a.E - 1)] + a.rank[i];
  a.order[p] = i;
  a.place[i] = p;
}

constexpr int RT_SMALL = 64;  // rows of the one-workgroup launch

template <int NR>
__global__ __launch_bounds__(1024) void route_small_kernel(RouteArgs a) {
  __shared__ int hist[EXPERTS_MAX], offs[EXPERTS_MAX + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  if (tid < EXPERTS_MAX) hist[tid] = 0;
  __syncthreads();
  for (int m0 = wave * 2; m0 < a.M; m0 += 32) {
    const int half = lane >> 5, l = lane & 31, m = m0 + half;
    route_row<NR>(a, m, m < a.M, l, half, [&](int t, int e) __attribute__((always_inline)) {
      if (l == 0) a.rank[(size_t)m * a.top + t] = atomicAdd(&hist[e], 1);
    });
  }
  __syncthreads();
  expert_offsets(hist, a.E, offs, tid);
  __syncthreads();
  for (int e = tid; e <= a.E; e += 1024) a.offs[e] = offs[e];
  for (int i = tid; i < a.M * a.top; i += 1024) {
    const int p = offs[min(max(a.idx[i], 0), a.E - 1)] + a.rank[i];
    a.order[p] = i;
    a.place[i] = p;
  }
}

// ---------------------------------------------------------------- few rows per expert
// grid (row tiles x column groups); a workgroup's four waves split K over
// 16 MT rows x 16 NT columns and reduce through LDS.
template <int ACT, int MT, int NT>
__global__ __launch_bounds__(256) void grouped_skinny_kernel(const bf16_t* __restrict__ A, int lda,
                                                             const uint8_t* __restrict__ wsh, bf16_t* __restrict__ C,
                                                             int ldc, int N, int K, GroupedRows g) {
  __shared__ f32x4 red[4][MT * NT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int nch = K / 32, ntn = N / (16 * NT);
  const GroupTile t = group_tile(g, 16 * MT, ntn, blockIdx.x, lane);
  if (t.expert < 0) return;
  const int r0 = t.tm * 16 * MT;
  const bf16_t* ap[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
    ap[i] = A + g.a_off(t.expert) + (size_t)g.row(t.first, min(r0 + i * 16 + (lane & 15), t.rows - 1)) * lda + (lane >> 4) * 8;
  const uint8_t* wp = wsh + ((size_t)t.expert * (N / 16) + (size_t)t.tn * NT) * nch * 1024 + lane * 16;
  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = MT * NT >= 4 ? 4 : 8;
  for (int c0 = wave; c0 < nch; c0 += 4 * U) {
    bf16x8 w[U][NT], x[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + u * 4, nch - 1);
#pragma unroll
      for (int j = 0; j < NT; ++j) w[u][j] = *reinterpret_cast<const bf16x8*>(wp + ((size_t)j * nch + c) * 1024);
#pragma unroll
      for (int i = 0; i < MT; ++i) x[u][i] = *reinterpret_cast<const bf16x8*>(ap[i] + c * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u * 4 < nch) {
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
          for (int j = 0; j < NT; ++j)
            acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][j], x[u][i], acc[i][j], 0, 0, 0);
      }
  }
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) red[wave][i * NT + j][lane] = acc[i][j];
  __syncthreads();
#pragma unroll
  for (int x = 0; x < MT * NT; ++x) {
    if ((x & 3) != wave) continue;
    f32x4 z = red[0][x][lane];
#pragma unroll
    for (int w = 1; w < 4; ++w) z += red[w][x][lane];
    const int i = x / NT, j = x % NT, r = r0 + i * 16 + (lane & 15), nb = (t.tn * NT + j) * 16;
    bf16_t* crow = C + g.c_off(t.expert, t.first, ldc) + (size_t)min(r, t.rows - 1) * ldc;
    if constexpr (is_glu(ACT)) {  // columns 0..7 of the tile are gates, 8..15 their partners
      f32x4 u;
#pragma unroll
      for (int q = 0; q < 4; ++q) u[q] = __shfl_xor(z[q], 32, 64);
      auto join = [&](float gate, float up) __attribute__((always_inline)) {
        if constexpr (ACT == ACT_CLAMP_MUL) return glu_clamped(gate, up, g.clamp);
        else return glu_gate<ACT>(gate) * up;
      };
      if (lane < 32 && r < t.rows)
        *reinterpret_cast<uint2*>(crow + nb / 2 + (lane >> 4) * 4) =
            make_uint2(pack2bf(join(z[0], u[0]), join(z[1], u[1])), pack2bf(join(z[2], u[2]), join(z[3], u[3])));
    } else {
      if (r < t.rows)
        *reinterpret_cast<uint2*>(crow + nb + (lane >> 4) * 4) = make_uint2(pack2bf(z[0], z[1]), pack2bf(z[2], z[3]));
    }
  }
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_route(const RouteArgs* a, hipStream_t st) {
  if (a->M <= 0 || a->E <= 0 || a->E > EXPERTS_MAX || a->ldl < a->E || a->groups <= 0 || a->E % a->groups != 0 ||
      a->keep < 1 || a->keep > a->groups || a->top < 1 || a->top > 64 || a->top > a->E / a->groups * a->keep || a->group_top < 1 || a->group_top > 2 ||
      a->M > (1 << 30) / a->top)
    return -1;
#define ROUTE(N)                                                                                                       \
  {                                                                                                                    \
    if (a->M <= RT_SMALL) hipLaunchKernelGGL(route_small_kernel<N>, dim3(1), dim3(1024), 0, st, *a);                   \
    else hipLaunchKernelGGL(route_kernel<N>, dim3((a->M + RT_ROWS - 1) / RT_ROWS), dim3(256), 0, st, *a);              \
  }
  if (a->E <= 32) ROUTE(1)
  else if (a->E <= 64) ROUTE(2)
  else ROUTE(EXPERTS_MAX / 32)
#undef ROUTE
  if (a->M > RT_SMALL) {
    hipLaunchKernelGGL(place_kernel, dim3((a->M * a->top + 255) / 256), dim3(256), 0, st, *a);
  }
  return (int)hipGetLastError();
}

template <int ACT>
static int grouped_launch(const GroupedArgs& a, const GroupedRows& g, hipStream_t st) {
  const bf16_t* A = (const bf16_t*)a.A;
  bf16_t* C = (bf16_t*)a.C;
  const int avg = (a.rows + a.E - 1) / a.E;
#define SKINNY(MT, NT)                                                                                              \
  {                                                                                                                 \
    const long n = (long)group_tiles_max(a.rows, 16 * MT, a.E) * (a.N / (16 * NT));                                 \
    if (n > 0x7fffffff) return -1;                                                                                  \
    hipLaunchKernelGGL((grouped_skinny_kernel<ACT, MT, NT>), dim3((unsigned)n), dim3(256), 0, st, A, a.lda,         \
                       (const uint8_t*)a.Wsh, C, a.ldc, a.N, a.K, g);                                               \
    return (int)hipGetLastError();                                                                                  \
  }
  const bool even = a.offs == nullptr;  // every expert has avg rows
  if (avg <= (even ? 16 : 12)) SKINNY(1, 1)
  if (avg <= (even ? 32 : 28)) SKINNY(2, 2)
  if (avg <= 64) SKINNY(4, 2)
#undef SKINNY
  const long n = (long)group_tiles_max(a.rows, BG_M, a.E) * ((a.N + BG_N - 1) / BG_N);
  if (n > 0x7fffffff) return -1;
  hipLaunchKernelGGL((gemm_bf16_256_kernel<ACT, false, false, 2, true>), dim3((unsigned)n), dim3(512), 0, st, A, a.lda,
                     (const bf16_t*)a.Wsh, a.K, (void*)C, a.ldc, nullptr, nullptr, 0, a.rows, a.N, a.K, 0, nullptr, nullptr,
                     QkvScatter{}, g);
  return (int)hipGetLastError();
}

extern "C" int dnn_grouped_gemm(const GroupedArgs* a, hipStream_t st) {
  const int nc = is_glu(a->act) ? a->N / 2 : a->N;
  if (a->rows <= 0 || a->E <= 0 || a->E > EXPERTS_MAX || a->N <= 0 || a->N % 32 != 0 || a->K <= 0 || a->K % 64 != 0 ||
      a->lda % 8 != 0 || a->lda < a->K || a->ldc % 8 != 0 || a->ldc < nc || a->div < 1 || a->arows < 1 || a->Wsh == nullptr ||
      (a->offs == nullptr && (a->rows % a->E != 0 || a->sa < 0 || a->sa % 8 != 0 || a->sc < 0 || a->sc % 8 != 0)))
    return -1;
  if ((((uintptr_t)a->A | (uintptr_t)a->Wsh | (uintptr_t)a->C) & 15) != 0) return -1;
  const GroupedRows g{a->offs, a->order, a->counts, a->E, a->div, a->arows, a->rows / a->E, a->sa, a->sc, a->clamp};
  if (a->act == ACT_SILU_MUL) return grouped_launch<ACT_SILU_MUL>(*a, g, st);
  if (a->act == ACT_CLAMP_MUL) return grouped_launch<ACT_CLAMP_MUL>(*a, g, st);
  if (a->act == ACT_NONE) return grouped_launch<ACT_NONE>(*a, g, st);
  return -1;
}
