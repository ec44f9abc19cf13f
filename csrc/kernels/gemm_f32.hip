// fp32 GEMM on the fp32 MFMA (no reduced-precision mode): C = A W^T + bias,
// A [M, lda], W [N, ldw] row-major, K a multiple of 16.  The exact mode of the
// decoder layers; 64 x 64 tiles, 4 waves of one 32 x 32 tile each, K in steps
// of 16 through LDS (k-major, so a fragment read is one row of 32 lanes).
#include "common.h"
#include "grouped_tile.h"
#include "mixer_api.h"
#include "residual_api.h"

namespace dnn {

constexpr int F32_T = 64, F32_K = 16, F32_LD = F32_T + 4;

// GRP: rows sorted by expert (grouped_tile.h), gathered; W [E][N][K]; C rows are places.
template <bool GRP>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const float* __restrict__ A, int lda, const float* __restrict__ W,
                                                       int ldw, float* __restrict__ C, int ldc,
                                                       const float* __restrict__ bias, int M, int N, int K,
                                                       GroupedRows grp) {
  __shared__ __attribute__((aligned(16))) float as[F32_K * F32_LD], ws[F32_K * F32_LD];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int n0 = blockIdx.x * F32_T, m0 = blockIdx.y * F32_T;
  const int row = tid >> 2, kc = (tid & 3) * 4;  // the 4 operand values this thread stages
  int arow = min(m0 + row, M - 1);
  if constexpr (GRP) {
    const GroupTile t = group_tile(grp, F32_T, (N + F32_T - 1) / F32_T, blockIdx.x, lane);
    if (t.expert < 0) return;
    n0 = t.tn * F32_T, m0 = t.tm * F32_T, M = t.rows;
    W += (size_t)t.expert * N * ldw;
    A += grp.a_off(t.expert);
    C += grp.c_off(t.expert, t.first, ldc);
    arow = grp.row(t.first, min(m0 + row, M - 1));
  }
  const float* ap = A + (size_t)arow * lda + kc;
  const float* wp = W + (size_t)min(n0 + row, N - 1) * ldw + kc;
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
  f32x16 acc = f32x16{};
  f32x4 ar = *reinterpret_cast<const f32x4*>(ap), wr = *reinterpret_cast<const f32x4*>(wp);
  for (int k = 0; k < K; k += F32_K) {
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      as[(kc + j) * F32_LD + row] = ar[j];
      ws[(kc + j) * F32_LD + row] = wr[j];
    }
    __syncthreads();
    if (k + F32_K < K) {
      ar = *reinterpret_cast<const f32x4*>(ap + k + F32_K);
      wr = *reinterpret_cast<const f32x4*>(wp + k + F32_K);
    }
#pragma unroll
    for (int s = 0; s < F32_K; s += 2) {
      const int kk = (s + (lane >> 5)) * F32_LD + (lane & 31);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(as[kk + wm], ws[kk + wn], acc, 0, 0, 0);
    }
  }
  const int n = n0 + wn + (lane & 31);
  if (n >= N) return;
  const float b = bias != nullptr ? bias[n] : 0.f;
#pragma unroll
  for (int g = 0; g < 16; ++g) {
    const int m = m0 + wm + (g & 3) + 8 * (g >> 2) + 4 * (lane >> 5);
    if (m < M) C[(size_t)m * ldc + n] = acc[g] + b;
  }
}

}  // namespace dnn

extern "C" int dnn_gemm_f32(const float* A, int lda, const float* W, int ldw, float* C, int ldc, const float* bias,
                            int M, int N, int K, hipStream_t st) {
  using namespace dnn;
  if (M <= 0 || N <= 0 || K <= 0 || K % F32_K != 0 || (lda | ldw) % 4 != 0 || lda < K || ldw < K || ldc < N) return -1;
  const dim3 grid((N + F32_T - 1) / F32_T, (M + F32_T - 1) / F32_T);
  if (grid.y > 65535) return -1;
  hipLaunchKernelGGL(gemm_f32_kernel<false>, grid, dim3(256), 0, st, A, lda, W, ldw, C, ldc, bias, M, N, K, GroupedRows{});
  return (int)hipGetLastError();
}

// Without an activation: C has all N columns (glu_f32 follows).
extern "C" int dnn_grouped_gemm_f32(const GroupedArgs* a, hipStream_t st) {
  using namespace dnn;
  if (a->rows <= 0 || a->E <= 0 || a->E > EXPERTS_MAX || a->N <= 0 || a->K <= 0 || a->K % F32_K != 0 || a->lda % 4 != 0 ||
      a->lda < a->K || a->ldc < a->N || a->div < 1 || a->arows < 1 || a->W == nullptr ||
      (a->offs == nullptr && (a->rows % a->E != 0 || a->sa < 0 || a->sa % 4 != 0 || a->sc < 0)))
    return -1;
  const long n = (long)group_tiles_max(a->rows, F32_T, a->E) * ((a->N + F32_T - 1) / F32_T);
  if (n > 0x7fffffff) return -1;
  const GroupedRows g{a->offs, a->order, a->counts, a->E, a->div, a->arows, a->rows / a->E, a->sa, a->sc, a->clamp};
  hipLaunchKernelGGL(gemm_f32_kernel<true>, dim3((unsigned)n), dim3(256), 0, st, (const float*)a->A, a->lda,
                     (const float*)a->W, a->K, (float*)a->C, a->ldc, (const float*)nullptr, a->rows, a->N, a->K, g);
  return (int)hipGetLastError();
}
