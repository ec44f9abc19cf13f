// Query and key norm over whole projections (all heads of a row at once), with
// a query temperature, and the cache write of keys that are the values too.
// The cache holds the keys as projected: the key's norm is one factor per
// token (kscale, applied to the scores by paged_attention.hip) and its weight
// is folded into the query's, so one pool serves scores and values.
// One workgroup per row.
#include "common.h"
#include "residual_api.h"
#include "vec16.h"

namespace dnn {

constexpr int QN_PG = 64;  // keys per page (paged_attention.hip PG)

template <typename T>
__global__ __launch_bounds__(256) void qk_norm_kernel(QkNormArgs a) {
  constexpr int E = Vec16<T>::N;
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x;
  T* row = reinterpret_cast<T*>(a.qkv) + (size_t)m * a.ldq;
  const int cq = a.H * a.DK / E, ck = a.G * a.DK / E;
  const int p = a.pos[m], blk = p / QN_PG;
  int page = blk < a.ldt ? a.table[(size_t)a.slots[m] * a.ldt + blk] : -1;
  if (page >= a.npages) page = -1;
  float sq = 0.f, sk = 0.f, v[E];
  for (int c = tid; c < cq; c += 256) {
    Vec16<T>::get(row + c * E, v);
#pragma unroll
    for (int j = 0; j < E; ++j) sq = fmaf(v[j], v[j], sq);
  }
  for (int c = tid; c < ck; c += 256) {
    const T* src = row + a.H * a.DK + c * E;
    Vec16<T>::get(src, v);
#pragma unroll
    for (int j = 0; j < E; ++j) sk = fmaf(v[j], v[j], sk);
    if (page >= 0) {
      const int g = c * E / a.DK, d = c * E % a.DK;
      *reinterpret_cast<uint4*>(reinterpret_cast<T*>(a.kp) + (((size_t)page * a.G + g) * QN_PG + p % QN_PG) * a.DK + d) =
          *reinterpret_cast<const uint4*>(src);
    }
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sk;
  __syncthreads();
  sq = red[0] + red[1] + red[2] + red[3];
  sk = red[4] + red[5] + red[6] + red[7];
  float f = 1.0f / sqrtf(sq / (float)a.nq + a.eps);
  if (a.t_every > 0) f *= fmaf(a.t_coef, logf((float)((p + 1) / a.t_every) + 1.0f), 1.0f);
  if (tid == 0 && page >= 0) a.kscale[(size_t)page * QN_PG + p % QN_PG] = 1.0f / sqrtf(sk / (float)a.nk + a.eps);
  for (int c = tid; c < cq; c += 256) {
    Vec16<T>::get(row + c * E, v);
#pragma unroll
    for (int j = 0; j < E; j += 4) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(a.qw + c * E + j);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[j + i] *= f * w[i];
    }
    Vec16<T>::put(row + c * E, v);
  }
}

}  // namespace dnn

extern "C" int dnn_qk_norm(const QkNormArgs* a, int f32, hipStream_t st) {
  using namespace dnn;
  const int e = f32 ? 4 : 8;
  if (a->M <= 0 || a->H <= 0 || a->G <= 0 || a->DK % 64 != 0 || a->ldq % e != 0 || a->ldq < (a->H + a->G) * a->DK ||
      a->nq <= 0 || a->nq > a->H * a->DK || a->nk <= 0 || a->nk > a->G * a->DK || a->ldt <= 0 || a->npages <= 0 ||
      a->t_every < 0)
    return -1;
  if (f32) hipLaunchKernelGGL(qk_norm_kernel<float>, dim3(a->M), dim3(256), 0, st, *a);
  else hipLaunchKernelGGL(qk_norm_kernel<bf16_t>, dim3(a->M), dim3(256), 0, st, *a);
  return (int)hipGetLastError();
}
