// Polynomial activation whose powers are normalised over the row (gfx950):
//   out = a N(z) + b N(z^2) + c N(z^3) + e,   N(y) = y / sqrt(mean(y^2) + eps)
// Rows are wider than n by zero padding that stays zero.  The means need the
// sums of z^2, z^4 and z^6 of a row: one workgroup per row.
#include "common.h"
#include "residual_api.h"
#include "vec16.h"

namespace dnn {

// NV pieces of a thread kept in registers (0: the row is read twice)
template <typename T, int NV>
__global__ __launch_bounds__(256) void poly_norm_kernel(PolyNormArgs a) {
  constexpr int E = Vec16<T>::N;
  __shared__ float red[12];
  const int tid = threadIdx.x, np = (a.n + E - 1) / E;  // pieces that hold a value
  T* row = reinterpret_cast<T*>(a.z) + (size_t)blockIdx.x * a.ld;
  float v[NV > 0 ? NV : 1][E], s2 = 0.f, s4 = 0.f, s6 = 0.f;
  auto sums = [&](const float (&x)[E]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < E; ++j) {
      const float q = x[j] * x[j], q2 = q * q;
      s2 += q;
      s4 += q2;
      s6 = fmaf(q2, q, s6);
    }
  };
  if constexpr (NV > 0) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (tid + i * 256 < np) Vec16<T>::get(row + (tid + i * 256) * E, v[i]);
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (tid + i * 256 < np) sums(v[i]);
  } else {
    for (int i = tid; i < np; i += 256) {
      Vec16<T>::get(row + i * E, v[0]);
      sums(v[0]);
    }
  }
  s2 = wave_sum(s2);
  s4 = wave_sum(s4);
  s6 = wave_sum(s6);
  if ((tid & 63) == 0) {
    const int w = tid >> 6;
    red[w] = s2, red[4 + w] = s4, red[8 + w] = s6;
  }
  __syncthreads();
  const float n = (float)a.n;
  const float c1 = a.w[0] / sqrtf((red[0] + red[1] + red[2] + red[3]) / n + a.eps);
  const float c2 = a.w[1] / sqrtf((red[4] + red[5] + red[6] + red[7]) / n + a.eps);
  const float c3 = a.w[2] / sqrtf((red[8] + red[9] + red[10] + red[11]) / n + a.eps);
  const float e = a.w[3];
  auto out = [&](int i, float (&x)[E]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < E; ++j) {
      x[j] = fmaf(x[j], fmaf(x[j], fmaf(x[j], c3, c2), c1), e);
      if (i * E + j >= a.n) x[j] = 0.f;
    }
    Vec16<T>::put(row + i * E, x);
  };
  if constexpr (NV > 0) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (tid + i * 256 < np) out(tid + i * 256, v[i]);
  } else {
    for (int i = tid; i < np; i += 256) {
      Vec16<T>::get(row + i * E, v[0]);
      out(i, v[0]);
    }
  }
}

}  // namespace dnn

extern "C" int dnn_poly_norm(const PolyNormArgs* a, int f32, hipStream_t st) {
  using namespace dnn;
  const int e = f32 ? 4 : 8, np = (a->n + e - 1) / e;
  if (a->M <= 0 || a->n <= 0 || a->ld % e != 0 || a->ld < np * e || ((uintptr_t)a->z & 15) != 0 || a->w == nullptr) return -1;
#define PN(T)                                                                                       \
  {                                                                                                 \
    if (np <= 256) hipLaunchKernelGGL((poly_norm_kernel<T, 1>), dim3(a->M), dim3(256), 0, st, *a);  \
    else if (np <= 512) hipLaunchKernelGGL((poly_norm_kernel<T, 2>), dim3(a->M), dim3(256), 0, st, *a); \
    else if (np <= 2048) hipLaunchKernelGGL((poly_norm_kernel<T, 8>), dim3(a->M), dim3(256), 0, st, *a); \
    else if (np <= 3072) hipLaunchKernelGGL((poly_norm_kernel<T, 12>), dim3(a->M), dim3(256), 0, st, *a); \
    else hipLaunchKernelGGL((poly_norm_kernel<T, 0>), dim3(a->M), dim3(256), 0, st, *a);            \
  }
  if (f32) PN(float)
  else PN(bf16_t)
#undef PN
  return (int)hipGetLastError();
}
