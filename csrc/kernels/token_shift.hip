// What a layer takes from the token before (gfx950): rows of a step whose
// sequences are cut anywhere, so the first row of a portion reads the last token
// of the portion before it from a state by slot.  A portion that begins at
// position 0 has no token before it.
//
//   pair_rows    row of a (previous token, token) table for every row
//   token_shift  several mixes of a row and the row before it,
//                out_i = x + (x_prev - x) * mu_i
//
// The thread that reads a sequence's state also writes what the next portion
// reads, so neither needs a second launch.
#include "common.h"
#include "mixer_api.h"
#include "vec16.h"

namespace dnn {

__global__ __launch_bounds__(256) void pair_rows_kernel(PairArgs a) {
  const int m = blockIdx.x * 256 + threadIdx.x;
  if (m >= a.M) return;
  int prev = -1;
  if (a.start[m] != m) {
    prev = a.ids[m - 1];
  } else {
    int* st = a.prev + min(max(a.slots[m], 0), a.nslots - 1);
    if (a.pos[m] > 0) prev = *st;
    *st = a.ids[min(max(a.last[m], m), a.M - 1)];
  }
  a.rows[m] = prev < 0 ? (int)a.buckets : (int)((prev * a.mul_prev + a.ids[m] * a.mul_cur) % a.buckets);
}

constexpr int SHIFT_MAX = 8;  // mixes of a launch

// grid ceil(M / R) * ceil(NP / 1024); a thread takes 4 channels of R rows.
template <typename T, int R, int N>
__global__ __launch_bounds__(256) void token_shift_kernel(ShiftArgs a) {
  const int gx = (a.NP + 1023) / 1024, m0 = (int)(blockIdx.x / gx) * R, c = ((int)(blockIdx.x % gx) * 256 + threadIdx.x) * 4;
  if (c >= a.NP) return;
  f32x4 mu[N], x[R], prev = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < N; ++i) mu[i] = *reinterpret_cast<const f32x4*>(a.mu + (size_t)i * a.NP + c);
#pragma unroll
  for (int r = 0; r < R; ++r) x[r] = *reinterpret_cast<const f32x4*>(a.x + (size_t)min(m0 + r, a.M - 1) * a.ldx + c);
  if (a.start[m0] != m0) prev = *reinterpret_cast<const f32x4*>(a.x + (size_t)(m0 - 1) * a.ldx + c);
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int m = m0 + r;
    if (m >= a.M) break;
    if (a.start[m] == m) {
      float* st = a.state + (size_t)min(max(a.slots[m], 0), a.nslots - 1) * a.NP + c;
      prev = f32x4{0.f, 0.f, 0.f, 0.f};
      if (a.pos[m] > 0) prev = *reinterpret_cast<const f32x4*>(st);
      *reinterpret_cast<f32x4*>(st) =
          *reinterpret_cast<const f32x4*>(a.x + (size_t)min(max(a.last[m], m), a.M - 1) * a.ldx + c);
    }
#pragma unroll
    for (int i = 0; i < N; ++i) {
      float v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = fmaf(prev[j] - x[r][j], mu[i][j], x[r][j]);
      T* o = reinterpret_cast<T*>(a.out) + (size_t)i * a.ostride + (size_t)m * a.ldo + c;
      if constexpr (sizeof(T) == 4) *reinterpret_cast<f32x4*>(o) = f32x4{v[0], v[1], v[2], v[3]};
      else *reinterpret_cast<uint2*>(o) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
    }
    prev = x[r];
  }
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_pair_rows(const PairArgs* a, hipStream_t st) {
  if (a->M <= 0 || a->nslots < 1 || a->buckets < 1 || a->buckets > 0x7ffffff0LL || a->mul_prev < 0 || a->mul_cur < 0 ||
      a->mul_prev > 0x3fffffffLL || a->mul_cur > 0x3fffffffLL)
    return -1;
  hipLaunchKernelGGL(pair_rows_kernel, dim3((a->M + 255) / 256), dim3(256), 0, st, *a);
  return (int)hipGetLastError();
}

extern "C" int dnn_token_shift(const ShiftArgs* a, int f32, hipStream_t st) {
  if (a->M <= 0 || a->NP <= 0 || a->NP % 4 != 0 || a->ldx % 4 != 0 || a->ldo % 4 != 0 || a->ldx < a->NP || a->ldo < a->NP ||
      a->ostride % 4 != 0 || a->n < 1 || a->n > SHIFT_MAX || a->nslots < 1)
    return -1;
  const int R = a->M > 256 ? 8 : 1;
  const long n = (long)((a->M + R - 1) / R) * ((a->NP + 1023) / 1024);
  if (n > 0x7fffffff) return -1;
#define TS(N)                                                                                                             \
  case N:                                                                                                                 \
    if (f32 && R > 1) hipLaunchKernelGGL((token_shift_kernel<float, 8, N>), dim3((unsigned)n), dim3(256), 0, st, *a);     \
    else if (f32) hipLaunchKernelGGL((token_shift_kernel<float, 1, N>), dim3((unsigned)n), dim3(256), 0, st, *a);         \
    else if (R > 1) hipLaunchKernelGGL((token_shift_kernel<bf16_t, 8, N>), dim3((unsigned)n), dim3(256), 0, st, *a);      \
    else hipLaunchKernelGGL((token_shift_kernel<bf16_t, 1, N>), dim3((unsigned)n), dim3(256), 0, st, *a);                 \
    break;
  switch (a->n) {
    TS(1) TS(2) TS(3) TS(4) TS(5) TS(6) TS(7) TS(8)
  }
#undef TS
  return (int)hipGetLastError();
}
