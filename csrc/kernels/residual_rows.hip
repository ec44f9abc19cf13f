// Row kernels of decoder layers with an fp32 residual stream.
//
// rows_update: one pass over a row that joins a sublayer's output into the
// residual and prepares the next projection's input,
//   x' = [x +] mult * y * [rsqrt(mean(y^2) + eps) * yw]      (fp32)
//   copy = T(x')              the residual as a GEMM operand
//   h    = T(x' * rsqrt(mean(x'^2) + eps) * nw)               RMS norm
// each part optional.  y rows may be gathered (the embedding: y = table,
// yidx = tokens, mult = the embedding scale), x rows too (the head's rows).
// Rows are NP wide (padded, zeros past N); means are over the true width N.
// bf16 y / T in serving, fp32 in the exact mode.
#include "common.h"
#include "residual_api.h"

namespace dnn {

__device__ __forceinline__ f32x4 ld4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 ld4(const bf16_t* p) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{bf2f_s(v[0]), bf2f_s(v[1]), bf2f_s(v[2]), bf2f_s(v[3])};
}
__device__ __forceinline__ void st4(float* p, const f32x4& v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void st4(bf16_t* p, const f32x4& v) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
}

// Sum over the TPR threads of a row (TPR = 64: the wave; 256: the workgroup).
template <int TPR>
__device__ __forceinline__ float row_sum(float v, float* red) {
  v = wave_sum(v);
  if constexpr (TPR == 64) return v;
  const int wave = threadIdx.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[wave] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

template <typename YT, typename OT, int TPR, int NC>
__global__ __launch_bounds__(256) void rows_update_kernel(RowsArgs a) {
  __shared__ float red[4];
  const int t = threadIdx.x % TPR;
  const int m = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (m >= a.M) return;  // TPR 256: uniform over the workgroup
  const int xr = a.xidx != nullptr ? min(max(a.xidx[m], 0), a.xrows - 1) : m;
  // few values per thread: the norm weights are issued with the row (one memory round trip)
  constexpr bool PF = NC <= 4;
  f32x4 x[NC], y[NC], yw[PF ? NC : 1], nw[PF ? NC : 1];
  const float* xp = a.x_in != nullptr ? a.x_in + (size_t)xr * a.ldx : nullptr;
  const YT* yp = nullptr;
  if (a.y != nullptr) {
    const int yr = a.yidx != nullptr ? min(max(a.yidx[m], 0), a.yrows - 1) : m;
    yp = reinterpret_cast<const YT*>(a.y) + (size_t)yr * a.ldy;
  }
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (t + TPR * i) * 4;
    x[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    y[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < a.NP) {
      if (xp != nullptr) x[i] = ld4(xp + c);
      if (yp != nullptr) y[i] = ld4(yp + c);
      if constexpr (PF) {
        if (a.y_w != nullptr) yw[i] = ld4(a.y_w + c);
        if (a.n_w != nullptr) nw[i] = ld4(a.n_w + c);
      }
    }
  }
  if (a.y_w != nullptr) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) s = fmaf(y[i][j], y[i][j], s);
    const float r = 1.0f / sqrtf(row_sum<TPR>(s, red) / (float)a.N + a.eps);
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (t + TPR * i) * 4;
      if (c < a.NP) y[i] = y[i] * r * (PF ? yw[PF ? i : 0] : ld4(a.y_w + c));
    }
  }
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (t + TPR * i) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      x[i][j] = fmaf(a.mult, y[i][j], x[i][j]);
      s = fmaf(x[i][j], x[i][j], s);
    }
    if (c < a.NP) {
      if (a.x_out != nullptr) st4(a.x_out + (size_t)m * a.ldx + c, x[i]);
      if (a.copy != nullptr) st4(reinterpret_cast<OT*>(a.copy) + (size_t)m * a.ldcopy + c, x[i]);
    }
  }
  if (a.n_w == nullptr) return;
  const float r = 1.0f / sqrtf(row_sum<TPR>(s, red) / (float)a.N + a.eps);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (t + TPR * i) * 4;
    if (c < a.NP) st4(reinterpret_cast<OT*>(a.h) + (size_t)m * a.ldh + c, x[i] * r * (PF ? nw[PF ? i : 0] : ld4(a.n_w + c)));
  }
}

template <typename YT, typename OT>
static int rows_launch(const RowsArgs& a, hipStream_t st) {
#define ROWS(TPR, NC)                                                                                             \
  {                                                                                                               \
    hipLaunchKernelGGL((rows_update_kernel<YT, OT, TPR, NC>), dim3((a.M + 256 / TPR - 1) / (256 / TPR)), dim3(256), \
                       0, st, a);                                                                                 \
    return (int)hipGetLastError();                                                                                \
  }
  // few rows (decode): a workgroup per row, so a row is one round trip deep
  if (a.M > 256) {
    if (a.NP <= 512) ROWS(64, 2)
    if (a.NP <= 1024) ROWS(64, 4)
  }
  if (a.NP <= 1024) ROWS(256, 1)
  if (a.NP <= 2048) ROWS(256, 2)
  if (a.NP <= 4096) ROWS(256, 4)
  if (a.NP <= 8192) ROWS(256, 8)
  if (a.NP <= 16384) ROWS(256, 16)
#undef ROWS
  return -1;
}

// fp32 gated activation of packed gate|up columns (8 gate, 8 up, ...): out = gelu_tanh(gate) * up.
__global__ __launch_bounds__(256) void glu_f32_kernel(const float* __restrict__ gu, int ldi, float* __restrict__ out,
                                                      int ldo, int M, int F) {
  const long i = blockIdx.x * 256L + threadIdx.x;
  if (i >= (long)M * F) return;
  const int m = (int)(i / F), c = (int)(i % F);
  const float* p = gu + (size_t)m * ldi + (c >> 3) * 16 + (c & 7);
  const float x = p[0];
  out[(size_t)m * ldo + c] = 0.5f * x * (1.0f + tanhf(0.797884560802865f * (x + 0.044715f * x * x * x))) * p[8];
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_rows_update(const RowsArgs* a, int y_f32, int out_f32, hipStream_t st) {
  if (a->M <= 0 || a->N <= 0 || a->N > a->NP || a->NP % 4 != 0 || (a->ldx | a->ldy | a->ldcopy | a->ldh) % 4 != 0)
    return -1;
  if ((a->xidx != nullptr && (a->xrows < 1 || a->x_out != nullptr)) || (a->yidx != nullptr && a->yrows < 1)) return -1;
  if (y_f32) return out_f32 ? rows_launch<float, float>(*a, st) : rows_launch<float, bf16_t>(*a, st);
  return out_f32 ? -1 : rows_launch<bf16_t, bf16_t>(*a, st);
}

extern "C" int dnn_glu_f32(const float* gu, int ldi, float* out, int ldo, int M, int F, hipStream_t st) {
  if (M <= 0 || F <= 0 || F % 8 != 0 || ldi < 2 * F || ldo < F) return -1;
  hipLaunchKernelGGL(glu_f32_kernel, dim3((unsigned)(((long)M * F + 255) / 256)), dim3(256), 0, st, gu, ldi, out, ldo,
                     M, F);
  return (int)hipGetLastError();
}
