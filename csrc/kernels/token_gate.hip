// Gated token input of a decoder layer: g = gelu_tanh(x W^T) * e[token], the
// projection and the product with the token's table row in one launch (bf16
// operands, fp32 accumulation; fp32 variant: the product alone, after
// gemm_f32).  W has few rows (the side dimension, padded to 64), so a plain
// GEMM grid would leave most CUs idle:
//
//   rows <= 256   a workgroup takes 16 columns of 16 rows; eight waves split
//                 K (one round trip for K <= 4096) over W in fragment order
//                 (ops/gemm.py shuffle_weight) and reduce through LDS
//   more rows     64 x 64 or 64 x 128 tiles, six LDS stages of the K loop,
//                 five in flight (the K loop is latency-bound at one workgroup per CU)
#include "common.h"
#include "residual_api.h"

namespace dnn {

struct TokenGate {
  const bf16_t* table;  // token rows, stride ldt; this layer's part starts at off
  const int* tok;
  bf16_t* g;
  int ldt, off, V, ldg, M, n;
};

// Table values of a lane's 4 consecutive columns c..c+3 of row m (transposed
// accumulators), 0 past the part; and the store of their products.
__device__ __forceinline__ void token_gate_row(const TokenGate& t, int m, int c, float (&e)[4]) {
  const bf16_t* p = t.table + (size_t)min(max(t.tok[min(m, t.M - 1)], 0), t.V - 1) * t.ldt + t.off;
#pragma unroll
  for (int r = 0; r < 4; ++r) e[r] = c + r < t.n ? bf2f(p[c + r]) : 0.f;
}
__device__ __forceinline__ void token_gate_store(const TokenGate& t, const f32x4& z, int m, int c,
                                                 const float (&e)[4]) {
  if (m >= t.M) return;
  *reinterpret_cast<uint2*>(t.g + (size_t)m * t.ldg + c) =
      make_uint2(pack2bf(gelu_tanh(z[0]) * e[0], gelu_tanh(z[1]) * e[1]),
                 pack2bf(gelu_tanh(z[2]) * e[2], gelu_tanh(z[3]) * e[3]));
}

constexpr int TG_WAVES = 8, TG_U = 16;  // waves that split K, 32-wide chunks each has in flight

// grid (columns / 16, rows / 16)
__global__ __launch_bounds__(64 * (TG_WAVES + 1)) void token_gate_skinny_kernel(const bf16_t* __restrict__ x, int ldx,
                                                                          const uint8_t* __restrict__ ws, int K,
                                                                          TokenGate t) {
  __shared__ f32x4 red[TG_WAVES][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int m0 = blockIdx.y * 16, nch = K / 32;
  const int m = m0 + (lane & 15);
  if (wave == TG_WAVES) {  // the last wave fetches the token rows meanwhile, then reduces
    const int c4 = blockIdx.x * 16 + (lane >> 4) * 4;
    float e[4];
    token_gate_row(t, m, c4, e);
    __syncthreads();
    f32x4 z = red[0][lane];
#pragma unroll
    for (int w = 1; w < TG_WAVES; ++w) z += red[w][lane];
    token_gate_store(t, z, m, c4, e);
    return;
  }
  const uint8_t* wp = ws + (size_t)blockIdx.x * nch * 1024 + lane * 16;
  const bf16_t* xp = x + (size_t)min(m, t.M - 1) * ldx + (lane >> 4) * 8;
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int c0 = wave; c0 < nch; c0 += TG_WAVES * TG_U) {
    bf16x8 w[TG_U], a[TG_U];
#pragma unroll
    for (int u = 0; u < TG_U; ++u) {
      const int c = min(c0 + u * TG_WAVES, nch - 1);
      w[u] = *reinterpret_cast<const bf16x8*>(wp + (size_t)c * 1024);
      a[u] = *reinterpret_cast<const bf16x8*>(xp + c * 32);
    }
#pragma unroll
    for (int u = 0; u < TG_U; ++u)
      if (c0 + u * TG_WAVES < nch) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u], a[u], acc, 0, 0, 0);
  }
  red[wave][lane] = acc;
  __syncthreads();
}

constexpr int TG_BM = 64, TG_BK = 64, TG_ST = 6;

// One wave-instruction copies 8 rows x 128 B; 16-B chunk p of row r holds
// logical chunk p ^ (r & 7).
__device__ __forceinline__ void tg_stage8(const bf16_t* src, int ld, int row0, int rows, int k, char* lds, int lane) {
  const int r = lane >> 3, c = (lane & 7) ^ r;
  glds16(src + (size_t)min(row0 + r, rows - 1) * ld + k + c * 8, lds);
}
__device__ __forceinline__ bf16x8 tg_frag(const char* lds, int r, int c) {
  return *reinterpret_cast<const bf16x8*>(lds + r * 128 + ((c ^ (r & 7)) << 4));
}

template <int BN>
__global__ __launch_bounds__(256) void token_gate_tile_kernel(const bf16_t* __restrict__ x, int ldx,
                                                              const bf16_t* __restrict__ w, int ldw, int np, int K,
                                                              TokenGate t) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int STAGE = (TG_BM + BN) * 128, NI = (TG_BM + BN) / 32;  // NI: copies per wave and stage
  constexpr int NJ = BN / 32;                                         // 16-column tiles of a wave
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int ntn = np / BN, b = xcd_remap(blockIdx.x, gridDim.x);
  const int m0 = b / ntn * TG_BM, n0 = b % ntn * BN, nk = K / TG_BK;
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * (BN / 2);
  // Every workgroup starts at another K tile: in step, the 64 rows of all of
  // them would ask the same few memory channels at a time (power-of-two strides)
  const int k0 = (int)((b * 7u) % (unsigned)nk);
  auto issue = [&](int s) __attribute__((always_inline)) {
    const int kt = (s + k0 < nk ? s + k0 : s + k0 - nk) * TG_BK;
    char* lds = smem + (s % TG_ST) * STAGE;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int q = wave * NI + i;  // 8-row group: first the x rows, then the weight rows
      if (q < TG_BM / 8) tg_stage8(x, ldx, m0 + q * 8, t.M, kt, lds + q * 1024, lane);
      else tg_stage8(w, ldw, n0 + (q - TG_BM / 8) * 8, np, kt, lds + q * 1024, lane);
    }
  };
  f32x4 acc[2][NJ];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int s = 0; s < TG_ST - 1 && s < nk; ++s) issue(s);
  for (int k = 0; k < nk; ++k) {
    // stage k has landed when only the stages issued after it are in flight
    if (k + TG_ST - 2 < nk) asm volatile("s_waitcnt vmcnt(%0)" ::"i"((TG_ST - 2) * NI) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    // every wave's part of stage k landed, and stage k - 1 is read
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
    if (k + TG_ST - 1 < nk) issue(k + TG_ST - 1);
    const char* as = smem + (k % TG_ST) * STAGE;
    const char* bs = as + TG_BM * 128;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int c = s * 4 + (lane >> 4);
      bf16x8 af[2], bf[NJ];
#pragma unroll
      for (int i = 0; i < 2; ++i) af[i] = tg_frag(as, wm + i * 16 + (lane & 15), c);
#pragma unroll
      for (int j = 0; j < NJ; ++j) bf[j] = tg_frag(bs, wn + j * 16 + (lane & 15), c);
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < NJ; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf[j], af[i], acc[i][j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int m = m0 + wm + i * 16 + (lane & 15), c = n0 + wn + j * 16 + (lane >> 4) * 4;
      float e[4];
      token_gate_row(t, m, c, e);
      token_gate_store(t, acc[i][j], m, c, e);
    }
}

// g[m, c] = gelu_tanh(z[m, c]) * table[token[m], off + c] for c < n, 0 up to np.
__global__ __launch_bounds__(256) void token_gate_f32_kernel(const float* __restrict__ z, int ldz,
                                                             const float* __restrict__ table, int ldt, int off,
                                                             const int* __restrict__ tok, int V, float* __restrict__ g,
                                                             int ldg, int M, int n, int np) {
  const long i = blockIdx.x * 256L + threadIdx.x;
  if (i >= (long)M * np) return;
  const int m = (int)(i / np), c = (int)(i % np);
  float v = 0.f;
  if (c < n) {
    const float x = z[(size_t)m * ldz + c];
    v = 0.5f * x * (1.0f + tanhf(0.797884560802865f * (x + 0.044715f * x * x * x))) *
        table[(size_t)min(max(tok[m], 0), V - 1) * ldt + off + c];
  }
  g[(size_t)m * ldg + c] = v;
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_token_gate(const void* x, int ldx, const void* w, int ldw, const void* wsh, int K, const void* table,
                              int ldt, int off, const int* tok, int V, void* g, int ldg, int M, int n, int np,
                              hipStream_t st) {
  if (M <= 0 || n <= 0 || n > np || np % 64 != 0 || K <= 0 || K % 64 != 0 || off < 0 || off + n > ldt || V < 1) return -1;
  if (ldx % 8 != 0 || ldw % 8 != 0 || ldx < K || ldw < K || ldg % 4 != 0 || ldg < np || wsh == nullptr) return -1;
  if ((((uintptr_t)x | (uintptr_t)w | (uintptr_t)wsh) & 15) != 0 || ((uintptr_t)g & 7) != 0) return -1;
  const TokenGate t{(const bf16_t*)table, tok, (bf16_t*)g, ldt, off, V, ldg, M, n};
#define TGT(BN)                                                                                                    \
  hipLaunchKernelGGL((token_gate_tile_kernel<BN>), dim3((unsigned)((M + TG_BM - 1) / TG_BM * (np / BN))), dim3(256), \
                     TG_ST * (TG_BM + BN) * 128, st, (const bf16_t*)x, ldx, (const bf16_t*)w, ldw, np, K, t)
  if (M <= 256)
    hipLaunchKernelGGL(token_gate_skinny_kernel, dim3(np / 16, (M + 15) / 16), dim3(64 * (TG_WAVES + 1)), 0, st,
                       (const bf16_t*)x, ldx, (const uint8_t*)wsh, K, t);
  else if (np % 128 == 0 && M > 4096) TGT(128);
  else TGT(64);
#undef TGT
  return (int)hipGetLastError();
}

extern "C" int dnn_token_gate_f32(const float* z, int ldz, const float* table, int ldt, int off, const int* tok, int V,
                                  float* g, int ldg, int M, int n, int np, hipStream_t st) {
  if (M <= 0 || n <= 0 || n > np || off < 0 || off + n > ldt || V < 1 || ldg < np || ldz < n) return -1;
  hipLaunchKernelGGL(token_gate_f32_kernel, dim3((unsigned)(((long)M * np + 255) / 256)), dim3(256), 0, st, z, ldz,
                     table, ldt, off, tok, V, g, ldg, M, n, np);
  return (int)hipGetLastError();
}
