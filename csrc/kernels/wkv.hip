// Recurrence with a decay per key channel and a bonus for the current token
// (gfx950), per head with a matrix state (fp32, [slot][H][value][key channel]):
//   y_t = (S + diag(u) k_t v_t^T)^T r_t,   S <- diag(exp(la_t)) S + k_t v_t^T
//
//   decay       la = -exp(W2 tanh(t) + w0) from the low-rank projection t
//   wkv_chunks  bf16, sequences of 2 tokens or more, on the MFMA
//   wkv_steps   token by token in fp32: single decoded tokens, and the exact mode
//
// States are fp32 in pools by slot; a portion that begins at position 0 starts
// from zero.
#include "common.h"
#include "mixer_api.h"
#include "vec16.h"

namespace dnn {

typedef short s16x4 __attribute__((ext_vector_type(4)));
constexpr float LOG2E = 1.4426950408889634f;
constexpr float LA_MIN = -88.f;  // exp(-88) is zero beside any state

__device__ __forceinline__ uint32_t wk_pack2(float a, float b) {
  typedef float f32x2v __attribute__((ext_vector_type(2)));
  return __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2v{a, b}), bf16x2v));
}
// Two values as bf16 and their remainders as bf16: about 16 bits of mantissa.
__device__ __forceinline__ void wk_split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = wk_pack2(a, b);
  lo = wk_pack2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}
__device__ __forceinline__ void wk_split4(const float* v, uint2& hi, uint2& lo) {
  wk_split2(v[0], v[1], hi.x, lo.x);
  wk_split2(v[2], v[3], hi.y, lo.y);
}
__device__ __forceinline__ bf16x8 wk_frag(const uint2& a, const uint2& b) {
  const i32x4 v = {(int)a.x, (int)a.y, (int)b.x, (int)b.y};
  return __builtin_bit_cast(bf16x8, v);
}

// ---------------------------------------------------------------- decay
// A wave takes 16 R rows x `cols` columns, grid (ceil(N / (4 cols)), ceil(M / 16 R));
// tanh in two bf16 terms, W2 rows [N][rank] in bf16.  KS: 32-column steps of the
// rank whose terms stay in registers (0: formed again for every 64 columns).
__device__ __forceinline__ void decay_terms(const float* tp, bf16x8& hi, bf16x8& lo) {
  float v[8];
#pragma unroll
  for (int j = 0; j < 8; j += 4) {
    const f32x4 x = *reinterpret_cast<const f32x4*>(tp + j);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      v[j + i] = 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x[i] * (2.0f * LOG2E)));
  }
  uint2 h0, h1, l0, l1;
  wk_split4(v, h0, l0);
  wk_split4(v + 4, h1, l1);
  hi = wk_frag(h0, h1), lo = wk_frag(l0, l1);
}

template <int KS, int R>
__global__ __launch_bounds__(256) void decay_kernel(DecayArgs a, int cols) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4;
  const int m0 = blockIdx.y * 16 * R + (lane & 15), first = (blockIdx.x * 4 + wave) * cols;
  const bf16_t* w2 = reinterpret_cast<const bf16_t*>(a.w2) + 8 * g;
  const float* tp[R];
  bf16x8 hi[R][KS > 0 ? KS : 1], lo[R][KS > 0 ? KS : 1];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    tp[r] = a.t + (size_t)min(m0 + 16 * r, a.M - 1) * a.ldt + 8 * g;
    if constexpr (KS > 0) {
#pragma unroll
      for (int k = 0; k < KS; ++k) decay_terms(tp[r] + k * 32, hi[r][k], lo[r][k]);
    }
  }
  for (int n0 = first; n0 < min(first + cols, a.N); n0 += 64) {
    f32x4 acc[R][4], w0[4];
    const bf16_t* wr[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int r = 0; r < R; ++r) acc[r][j] = f32x4{0.f, 0.f, 0.f, 0.f};
      wr[j] = w2 + (size_t)min(n0 + j * 16 + (lane & 15), a.N - 1) * a.rank;
      w0[j] = *reinterpret_cast<const f32x4*>(a.w0 + min(n0 + j * 16 + 4 * g, a.N - 4));
    }
    auto step = [&](int col, int k) __attribute__((always_inline)) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bf16x8 w = *reinterpret_cast<const bf16x8*>(wr[j] + col);
#pragma unroll
        for (int r = 0; r < R; ++r) {
          acc[r][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, hi[r][k], acc[r][j], 0, 0, 0);
          acc[r][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, lo[r][k], acc[r][j], 0, 0, 0);
        }
      }
    };
    if constexpr (KS > 0) {
#pragma unroll
      for (int k = 0; k < KS; ++k) step(k * 32, k);
    } else {
      for (int k = 0; k < a.rank; k += 32) {
#pragma unroll
        for (int r = 0; r < R; ++r) decay_terms(tp[r] + k, hi[r][0], lo[r][0]);
        step(k, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
      if (m0 + 16 * r >= a.M) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int n = n0 + j * 16 + 4 * g;
        if (n >= a.N) continue;
        f32x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = fmaxf(-__builtin_amdgcn_exp2f((acc[r][j][i] + w0[j][i]) * LOG2E), LA_MIN);
        *reinterpret_cast<f32x4*>(a.la + (size_t)(m0 + 16 * r) * a.N + n) = o;
      }
    }
  }
}

// grid (ceil(N / 256), M); W2 in fp32
__global__ __launch_bounds__(256) void decay_f32_kernel(DecayArgs a) {
  __shared__ float th[256];
  const int m = blockIdx.y, n = blockIdx.x * 256 + threadIdx.x;
  const float* w2 = reinterpret_cast<const float*>(a.w2) + (size_t)min(n, a.N - 1) * a.rank;
  float s = 0.f;
  for (int k0 = 0; k0 < a.rank; k0 += 256) {
    const int len = min(256, a.rank - k0);
    __syncthreads();
    if ((int)threadIdx.x < len) th[threadIdx.x] = tanhf(a.t[(size_t)m * a.ldt + k0 + threadIdx.x]);
    __syncthreads();
    for (int k = 0; k < len; ++k) s = fmaf(th[k], w2[k0 + k], s);
  }
  if (n < a.N) a.la[(size_t)m * a.N + n] = fmaxf(-expf(s + a.w0[n]), LA_MIN);
}

// ---------------------------------------------------------------- token by token
// grid (H, NP / 64, sequences); LPR lanes share a state row (one value column),
// each holding float4s of it.
template <typename T, int NP>
__global__ __launch_bounds__(256) void wkv_steps_kernel(WkvArgs a) {
  constexpr int LPR = 16, NI = NP / (4 * LPR);
  constexpr int RPP = 256 / LPR, NR = 64 / RPP;
  const int h = blockIdx.x, v0 = blockIdx.y * 64;
  const int4 e = a.ent[blockIdx.z];
  const int slot = min(max(e.z, 0), a.nslots - 1);
  const int l = threadIdx.x % LPR, r0 = threadIdx.x / LPR;
  float* st = a.state + (((size_t)slot * a.H + h) * NP + v0) * NP;
  f32x4 S[NR][NI], u[NI];
  const bool fresh = a.pos[e.x] == 0;
#pragma unroll
  for (int i = 0; i < NI; ++i) u[i] = *reinterpret_cast<const f32x4*>(a.u + h * NP + i * 4 * LPR + l * 4);
#pragma unroll
  for (int r = 0; r < NR; ++r)
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      S[r][i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!fresh) S[r][i] = *reinterpret_cast<const f32x4*>(st + (size_t)(r0 + r * RPP) * NP + i * 4 * LPR + l * 4);
    }
  for (int t = 0; t < e.y; ++t) {
    const int m = e.x + t;
    const size_t o = (size_t)m * a.ld + h * NP;
    const T* rp = reinterpret_cast<const T*>(a.r) + o + l * 4;
    const T* kp = reinterpret_cast<const T*>(a.k) + o + l * 4;
    const T* vp = reinterpret_cast<const T*>(a.v) + o;
    const float* lp = a.la + ((size_t)m * a.H + h) * NP + l * 4;
    f32x4 q[NI], k[NI], w[NI], qu[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const f32x4 la = *reinterpret_cast<const f32x4*>(lp + i * 4 * LPR);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        q[i][j] = to_f32(rp[i * 4 * LPR + j]);
        k[i][j] = to_f32(kp[i * 4 * LPR + j]);
        w[i][j] = expf(la[j]);
        qu[i][j] = q[i][j] * u[i][j];
      }
    }
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const int v = v0 + r0 + r * RPP;
      const float x = to_f32(vp[v]);
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float kv = k[i][j] * x;
          y = fmaf(S[r][i][j], q[i][j], y);
          y = fmaf(kv, qu[i][j], y);
          S[r][i][j] = fmaf(w[i][j], S[r][i][j], kv);
        }
      y = group_sum<LPR>(y);
      if (l == 0 && v < a.dim) reinterpret_cast<T*>(a.y)[(size_t)m * a.ldy + h * a.dim + v] = from_f32<T>(y);
    }
  }
#pragma unroll
  for (int r = 0; r < NR; ++r)
#pragma unroll
    for (int i = 0; i < NI; ++i)
      *reinterpret_cast<f32x4*>(st + (size_t)(r0 + r * RPP) * NP + i * 4 * LPR + l * 4) = S[r][i];
}

// ---------------------------------------------------------------- chunks
// 64 tokens at a time as four parts of 16.  With L_t the running sum of la
// within a part, E_t = L_t - la_t and L the sum over the whole part,
//   y_t = (r_t exp(E_t)) S + sum_{s < t} A_ts v_s + (r_t . u k_t) v_t
//   S  <- exp(L) S + sum_s (k_s exp(L - L_s)) v_s^T,   A_ts = sum_c r_t k_s exp(E_t - L_s)
// First wave w prepares part w (all factors at most 1, except in A); then every
// wave walks the parts in order with 16 value columns of the state in its
// accumulators, which are the next product's operand as they lie.
//
// A factorises around the middle of the part: exp(E_t - M) exp(M - L_s) where
// neither half decays by more than 2^-60; else it is summed pair by pair.
// Whatever carries a decay, and the state, enters the MFMA as two bf16 terms.
//
// PIPE: 8 waves, four prepare 64 tokens while the other four walk the 64 before
// (two sets of parts in LDS); else 4 waves do both in turn.
//
// A lane of a preparing wave has token lane & 15 and, of every 32 channels, the
// 8 that a fragment of the products holds: 4 g + {0..3} and 16 + 4 g + {0..3},
// g = lane >> 4.
template <int NP>
struct WkvLds {
  static constexpr int PAIRS = NP / 32;
  static constexpr int R = PAIRS * 2 * 1024, A = 1024;    // fragments by lane: r (two terms), A (both terms)
  static constexpr int KST = NP * 2 + 32, K = 16 * KST;   // rows of k, per term
  static constexpr int VST = 160, V = 16 * VST;
  static constexpr int O_A = R, O_K = R + A, O_D = O_K + 2 * K, O_V = O_D + NP * 4;
  static constexpr int PART = O_V + V, TOTAL = 4 * PART;
};
constexpr float WK_HALF = 60.f;

// 4 rows of one column: rows 4 g.., column (lane & 15) of the 16 from `col`
__device__ __forceinline__ s16x4 wk_tr(const char* rows, int stride, int col, int lane) {
  const int r = 4 * (lane >> 4) + ((lane & 15) >> 2);
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(rows + r * stride + (col + 4 * (lane & 3)) * 2));
}
// x of the lane n to the left within 16 lanes, 0 past the edge
template <int N>
__device__ __forceinline__ float wk_left(float x) {
  return __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(x), 0x110 | N, 0xf, 0xf, true));
}

template <int NP, bool PIPE>
__global__ __launch_bounds__(PIPE ? 512 : 256, 1) void wkv_chunks_kernel(WkvArgs a) {
  using L = WkvLds<NP>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int PAIRS = L::PAIRS;
  const int tid = threadIdx.x, lane = tid & 63, wave = (tid >> 6) & 3, t16 = lane & 15, g = lane >> 4;
  const bool prepares = !PIPE || tid >= 256, walks = !PIPE || tid < 256;
  const int h = blockIdx.x, v0 = blockIdx.y * 64;
  const int4 e = a.ent[blockIdx.z];
  const int n = e.y, slot = min(max(e.z, 0), a.nslots - 1);
  float* state = a.state + (((size_t)slot * a.H + h) * NP + v0 + wave * 16 + t16) * NP + 4 * g;
  const bool fresh = a.pos[e.x] == 0;
  f32x4 S[2 * PAIRS];
#pragma unroll
  for (int i = 0; i < 2 * PAIRS; ++i) {
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (walks && !fresh) S[i] = *reinterpret_cast<const f32x4*>(state + 16 * i);
  }
  const bf16_t* rb = reinterpret_cast<const bf16_t*>(a.r) + h * NP + 4 * g;
  const bf16_t* kb = reinterpret_cast<const bf16_t*>(a.k) + h * NP + 4 * g;
  const bf16_t* vb = reinterpret_cast<const bf16_t*>(a.v) + h * NP + v0 + (lane & 3) * 16;
  const float* lb = a.la + h * NP + 4 * g;
  const float* ub = a.u + h * NP + 4 * g;

  s16x4 pr[PAIRS][2], pk[PAIRS][2];
  f32x4 pl[PAIRS][2];
  i32x4 pv[2];
  auto fetch = [&](int c0) __attribute__((always_inline)) {
    const size_t m = (size_t)e.x + min(c0 + wave * 16 + t16, n - 1);
#pragma unroll
    for (int p = 0; p < PAIRS; ++p)
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        pr[p][q] = *reinterpret_cast<const s16x4*>(rb + m * a.ld + p * 32 + q * 16);
        pk[p][q] = *reinterpret_cast<const s16x4*>(kb + m * a.ld + p * 32 + q * 16);
        pl[p][q] = *reinterpret_cast<const f32x4*>(lb + m * a.H * NP + p * 32 + q * 16);
      }
    const size_t mv = (size_t)e.x + min(c0 + wave * 16 + (lane >> 2), n - 1);
#pragma unroll
    for (int q = 0; q < 2; ++q) pv[q] = *reinterpret_cast<const i32x4*>(vb + mv * a.ld + q * 8);
  };
  auto prepare = [&](int c0, char* buf) __attribute__((always_inline)) {  // this wave's part
    char* part = buf + wave * L::PART;
    s16x4 cr[PAIRS][2], ck[PAIRS][2];
    f32x4 cl[PAIRS][2];
    i32x4 cv[2] = {pv[0], pv[1]};
#pragma unroll
    for (int p = 0; p < PAIRS; ++p)
#pragma unroll
      for (int q = 0; q < 2; ++q) cr[p][q] = pr[p][q], ck[p][q] = pk[p][q], cl[p][q] = pl[p][q];
    if (PIPE && c0 + 64 < n) fetch(c0 + 64);
    const bool live = c0 + wave * 16 + t16 < n;  // past the end: no decay, no key
    f32x4 A = f32x4{0.f, 0.f, 0.f, 0.f};
    float own = 0.f;
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      float r[8], k[8], Lc[8], E[8], tot[8], mid[8], x[8], y[8];
      float span = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int q = j >> 2, i = j & 3;
        r[j] = bf2f_s(cr[p][q][i]);
        k[j] = live ? bf2f_s(ck[p][q][i]) : 0.f;
        const float la = live ? cl[p][q][i] * LOG2E : 0.f;
        float s = la;
        s += wk_left<1>(s);
        s += wk_left<2>(s);
        s += wk_left<4>(s);
        s += wk_left<8>(s);
        Lc[j] = s;
        E[j] = s - la;
        tot[j] = __shfl(s, (lane & 48) | 15, 64);
        mid[j] = __shfl(s, (lane & 48) | 7, 64);
        span = fmaxf(span, fmaxf(-mid[j], mid[j] - tot[j]));
      }
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        const f32x4 u = *reinterpret_cast<const f32x4*>(ub + p * 32 + q * 16);
#pragma unroll
        for (int i = 0; i < 4; ++i) own = fmaf(r[q * 4 + i] * u[i], k[q * 4 + i], own);
      }
      uint2 h0, h1, l0, l1;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        x[j] = r[j] * __builtin_amdgcn_exp2f(E[j]);
        y[j] = k[j] * __builtin_amdgcn_exp2f(tot[j] - Lc[j]);
      }
      wk_split4(x, h0, l0);
      wk_split4(x + 4, h1, l1);
      *reinterpret_cast<bf16x8*>(part + (p * 2) * 1024 + lane * 16) = wk_frag(h0, h1);
      *reinterpret_cast<bf16x8*>(part + (p * 2 + 1) * 1024 + lane * 16) = wk_frag(l0, l1);
      wk_split4(y, h0, l0);
      wk_split4(y + 4, h1, l1);
      char* kr = part + L::O_K + t16 * L::KST + (p * 32 + 4 * g) * 2;
      *reinterpret_cast<uint2*>(kr) = h0;
      *reinterpret_cast<uint2*>(kr + 32) = h1;
      *reinterpret_cast<uint2*>(kr + L::K) = l0;
      *reinterpret_cast<uint2*>(kr + L::K + 32) = l1;
      if (t16 == 0) {
        float* d = reinterpret_cast<float*>(part + L::O_D) + p * 32 + 4 * g;
#pragma unroll
        for (int j = 0; j < 8; ++j) d[(j >> 2) * 16 + (j & 3)] = __builtin_amdgcn_exp2f(tot[j]);
      }
      if (__all(span <= WK_HALF)) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          x[j] = r[j] * __builtin_amdgcn_exp2f(E[j] - mid[j]);
          y[j] = k[j] * __builtin_amdgcn_exp2f(mid[j] - Lc[j]);
        }
        wk_split4(x, h0, l0);
        wk_split4(x + 4, h1, l1);
        const bf16x8 xh = wk_frag(h0, h1), xl = wk_frag(l0, l1);
        wk_split4(y, h0, l0);
        wk_split4(y + 4, h1, l1);
        const bf16x8 yh = wk_frag(h0, h1), yl = wk_frag(l0, l1);
        f32x4 d = f32x4{0.f, 0.f, 0.f, 0.f};
        d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(yh, xh, d, 0, 0, 0);
        d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(yh, xl, d, 0, 0, 0);
        d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(yl, xh, d, 0, 0, 0);
        A += d;
      } else {
        for (int sq = 0; sq < 4; ++sq)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int src = (lane & 48) | (sq * 4 + i);
            float v = 0.f;
#pragma unroll
            for (int j = 0; j < 8; ++j)
              v = fmaf(r[j] * __shfl(k[j], src, 64), __builtin_amdgcn_exp2f(fminf(E[j] - __shfl(Lc[j], src, 64), 0.f)), v);
            v += __shfl_xor(v, 16, 64);
            v += __shfl_xor(v, 32, 64);
            if (g == sq) A[i] += v;
          }
      }
    }
    own += __shfl_xor(own, 16, 64);
    own += __shfl_xor(own, 32, 64);
    float m[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) m[i] = 4 * g + i < t16 ? A[i] : 4 * g + i == t16 ? own : 0.f;
    uint2 hi, lo;
    wk_split4(m, hi, lo);
    *reinterpret_cast<bf16x8*>(part + L::O_A + lane * 16) = wk_frag(hi, lo);
#pragma unroll
    for (int q = 0; q < 2; ++q)
      *reinterpret_cast<i32x4*>(part + L::O_V + (lane >> 2) * L::VST + (lane & 3) * 32 + q * 16) = cv[q];
  };
  auto walk = [&](int c0, const char* buf) __attribute__((always_inline)) {  // the parts in order
    const int parts = min(4, (n - c0 + 15) >> 4);
    for (int s = 0; s < parts; ++s) {
      const char* part = buf + s * L::PART;
      const s16x4 v4 = wk_tr(part + L::O_V, L::VST, wave * 16, lane);
      const bf16x8 vv = {v4[0], v4[1], v4[2], v4[3], v4[0], v4[1], v4[2], v4[3]};
      f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
      o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(part + L::O_A + lane * 16), vv, o, 0, 0, 0);
#pragma unroll
      for (int p = 0; p < PAIRS; ++p) {
        const bf16x8 rh = *reinterpret_cast<const bf16x8*>(part + (p * 2) * 1024 + lane * 16);
        const bf16x8 rl = *reinterpret_cast<const bf16x8*>(part + (p * 2 + 1) * 1024 + lane * 16);
        uint2 h0, h1, l0, l1;
        const float s0[4] = {S[2 * p][0], S[2 * p][1], S[2 * p][2], S[2 * p][3]};
        const float s1[4] = {S[2 * p + 1][0], S[2 * p + 1][1], S[2 * p + 1][2], S[2 * p + 1][3]};
        wk_split4(s0, h0, l0);
        wk_split4(s1, h1, l1);
        const bf16x8 sh = wk_frag(h0, h1), sl = wk_frag(l0, l1);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rh, sh, o, 0, 0, 0);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rh, sl, o, 0, 0, 0);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rl, sh, o, 0, 0, 0);
      }
      const float* dec = reinterpret_cast<const float*>(part + L::O_D) + 4 * g;
#pragma unroll
      for (int i = 0; i < 2 * PAIRS; ++i) {
        const s16x4 kh = wk_tr(part + L::O_K, L::KST, i * 16, lane), kl = wk_tr(part + L::O_K + L::K, L::KST, i * 16, lane);
        const bf16x8 kf = {kh[0], kh[1], kh[2], kh[3], kl[0], kl[1], kl[2], kl[3]};
        S[i] *= *reinterpret_cast<const f32x4*>(dec + 16 * i);
        S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vv, S[i], 0, 0, 0);
      }
      const int v = v0 + wave * 16 + t16;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = c0 + s * 16 + 4 * g + i;
        if (t < n && v < a.dim) reinterpret_cast<bf16_t*>(a.y)[(size_t)(e.x + t) * a.ldy + h * a.dim + v] = f2bf(o[i]);
      }
    }
  };
  if (prepares) fetch(0);
  if constexpr (PIPE) {
    const int chunks = (n + 63) / 64;
    for (int i = 0; i <= chunks; ++i) {
      if (prepares && i < chunks) prepare(i * 64, smem + (i & 1) * L::TOTAL);
      if (walks && i > 0) walk((i - 1) * 64, smem + ((i - 1) & 1) * L::TOTAL);
      __syncthreads();
    }
  } else {
    for (int c0 = 0; c0 < n; c0 += 64) {
      __syncthreads();  // the last 64 tokens are read
      prepare(c0, smem);
      __syncthreads();
      if (c0 + 64 < n) fetch(c0 + 64);
      walk(c0, smem);
    }
  }
  if (!walks) return;
#pragma unroll
  for (int i = 0; i < 2 * PAIRS; ++i) *reinterpret_cast<f32x4*>(state + 16 * i) = S[i];
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_decay(const DecayArgs* a, int f32, hipStream_t st) {
  if (a->M <= 0 || a->N <= 0 || a->N % 4 != 0 || a->rank <= 0 || a->ldt % 4 != 0 || a->ldt < a->rank) return -1;
  if (f32) {
    if (a->M > 65535) return -1;
    hipLaunchKernelGGL(decay_f32_kernel, dim3((a->N + 255) / 256, a->M), dim3(256), 0, st, *a);
  } else {
    const int R = a->M >= 1024 ? 4 : 1, rows = (a->M + 16 * R - 1) / (16 * R);
    if (a->N % 64 != 0 || a->rank % 32 != 0 || rows > 65535) return -1;
    int cols = 64;  // per wave: wide where the rows alone fill the chip
    while (cols < 256 && (long)rows * (a->N / (8 * cols)) >= 512) cols *= 2;
    const dim3 grid((a->N + 4 * cols - 1) / (4 * cols), rows);
#define DECAY(K)                                                                                   \
  {                                                                                                \
    if (R == 1) hipLaunchKernelGGL((decay_kernel<K, 1>), grid, dim3(256), 0, st, *a, cols);        \
    else hipLaunchKernelGGL((decay_kernel<K, 4>), grid, dim3(256), 0, st, *a, cols);               \
  }
    if (a->rank == 64) DECAY(2)
    else if (a->rank == 128) DECAY(4)
    else DECAY(0)
#undef DECAY
  }
  return (int)hipGetLastError();
}

static bool wkv_ok(const WkvArgs& a) {
  return a.M > 0 && a.H > 0 && (a.NP == 64 || a.NP == 128 || a.NP == 256) && a.dim > 0 && a.dim <= a.NP && a.nent > 0 &&
         a.nent <= 65535 && a.nslots > 0 && a.ld >= a.H * a.NP && a.ld % 8 == 0 && a.ldy >= a.H * a.dim &&
         ((uintptr_t)a.ent & 15) == 0 && (((uintptr_t)a.r | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)a.la | (uintptr_t)a.u) & 15) == 0 &&
         a.state != nullptr && a.pos != nullptr && a.la != nullptr && a.u != nullptr;
}

extern "C" int dnn_wkv_steps(const WkvArgs* a, int f32, hipStream_t st) {
  if (!wkv_ok(*a)) return -1;
  const dim3 grid(a->H, a->NP / 64, a->nent);
#define WS(N)                                                                                \
  {                                                                                          \
    if (f32) hipLaunchKernelGGL((wkv_steps_kernel<float, N>), grid, dim3(256), 0, st, *a);   \
    else hipLaunchKernelGGL((wkv_steps_kernel<bf16_t, N>), grid, dim3(256), 0, st, *a);      \
  }
  if (a->NP == 64) WS(64) else if (a->NP == 128) WS(128) else WS(256)
#undef WS
  return (int)hipGetLastError();
}

extern "C" int dnn_wkv_chunks(const WkvArgs* a, hipStream_t st) {
  if (!wkv_ok(*a)) return -1;
  const dim3 grid(a->H, a->NP / 64, a->nent);
#define WC(N, P) hipLaunchKernelGGL((wkv_chunks_kernel<N, P>), grid, dim3(P ? 512 : 256), (P ? 2 : 1) * WkvLds<N>::TOTAL, st, *a)
  if (a->NP == 64) WC(64, true);
  else if (a->NP == 128) WC(128, false);
  else WC(256, false);
#undef WC
  return (int)hipGetLastError();
}
