// Attention over a latent cache, for batches of unequal sequences (gfx950).
//
// The cache holds one row per token for all heads, [page][64][CP + RP]: a normed
// latent of CP columns and a rotated key part of RP.  A head's unrotated key and
// its value are linear in the latent, so the key projection is moved to the
// query (q . W_uk c = (W_uk^T q) . c) and the value projection behind the
// softmax: every head scores whole cache rows and sums their latents.
//
//   latent_prep      norms of the query's and the cache's latent, rotation of the
//                    shared key part, cache write
//   rope_rows        rotation of every head's rotated part, in place
//   latent_attn      bf16; a workgroup takes 64 packed (token, head) rows and
//                    walks the pages: its 4 waves take a quarter each of the
//                    64 x 64 scores, then a quarter each of the latent columns.
//                    Portions of prompts, and single tokens (over `splits`
//                    workgroups, then a combine)
//   latent_attn_f32  fp32, one wave per (row, head): the exact mode
//
// Scores, softmax and accumulation are fp32.
#include "common.h"
#include "residual_api.h"
#include "vec16.h"

namespace dnn {

typedef short s16x4 __attribute__((ext_vector_type(4)));
constexpr int PG = 64;  // keys per page
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ int la_page(const int* table, int ldt, int npages, int slot, int blk) {
  if (blk < 0 || blk >= ldt) return -1;
  const int p = table[(size_t)slot * ldt + blk];
  return p < npages ? p : -1;
}

// ---------------------------------------------------------------- rotation
// cos and sin of pair i at position p times `mag`; the angle is in turns and
// reduced in fp64.
template <typename T>
__device__ __forceinline__ void rope_pair(int p, double freq, float mag, float& u, float& v) {
  double t = (double)p * freq;
  t -= floor(t);
  const float a = (float)t;
  const float c = mag * (sizeof(T) == 2 ? __builtin_amdgcn_cosf(a) : cosf(6.283185307179586f * a));
  const float s = mag * (sizeof(T) == 2 ? __builtin_amdgcn_sinf(a) : sinf(6.283185307179586f * a));
  const float x = u * c - v * s;
  v = v * c + u * s;
  u = x;
}
// A 16-byte piece of neighbouring pairs from pair i0 on; pairs past `pairs` pass.
template <typename T>
__device__ __forceinline__ void rope_piece(const RopeTable& r, int p, int i0, float (&v)[Vec16<T>::N]) {
#pragma unroll
  for (int j = 0; j < Vec16<T>::N / 2; ++j)
    if (i0 + j < r.pairs) rope_pair<T>(p, r.freq[i0 + j], r.mag, v[2 * j], v[2 * j + 1]);
}

template <typename T>
__global__ __launch_bounds__(256) void rope_rows_kernel(T* __restrict__ x, int ld, int hs, int M, int H, int RP,
                                                        const int* __restrict__ pos, RopeTable r) {
  constexpr int E = Vec16<T>::N;
  const int pc = (2 * r.pairs + E - 1) / E;  // pieces of a head that turn
  const long i = blockIdx.x * 256L + threadIdx.x;
  if (i >= (long)M * H * pc) return;
  const int c = (int)(i % pc), h = (int)(i / pc % H), m = (int)(i / pc / H);
  T* p = x + (size_t)m * ld + h * hs + c * E;
  float v[E];
  Vec16<T>::get(p, v);
  rope_piece<T>(r, pos[m], c * (E / 2), v);
  Vec16<T>::put(p, v);
}

// ---------------------------------------------------------------- norms and cache write
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrepArgs a) {
  constexpr int E = Vec16<T>::N;
  __shared__ float red[8];
  const int m = blockIdx.x, tid = threadIdx.x, p = a.pos[m];
  T* row = reinterpret_cast<T*>(a.rows) + (size_t)m * a.ld;
  T* cr = row + a.QP;
  T* rr = cr + a.CP;
  const int page = la_page(a.table, a.ldt, a.npages, a.slots[m], p / PG);
  T* kd = page >= 0 ? reinterpret_cast<T*>(a.kp) + ((size_t)page * PG + p % PG) * (a.CP + a.RP) : nullptr;
  float sq = 0.f, sc = 0.f, v[E];
  for (int c = tid * E; c < a.QP; c += 256 * E) {
    Vec16<T>::get(row + c, v);
#pragma unroll
    for (int j = 0; j < E; ++j) sq = fmaf(v[j], v[j], sq);
  }
  for (int c = tid * E; c < a.CP; c += 256 * E) {
    Vec16<T>::get(cr + c, v);
#pragma unroll
    for (int j = 0; j < E; ++j) sc = fmaf(v[j], v[j], sc);
  }
  for (int c = tid * E; c < a.RP; c += 256 * E) {
    Vec16<T>::get(rr + c, v);
    rope_piece<T>(a.rope, p, c / 2, v);
    Vec16<T>::put(rr + c, v);
    if (kd != nullptr) Vec16<T>::put(kd + a.CP + c, v);
  }
  sq = wave_sum(sq);
  sc = wave_sum(sc);
  if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sc;
  __syncthreads();
  const float fq = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.QN + a.eps);
  const float fc = 1.0f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)a.CN + a.eps);
  auto scale = [&](T* src, const float* w, float f) __attribute__((always_inline)) {
    Vec16<T>::get(src, v);
#pragma unroll
    for (int j = 0; j < E; j += 4) {
      const f32x4 w4 = *reinterpret_cast<const f32x4*>(w + j);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[j + i] *= f * w4[i];
    }
    Vec16<T>::put(src, v);
  };
  for (int c = tid * E; c < a.QP; c += 256 * E) scale(row + c, a.qw + c, fq);
  for (int c = tid * E; c < a.CP; c += 256 * E) {
    scale(cr + c, a.cw + c, fc);
    if (kd != nullptr) Vec16<T>::put(kd + c, v);
  }
}

// ---------------------------------------------------------------- MFMA attention
template <int CP, int RP>
struct LaLds {
  static constexpr int DK = CP + RP;
  static constexpr int RS = (DK * 2 + 255) / 256 * 256;  // bytes of a key row: whole groups of 16 pieces
  static constexpr int K = PG * RS, P = 8 * 1024, TOTAL = K + P + 2 * 2 * 32 * 4;
};
// Byte of 16-B piece c of key r; swizzled within groups of 16 pieces so that a
// fragment read (one piece of 16 rows) and a transposing read (4 pieces of 4
// rows) spread over all banks.
template <int RS>
__device__ __forceinline__ int la_at(int r, int c) {
  return r * RS + ((c ^ (((r & 3) << 2) | ((r >> 2) & 3))) << 4);
}
// 8 values of column col0 + (lane & 31) at rows 16 s + 4 h + {0..3, 8..11}
template <int RS>
__device__ __forceinline__ bf16x8 la_tr(const char* tile, int s, int col0, int lane) {
  const int r = 16 * s + 4 * (lane >> 5) + ((lane & 15) >> 2);
  const int c = (col0 >> 3) + ((lane >> 4) & 1) * 2 + ((lane >> 1) & 1), b = (lane & 1) * 8;
  const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(tile + la_at<RS>(r, c) + b));
  const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(tile + la_at<RS>(r + 8, c) + b));
  return bf16x8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
}

__device__ __forceinline__ float la_gate(const LatentAttnArgs& a, int row, int head) {
  if (a.gate == nullptr) return 1.f;
  return 1.0f / (1.0f + __expf(-bf2f(reinterpret_cast<const bf16_t*>(a.gate)[(size_t)row * a.ldg + head])));
}

// grid (tiles, splits); tiles: {first batch row, tokens, slot, first packed row}.
// With splits the tiles are single tokens, per_token tiles each, and
// ws = [token][H][splits][CP + 2] takes {max, sum, O} partials.
template <int CP, int RP>
__global__ __launch_bounds__(256, 1) void latent_attn_kernel(LatentAttnArgs a, const int4* __restrict__ tiles,
                                                             int per_token, float* __restrict__ ws) {
  using L = LaLds<CP, RP>;
  constexpr int DK = L::DK, RS = L::RS, NKS = DK / 16, CK = DK / 8, NI = PG * CK / 256, NC = CP / 128;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ks = smem;
  char* ps = smem + L::K;
  float* red = reinterpret_cast<float*>(ps + L::P);  // [row half][key half][32]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = lane >> 5, r32 = lane & 31;
  const int rh = wave >> 1, kh = wave & 1, ns = gridDim.y;
  const int4 t = tiles[blockIdx.x];
  const int tok0 = t.x, n = t.y, slot = t.z, row0 = t.w, last = n - 1;
  const int p0 = a.pos[tok0];
  const int row = row0 + rh * 32 + r32, tk = min(row / a.H, last), head = row % a.H, q_abs = p0 + tk;
  const int q_min = p0 + min((row0 + rh * 32) / a.H, last);
  const int total = (p0 + min((row0 + 63) / a.H, last)) / PG + 1;
  const int ub = (int)((long)total * blockIdx.y / ns), ue = (int)((long)total * (blockIdx.y + 1) / ns);

  bf16x8 qf[NKS];
  {
    const bf16_t* ql = reinterpret_cast<const bf16_t*>(a.qlat) + (size_t)(tok0 + tk) * a.ldql + head * CP + 8 * h;
    const bf16_t* qr = reinterpret_cast<const bf16_t*>(a.qrot) + (size_t)(tok0 + tk) * a.ldqr + head * a.hs + 8 * h;
#pragma unroll
    for (int s = 0; s < CP / 16; ++s) qf[s] = *reinterpret_cast<const bf16x8*>(ql + s * 16);
#pragma unroll
    for (int s = 0; s < RP / 16; ++s) qf[CP / 16 + s] = *reinterpret_cast<const bf16x8*>(qr + s * 16);
  }
  f32x16 o[2][NC];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < NC; ++j) o[i][j] = f32x16{};
  float m0 = -INFINITY, m1 = -INFINITY, l_i = 0.f;
  const float sc = a.scale * LOG2E;

  i32x4 pk[NI];
  auto fetch = [&](int i) __attribute__((always_inline)) {
    const int page = max(la_page(a.table, a.ldt, a.npages, slot, i), 0);  // a missing page is never visible; stay in the pool
    const bf16_t* kb = reinterpret_cast<const bf16_t*>(a.kp) + (size_t)page * PG * DK;
#pragma unroll
    for (int it = 0; it < NI; ++it) pk[it] = *reinterpret_cast<const i32x4*>(kb + (it * 256 + tid) * 8);
  };
  if (ub < ue) fetch(ub);
  for (int i = ub; i < ue; ++i) {
    const int kb0 = i * PG + kh * 32;
    __syncthreads();  // the last page is read
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int x = it * 256 + tid;
      *reinterpret_cast<i32x4*>(ks + la_at<RS>(x / CK, x % CK)) = pk[it];
    }
    __syncthreads();
    if (i + 1 < ue) fetch(i + 1);
    f32x16 s = f32x16{};
#pragma unroll
    for (int k = 0; k < NKS; ++k)
      s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(ks + la_at<RS>(kh * 32 + r32, 2 * k + h)),
                                                 qf[k], s, 0, 0, 0);
    if (kb0 + 31 > q_min) {
#pragma unroll
      for (int e = 0; e < 16; ++e)
        if (kb0 + (e & 3) + 8 * (e >> 2) + 4 * h > q_abs) s[e] = -INFINITY;
    }
    float mx = -INFINITY;
#pragma unroll
    for (int e = 0; e < 16; ++e) mx = fmaxf(mx, s[e]);
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (h == 0) red[wave * 32 + r32] = mx;
    __syncthreads();
    const float n0 = fmaxf(m0, fmaxf(red[r32], red[32 + r32]) * sc), n1 = fmaxf(m1, fmaxf(red[64 + r32], red[96 + r32]) * sc);
    const float u0 = n0 == -INFINITY ? 0.f : n0, u1 = n1 == -INFINITY ? 0.f : n1;
    const float a0 = __builtin_amdgcn_exp2f(m0 - u0), a1 = __builtin_amdgcn_exp2f(m1 - u1);
    m0 = n0, m1 = n1;
    const float mu = rh == 0 ? u0 : u1;
    float rs = 0.f;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      s[e] = __builtin_amdgcn_exp2f(fmaf(s[e], sc, -mu));
      rs += s[e];
    }
    rs += __shfl_xor(rs, 32, 64);
    l_i = fmaf(l_i, rh == 0 ? a0 : a1, rs);
#pragma unroll
    for (int x = 0; x < 2; ++x)
      *reinterpret_cast<uint4*>(ps + (wave * 2 + x) * 1024 + lane * 16) =
          make_uint4(pack2bf(s[8 * x], s[8 * x + 1]), pack2bf(s[8 * x + 2], s[8 * x + 3]), pack2bf(s[8 * x + 4], s[8 * x + 5]),
                     pack2bf(s[8 * x + 6], s[8 * x + 7]));
    __syncthreads();
    if (!__all(a0 == 1.f && a1 == 1.f)) {
#pragma unroll
      for (int j = 0; j < NC; ++j) {
        o[0][j] *= a0;
        o[1][j] *= a1;
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {  // 16 keys each
      const bf16x8 f0 = *reinterpret_cast<const bf16x8*>(ps + x * 1024 + lane * 16);
      const bf16x8 f1 = *reinterpret_cast<const bf16x8*>(ps + (4 + x) * 1024 + lane * 16);
#pragma unroll
      for (int j = 0; j < NC; ++j) {
        const bf16x8 vf = la_tr<RS>(ks, x, (wave * NC + j) * 32, lane);
        o[0][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, f0, o[0][j], 0, 0, 0);
        o[1][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, f1, o[1][j], 0, 0, 0);
      }
    }
  }
  __syncthreads();
  if (h == 0) red[wave * 32 + r32] = l_i;
  __syncthreads();
#pragma unroll
  for (int x = 0; x < 2; ++x) {
    const int rw = row0 + x * 32 + r32;
    if (rw >= n * a.H) continue;
    const int tok = tok0 + rw / a.H, hd = rw % a.H;
    const float l = red[x * 64 + r32] + red[x * 64 + 32 + r32];
    if (ns > 1) {
      float* d = ws + (((size_t)(blockIdx.x / per_token) * a.H + hd) * ns + blockIdx.y) * (CP + 2);
      if (wave == 0 && h == 0) {
        d[0] = x == 0 ? m0 : m1;
        d[1] = l;
      }
#pragma unroll
      for (int j = 0; j < NC; ++j)
#pragma unroll
        for (int e = 0; e < 16; ++e) d[2 + (wave * NC + j) * 32 + (e & 3) + 8 * (e >> 2) + 4 * h] = o[x][j][e];
      continue;
    }
    const float f = (l > 0.f ? 1.f / l : 0.f) * la_gate(a, tok, hd);
    bf16_t* op = reinterpret_cast<bf16_t*>(a.out) + (size_t)tok * a.ldo + hd * CP + wave * NC * 32 + 4 * h;
#pragma unroll
    for (int j = 0; j < NC; ++j)
#pragma unroll
      for (int q = 0; q < 4; ++q)
        *reinterpret_cast<uint2*>(op + j * 32 + 8 * q) =
            make_uint2(pack2bf(o[x][j][4 * q] * f, o[x][j][4 * q + 1] * f), pack2bf(o[x][j][4 * q + 2] * f, o[x][j][4 * q + 3] * f));
  }
}

// grid (tokens * H, CP / 128): a wave takes every fourth split of 128 columns
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentAttnArgs a, const int4* __restrict__ tiles, int per_token,
                                                             int ns, const float* __restrict__ ws) {
  __shared__ float acc[4][130];
  const int e = blockIdx.x / a.H, head = blockIdx.x % a.H, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = tiles[(size_t)e * per_token].x, c0 = blockIdx.y * 128;
  const float* d = ws + ((size_t)e * a.H + head) * ns * (a.CP + 2);
  float m = -INFINITY;
  for (int s = lane; s < ns; s += 64) m = fmaxf(m, d[(size_t)s * (a.CP + 2)]);
  m = wave_max(m);
  float l = 0.f, v[2] = {0.f, 0.f};
  for (int s = wave; s < ns; s += 4) {
    const float* q = d + (size_t)s * (a.CP + 2);
    const float f = q[0] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(q[0] - m);
    l = fmaf(q[1], f, l);
    v[0] = fmaf(q[2 + c0 + lane], f, v[0]);
    v[1] = fmaf(q[2 + c0 + 64 + lane], f, v[1]);
  }
  acc[wave][lane] = v[0];
  acc[wave][64 + lane] = v[1];
  if (lane == 0) acc[wave][128] = l;
  __syncthreads();
  const int c = threadIdx.x;
  if (c >= 128) return;
  l = acc[0][128] + acc[1][128] + acc[2][128] + acc[3][128];
  const float o = acc[0][c] + acc[1][c] + acc[2][c] + acc[3][c];
  reinterpret_cast<bf16_t*>(a.out)[(size_t)row * a.ldo + head * a.CP + c0 + c] =
      f2bf((l > 0.f ? o / l : 0.f) * la_gate(a, row, head));
}

// ---------------------------------------------------------------- fp32
constexpr int LA_DK_MAX = 640;

__global__ __launch_bounds__(256) void latent_attn_f32_kernel(LatentAttnArgs a) {
  __shared__ float qs[4][LA_DK_MAX], ps[4][PG];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, DK = a.CP + a.RP;
  const int x = min((int)(blockIdx.x * 4 + wave), a.M * a.H - 1);  // surplus waves repeat the last row
  const int row = x / a.H, head = x % a.H, slot = a.slots[row], p = a.pos[row];
  const float* ql = reinterpret_cast<const float*>(a.qlat) + (size_t)row * a.ldql + head * a.CP;
  const float* qr = reinterpret_cast<const float*>(a.qrot) + (size_t)row * a.ldqr + head * a.hs;
  for (int d = lane; d < DK; d += 64) qs[wave][d] = d < a.CP ? ql[d] : qr[d - a.CP];
  __syncthreads();
  float m = -INFINITY, l = 0.f, o[8];
#pragma unroll
  for (int c = 0; c < 8; ++c) o[c] = 0.f;
  for (int blk = 0; blk <= p / PG; ++blk) {
    const int page = la_page(a.table, a.ldt, a.npages, slot, blk);
    if (page < 0) continue;
    const float* kb = reinterpret_cast<const float*>(a.kp) + (size_t)page * PG * DK;
    float s = -INFINITY;
    if (blk * PG + lane <= p) {
      s = 0.f;
      for (int d = 0; d < DK; d += 4) {
        const f32x4 k4 = *reinterpret_cast<const f32x4*>(kb + (size_t)lane * DK + d);
#pragma unroll
        for (int i = 0; i < 4; ++i) s = fmaf(k4[i], qs[wave][d + i], s);
      }
      s *= a.scale;
    }
    const float m_new = fmaxf(m, wave_max(s));
    const float alpha = expf(m - m_new), pr = expf(s - m_new);
    l = l * alpha + wave_sum(pr);
    m = m_new;
    ps[wave][lane] = pr;
    __builtin_amdgcn_wave_barrier();
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int c = 0; c < 8; ++c) {
      const int d = lane + 64 * c;
      if (d >= a.CP) break;
      float v = o[c] * alpha;
      for (int j = 0; j < PG; ++j) v = fmaf(ps[wave][j], kb[(size_t)j * DK + d], v);
      o[c] = v;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }
  float f = l > 0.f ? 1.f / l : 0.f;
  if (a.gate != nullptr) f *= 1.0f / (1.0f + expf(-reinterpret_cast<const float*>(a.gate)[(size_t)row * a.ldg + head]));
  float* op = reinterpret_cast<float*>(a.out) + (size_t)row * a.ldo + head * a.CP;
#pragma unroll
  for (int c = 0; c < 8; ++c)
    if (lane + 64 * c < a.CP) op[lane + 64 * c] = o[c] * f;
}

}  // namespace dnn

using namespace dnn;

extern "C" int dnn_rope_rows(void* x, int ld, int hs, int M, int H, int RP, const int* pos, const RopeTable* r, int f32,
                             hipStream_t st) {
  const int e = f32 ? 4 : 8;
  if (M <= 0 || H <= 0 || RP % 8 != 0 || hs < RP || hs % e != 0 || ld % e != 0 || ld < (H - 1) * hs + RP || r->pairs < 1 ||
      2 * r->pairs > RP || ((uintptr_t)x & 15) != 0)
    return -1;
  const long n = ((long)M * H * ((2 * r->pairs + e - 1) / e) + 255) / 256;
  if (n > 0x7fffffff) return -1;
  if (f32) hipLaunchKernelGGL(rope_rows_kernel<float>, dim3((unsigned)n), dim3(256), 0, st, (float*)x, ld, hs, M, H, RP, pos, *r);
  else hipLaunchKernelGGL(rope_rows_kernel<bf16_t>, dim3((unsigned)n), dim3(256), 0, st, (bf16_t*)x, ld, hs, M, H, RP, pos, *r);
  return (int)hipGetLastError();
}

extern "C" int dnn_latent_prep(const LatentPrepArgs* a, int f32, hipStream_t st) {
  const int e = f32 ? 4 : 8;
  if (a->M <= 0 || (a->QP | a->CP | a->RP | a->ld) % e != 0 || a->ld < a->QP + a->CP + a->RP || a->QN <= 0 || a->QN > a->QP ||
      a->CN <= 0 || a->CN > a->CP || a->rope.pairs < 1 || 2 * a->rope.pairs > a->RP || a->ldt <= 0 || a->npages <= 0)
    return -1;
  if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(a->M), dim3(256), 0, st, *a);
  else hipLaunchKernelGGL(latent_prep_kernel<bf16_t>, dim3(a->M), dim3(256), 0, st, *a);
  return (int)hipGetLastError();
}

static bool la_ok(const LatentAttnArgs& a, int e) {
  return a.M > 0 && a.H > 0 && (a.CP == 128 || a.CP == 256 || a.CP == 512) && (a.RP == 64 || a.RP == 128) &&
         (a.ldql | a.ldqr | a.hs) % e == 0 && a.ldql >= a.H * a.CP && a.hs >= a.RP && a.ldqr >= (a.H - 1) * a.hs + a.RP &&
         a.ldo % 4 == 0 && a.ldo >= a.H * a.CP && (a.gate == nullptr || a.ldg >= a.H) && a.ldt > 0 && a.npages > 0 &&
         (((uintptr_t)a.qlat | (uintptr_t)a.qrot | (uintptr_t)a.kp | (uintptr_t)a.out) & 15) == 0 && a.scale > 0.f &&
         a.table != nullptr && a.slots != nullptr && a.pos != nullptr;
}

extern "C" int dnn_latent_attn(const LatentAttnArgs* a, const int* tiles, int ntiles, int splits, int per_token, float* ws,
                               long long ws_elems, hipStream_t st) {
  if (!la_ok(*a, 8) || ntiles <= 0 || splits < 1 || splits > 256 || per_token < 1 || ntiles % per_token != 0 ||
      ((uintptr_t)tiles & 15) != 0)
    return -1;
  const int tokens = ntiles / per_token;
  if (splits > 1 && (ws == nullptr || per_token != (a->H + 63) / 64 || (long)tokens * a->H > 0x7fffffff ||
                     ws_elems < (long long)tokens * a->H * splits * (a->CP + 2)))
    return -1;
  const dim3 grid(ntiles, splits);
#define LA(C, R) hipLaunchKernelGGL((latent_attn_kernel<C, R>), grid, dim3(256), (LaLds<C, R>::TOTAL), st, *a, (const int4*)tiles, per_token, ws)
  if (a->RP == 64) {
    if (a->CP == 128) LA(128, 64);
    else if (a->CP == 256) LA(256, 64);
    else LA(512, 64);
  } else {
    if (a->CP == 128) LA(128, 128);
    else if (a->CP == 256) LA(256, 128);
    else LA(512, 128);
  }
#undef LA
  if (splits > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)(tokens * a->H), a->CP / 128), dim3(256), 0, st, *a,
                       (const int4*)tiles, per_token, splits, ws);
  return (int)hipGetLastError();
}

extern "C" int dnn_latent_attn_f32(const LatentAttnArgs* a, hipStream_t st) {
  if (!la_ok(*a, 4)) return -1;
  hipLaunchKernelGGL(latent_attn_f32_kernel, dim3((unsigned)(((long)a->M * a->H + 3) / 4)), dim3(256), 0, st, *a);
  return (int)hipGetLastError();
}
