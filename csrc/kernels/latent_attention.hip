// Attention over a latent cache, for batches of unequal sequences (gfx950).
//
// The cache holds one row per token for all heads, [page][64][CP + RP]: a normed
// latent of CP columns and a rotated key part of RP.  A head's unrotated key and
// its value are linear in the latent.  Two ways to score:
//   over latents   the key projection is moved to the query (q . W_uk c =
//                  (W_uk^T q) . c) and the value projection behind the softmax:
//                  every head reads whole cache rows and sums their latents.
//                  Single tokens, short portions
//   over keys      the sequence's cache rows are gathered and projected to the
//                  heads' keys and values first: fewer operations per score
//                  where many queries share them.  Long portions
//
//   latent_prep      norms of the query's and the cache's latent, rotation of the
//                    shared key part, cache write
//   rope_rows        rotation of every head's rotated part, in place
//   latent_attn      bf16, over latents; a workgroup takes 32 or 64 packed (token,
//                    head) rows and walks the pages.  Its 8 waves take a part each
//                    of keys, rows and columns of the scores, then a part of the
//                    latent columns.  Single tokens may be split over workgroups
//                    (then a combine)
//   latent_gather    cache pages -> rows
//   latent_prefill   bf16, over keys; a workgroup takes 128 tokens of a head
//   latent_attn_f32  fp32, one wave per (row, head): the exact mode
//
// Scores, softmax and accumulation are fp32.
#include "attention_tile.h"
#include "residual_api.h"
#include "vec16.h"

namespace dnn {

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

// ---------------------------------------------------------------- over latents
// ROWS packed rows and 64 keys of a page, 8 waves.  Scores: wave (kh, rh, kq) of
// 2 key halves x RH row halves x KQ parts of the columns; the parts are summed
// through LDS, where each wave of a group ends with EN of the 16 keys of a lane.
template <int CP, int RP, int ROWS>
struct LaTile {
  static constexpr int DK = CP + RP, RH = ROWS / 32, KQ = 4 / RH, EN = 16 / KQ;
  static constexpr int RS = (DK * 2 + 255) / 256 * 256;  // bytes of a key row: whole groups of 16 pieces
  static constexpr int NK = DK / 16 / KQ;                // MFMA steps of a wave's part
  static constexpr int NI = PG * (DK / 8) / 512;         // 16-byte pieces of a page per thread
  static constexpr int NC = CP >= 256 ? CP / 256 : 1;    // 32-column groups of the latent per wave
  static constexpr int O_X = PG * RS, O_P = O_X + 8 * 4 * 1024, O_R = O_P + RH * 4 * 1024;
  static constexpr int TOTAL = O_R + 8 * 32 * 4;
  static_assert(DK % (16 * KQ) == 0 && PG * (DK / 8) % 512 == 0, "tile");
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

constexpr int LA_WS = 4;  // floats of a partial before its columns: {max, sum, -, -}

// grid (tiles, splits); tiles: {first batch row, tokens, slot, first packed row}.
// With splits the tiles are single tokens, per_token tiles each, and
// ws = [token][H][splits][LA_WS + CP] takes the partials.
template <int CP, int RP, int ROWS>
__global__ __launch_bounds__(512, 1) void latent_attn_kernel(LatentAttnArgs a, const int4* __restrict__ tiles,
                                                             int per_token, float* __restrict__ ws) {
  using L = LaTile<CP, RP, ROWS>;
  constexpr int DK = L::DK, RS = L::RS, CK = DK / 8, RH = L::RH, KQ = L::KQ, EN = L::EN, NK = L::NK, NI = L::NI, NC = L::NC;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ks = smem;
  char* xs = smem + L::O_X;
  char* ps = smem + L::O_P;
  float* red = reinterpret_cast<float*>(smem + L::O_R);  // [wave][32]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = lane >> 5, r32 = lane & 31;
  const int kh = wave & 1, rh = (wave >> 1) & (RH - 1), kq = wave / (2 * RH), ns = gridDim.y;
  const int4 t = tiles[blockIdx.x];
  const int tok0 = t.x, n = t.y, slot = t.z, row0 = t.w, last = n - 1;
  const int p0 = a.pos[tok0];
  const int row = row0 + rh * 32 + r32, tk = min(row / a.H, last), head = row % a.H, q_abs = p0 + tk;
  const int q_min = p0 + min((row0 + rh * 32) / a.H, last);
  const int total = (p0 + min((row0 + ROWS - 1) / a.H, last)) / PG + 1;
  const int ub = (int)((long)total * blockIdx.y / ns), ue = (int)((long)total * (blockIdx.y + 1) / ns);

  i32x4 pk[NI];
  auto fetch = [&](int i) __attribute__((always_inline)) {
    const int page = max(la_page(a.table, a.ldt, a.npages, slot, i), 0);  // a missing page is never visible; stay in the pool
    const bf16_t* kb = reinterpret_cast<const bf16_t*>(a.kp) + (size_t)page * PG * DK;
#pragma unroll
    for (int it = 0; it < NI; ++it) pk[it] = *reinterpret_cast<const i32x4*>(kb + (it * 512 + tid) * 8);
  };
  if (ub < ue) fetch(ub);
  bf16x8 qf[NK];
  {
    const bf16_t* ql = reinterpret_cast<const bf16_t*>(a.qlat) + (size_t)(tok0 + tk) * a.ldql + head * CP + 8 * h;
    const bf16_t* qr = reinterpret_cast<const bf16_t*>(a.qrot) + (size_t)(tok0 + tk) * a.ldqr + head * a.hs + 8 * h;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int k = kq * NK + s;
      qf[s] = *reinterpret_cast<const bf16x8*>(k < CP / 16 ? ql + k * 16 : qr + (k - CP / 16) * 16);
    }
  }
  f32x16 o[RH][NC];
  float m[RH], l_i = 0.f;
#pragma unroll
  for (int i = 0; i < RH; ++i) {
    m[i] = -INFINITY;
#pragma unroll
    for (int j = 0; j < NC; ++j) o[i][j] = f32x16{};
  }
  const float sc = a.scale * LOG2E;
  const bool has_cols = wave * NC * 32 < CP;

  for (int i = ub; i < ue; ++i) {
    __syncthreads();  // the last page is read
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int x = it * 512 + tid;
      *reinterpret_cast<i32x4*>(ks + la_at<RS>(x / CK, x % CK)) = pk[it];
    }
    __syncthreads();
    if (i + 1 < ue) fetch(i + 1);
    {
      f32x16 s = f32x16{};
#pragma unroll
      for (int k = 0; k < NK; ++k)
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
            *reinterpret_cast<const bf16x8*>(ks + la_at<RS>(kh * 32 + r32, 2 * (kq * NK + k) + h)), qf[k], s, 0, 0, 0);
#pragma unroll
      for (int q = 0; q < 4; ++q)
        *reinterpret_cast<f32x4*>(xs + (wave * 4 + q) * 1024 + lane * 16) = f32x4{s[4 * q], s[4 * q + 1], s[4 * q + 2], s[4 * q + 3]};
    }
    __syncthreads();
    float s[EN];
#pragma unroll
    for (int q = 0; q < EN / 4; ++q) {
      f32x4 z = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < KQ; ++w)
        z += *reinterpret_cast<const f32x4*>(xs + ((w * 2 * RH + rh * 2 + kh) * 4 + kq * (EN / 4) + q) * 1024 + lane * 16);
#pragma unroll
      for (int j = 0; j < 4; ++j) s[4 * q + j] = z[j];
    }
    const int kb0 = i * PG + kh * 32 + kq * (EN / 4) * 8 + 4 * h;  // key of s[0]; s[4 q + j]: + 8 q + j
    if (i * PG + kh * 32 + 31 > q_min) {
#pragma unroll
      for (int e = 0; e < EN; ++e)
        if (kb0 + 8 * (e >> 2) + (e & 3) > q_abs) s[e] = -INFINITY;
    }
    float mx = -INFINITY;
#pragma unroll
    for (int e = 0; e < EN; ++e) mx = fmaxf(mx, s[e]);
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (h == 0) red[wave * 32 + r32] = mx;
    __syncthreads();
    float al[RH], mu = 0.f, mine = 1.f;
    bool same = true;
#pragma unroll
    for (int x = 0; x < RH; ++x) {
      float v = -INFINITY;
#pragma unroll
      for (int w = 0; w < KQ; ++w)
        v = fmaxf(v, fmaxf(red[((w * RH + x) * 2) * 32 + r32], red[((w * RH + x) * 2 + 1) * 32 + r32]));
      const float nx = fmaxf(m[x], v * sc), u = nx == -INFINITY ? 0.f : nx;
      al[x] = __builtin_amdgcn_exp2f(m[x] - u);
      m[x] = nx;
      same = same && al[x] == 1.f;
      if (x == rh) mu = u, mine = al[x];
    }
    float rs = 0.f;
#pragma unroll
    for (int e = 0; e < EN; ++e) {
      s[e] = __builtin_amdgcn_exp2f(fmaf(s[e], sc, -mu));
      rs += s[e];
    }
    rs += __shfl_xor(rs, 32, 64);
    l_i = fmaf(l_i, mine, rs);
    {  // fragment of 16 keys: this lane's 8, of which a wave has EN
      char* d = ps + ((rh * 4 + kh * 2 + kq * EN / 8) * 64 + lane) * 16;
      if constexpr (EN == 8)
        *reinterpret_cast<uint4*>(d) = make_uint4(pack2bf(s[0], s[1]), pack2bf(s[2], s[3]), pack2bf(s[4], s[5]), pack2bf(s[6], s[7]));
      else
        *reinterpret_cast<uint2*>(d + (kq & 1) * 8) = make_uint2(pack2bf(s[0], s[1]), pack2bf(s[2], s[3]));
    }
    __syncthreads();
    if (!has_cols) continue;
    if (!__all(same)) {
#pragma unroll
      for (int x = 0; x < RH; ++x)
#pragma unroll
        for (int j = 0; j < NC; ++j) o[x][j] *= al[x];
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {  // 16 keys each
      bf16x8 f[RH];
#pragma unroll
      for (int r = 0; r < RH; ++r) f[r] = *reinterpret_cast<const bf16x8*>(ps + ((r * 4 + x) * 64 + lane) * 16);
#pragma unroll
      for (int j = 0; j < NC; ++j) {
        const bf16x8 vf = la_tr<RS>(ks, x, (wave * NC + j) * 32, lane);
#pragma unroll
        for (int r = 0; r < RH; ++r) o[r][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, f[r], o[r][j], 0, 0, 0);
      }
    }
  }
  __syncthreads();
  if (h == 0) red[wave * 32 + r32] = l_i;
  __syncthreads();
#pragma unroll
  for (int x = 0; x < RH; ++x) {
    const int rw = row0 + x * 32 + r32;
    if (!has_cols || rw >= n * a.H) continue;
    const int tok = tok0 + rw / a.H, hd = rw % a.H, c0 = wave * NC * 32 + 4 * h;
    float l = 0.f;
#pragma unroll
    for (int w = 0; w < KQ; ++w) l += red[((w * RH + x) * 2) * 32 + r32] + red[((w * RH + x) * 2 + 1) * 32 + r32];
    if (ns > 1) {
      float* d = ws + (((size_t)(blockIdx.x / per_token) * a.H + hd) * ns + blockIdx.y) * (LA_WS + CP);
      if (wave == 0 && h == 0) {
        d[0] = m[x];
        d[1] = l;
      }
#pragma unroll
      for (int j = 0; j < NC; ++j)
#pragma unroll
        for (int q = 0; q < 4; ++q)
          *reinterpret_cast<f32x4*>(d + LA_WS + c0 + j * 32 + 8 * q) =
              f32x4{o[x][j][4 * q], o[x][j][4 * q + 1], o[x][j][4 * q + 2], o[x][j][4 * q + 3]};
      continue;
    }
    const float f = (l > 0.f ? 1.f / l : 0.f) * la_gate(a, tok, hd);
    bf16_t* op = reinterpret_cast<bf16_t*>(a.out) + (size_t)tok * a.ldo + hd * CP + c0;
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
  const int row = tiles[(size_t)e * per_token].x, c0 = blockIdx.y * 128, st = LA_WS + a.CP;
  const float* d = ws + ((size_t)e * a.H + head) * ns * st;
  float m = -INFINITY;
  for (int s = lane; s < ns; s += 64) m = fmaxf(m, d[(size_t)s * st]);
  m = wave_max(m);
  float l = 0.f, v[2] = {0.f, 0.f};
  for (int s = wave; s < ns; s += 4) {
    const float* q = d + (size_t)s * st;
    const float f = q[0] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(q[0] - m);
    l = fmaf(q[1], f, l);
    v[0] = fmaf(q[LA_WS + c0 + lane], f, v[0]);
    v[1] = fmaf(q[LA_WS + c0 + 64 + lane], f, v[1]);
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

// ---------------------------------------------------------------- over keys
// grid (pages, 4): 16 rows each; ent: {first row of the 64, slot, block, -}
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint4* __restrict__ kp, const int* __restrict__ table, int ldt,
                                                            int npages, const int4* __restrict__ ent, int rows, int pieces,
                                                            uint4* __restrict__ out) {
  const int4 e = ent[blockIdx.x];
  const int page = la_page(table, ldt, npages, e.y, e.z);
  const int n = min(PG, rows - e.x) * pieces, part = PG / 4 * pieces;
  const uint4* src = kp + (size_t)max(page, 0) * PG * pieces;
  uint4* dst = out + (size_t)e.x * pieces;
  for (int i = blockIdx.y * part + threadIdx.x; i < min(n, (int)(blockIdx.y + 1) * part); i += 256) dst[i] = page >= 0 ? src[i] : make_uint4(0, 0, 0, 0);
}

template <int DP, int RP, int VP>
struct LpTile {
  static constexpr int D = DP + RP, RS = (D * 2 + 255) / 256 * 256, O_V = PG * RS, TOTAL = O_V + PG * PaV<VP>::STRIDE;
};

// grid (H, tiles); tiles: {first batch row, tokens, first key row, first token}
template <int DP, int RP, int VP>
__global__ __launch_bounds__(256, DP + RP + VP > 320 ? 1 : 2) void latent_prefill_kernel(LatentKeysArgs a, const int4* __restrict__ tiles) {
  using L = LpTile<DP, RP, VP>;
  constexpr int D = L::D, RS = L::RS, NKS = D / 16, NDT = VP / 32;
  constexpr int CU = DP / 8, CR = RP / 8, CV = VP / 8, NU = PG * CU / 256, NR = PG * CR / 256, NV = PG * CV / 256;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ks = smem;
  char* vs = smem + L::O_V;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = lane >> 5, r32 = lane & 31, head = blockIdx.x;
  const int4 t = tiles[blockIdx.y];
  const int tok0 = t.x, n = t.y, key0 = t.z, last = n - 1;
  const int p0 = a.pos[tok0], w0 = t.w + wave * 32, tk = min(w0 + r32, last), q_abs = p0 + tk;
  const int q_min = p0 + min(w0, last), q_max = p0 + min(w0 + 31, last);
  const int total = (p0 + min(t.w + 127, last)) / PG + 1;
  bf16x8 qf[NKS];
  {
    const bf16_t* qp = reinterpret_cast<const bf16_t*>(a.q) + (size_t)(tok0 + tk) * a.ldq + head * D + 8 * h;
#pragma unroll
    for (int s = 0; s < NKS; ++s) qf[s] = *reinterpret_cast<const bf16x8*>(qp + s * 16);
  }
  f32x16 o[NDT];
#pragma unroll
  for (int i = 0; i < NDT; ++i) o[i] = f32x16{};
  float m_i = -INFINITY, l_i = 0.f;
  const float sc = a.scale * LOG2E;
  const bf16_t* kv = reinterpret_cast<const bf16_t*>(a.kv) + head * (DP + VP);
  const bf16_t* kr = reinterpret_cast<const bf16_t*>(a.krot);
  i32x4 pu[NU], pr[NR], pv[NV];
  auto fetch = [&](int i) __attribute__((always_inline)) {
    const int k0 = key0 + i * PG;
#pragma unroll
    for (int it = 0; it < NU; ++it) {
      const int x = it * 256 + tid;
      pu[it] = *reinterpret_cast<const i32x4*>(kv + (size_t)min(k0 + x / CU, a.keys - 1) * a.ldkv + x % CU * 8);
    }
#pragma unroll
    for (int it = 0; it < NR; ++it) {
      const int x = it * 256 + tid;
      pr[it] = *reinterpret_cast<const i32x4*>(kr + (size_t)min(k0 + x / CR, a.keys - 1) * a.ldr + x % CR * 8);
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int x = it * 256 + tid;
      pv[it] = *reinterpret_cast<const i32x4*>(kv + (size_t)min(k0 + x / CV, a.keys - 1) * a.ldkv + DP + x % CV * 8);
    }
  };
  fetch(0);
  for (int i = 0; i < total; ++i) {
    const int kb0 = i * PG;
    __syncthreads();
#pragma unroll
    for (int it = 0; it < NU; ++it) {
      const int x = it * 256 + tid;
      *reinterpret_cast<i32x4*>(ks + la_at<RS>(x / CU, x % CU)) = pu[it];
    }
#pragma unroll
    for (int it = 0; it < NR; ++it) {
      const int x = it * 256 + tid;
      *reinterpret_cast<i32x4*>(ks + la_at<RS>(x / CR, CU + x % CR)) = pr[it];
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int x = it * 256 + tid;
      *reinterpret_cast<i32x4*>(vs + x / CV * PaV<VP>::STRIDE + x % CV * 16) = pv[it];
    }
    __syncthreads();
    if (i + 1 < total) fetch(i + 1);
    if (kb0 > q_max) continue;
    f32x16 s[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      s[kt] = f32x16{};
#pragma unroll
      for (int k = 0; k < NKS; ++k)
        s[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
            *reinterpret_cast<const bf16x8*>(ks + la_at<RS>(kt * 32 + r32, 2 * k + h)), qf[k], s[kt], 0, 0, 0);
    }
    if (kb0 + PG - 1 > q_min) {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int e = 0; e < 16; ++e)
          if (kb0 + kt * 32 + (e & 3) + 8 * (e >> 2) + 4 * h > q_abs) s[kt][e] = -INFINITY;
    }
    const float alpha = pa_softmax<2>(s, sc, m_i, l_i);
    if (!__all(alpha == 1.f)) {
#pragma unroll
      for (int d = 0; d < NDT; ++d) o[d] *= alpha;
    }
    pa_pv<VP>(vs, s[0], o, lane);
    pa_pv<VP>(vs + 32 * PaV<VP>::STRIDE, s[1], o, lane);
  }
  if (w0 + r32 >= n) return;
  float f = l_i > 0.f ? 1.f / l_i : 0.f;
  if (a.gate != nullptr)
    f /= 1.0f + __expf(-bf2f(reinterpret_cast<const bf16_t*>(a.gate)[(size_t)(tok0 + tk) * a.ldg + head]));
  bf16_t* op = reinterpret_cast<bf16_t*>(a.out) + (size_t)(tok0 + tk) * a.ldo + head * VP + 4 * h;
#pragma unroll
  for (int d = 0; d < NDT; ++d)
#pragma unroll
    for (int q = 0; q < 4; ++q)
      *reinterpret_cast<uint2*>(op + d * 32 + 8 * q) =
          make_uint2(pack2bf(o[d][4 * q] * f, o[d][4 * q + 1] * f), pack2bf(o[d][4 * q + 2] * f, o[d][4 * q + 3] * f));
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

extern "C" int dnn_latent_attn(const LatentAttnArgs* a, const int* tiles, int ntiles, int rows, int splits, int per_token,
                               float* ws, long long ws_elems, hipStream_t st) {
  if (!la_ok(*a, 8) || ntiles <= 0 || (rows != 32 && rows != 64) || splits < 1 || splits > 256 || per_token < 1 ||
      ntiles % per_token != 0 || ((uintptr_t)tiles & 15) != 0)
    return -1;
  const int tokens = ntiles / per_token;
  if (splits > 1 && (ws == nullptr || ((uintptr_t)ws & 15) != 0 || per_token != (a->H + rows - 1) / rows ||
                     (long)tokens * a->H > 0x7fffffff || ws_elems < (long long)tokens * a->H * splits * (LA_WS + a->CP)))
    return -1;
  const dim3 grid(ntiles, splits);
#define LA(C, R, N)                                                                                                           \
  hipLaunchKernelGGL((latent_attn_kernel<C, R, N>), grid, dim3(512), (LaTile<C, R, N>::TOTAL), st, *a, (const int4*)tiles, \
                     per_token, ws)
#define LAR(C, R)             \
  {                           \
    if (rows == 32) LA(C, R, 32); \
    else LA(C, R, 64);        \
  }
  if (a->RP == 64) {
    if (a->CP == 128) LAR(128, 64)
    else if (a->CP == 256) LAR(256, 64)
    else LAR(512, 64)
  } else {
    if (a->CP == 128) LAR(128, 128)
    else if (a->CP == 256) LAR(256, 128)
    else LAR(512, 128)
  }
#undef LAR
#undef LA
  if (splits > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)(tokens * a->H), a->CP / 128), dim3(256), 0, st, *a,
                       (const int4*)tiles, per_token, splits, ws);
  return (int)hipGetLastError();
}

extern "C" int dnn_latent_gather(const void* kp, int cols, const int* table, int ldt, int npages, const int* ent, int nent,
                                 void* out, int rows, hipStream_t st) {
  if (cols <= 0 || cols % 8 != 0 || ldt <= 0 || npages <= 0 || nent <= 0 || rows <= 0 ||
      (((uintptr_t)kp | (uintptr_t)out | (uintptr_t)ent) & 15) != 0)
    return -1;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(nent, 4), dim3(256), 0, st, (const uint4*)kp, table, ldt, npages, (const int4*)ent,
                     rows, cols / 8, (uint4*)out);
  return (int)hipGetLastError();
}

extern "C" int dnn_latent_prefill(const LatentKeysArgs* a, const int* tiles, int ntiles, hipStream_t st) {
  const int D = a->DP + a->RP;
  if (a->M <= 0 || a->H <= 0 || a->keys <= 0 || ntiles <= 0 || ntiles > 65535 || (a->DP != 64 && a->DP != 128) ||
      (a->RP != 64 && a->RP != 128) || (a->VP != 64 && a->VP != 128) || (a->ldq | a->ldkv | a->ldr) % 8 != 0 ||
      a->ldq < a->H * D || a->ldkv < a->H * (a->DP + a->VP) || a->ldr < a->RP || a->ldo % 4 != 0 || a->ldo < a->H * a->VP ||
      (a->gate != nullptr && a->ldg < a->H) || !(a->scale > 0.f) || a->pos == nullptr ||
      (((uintptr_t)a->q | (uintptr_t)a->kv | (uintptr_t)a->krot | (uintptr_t)a->out | (uintptr_t)tiles) & 15) != 0)
    return -1;
#define LP(X, R, V)                                                                                                       \
  if (a->DP == X && a->RP == R && a->VP == V)                                                                             \
  hipLaunchKernelGGL((latent_prefill_kernel<X, R, V>), dim3(a->H, ntiles), dim3(256), (LpTile<X, R, V>::TOTAL), st, *a, \
                     (const int4*)tiles)
  LP(64, 64, 64);
  LP(64, 64, 128);
  LP(64, 128, 64);
  LP(64, 128, 128);
  LP(128, 64, 64);
  LP(128, 64, 128);
  LP(128, 128, 64);
  LP(128, 128, 128);
#undef LP
  return (int)hipGetLastError();
}

extern "C" int dnn_latent_attn_f32(const LatentAttnArgs* a, hipStream_t st) {
  if (!la_ok(*a, 4)) return -1;
  hipLaunchKernelGGL(latent_attn_f32_kernel, dim3((unsigned)(((long)a->M * a->H + 3) / 4)), dim3(256), 0, st, *a);
  return (int)hipGetLastError();
}
