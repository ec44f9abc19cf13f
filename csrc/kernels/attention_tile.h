// Pieces of the flash-attention kernels over 64-key tiles staged in LDS
// (paged_attention.hip, latent_attention.hip): S^T = K Q^T by the 32x32x16 MFMA
// keeps a query on one lane pair, P stays in the score registers, V^T comes by
// transposing LDS reads.
#pragma once
#include "common.h"

namespace dnn {

typedef short s16x4 __attribute__((ext_vector_type(4)));

constexpr int PG = 64;  // keys per page
constexpr float LOG2E = 1.4426950408889634f;

template <int D>
__device__ __forceinline__ int pa_swz(int key, int chunk) {  // 16-B chunk of a K row in LDS
  return D == 64 ? (chunk ^ ((key >> 1) & 7)) : (chunk ^ (key & 15));
}
template <int DV>
struct PaV {
  static constexpr int STRIDE = DV * 2 + 64;  // padded rows: conflict-free transposing reads
};

// Online softmax of 16 score registers per 32-key tile (NT tiles); returns the
// rescale of what was accumulated so far.  sc: scale * log2(e).
template <int NT>
__device__ __forceinline__ float pa_softmax(f32x16 (&s)[NT], float sc, float& m_i, float& l_i) {
  float mx = -INFINITY;
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int g = 0; g < 16; g += 2) mx = fmax_nan(mx, fmax_nan(s[t][g], s[t][g + 1]));
  mx = fmax_nan(mx, __shfl_xor(mx, 32, 64));
  const float m_new = fmax_nan(m_i, mx * sc);
  const float m_use = m_new == -INFINITY ? 0.f : m_new;
  const float alpha = __builtin_amdgcn_exp2f(m_i - m_use);
  float rs = 0.f;
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int g = 0; g < 16; ++g) {
      s[t][g] = __builtin_amdgcn_exp2f(fmaf(s[t][g], sc, -m_use));
      rs += s[t][g];
    }
  rs += __shfl_xor(rs, 32, 64);
  l_i = fmaf(l_i, alpha, rs);
  m_i = m_new;
  return alpha;
}

// O^T += V^T P^T for one 32-key tile staged at vbuf (row 0 = the tile's first key).
template <int DV>
__device__ __forceinline__ void pa_pv(const char* vbuf, const f32x16& p, f32x16 (&o)[DV / 32], int lane) {
  const int h = lane >> 5;
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    bf16x8 pf;
#pragma unroll
    for (int j = 0; j < 8; ++j) pf[j] = (short)f2bf(p[8 * s + j]);
    const int krow = 16 * s + 4 * h + ((lane & 15) >> 2);
    const int gsub = (lane >> 4) & 1;
#pragma unroll
    for (int dt = 0; dt < DV / 32; ++dt) {
      const char* a0 = vbuf + krow * PaV<DV>::STRIDE + (dt * 32 + gsub * 16 + 4 * (lane & 3)) * 2;
      const s16x4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(a0));
      const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(a0 + 8 * PaV<DV>::STRIDE));
      const bf16x8 vf = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
      o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf, o[dt], 0, 0, 0);
    }
  }
}

}  // namespace dnn
