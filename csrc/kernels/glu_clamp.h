// Constants of the clamped gated activation (ACT_CLAMP_MUL, gemm_epilogue.h):
//   g = min(gate, limit), u = clamp(up, -limit, limit), y = g sigmoid(alpha g) (u + shift)
#pragma once

struct GluClamp {
  float limit = 0.f, alpha = 0.f, shift = 0.f;
};
