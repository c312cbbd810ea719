// How a gated feed-forward makes one value of a gate value g and an up value u:
//   0 silu(g) u;   1 gelu(g) u in gelu's tanh form, 0.5 g (1 + tanh(sqrt(2 / pi) (g + 0.044715 g^3)));   2 relu(g) u;
//   3 with g' = min(g, limit) and u' = u held between -limit and limit: g' sigmoid(slope g') (u' + 1).
// limit and slope are read by kind 3 only.
#pragma once
#include "common.h"

namespace atoma {

constexpr int kGateKinds = 4;

struct GateAct {
  int kind;
  float limit, slope;
};

__device__ __forceinline__ float gated(float g, float u, const GateAct& act) {
  if (act.kind == 1) return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
  if (act.kind == 2) return fmaxf(g, 0.f) * u;
  if (act.kind == 3) {
    const float gc = fminf(g, act.limit), uc = fminf(fmaxf(u, -act.limit), act.limit);
    return gc / (1.0f + expf(-act.slope * gc)) * (uc + 1.0f);
  }
  return g / (1.0f + expf(-g)) * u;
}

inline bool gate_act_ok(int kind, float limit) { return kind >= 0 && kind < kGateKinds && (kind != 3 || limit > 0.f); }

}  // namespace atoma
