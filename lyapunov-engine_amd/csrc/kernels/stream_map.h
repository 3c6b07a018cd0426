// What a branch reads of the residual stream when every feature is worked out
// by itself (no sum over the row): the value as it is, or bent through a tanh,
//     out = v        or        out = tanh(alpha v) * w + b.
// Being feature by feature it can be the last step of whatever kernel forms v:
// the row kernel in stream_rows.hip, a product of few rows (gemm.hip), the
// weighted sum of a token's experts (moe.hip).
#pragma once

#include "common.h"

namespace lyp {

enum StreamMapKind : int { kMapCopy = 0, kMapTanh = 1 };

struct StreamMap {
  int kind;
  float alpha;
  const float* w;   // kMapTanh: one per feature
  const float* b;
};

__device__ __forceinline__ float map_feature(int kind, float alpha, float v, float w, float b) {
  return kind == kMapTanh ? tanhf(alpha * v) * w + b : v;
}

// A logit after its product: scaled, then bent so that it stays within +- cap (cap 0: not bent).
__device__ __forceinline__ float shaped_logit(float z, float scale, float cap) {
  z *= scale;
  return cap > 0.f ? cap * tanhf(z / cap) : z;
}

inline bool stream_map_ok(const StreamMap& m) {
  return m.kind == kMapCopy || (m.kind == kMapTanh && m.w != nullptr && m.b != nullptr);
}

}  // namespace lyp
