// router_device.h — the choice of experts that the sequence models' router launches share.
#pragma once
#include "common.h"

// One wave: `top` rounds of arg-max over z[0 .. E) (ties: the lower index), then the softmax over the chosen logits (SIGMOID: every chosen
// logit's sigmoid as it is).  Lane l owns the logits l, l + 64, ... and a bit per owned logit that says it has been chosen (E <= 4096).
template <bool SIGMOID>
__device__ __forceinline__ void wave_topk(const float* z, int E, int top, int lane, int32_t* ir, float* wr) {
  uint64_t taken = 0;
  float first = 0.f, sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane, i = 0; e < E; e += 64, ++i) {
      const float v = z[e];
      if (!((taken >> i) & 1) && (v > best || (v == best && e < bi) || bi == 0x7fffffff)) { best = v; bi = e; }
    }
    for (int off = 32; off >= 1; off >>= 1) {
      const float ob = __shfl_xor(best, off);
      const int oi = __shfl_xor(bi, off);
      if (oi != 0x7fffffff && (bi == 0x7fffffff || ob > best || (ob == best && oi < bi))) { best = ob; bi = oi; }
    }
    if ((bi & 63) == lane) taken |= (uint64_t)1 << (bi >> 6);
    if (k == 0) first = best;
    const float p = SIGMOID ? 1.0f / (1.0f + expf(-best)) : expf(best - first);
    sum += p;
    if (lane == 0) { ir[k] = bi; wr[k] = p; }
  }
  if (SIGMOID) return;
  // lane 0 wrote the unnormalised weights and is the one that scales them
  if (lane == 0)
    for (int k = 0; k < top; ++k) wr[k] = wr[k] / sum;
}
