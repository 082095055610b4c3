// Chain over the chunks of linear recurrences whose transition is diagonal in the key index (plain
// writes): init_{c+1} = decay_c * init_c + local_c.  One thread per state element walks its
// portion's chunks; init_c replaces local_c in `cs` [chunks, H, D, V], the end goes to the slot.
// decay [chunks, H, D]; cent: per portion (first chunk, chunks, first position, slot).
#pragma once
#include "common.h"

namespace sm {

static __global__ void __launch_bounds__(256)
diag_chain_k(float* __restrict__ cs, const float* __restrict__ decay, float* __restrict__ state,
             const int* __restrict__ cent, int H, int D, int V) {
  const int e = blockIdx.y / H, h = blockIdx.y % H;
  const int idx = blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= D * V) return;
  const int i = idx / V;
  const int c0 = cent[4 * e], nc = cent[4 * e + 1], start = cent[4 * e + 2], slot = cent[4 * e + 3];
  float* sg = state + ((size_t)slot * H + h) * D * V + idx;
  float cur = start > 0 ? *sg : 0.0f;
  float* q = cs + ((size_t)c0 * H + h) * D * V + idx;
  const float* dq = decay + ((size_t)c0 * H + h) * D + i;
  const size_t step = (size_t)H * D * V, dstep = (size_t)H * D;
  for (int k = 0; k < nc; k += 8) {
    float loc[8], dec[8];   // eight chunks' loads in flight
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int kk = min(k + u, nc - 1);
      loc[u] = q[kk * step];
      dec[u] = dq[kk * dstep];
    }
#pragma unroll
    for (int u = 0; u < 8; u++)
      if (k + u < nc) {
        q[(k + u) * step] = cur;
        cur = dec[u] * cur + loc[u];
      }
  }
  *sg = cur;
}

}  // namespace sm
