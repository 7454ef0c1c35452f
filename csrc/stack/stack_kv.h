// K/V store of one (row, key/value head) by one wave, shared by the launches that carry it.
#pragma once
#include "stack_device.h"
#include "stack_ops.h"

namespace omx {
namespace stack {

// the key as it is, the value as it is or divided by its root mean square, into the row's cache slot
template <typename T>
__device__ __forceinline__ void kv_store_item(const KvStoreParams& P, const StepRows& R, int b, int g, int lane) {
  const float* k = P.proj + (long long)b * P.ld + P.off_k + g * P.D;
  const float* v = P.proj + (long long)b * P.ld + P.off_v + g * P.Dv;
  const int slot = R.slot[b];
  const long long at = ((long long)(slot / R.bs) * P.G + g) * R.bs + slot % R.bs;
  for (int d = lane; d < P.D; d += 64) st((T*)P.kc + at * P.D + d, k[d]);
  float f = 1.f;
  if (P.v_unit) {
    float ss = 0.f;
    for (int d = lane; d < P.Dv; d += 64) ss += v[d] * v[d];
    f = 1.f / sqrtf(wave_sum(ss) / (float)P.Dv + P.eps);
  }
  for (int d = lane; d < P.Dv; d += 64) st((T*)P.vc + at * P.Dv + d, v[d] * f);
}

}  // namespace stack
}  // namespace omx
