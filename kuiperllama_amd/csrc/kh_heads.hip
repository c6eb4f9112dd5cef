// kh_heads.hip — launcher and instantiations of the attention over grouped heads (kh_heads.h).
#include <vector>

#include "kh_heads.h"

namespace khm {

template <class T>
int heads_attn_launch(hipStream_t s, HeadsArgs a, int ntiles, int rows) {
  if (a.dkp % 64 || a.dvp % 64 || a.dkp > KH_HEADS_MAX_DIM || a.dvp > KH_HEADS_MAX_DIM || a.dkr > a.dkp || a.dvr > a.dvp ||
      a.dkr % 16 || a.dvr % 16 || a.ldr % 16 || a.G <= 0 || a.H % a.G || a.ring <= 0 || a.nsplit < 1 || ntiles <= 0)
    return KH_ERR_INTERNAL;
  const size_t table = (size_t)(a.H / a.G) * a.nbias * sizeof(float);
  a.bias_lds = a.bias && table <= KH_HEADS_BIAS_LDS;
  auto go = [&](auto kern, size_t stage) -> int {
    const size_t lds = stage * (stage <= 24 * 1024 ? 3 : 2) + (a.bias_lds ? table : 0);
    if (lds > 64 * 1024) {
      struct Done { int dev; const void* fn; size_t lds; };
      static thread_local std::vector<Done> done;
      int dev = 0;
      (void)hipGetDevice(&dev);
      bool hit = false;
      for (const auto& d : done) hit = hit || (d.dev == dev && d.fn == (const void*)kern && d.lds >= lds);
      if (!hit) {
        const hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        done.push_back({dev, (const void*)kern, lds});
      }
    }
    hipLaunchKernelGGL(kern, dim3(a.G, ntiles, a.nsplit), dim3(256), lds, s, a);
    return KH_OK;
  };
  auto by_rows = [&](auto kn, auto kv) -> int {
    constexpr int KN = decltype(kn)::value, KV = decltype(kv)::value;
    const size_t stage = (size_t)4 * Tile<T>::N * (a.dkp + a.dvp) * sizeof(T);
    if (rows == 16) return go(k_heads_attn<T, KN, KV, 4, 1>, stage);
    if (rows == 64) return go(k_heads_attn<T, KN, KV, 1, 1>, stage);
    if constexpr (sizeof(T) == 2 && KN <= 2 && KV <= 2)
      if (rows == 128) return go(k_heads_attn<T, KN, KV, 1, 2>, stage);
    return KH_ERR_INTERNAL;
  };
  auto by_value = [&](auto kn) -> int {
    switch (a.dvp / 64) {
      case 1: return by_rows(kn, std::integral_constant<int, 1>());
      case 2: return by_rows(kn, std::integral_constant<int, 2>());
      case 3: return by_rows(kn, std::integral_constant<int, 3>());
      default: return by_rows(kn, std::integral_constant<int, 4>());
    }
  };
  switch (a.dkp / 64) {
    case 1: return by_value(std::integral_constant<int, 1>());
    case 2: return by_value(std::integral_constant<int, 2>());
    case 3: return by_value(std::integral_constant<int, 3>());
    default: return by_value(std::integral_constant<int, 4>());
  }
}
template int heads_attn_launch<bf16>(hipStream_t, HeadsArgs, int, int);
template int heads_attn_launch<float>(hipStream_t, HeadsArgs, int, int);

}  // namespace khm
