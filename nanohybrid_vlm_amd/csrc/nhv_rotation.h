// The angle by which a pair of entries is turned at a position: position * frequency, the frequency a double. The product is
// taken and brought into [-pi, pi] in double (a float product of a position in the thousands is off by 1e-4 of a turn).
#pragma once
#include "nhv_common.h"

// The sine and cosine are float's own for float rows; for bfloat16 rows, whose rounding is a thousand times coarser, they
// are the hardware's (which takes turns).
template <typename T>
__device__ __forceinline__ void nhv_turn_angle(int pos, double f, float gain, float* sn, float* cs) {
  const double a = (double)pos * f;
  const double turns = a * 0.15915494309189535;
  if (sizeof(T) == 2) {
    const float part = (float)(turns - rint(turns));
    *sn = __builtin_amdgcn_sinf(part) * gain;
    *cs = __builtin_amdgcn_cosf(part) * gain;
    return;
  }
  sincosf((float)(a - rint(turns) * 6.283185307179586), sn, cs);
  *sn *= gain;
  *cs *= gain;
}
