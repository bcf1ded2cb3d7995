// What the recurrences with a matrix per head share: the functions that make decays, and how a
// column of the state [d] is spread over KS neighbouring lanes of a wave, R rows a lane, in groups
// of four: rows 4 (j KS + s) .. + 3 for j = 0 .. R / 4 - 1.  In memory a head's matrix lies column
// by column.
#pragma once
#include "common.h"

__device__ __forceinline__ float la_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float la_softplus(float x) {
  return x > 20.f ? x : log1pf(expf(x));
}

// the r-th of a lane's rows
template <int KS>
__device__ __forceinline__ int la_row(int s, int r) { return 4 * ((r / 4) * KS + s) + r % 4; }

template <int KS>
__device__ __forceinline__ float ks_sum(float v) {
  if (KS >= 2) v += dpp_move<0xB1>(v);      // quad_perm [1, 0, 3, 2]
  if (KS >= 4) v += dpp_move<0x4E>(v);      // quad_perm [2, 3, 0, 1]
  if (KS >= 8) v += dpp_move<0x141>(v);     // the other quad of a half row (row_half_mirror)
  if (KS >= 16) v += dpp_move<0x140>(v);    // the other half of a row (row_mirror)
  if (KS >= 32) v += lane_xor16(v);
  if (KS >= 64) v += lane_xor32(v);
  return v;
}

template <int KS, int R>
__device__ __forceinline__ void la_load_rows(const float* __restrict__ st, int s, int d,
                                             bool carry, float (&S)[R]) {
#pragma unroll
  for (int r = 0; r < R; ++r) S[r] = 0.f;
  if (!carry) return;
  if (d % 4 == 0) {
#pragma unroll
    for (int r4 = 0; r4 < R; r4 += 4) {
      const int row = la_row<KS>(s, r4);
      if (row < d) {
        const float4 x = *reinterpret_cast<const float4*>(st + row);
        S[r4] = x.x; S[r4 + 1] = x.y; S[r4 + 2] = x.z; S[r4 + 3] = x.w;
      }
    }
  } else {
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (la_row<KS>(s, r) < d) S[r] = st[la_row<KS>(s, r)];
  }
}

template <int KS, int R>
__device__ __forceinline__ void la_store_rows(float* __restrict__ st, int s, int d,
                                              const float (&S)[R]) {
  if (d % 4 == 0) {
#pragma unroll
    for (int r4 = 0; r4 < R; r4 += 4) {
      const int row = la_row<KS>(s, r4);
      if (row < d)
        *reinterpret_cast<float4*>(st + row) =
            make_float4(S[r4], S[r4 + 1], S[r4 + 2], S[r4 + 3]);
    }
  } else {
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (la_row<KS>(s, r) < d) st[la_row<KS>(s, r)] = S[r];
  }
}
