// What an attention kernel may do to a score between the scaled dot product and the softmax, and a
// sink: one more term of the softmax's denominator that has no key and no value.
//   softcap     0: nothing; else score <- softcap * tanh(score / softcap)
//   dist_bias   [heads, dist_cols] float32, added after the cap: column min(i - j, dist_cols - 1)
//               for query position i and key position j; null: nothing.  In memory a head's row
//               has KAPPAI_BIAS_PAD more columns on either side (zeros in front, the last column
//               repeated behind), so that the biases of eight keys in a row are eight neighbours
//               wherever the row begins or ends
//   sink        [heads] float32: exp(sink[h]) joins the denominator once; null: nothing
//   keep_first  the first keep_first positions of a sequence are seen by every later one, whatever
//               the window or chunk; 0: nothing is kept
#pragma once
#include <hip/hip_runtime.h>

// Which keys a position sees, as one number that every attention kernel takes in its `window`
// place: 0: all keys up to its own; n > 0: the last n (a sliding window); n < 0: those of its
// own chunk of -n positions, chunks counted from position 0 of the sequence.  The first key seen
// never moves back as the position grows, which is all the kernels' tile bounds rely on.
__host__ __device__ __forceinline__ int kappai_first_key(int pos, int window) {
  if (window > 0) return pos + 1 > window ? pos + 1 - window : 0;
  if (window < 0) return pos < 0 ? 0 : pos - pos % (-window);
  return 0;
}

#define KAPPAI_BIAS_PAD 8

struct kappai_score_mods {
  float softcap;
  const float* dist_bias;
  int dist_cols;
  const float* sink;
  int keep_first;
};

// With kept first positions a row's keys are two runs: [0, keep) and [lo, pos], lo from
// kappai_first_key.  The matrix-core kernels walk tiles of 32 keys; the tiles of the first run that
// lie before the window's first tile (lo32 = lo rounded down to 32) are put right in front of it:
// tile address kb >= lo32 holds the keys from kb on, the `kept` places before lo32 hold the keys
// from 0 on.  With nothing kept (or a window that still reaches the beginning) kept is 0.
__device__ __forceinline__ int kappai_kept_places(int keep, int lo32) {
  return (min(keep, lo32) + 31) / 32 * 32;
}
__device__ __forceinline__ int kappai_key_at(int place, int lo32, int kept) {
  return place >= lo32 ? place : place - (lo32 - kept);
}

__host__ __device__ __forceinline__ bool kappai_mods_on(const kappai_score_mods* m) {
  return m != nullptr && (m->softcap > 0.f || m->dist_bias != nullptr || m->sink != nullptr ||
                          m->keep_first > 0);
}

// (a cap, a bias or kept positions: the scores themselves change or a row's keys are two runs; a
// sink alone leaves them as they are)
__host__ __device__ __forceinline__ bool kappai_mods_change_scores(const kappai_score_mods* m) {
  return m != nullptr && (m->softcap > 0.f || m->dist_bias != nullptr || m->keep_first > 0);
}

__device__ __forceinline__ const float* kappai_bias_row(const kappai_score_mods& m, int h) {
  return m.dist_bias + (size_t)h * (m.dist_cols + 2 * KAPPAI_BIAS_PAD) + KAPPAI_BIAS_PAD;
}

// cap * tanh(s / cap) for the kernels that work in bfloat16: tanh(x) = 1 - 2 / (1 + e^(2x)) by the
// hardware's exponential and reciprocal (absolute error of a few 1e-7 of the cap).
__device__ __forceinline__ float kappai_fast_cap(float s, float cap) {
  const float e = __builtin_amdgcn_exp2f(s * (2.885390081777927f / cap));    // 2 log2(e) / cap
  return cap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + e));
}

// `s` is the scaled dot product; the result is what the softmax sees (natural-logarithm units).
__device__ __forceinline__ float kappai_modified_score(const kappai_score_mods& m, float s, int h,
                                                       int dist) {
  if (m.softcap > 0.f) s = m.softcap * tanhf(s / m.softcap);
  if (m.dist_bias != nullptr)
    s += kappai_bias_row(m, h)[max(0, min(dist, m.dist_cols - 1))];
  return s;
}
