// Embedding rows, (residual add +) RMSNorm, SwiGLU gate, casts and row gathers.
//
// The residual stream is float in every run; `T` is the run's compute type (float or
// bf16_t) in which normalised activations and GEMM outputs are stored.
#include "common.h"

// ---------------------------------------------------------------------------------------
// out[t, :] = table[ids[t], :]  widened to float        (kappai: src/recipe/scratch.c:195-235)
// ---------------------------------------------------------------------------------------
template <typename TW>
__global__ void embed_rows_kernel(const int* __restrict__ ids, const TW* __restrict__ table,
                                  float* __restrict__ out, int D, float scale) {
  const int t = blockIdx.x;
  const TW* src = table + (size_t)ids[t] * D;
  float* dst = out + (size_t)t * D;
  for (int i = threadIdx.x; i < D; i += blockDim.x) dst[i] = to_f32(src[i]) * scale;
}

// The same from a bfloat16 table that is kept in the order of the matrix cores' fragments (a
// tied output head's matrix, see gemm.hip: pieces of 16 rows x 32 columns, a lane's 8 values at
// lane = (column % 32) / 8 * 16 + row % 16); D a multiple of 32.
__global__ void embed_rows_fragments_kernel(const int* __restrict__ ids,
                                            const bf16_t* __restrict__ table,
                                            float* __restrict__ out, int D, float scale) {
  const int t = blockIdx.x;
  const size_t r = (size_t)ids[t];
  const bf16_t* src = table + (r / 16) * 16 * D + (r % 16) * 8;
  float* dst = out + (size_t)t * D;
  // a thread takes 8 neighbouring columns: 16 bytes of the piece, 32 bytes of the row
  for (int c = threadIdx.x; c < D / 8; c += blockDim.x) {
    const uint4 v = *reinterpret_cast<const uint4*>(src + (size_t)(c / 4) * 512 + (c % 4) * 128);
    const uint32_t u[4] = {v.x, v.y, v.z, v.w};
    float4 lo, hi;
    lo.x = __uint_as_float(u[0] << 16), lo.y = __uint_as_float(u[0] & 0xffff0000u);
    lo.z = __uint_as_float(u[1] << 16), lo.w = __uint_as_float(u[1] & 0xffff0000u);
    hi.x = __uint_as_float(u[2] << 16), hi.y = __uint_as_float(u[2] & 0xffff0000u);
    hi.z = __uint_as_float(u[3] << 16), hi.w = __uint_as_float(u[3] & 0xffff0000u);
    lo.x *= scale, lo.y *= scale, lo.z *= scale, lo.w *= scale;
    hi.x *= scale, hi.y *= scale, hi.z *= scale, hi.w *= scale;
    *reinterpret_cast<float4*>(dst + 8 * c) = lo;
    *reinterpret_cast<float4*>(dst + 8 * c + 4) = hi;
  }
}

// table_is_bf16: 0 = float32 rows, 1 = bfloat16 rows, 2 = bfloat16 in fragment order; `scale`: a
// factor on every row
extern "C" int kappai_embed_rows_scaled(const int* ids, const void* table, int table_is_bf16,
                                        float* out, int T, int D, float scale,
                                        hipStream_t stream) {
  if (T <= 0) return 0;
  const int threads = D >= 1024 ? 256 : (D >= 256 ? 128 : 64);
  if (table_is_bf16 == 2) {
    if (D % 32 || ((uintptr_t)table % 16) || ((uintptr_t)out % 16)) return (int)hipErrorInvalidValue;
    hipLaunchKernelGGL(embed_rows_fragments_kernel, dim3(T), dim3(threads), 0, stream, ids,
                       (const bf16_t*)table, out, D, scale);
  } else if (table_is_bf16)
    hipLaunchKernelGGL(embed_rows_kernel<bf16_t>, dim3(T), dim3(threads), 0, stream, ids,
                       (const bf16_t*)table, out, D, scale);
  else
    hipLaunchKernelGGL(embed_rows_kernel<float>, dim3(T), dim3(threads), 0, stream, ids,
                       (const float*)table, out, D, scale);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

extern "C" int kappai_embed_rows(const int* ids, const void* table, int table_is_bf16, float* out,
                                 int T, int D, hipStream_t stream) {
  return kappai_embed_rows_scaled(ids, table, table_is_bf16, out, T, D, 1.0f, stream);
}

// ---------------------------------------------------------------------------------------
// A norm on what a sublayer returns: y = scale_a * a (+ scale_b * b), n = y / sqrt(mean(y^2) + eps)
// * w, then resid += n (or resid = n), and the new resid again in the compute dtype for the next
// sublayer to read.  a may come as `a_parts` float planes [parts][T][D] that are added in order
// first (a product cut over its input dimension).  Everything in float32; a block a row, the row
// kept in LDS between the sum of squares and the scaling.  `vec`: D is a multiple of eight and
// every pointer of 32 bytes, so a thread takes eight values at a time and asks for the planes
// four at a time (same sums in the same order).
// ---------------------------------------------------------------------------------------
template <typename TA, typename TO>
__global__ __launch_bounds__(256) void output_norm_add_kernel(
    const TA* __restrict__ a, int a_parts, size_t a_plane, float scale_a, const TA* __restrict__ b,
    float scale_b, const float* __restrict__ w, float eps, float* __restrict__ resid, int add,
    TO* __restrict__ rows, int D, int vec) {
  extern __shared__ __attribute__((aligned(16))) float ys[];
  __shared__ float red[16];
  const size_t at = (size_t)blockIdx.x * D;
  float ss = 0.f;
  if (vec) {
    for (int e = 8 * threadIdx.x; e < D; e += 8 * 256) {
      float v[8];
      load8(a + at + e, v);
#pragma unroll 4
      for (int k = 1; k < a_parts; ++k) {
        float u[8];
        load8(a + k * a_plane + at + e, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] += u[i];
      }
      float bb[8];
      if (b != nullptr) load8(b + at + e, bb);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        v[i] *= scale_a;
        if (b != nullptr) v[i] = fmaf(scale_b, bb[i], v[i]);
        ss = fmaf(v[i], v[i], ss);
      }
      store8(ys + e, v);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)D + eps);
    for (int e = 8 * threadIdx.x; e < D; e += 8 * 256) {
      float y[8], ww[8], r[8];
      load8(ys + e, y);
      load8(w + e, ww);
      if (add) load8(resid + at + e, r);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        y[i] = y[i] * inv * ww[i];
        if (add) y[i] += r[i];
      }
      store8(resid + at + e, y);
      if (rows != nullptr) store8(rows + at + e, y);
    }
    return;
  }
  for (int e = threadIdx.x; e < D; e += 256) {
    float v = to_f32(a[at + e]);
    for (int k = 1; k < a_parts; ++k) v += to_f32(a[k * a_plane + at + e]);
    v *= scale_a;
    if (b != nullptr) v = fmaf(scale_b, to_f32(b[at + e]), v);
    ys[e] = v;
    ss = fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)D + eps);
  for (int e = threadIdx.x; e < D; e += 256) {
    float n = ys[e] * inv * w[e];
    if (add) n += resid[at + e];
    resid[at + e] = n;
    if (rows != nullptr) from_f32(rows + at + e, n);
  }
}

extern "C" int kappai_output_norm_add(const void* a, int a_is_bf16, int a_parts, float scale_a,
                                      const void* b, float scale_b, const float* w, float eps,
                                      float* resid, int add, void* rows, int rows_is_bf16, int T,
                                      int D, hipStream_t stream) {
  if (T <= 0) return 0;
  if (D < 1 || D > 15 * 1024 || a_parts < 1 || (a_is_bf16 && a_parts != 1))
    return (int)hipErrorInvalidValue;
  const size_t lds = (size_t)D * sizeof(float), plane = (size_t)T * D;
  const int vec = D % 8 == 0 && ((uintptr_t)a | (uintptr_t)b | (uintptr_t)w | (uintptr_t)resid |
                                 (uintptr_t)rows) % 32 == 0;
#define KAPPAI_OUT_NORM(TA, TO)                                                                  \
  hipLaunchKernelGGL((output_norm_add_kernel<TA, TO>), dim3(T), dim3(256), lds, stream,          \
                     (const TA*)a, a_parts, plane, scale_a, (const TA*)b, scale_b, w, eps, resid, \
                     add, (TO*)rows, D, vec)
  if (a_is_bf16) {
    if (rows_is_bf16) KAPPAI_OUT_NORM(bf16_t, bf16_t); else KAPPAI_OUT_NORM(bf16_t, float);
  } else {
    if (rows_is_bf16) KAPPAI_OUT_NORM(float, bf16_t); else KAPPAI_OUT_NORM(float, float);
  }
#undef KAPPAI_OUT_NORM
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// Pointwise norms that saturate, n(x) = tanh(alpha x) w + b (one alpha a row, w and b [D]), on both
// sides of a sublayer in one pass over the stream: resid += n_post(y), rows = n_pre(resid).  No place
// looks at another, so there is nothing to sum and a thread works on its own VEC columns from the
// loads to the store.  y comes as
//   TY rows, or float planes [parts][T][D] that are added in order (a product cut over its input
//   dimension), or, with slot_of_pair, as a mixture's experts left it: the sum over the row's `top`
//   choices of wts[t, k] * y[slot of (t, k)], in the order of k.
// post.w null: y is added as it is; pre.w null: no rows are wanted.  `pick`: only these rows are
// normalised, and the stream keeps its old values.  Everything in float32.
// ---------------------------------------------------------------------------------------
struct kappai_tanh_norm {
  float alpha;
  const float* w;
  const float* b;
};

template <int VEC>
__device__ __forceinline__ void load_cols(const float* p, float (&v)[VEC]) {
  if (VEC == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    v[0] = a.x; v[VEC > 1 ? 1 : 0] = a.y; v[VEC > 2 ? 2 : 0] = a.z; v[VEC > 3 ? 3 : 0] = a.w;
  } else {
    v[0] = p[0];
  }
}
template <int VEC>
__device__ __forceinline__ void load_cols(const bf16_t* p, float (&v)[VEC]) {
  if (VEC == 4) {
    const uint2 a = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(a.x << 16); v[VEC > 1 ? 1 : 0] = __uint_as_float(a.x & 0xffff0000u);
    v[VEC > 2 ? 2 : 0] = __uint_as_float(a.y << 16);
    v[VEC > 3 ? 3 : 0] = __uint_as_float(a.y & 0xffff0000u);
  } else {
    v[0] = to_f32(p[0]);
  }
}
template <int VEC>
__device__ __forceinline__ void store_cols(float* p, const float (&v)[VEC]) {
  if (VEC == 4)
    *reinterpret_cast<float4*>(p) =
        make_float4(v[0], v[VEC > 1 ? 1 : 0], v[VEC > 2 ? 2 : 0], v[VEC > 3 ? 3 : 0]);
  else
    p[0] = v[0];
}
template <int VEC>
__device__ __forceinline__ void store_cols(bf16_t* p, const float (&v)[VEC]) {
  if (VEC == 4)
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[VEC > 1 ? 1 : 0]),
                                              pack_bf16x2(v[VEC > 2 ? 2 : 0], v[VEC > 3 ? 3 : 0]));
  else
    from_f32(p, v[0]);
}

template <typename TY, typename TO, int VEC>
__global__ __launch_bounds__(256) void tanh_norm_kernel(
    float* __restrict__ resid, const TY* __restrict__ y, int parts, size_t plane,
    const int* __restrict__ slot_of_pair, const float* __restrict__ wts, int top,
    kappai_tanh_norm post, kappai_tanh_norm pre, const int* __restrict__ pick, long n_pieces,
    int D, int store, TO* __restrict__ rows) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n_pieces) return;
  const int per_row = D / VEC;
  const long r = i / per_row;
  const int c = (int)(i - r * per_row) * VEC;
  const size_t t = pick != nullptr ? (size_t)pick[r] : (size_t)r;
  float x[VEC];
  load_cols<VEC>(resid + t * D + c, x);
  if (y != nullptr) {
    float u[VEC], w[VEC], b[VEC];
    if (slot_of_pair != nullptr) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = 0.f;
#pragma unroll 4
      for (int k = 0; k < top; ++k) {
        float v[VEC];
        load_cols<VEC>(y + (size_t)slot_of_pair[t * top + k] * D + c, v);
        const float f = wts[t * top + k];
#pragma unroll
        for (int j = 0; j < VEC; ++j) u[j] = fmaf(f, v[j], u[j]);
      }
    } else {
      load_cols<VEC>(y + t * D + c, u);
#pragma unroll 4
      for (int k = 1; k < parts; ++k) {
        float v[VEC];
        load_cols<VEC>(y + k * plane + t * D + c, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) u[j] += v[j];
      }
    }
    if (post.w != nullptr) {
      load_cols<VEC>(post.w + c, w);
      load_cols<VEC>(post.b + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = fmaf(tanhf(post.alpha * u[j]), w[j], b[j]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[j] += u[j];
    if (store) store_cols<VEC>(resid + t * D + c, x);
  }
  if (rows == nullptr) return;
  float w[VEC], b[VEC];
  load_cols<VEC>(pre.w + c, w);
  load_cols<VEC>(pre.b + c, b);
#pragma unroll
  for (int j = 0; j < VEC; ++j) x[j] = fmaf(tanhf(pre.alpha * x[j]), w[j], b[j]);
  store_cols<VEC>(rows + r * D + c, x);
}

extern "C" int kappai_tanh_norm_step(float* resid, const void* y, int y_is_bf16, int parts,
                                     const int* slot_of_pair, const float* wts, int top,
                                     float post_alpha, const float* post_w, const float* post_b,
                                     float pre_alpha, const float* pre_w, const float* pre_b,
                                     const int* pick, int n_rows, int T, int D, void* rows,
                                     int rows_is_bf16, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (D < 1 || (y && parts < 1) || (y_is_bf16 && (parts != 1 || slot_of_pair)) ||
      (slot_of_pair && (!y || !wts || top < 1)) || (post_w && !post_b) ||
      (rows && (!pre_w || !pre_b)) || (!pick && n_rows != T))
    return (int)hipErrorInvalidValue;
  const bool vec = D % 4 == 0 &&
                   ((uintptr_t)resid | (uintptr_t)y | (uintptr_t)post_w | (uintptr_t)post_b |
                    (uintptr_t)pre_w | (uintptr_t)pre_b | (uintptr_t)rows) % 16 == 0;
  const long pieces = (long)n_rows * (vec ? D / 4 : D);
  // few rows: blocks of one wave, so that the pieces spread over the chip
  const int threads = pieces <= 64 * 1024 ? 64 : 256;
  const long blocks = (pieces + threads - 1) / threads;
  if (blocks > 0x7fffffffL) return (int)hipErrorInvalidValue;
  const kappai_tanh_norm post{post_alpha, post_w, post_b}, pre{pre_alpha, pre_w, pre_b};
#define KAPPAI_TANH_NORM(TY, TO, V)                                                              \
  hipLaunchKernelGGL((tanh_norm_kernel<TY, TO, V>), dim3((unsigned)blocks), dim3(threads), 0,    \
                     stream, resid, (const TY*)y, parts, (size_t)T * D, slot_of_pair, wts, top,  \
                     post, pre, pick, pieces, D, pick ? 0 : 1, (TO*)rows)
#define KAPPAI_TANH_NORM_V(TY, TO)                                                               \
  if (vec) KAPPAI_TANH_NORM(TY, TO, 4); else KAPPAI_TANH_NORM(TY, TO, 1)
  if (y_is_bf16) {
    if (rows_is_bf16) { KAPPAI_TANH_NORM_V(bf16_t, bf16_t); } else { KAPPAI_TANH_NORM_V(bf16_t, float); }
  } else {
    if (rows_is_bf16) { KAPPAI_TANH_NORM_V(float, bf16_t); } else { KAPPAI_TANH_NORM_V(float, float); }
  }
#undef KAPPAI_TANH_NORM_V
#undef KAPPAI_TANH_NORM
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// RMS norms n(x) = x / sqrt(mean(x^2) + eps) * w on both sides of a sublayer in one pass over the
// stream: resid += n_post(y), rows = n_pre(resid).  A block a row; the row stays in registers from
// the loads over both sums of squares to the stores.  y comes as
//   rows (float32 or bfloat16), or float planes [parts][T][D] that are added in order, or, with
//   slot_of_pair, as a mixture's experts left it: also[t] * gate[t] first (what every row gets: rows
//   or planes; a gate or none), then the sum over the row's `top` choices of wts[t, k] * y[slot of
//   (t, k)], in the order of k; slot -1 stands for the row x[t] itself.
// post_w null: y is added as it is; pre_w null: no rows are wanted.  `pick`: only these rows are
// normalised, and the stream keeps its old values.  Everything in float32.
// ---------------------------------------------------------------------------------------
struct kappai_update {
  const void* y;
  int y_is_bf16, parts;
  const int* slot_of_pair;
  const float* wts;
  int top;
  const void* also;
  int also_is_bf16, also_parts;
  const float* also_gate;
  const void* x;
  int ldx, x_is_bf16;
};

template <int VEC>
__device__ __forceinline__ void load_cols(const void* p, int is_bf16, size_t at, float (&v)[VEC]) {
  if (is_bf16) load_cols<VEC>((const bf16_t*)p + at, v);
  else load_cols<VEC>((const float*)p + at, v);
}

// rows, or planes added in order
template <int VEC>
__device__ __forceinline__ void load_planes(const void* p, int is_bf16, int parts, size_t plane,
                                            size_t at, float (&u)[VEC]) {
  load_cols<VEC>(p, is_bf16, at, u);
#pragma unroll 4
  for (int k = 1; k < parts; ++k) {
    float v[VEC];
    load_cols<VEC>((const float*)p + k * plane + at, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] += v[j];
  }
}

template <int VEC>
__device__ __forceinline__ void load_update(const kappai_update& up, size_t t, int c, int D,
                                            size_t plane, float (&u)[VEC]) {
  if (up.slot_of_pair == nullptr) {
    load_planes<VEC>(up.y, up.y_is_bf16, up.parts, plane, t * D + c, u);
    return;
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) u[j] = 0.f;
  if (up.also != nullptr) {
    load_planes<VEC>(up.also, up.also_is_bf16, up.also_parts, plane, t * D + c, u);
    const float g = up.also_gate != nullptr ? up.also_gate[t] : 1.f;
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] *= g;
  }
  float own[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) own[j] = 0.f;
  if (up.x != nullptr) load_cols<VEC>(up.x, up.x_is_bf16, t * up.ldx + c, own);
#pragma unroll 4
  for (int k = 0; k < up.top; ++k) {
    const int slot = up.slot_of_pair[t * up.top + k];
    const float f = up.wts[t * up.top + k];
    float v[VEC];
    if (slot >= 0) {
      load_cols<VEC>((const float*)up.y + (size_t)slot * D + c, v);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = own[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] = fmaf(f, v[j], u[j]);
  }
}

// NC pieces of VEC columns a thread, a block's width apart
template <int VEC, int NC>
__global__ __launch_bounds__(1024) void rms_norm_step_kernel(
    float* __restrict__ resid, const kappai_update up, size_t plane,
    const float* __restrict__ post_w, float post_eps, const float* __restrict__ pre_w,
    float pre_eps, const int* __restrict__ pick, int D, int store, void* __restrict__ rows,
    int rows_is_bf16) {
  __shared__ float red[16];
  const size_t r = blockIdx.x;
  const size_t t = pick != nullptr ? (size_t)pick[r] : r;
  float x[NC][VEC], u[NC][VEC], w[NC][VEC];
  float ss = 0.f;
  const bool update = up.y != nullptr;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[i][j] = u[i][j] = w[i][j] = 0.f;
    if (c >= D) continue;
    load_cols<VEC>(resid + t * D + c, x[i]);
    if (update) {
      if (post_w != nullptr) load_cols<VEC>(post_w + c, w[i]);
      load_update<VEC>(up, t, c, D, plane, u[i]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(u[i][j], u[i][j], ss);
  }
  if (update) {
    float inv = 1.f;
    if (post_w != nullptr) inv = 1.0f / sqrtf(block_sum(ss, red) / (float)D + post_eps);
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (i * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[i][j] += post_w != nullptr ? u[i][j] * inv * w[i][j] : u[i][j];
      if (store && c < D) store_cols<VEC>(resid + t * D + c, x[i]);
    }
  }
  if (rows == nullptr) return;
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * VEC;
    if (c < D) load_cols<VEC>(pre_w + c, w[i]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(x[i][j], x[i][j], ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)D + pre_eps);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * VEC;
    if (c >= D) continue;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[i][j] = x[i][j] * inv * w[i][j];
    if (rows_is_bf16) store_cols<VEC>((bf16_t*)rows + r * D + c, x[i]);
    else store_cols<VEC>((float*)rows + r * D + c, x[i]);
  }
}

extern "C" int kappai_rms_norm_step(
    float* resid, const void* y, int y_is_bf16, int parts, const int* slot_of_pair,
    const float* wts, int top, const void* also, int also_is_bf16, int also_parts,
    const float* also_gate, const void* x, int ldx, int x_is_bf16, const float* post_w,
    float post_eps, const float* pre_w, float pre_eps, const int* pick, int n_rows, int T, int D,
    void* rows, int rows_is_bf16, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (D < 1 || D > 8192 || (y && parts < 1) || (y_is_bf16 && (parts != 1 || slot_of_pair)) ||
      (slot_of_pair && (!y || !wts || top < 1)) || (rows && !pre_w) || (!pick && n_rows != T) ||
      (also && (also_parts < 1 || (also_is_bf16 && also_parts != 1))) || (x && ldx < D))
    return (int)hipErrorInvalidValue;
  const kappai_update up{y, y_is_bf16, parts, slot_of_pair, wts, top, also, also_is_bf16,
                         also_parts, also_gate, x, ldx, x_is_bf16};
  const bool vec = D % 4 == 0 && ldx % 4 == 0 &&
                   ((uintptr_t)resid | (uintptr_t)y | (uintptr_t)post_w | (uintptr_t)pre_w |
                    (uintptr_t)rows | (uintptr_t)also | (uintptr_t)x) % 16 == 0;
  const int pieces = vec ? D / 4 : D;
  const int threads = pieces >= 1024 ? 1024 : (pieces + WAVE - 1) / WAVE * WAVE;
#define KAPPAI_RMS_STEP(V, N)                                                                    \
  hipLaunchKernelGGL((rms_norm_step_kernel<V, N>), dim3(n_rows), dim3(threads), 0, stream, resid, \
                     up, (size_t)T * D, post_w, post_eps, pre_w, pre_eps, pick, D, pick ? 0 : 1,  \
                     rows, rows_is_bf16)
  if (vec) {
    if (pieces <= 1024) KAPPAI_RMS_STEP(4, 1); else KAPPAI_RMS_STEP(4, 2);
  } else {
    if (pieces <= 1024) KAPPAI_RMS_STEP(1, 1); else KAPPAI_RMS_STEP(1, 8);
  }
#undef KAPPAI_RMS_STEP
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// Two sublayers' results side by side, made one update of the stream in float32:
// out = scale_a * n_a(a) + scale_b * n_b(b), with n(y) = y / sqrt(mean(y^2) + eps) * w when a
// weight is given and y itself when not.  a, b [T, D] in float32 or bfloat16 (one dtype); a block
// a row, both rows in LDS between the sums of squares and the scaling.
// ---------------------------------------------------------------------------------------
template <typename TA>
__global__ __launch_bounds__(256) void pair_norm_sum_kernel(
    const TA* __restrict__ a, float scale_a, const float* __restrict__ wa,
    const TA* __restrict__ b, float scale_b, const float* __restrict__ wb, float eps, int D,
    float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float ys[];
  __shared__ float red[16];
  const size_t at = (size_t)blockIdx.x * D;
  float sa = 0.f, sb = 0.f;
  for (int e = threadIdx.x; e < D; e += 256) {
    const float x = to_f32(a[at + e]), y = to_f32(b[at + e]);
    ys[e] = x;
    ys[D + e] = y;
    sa = fmaf(x, x, sa);
    sb = fmaf(y, y, sb);
  }
  float fa = scale_a, fb = scale_b;
  if (wa != nullptr) fa *= 1.0f / sqrtf(block_sum(sa, red) / (float)D + eps);
  if (wb != nullptr) fb *= 1.0f / sqrtf(block_sum(sb, red) / (float)D + eps);
  for (int e = threadIdx.x; e < D; e += 256) {
    const float x = ys[e] * fa * (wa != nullptr ? wa[e] : 1.f);
    const float y = ys[D + e] * fb * (wb != nullptr ? wb[e] : 1.f);
    out[at + e] = x + y;
  }
}

extern "C" int kappai_pair_norm_sum(const void* a, float scale_a, const float* wa, const void* b,
                                    float scale_b, const float* wb, float eps, int T, int D,
                                    float* out, int is_bf16, hipStream_t stream) {
  if (T <= 0) return 0;
  if (D < 1 || D > 7 * 1024) return (int)hipErrorInvalidValue;
  const size_t lds = 2 * (size_t)D * sizeof(float);
  if (is_bf16)
    hipLaunchKernelGGL(pair_norm_sum_kernel<bf16_t>, dim3(T), dim3(256), lds, stream,
                       (const bf16_t*)a, scale_a, wa, (const bf16_t*)b, scale_b, wb, eps, D, out);
  else
    hipLaunchKernelGGL(pair_norm_sum_kernel<float>, dim3(T), dim3(256), lds, stream,
                       (const float*)a, scale_a, wa, (const float*)b, scale_b, wb, eps, D, out);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// What a pass over a run of layers starts with: resid += delta (the update that the layer before
// left pending; float32 or the compute dtype; may be null), then += again (rows of the same
// shape, float32; may be null), then += row (one row [D] for all; may be null), in this order.
// ---------------------------------------------------------------------------------------
template <typename TD>
__global__ __launch_bounds__(256) void stream_enter_kernel(
    float* __restrict__ resid, const TD* __restrict__ delta, const float* __restrict__ again,
    const float* __restrict__ row, long n, int D) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  float x = resid[i];
  if (delta != nullptr) x += to_f32(delta[i]);
  if (again != nullptr) x += again[i];
  if (row != nullptr) x += row[i % D];
  resid[i] = x;
}

extern "C" int kappai_stream_enter(float* resid, const void* delta, int delta_is_bf16,
                                   const float* again, const float* row, int T, int D,
                                   hipStream_t stream) {
  if (T <= 0) return 0;
  if (D < 1) return (int)hipErrorInvalidValue;
  const long n = (long)T * D;
  const dim3 grid((unsigned)((n + 255) / 256));
  if (delta_is_bf16)
    hipLaunchKernelGGL(stream_enter_kernel<bf16_t>, grid, dim3(256), 0, stream, resid,
                       (const bf16_t*)delta, again, row, n, D);
  else
    hipLaunchKernelGGL(stream_enter_kernel<float>, grid, dim3(256), 0, stream, resid,
                       (const float*)delta, again, row, n, D);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// tokens[dst_rows[i]] = chosen[src_idx[i]]: token ids that the last step's sampling kernels
// left on the GPU go to their rows of this step's token table without a trip through the host.
// ---------------------------------------------------------------------------------------
__global__ void place_tokens_kernel(int* __restrict__ tokens, const int* __restrict__ dst_rows,
                                    const int* __restrict__ chosen,
                                    const int* __restrict__ src_idx, int n) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) tokens[dst_rows[i]] = chosen[src_idx[i]];
}

extern "C" int kappai_place_tokens(int* tokens, const int* dst_rows, const int* chosen,
                                   const int* src_idx, int n, hipStream_t stream) {
  if (n <= 0) return 0;
  hipLaunchKernelGGL(place_tokens_kernel, dim3((n + 255) / 256), dim3(256), 0, stream, tokens,
                     dst_rows, chosen, src_idx, n);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// dst[i] = src[i]: token ids to pinned host memory by a kernel.  (A copy command from device to
// host that is still pending makes the host wait when the next copy from host to device is
// queued behind it; a kernel that writes to host memory does not.)
// ---------------------------------------------------------------------------------------
__global__ void copy_ints_kernel(int* __restrict__ dst, const int* __restrict__ src, int n) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) dst[i] = src[i];
}

extern "C" int kappai_copy_ints(int* dst, const int* src, int n, hipStream_t stream) {
  if (n <= 0) return 0;
  hipLaunchKernelGGL(copy_ints_kernel, dim3((n + 255) / 256), dim3(256), 0, stream, dst, src, n);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// Rows that lie in the order of the matrix cores' fragments ([D / 32][4 groups of 8 of K][16
// rows][8 values], what the norm writes for the product kernel of 1 to 16 rows) as ordinary rows
// [n_rows, D], for a consumer that reads rows: 16-byte chunk c of row m lies at chunk c * 16 + m.
__global__ void rows_from_fragments_kernel(const uint4* __restrict__ frag, uint4* __restrict__ out,
                                           int n_rows, int chunks) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n_rows * chunks) return;
  const int m = i / chunks, c = i % chunks;
  out[i] = frag[(size_t)c * 16 + m];
}
extern "C" int kappai_rows_from_fragments(const void* frag, void* out, int n_rows, int D,
                                          hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (n_rows > 16 || D % 32 || ((uintptr_t)frag % 16) || ((uintptr_t)out % 16))
    return (int)hipErrorInvalidValue;
  const int chunks = D / 8;                               // 8 bfloat16 values a chunk
  hipLaunchKernelGGL(rows_from_fragments_kernel, dim3((n_rows * chunks + 255) / 256), dim3(256), 0,
                     stream, (const uint4*)frag, (uint4*)out, n_rows, chunks);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// RMSNorm with the residual sum folded in:
//   x = resid[r] (+ delta[r]);  if write_resid: resid[r] = x;
//   out[i] = x * rsqrt(mean(x^2) + eps) * w           (src/backend/cpu/scalar/quants.c:1507-1512)
// r = rows ? rows[i] : i.  Sum of squares and scaling in float.  delta may be n_part partial
// sums (a product split over K), `pstride` elements apart; they are added in order.
// ---------------------------------------------------------------------------------------
template <typename T, typename TD>
__global__ void add_rmsnorm_kernel(float* __restrict__ resid, const TD* __restrict__ delta,
                                   int n_part, size_t pstride, const float* __restrict__ w,
                                   T* __restrict__ out, const int* __restrict__ rows, int D,
                                   float eps, int write_resid) {
  __shared__ float red[16];
  const int i = blockIdx.x;
  const int r = rows ? rows[i] : i;
  float* x = resid + (size_t)r * D;
  const TD* dl = delta ? delta + (size_t)r * D : nullptr;
  T* o = out + (size_t)i * D;
  float ss = 0.f;
  for (int j = threadIdx.x; j < D; j += blockDim.x) {
    float v = x[j];
    if (dl) {
      for (int p = 0; p < n_part; ++p) v += to_f32(dl[p * pstride + j]);
      if (write_resid) x[j] = v;
    }
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float scale = 1.0f / sqrtf(ss / (float)D + eps);
  for (int j = threadIdx.x; j < D; j += blockDim.x) {
    float v = x[j];
    if (dl && !write_resid)
      for (int p = 0; p < n_part; ++p) v += to_f32(dl[p * pstride + j]);
    from_f32(o + j, v * scale * w[j]);
  }
}

// The same for widths that are multiples of 8 up to 8192: one block per row, eight elements per
// thread kept in registers between the sum of squares and the scaling, 16/32-byte loads and
// stores, all loads (the row, every partial sum, the weights) issued before anything waits.
#define RN_MAX_PART 8

template <typename T, typename TD>
__global__ __launch_bounds__(1024) void add_rmsnorm_row_kernel(
    float* __restrict__ resid, const TD* __restrict__ delta, int n_part, size_t pstride,
    const float* __restrict__ w, T* __restrict__ out, const int* __restrict__ rows, int D,
    float eps, int write_resid, int out_frag) {
  __shared__ float red[16];
  const int i = blockIdx.x;
  const int r = rows ? rows[i] : i;
  const int j = threadIdx.x * 8;
  const bool in = j < D;
  float* x = resid + (size_t)r * D;
  const TD* dl = delta ? delta + (size_t)r * D : nullptr;
  float v[8], w8[8], d8[RN_MAX_PART][8];
  float ss = 0.f;
  if (in) {
    load8(w + j, w8);
    load8(x + j, v);
    if (dl) {
#pragma unroll
      for (int p = 0; p < RN_MAX_PART; ++p)
        if (p < n_part) load8(dl + p * pstride + j, d8[p]);
#pragma unroll
      for (int p = 0; p < RN_MAX_PART; ++p)
        if (p < n_part)
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] += d8[p][e];
      if (write_resid) store8(x + j, v);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
  }
  ss = block_sum(ss, red);
  const float scale = 1.0f / sqrtf(ss / (float)D + eps);
  if (in) {
#pragma unroll
    for (int e = 0; e < 8; ++e) w8[e] = v[e] * scale * w8[e];
    // out_frag (at most 16 rows, D a multiple of 32): the rows in the order in which the product
    // kernel for 1 to 16 rows loads its activations, [D / 32][(k % 32) / 8][16 rows][8 values]:
    // its load instructions then touch whole cache lines of neighbouring rows
    const size_t at = out_frag ? (size_t)(j / 32) * 512 + ((size_t)((j % 32) / 8) * 16 + i) * 8
                               : (size_t)i * D + j;
    store8(out + at, w8);
  }
}

template <typename T, typename TD>
static void launch_add_rmsnorm(float* resid, const void* delta, int n_part, size_t pstride,
                               const float* w, void* out, const int* rows, int n_rows, int D,
                               float eps, int write_resid, int out_frag, hipStream_t stream) {
  if (D % 8 == 0 && D <= 8192 && n_part <= RN_MAX_PART) {
    const int threads = ((D / 8 + WAVE - 1) / WAVE) * WAVE;
    hipLaunchKernelGGL((add_rmsnorm_row_kernel<T, TD>), dim3(n_rows), dim3(threads), 0, stream,
                       resid, (const TD*)delta, n_part, pstride, w, (T*)out, rows, D, eps,
                       write_resid, out_frag);
    return;
  }
  const int threads = D >= 2048 ? 512 : (D >= 512 ? 256 : (D >= 128 ? 128 : 64));
  hipLaunchKernelGGL((add_rmsnorm_kernel<T, TD>), dim3(n_rows), dim3(threads), 0, stream, resid,
                     (const TD*)delta, n_part, pstride, w, (T*)out, rows, D, eps, write_resid);
}

// out is bf16 or float (is_bf16); delta is of out's type, or float when delta_is_f32 (then it
// may consist of n_part partial sums, pstride elements apart).
extern "C" int kappai_add_rmsnorm(float* resid, const void* delta, int delta_is_f32, int n_part,
                                  long pstride, const float* w, void* out, const int* rows,
                                  int n_rows, int D, float eps, int write_resid, int is_bf16,
                                  int out_frag, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (n_part < 1 || (n_part > 1 && !delta_is_f32)) return (int)hipErrorInvalidValue;
  // rows in fragment order: bfloat16, at most 16 of them, in the kernel that keeps a row in
  // registers; out holds 16 x D values
  if (out_frag && (!is_bf16 || n_rows > 16 || (D % 32) || D > 8192 || n_part > RN_MAX_PART))
    return (int)hipErrorInvalidValue;
  if (!is_bf16)
    launch_add_rmsnorm<float, float>(resid, delta, n_part, (size_t)pstride, w, out, rows, n_rows,
                                     D, eps, write_resid, out_frag, stream);
  else if (delta_is_f32)
    launch_add_rmsnorm<bf16_t, float>(resid, delta, n_part, (size_t)pstride, w, out, rows, n_rows,
                                      D, eps, write_resid, out_frag, stream);
  else
    launch_add_rmsnorm<bf16_t, bf16_t>(resid, delta, n_part, (size_t)pstride, w, out, rows, n_rows,
                                       D, eps, write_resid, out_frag, stream);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// The embedding and the first norm in one kernel: resid[i] = table[ids[i]] (float32) and
// out[i] = resid[i] * rsqrt(mean(resid[i]^2) + eps) * w, the arithmetic of embed_rows followed by
// add_rmsnorm_row, bit for bit.  KIND: the table's layout as in kappai_embed_rows.
template <typename T, int KIND>
__global__ __launch_bounds__(1024) void embed_rmsnorm_row_kernel(
    const int* __restrict__ ids, const void* __restrict__ table, float* __restrict__ resid,
    const float* __restrict__ w, T* __restrict__ out, int D, float eps, int out_frag) {
  __shared__ float red[16];
  const int i = blockIdx.x;
  const size_t r = (size_t)ids[i];
  const int j = threadIdx.x * 8;
  const bool in = j < D;
  float v[8], w8[8];
  float ss = 0.f;
  if (in) {
    load8(w + j, w8);
    if (KIND == 0) {
      load8((const float*)table + r * D + j, v);
    } else if (KIND == 1) {
      load8((const bf16_t*)table + r * D + j, v);
    } else {
      const int c = j / 8;                      // the row's 16-byte chunk: piece c / 4, group c % 4
      load8((const bf16_t*)table + (r / 16) * 16 * D + (r % 16) * 8 + (size_t)(c / 4) * 512 +
                (c % 4) * 128, v);
    }
    store8(resid + (size_t)i * D + j, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
  }
  ss = block_sum(ss, red);
  const float scale = 1.0f / sqrtf(ss / (float)D + eps);
  if (in) {
#pragma unroll
    for (int e = 0; e < 8; ++e) w8[e] = v[e] * scale * w8[e];
    const size_t at = out_frag ? (size_t)(j / 32) * 512 + ((size_t)((j % 32) / 8) * 16 + i) * 8
                               : (size_t)i * D + j;
    store8(out + at, w8);
  }
}

// Refuses (hipErrorInvalidValue) what the row kernel does not take: the caller then runs
// kappai_embed_rows and kappai_add_rmsnorm.
extern "C" int kappai_embed_rmsnorm(const int* ids, const void* table, int table_is_bf16,
                                    float* resid, const float* w, void* out, int T, int D,
                                    float eps, int is_bf16, int out_frag, hipStream_t stream) {
  if (T <= 0) return 0;
  if (D % 8 || D > 8192 || (table_is_bf16 == 2 && D % 32) || ((uintptr_t)table % 16) ||
      ((uintptr_t)resid % 16) || ((uintptr_t)out % 16) || ((uintptr_t)w % 16) ||
      table_is_bf16 < 0 || table_is_bf16 > 2)
    return (int)hipErrorInvalidValue;
  if (out_frag && (!is_bf16 || T > 16 || D % 32)) return (int)hipErrorInvalidValue;
  const int threads = ((D / 8 + WAVE - 1) / WAVE) * WAVE;
#define KAPPAI_EMBED_NORM(TT, KIND)                                                              \
  hipLaunchKernelGGL((embed_rmsnorm_row_kernel<TT, KIND>), dim3(T), dim3(threads), 0, stream,    \
                     ids, table, resid, w, (TT*)out, D, eps, out_frag)
  if (is_bf16) {
    if (table_is_bf16 == 0) KAPPAI_EMBED_NORM(bf16_t, 0);
    else if (table_is_bf16 == 1) KAPPAI_EMBED_NORM(bf16_t, 1);
    else KAPPAI_EMBED_NORM(bf16_t, 2);
  } else {
    if (table_is_bf16 == 0) KAPPAI_EMBED_NORM(float, 0);
    else if (table_is_bf16 == 1) KAPPAI_EMBED_NORM(float, 1);
    else KAPPAI_EMBED_NORM(float, 2);
  }
#undef KAPPAI_EMBED_NORM
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// resid[r] += delta[r] without a norm (the last residual sum of a model whose output is
// the hidden state itself)
template <typename T>
__global__ void add_residual_kernel(float* __restrict__ resid, const T* __restrict__ delta,
                                    size_t n) {
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) resid[i] += to_f32(delta[i]);
}

extern "C" int kappai_add_residual(float* resid, const void* delta, long n, int is_bf16,
                                   hipStream_t stream) {
  if (n <= 0) return 0;
  const int threads = 256;
  const unsigned blocks = (unsigned)((n + threads - 1) / threads);
  if (is_bf16)
    hipLaunchKernelGGL(add_residual_kernel<bf16_t>, dim3(blocks), dim3(threads), 0, stream, resid,
                       (const bf16_t*)delta, (size_t)n);
  else
    hipLaunchKernelGGL(add_residual_kernel<float>, dim3(blocks), dim3(threads), 0, stream, resid,
                       (const float*)delta, (size_t)n);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// out[i] = parts[0][i] + parts[1][i] + ... in this order, in float: the partial sums of a
// product split over K, for a consumer that does not add them itself
__global__ void sum_partials_kernel(const float* __restrict__ parts, int n_parts, size_t n,
                                    float* __restrict__ out) {
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  float acc = parts[i];
  for (int s = 1; s < n_parts; ++s) acc += parts[(size_t)s * n + i];
  out[i] = acc;
}

extern "C" int kappai_sum_partials(const float* parts, int n_parts, long n, float* out,
                                   hipStream_t stream) {
  if (n <= 0 || n_parts < 1) return n_parts < 1 ? (int)hipErrorInvalidValue : 0;
  const int threads = 256;
  const unsigned blocks = (unsigned)((n + threads - 1) / threads);
  hipLaunchKernelGGL(sum_partials_kernel, dim3(blocks), dim3(threads), 0, stream, parts, n_parts,
                     (size_t)n, out);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// act[t, f] = silu(gu[t, f]) * gu[t, F + f],  silu(z) = z / (1 + exp(-z))
//                                                      (src/backend/cpu/quants.h:369-371)
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void swiglu_kernel(const T* __restrict__ gu, T* __restrict__ act, int F, size_t n) {
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  const size_t t = i / F;
  const int f = (int)(i - t * F);
  const float g = to_f32(gu[t * 2 * F + f]);
  const float u = to_f32(gu[t * 2 * F + F + f]);
  from_f32(act + i, g / (1.0f + expf(-g)) * u);
}

extern "C" int kappai_swiglu(const void* gu, void* act, int T, int F, int is_bf16,
                             hipStream_t stream) {
  const size_t n = (size_t)T * F;
  if (n == 0) return 0;
  const int threads = 256;
  const unsigned blocks = (unsigned)((n + threads - 1) / threads);
  if (is_bf16)
    hipLaunchKernelGGL(swiglu_kernel<bf16_t>, dim3(blocks), dim3(threads), 0, stream,
                       (const bf16_t*)gu, (bf16_t*)act, F, n);
  else
    hipLaunchKernelGGL(swiglu_kernel<float>, dim3(blocks), dim3(threads), 0, stream,
                       (const float*)gu, (float*)act, F, n);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// out[i] = f(in[i]) for one of a few functions: 0 tanh.
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void unary_kernel(const T* __restrict__ in, T* __restrict__ out, size_t n, int kind) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  const float x = to_f32(in[i]);
  from_f32(out + i, kind == 0 ? tanhf(x) : x);
}

extern "C" int kappai_unary(const void* in, void* out, long n, int kind, int is_bf16,
                            hipStream_t stream) {
  if (n <= 0) return 0;
  if (kind != 0) return (int)hipErrorInvalidValue;
  const unsigned blocks = (unsigned)((n + 255) / 256);
  if (is_bf16)
    hipLaunchKernelGGL(unary_kernel<bf16_t>, dim3(blocks), dim3(256), 0, stream,
                       (const bf16_t*)in, (bf16_t*)out, (size_t)n, kind);
  else
    hipLaunchKernelGGL(unary_kernel<float>, dim3(blocks), dim3(256), 0, stream, (const float*)in,
                       (float*)out, (size_t)n, kind);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// act(gate) * up with a choice of act: 0 silu, 1 the tanh form of gelu,
// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), 2 the clamped gate: g = min(gate, limit),
// u = clamp(up, -limit, limit), g sigmoid(slope g) (u + shift).
struct kappai_clamp { float limit, slope, shift; };

__device__ __forceinline__ float glu_value(float g, float u, int kind, const kappai_clamp& c) {
  if (kind == 2) {
    g = fminf(g, c.limit);
    u = fminf(fmaxf(u, -c.limit), c.limit);
    return g / (1.0f + expf(-c.slope * g)) * (u + c.shift);
  }
  if (kind == 1)
    return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
  return g / (1.0f + expf(-g)) * u;
}

// VEC columns a thread (4: F a multiple of four and 16-byte aligned pointers)
template <typename T, int VEC>
__global__ void glu_kernel(const T* __restrict__ gu, T* __restrict__ act, int F, size_t n,
                           int kind, kappai_clamp clamp) {
  const size_t i = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (i >= n) return;
  const size_t t = i / F;
  const int f = (int)(i - t * F);
  float g[VEC], u[VEC];
  load_cols<VEC>(gu + t * 2 * F + f, g);
  load_cols<VEC>(gu + t * 2 * F + F + f, u);
#pragma unroll
  for (int j = 0; j < VEC; ++j) g[j] = glu_value(g[j], u[j], kind, clamp);
  store_cols<VEC>(act + i, g);
}

extern "C" int kappai_glu(const void* gu, void* act, int T, int F, int is_bf16, int kind,
                          float limit, float slope, float shift, hipStream_t stream) {
  const size_t n = (size_t)T * F;
  if (n == 0) return 0;
  if (kind < 0 || kind > 2) return (int)hipErrorInvalidValue;
  const kappai_clamp clamp{limit, slope, shift};
  const int vec = F % 4 == 0 && ((uintptr_t)gu | (uintptr_t)act) % 16 == 0 ? 4 : 1;
  const int threads = 256;
  const unsigned blocks = (unsigned)((n / vec + threads - 1) / threads);
#define KAPPAI_GLU(TT, V)                                                                        \
  hipLaunchKernelGGL((glu_kernel<TT, V>), dim3(blocks), dim3(threads), 0, stream, (const TT*)gu, \
                     (TT*)act, F, n, kind, clamp)
  if (is_bf16) {
    if (vec == 4) KAPPAI_GLU(bf16_t, 4); else KAPPAI_GLU(bf16_t, 1);
  } else {
    if (vec == 4) KAPPAI_GLU(float, 4); else KAPPAI_GLU(float, 1);
  }
#undef KAPPAI_GLU
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// casts between float and bf16 (activations that meet a matrix stored in 32 bits)
// ---------------------------------------------------------------------------------------
template <typename TI, typename TO>
__global__ void cast_kernel(const TI* __restrict__ in, TO* __restrict__ out, size_t n) {
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) from_f32(out + i, to_f32(in[i]));
}

extern "C" int kappai_cast(const void* in, void* out, long n, int in_is_bf16, int out_is_bf16,
                           hipStream_t stream) {
  if (n <= 0) return 0;
  const int threads = 256;
  const unsigned blocks = (unsigned)((n + threads - 1) / threads);
  if (in_is_bf16 && !out_is_bf16)
    hipLaunchKernelGGL((cast_kernel<bf16_t, float>), dim3(blocks), dim3(threads), 0, stream,
                       (const bf16_t*)in, (float*)out, (size_t)n);
  else if (!in_is_bf16 && out_is_bf16)
    hipLaunchKernelGGL((cast_kernel<float, bf16_t>), dim3(blocks), dim3(threads), 0, stream,
                       (const float*)in, (bf16_t*)out, (size_t)n);
  else
    return (int)hipErrorInvalidValue;
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// a plain read of a buffer: what the memory delivers to a kernel that does nothing else
// (the yardstick beside the published peak for the kernels that stream weights and cache)
// ---------------------------------------------------------------------------------------
typedef uint32_t stream_u32x4_t __attribute__((ext_vector_type(4)));
__global__ __launch_bounds__(256) void stream_read_kernel(const stream_u32x4_t* __restrict__ p,
                                                          size_t n_per_block,
                                                          uint32_t* __restrict__ sink) {
  // every block reads its own contiguous range, 8 loads of 16 bytes a lane in flight
  const stream_u32x4_t* b = p + n_per_block * blockIdx.x;
  stream_u32x4_t acc = {0u, 0u, 0u, 0u};
  for (size_t i = threadIdx.x; i + 7 * 256 < n_per_block; i += 8 * 256) {
    stream_u32x4_t v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = b[i + u * 256];
#pragma unroll
    for (int u = 0; u < 8; ++u) acc ^= v[u];
  }
  // never true for data the host made, but the compiler cannot know: the loads stay
  if ((acc.x ^ acc.y ^ acc.z ^ acc.w) == 0x9e3779b9u && sink != nullptr) sink[0] = acc.x;
}

// Reads the first `bytes` of `p` (rounded down to what `blocks` blocks share evenly in pieces of
// 32 KB) once.  Returns the bytes read through *bytes_read.  blocks: 0 for 512, else how many
// blocks share the read (the bench takes the best of several).
extern "C" int kappai_stream_read(const void* p, long bytes, uint32_t* sink, long* bytes_read,
                                  int blocks, hipStream_t stream) {
  if (blocks == 0) blocks = 512;
  if (blocks < 1 || blocks > 65535) return (int)hipErrorInvalidValue;
  const size_t piece = 8 * 256;                                  // 16-byte elements a block and turn
  const size_t n_per_block = ((size_t)bytes / 16 / blocks / piece) * piece;
  if (bytes_read) *bytes_read = (long)(n_per_block * blocks * 16);
  if (n_per_block == 0 || ((uintptr_t)p % 16)) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(stream_read_kernel, dim3(blocks), dim3(256), 0, stream,
                     (const stream_u32x4_t*)p, n_per_block, sink);
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------------
// The other yardstick: what the matrix cores do when nothing feeds them but registers.  Every
// wave issues `iters` rounds of eight independent v_mfma_f32_32x32x16_bf16 (32 x 32 x 16
// multiply-adds each); 1024 blocks of four waves keep every SIMD of the chip busy.
// ---------------------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(8))) __bf16 probe_bf16x8_t;
typedef __attribute__((ext_vector_type(16))) float probe_f32x16_t;
__global__ __launch_bounds__(256) void mfma_probe_kernel(float* __restrict__ out, int iters) {
  probe_bf16x8_t a, b;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    a[i] = (__bf16)(threadIdx.x * 0.001f + i);
    b[i] = (__bf16)(1.0f + i * 0.01f);
  }
  probe_f32x16_t acc[8];
#pragma unroll
  for (int j = 0; j < 8; ++j)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[j][v] = 0.f;
  for (int it = 0; it < iters; ++it) {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      acc[j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, acc[j], 0, 0, 0);
  }
  float sum = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j)
#pragma unroll
    for (int v = 0; v < 16; ++v) sum += acc[j][v];
  out[(size_t)blockIdx.x * 256 + threadIdx.x] = sum;
}

// Launches the probe; `out` holds 1024 * 256 floats.  *flops receives the multiply-adds x 2.
extern "C" int kappai_mfma_probe(float* out, int iters, double* flops, hipStream_t stream) {
  const int blocks = 1024;
  if (iters < 1 || out == nullptr) return (int)hipErrorInvalidValue;
  if (flops) *flops = (double)blocks * 4 * (double)iters * 8 * (2.0 * 32 * 32 * 16);
  hipLaunchKernelGGL(mfma_probe_kernel, dim3(blocks), dim3(256), 0, stream, out, iters);
  KAPPAI_RETURN_LAUNCH_STATUS();
}
