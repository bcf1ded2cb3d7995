// State-space recurrence with one decay a head and token ("state-space duality"): per head a state
// S [dv, N] in float32 (a slot per request, column by column: N consecutive for a value channel),
//   dt = softplus(z + z_bias[h]),  a = exp(-rate[h] dt),
//   S <- a S + x (dt B)^T,         y = S C + D[h] x,
// with B and C [N] of the head's group (head h reads group h / (H / G)) and x [dv].  x, B and C are
// read from the rows the short convolution left (columns x_at + h dv, b_at + g N, c_at + g N), z from
// the projection; everything made of them is float32.
//
// Two forms.  The walk: a column of S over KS neighbouring lanes, tokens in order (decoding, short
// portions, float32, any size).  The chunks: runs of up to SS_L rows, inside which no token waits for
// another (long portions in bfloat16), three passes on the matrix cores.  A segment that starts at
// position 0 starts from zero, whatever the slot holds.
#include "matrix_state.h"

#define SS_THREADS 256

struct ss_columns {
  int stride, x_at, b_at, c_at;      // of the convolution's rows
};

// R values of a row of B or C from `p`: the lane's rows of la_row, zeros beyond n
template <int KS, int R, typename T>
__device__ __forceinline__ void ss_rows(const T* __restrict__ p, int s, int n, int vec,
                                        float (&v)[R]) {
#pragma unroll
  for (int r4 = 0; r4 < R; r4 += 4) {
    const int row = la_row<KS>(s, r4);
    if (vec && sizeof(T) == 2) {
      uint2 q = make_uint2(0u, 0u);
      if (row < n) q = *reinterpret_cast<const uint2*>(p + row);
      v[r4] = __uint_as_float(q.x << 16);
      v[r4 + 1] = __uint_as_float(q.x & 0xffff0000u);
      v[r4 + 2] = __uint_as_float(q.y << 16);
      v[r4 + 3] = __uint_as_float(q.y & 0xffff0000u);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[r4 + i] = row + i < n ? to_f32(p[row + i]) : 0.f;
    }
  }
}

// grid: (columns, heads, segments), four waves a block, 64 / KS columns a wave.  The next token's
// loads are on their way while this one is worked on.  `vec`: N, the row stride and the columns are
// multiples of four values.
template <int KS, int R, typename T>
__global__ __launch_bounds__(SS_THREADS) void state_space_walk_kernel(
    const T* __restrict__ xbc, ss_columns at, const T* __restrict__ z, int z_stride,
    const float* __restrict__ z_bias, const float* __restrict__ rate,
    const float* __restrict__ skip, float* __restrict__ state, const int* __restrict__ seg_start,
    const int* __restrict__ seg_pos0, const int* __restrict__ seg_slot, int H, int G, int N,
    int dv, int vec, float* __restrict__ out) {
  constexpr int COLS = WAVE / KS;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int seg = blockIdx.z, h = blockIdx.y, g = h / (H / G), s = lane % KS;
  const int c = (blockIdx.x * (SS_THREADS / WAVE) + wave) * COLS + lane / KS;
  const bool col_ok = c < dv;
  const int cc = col_ok ? c : dv - 1;
  const int first = seg_start[seg], last = seg_start[seg + 1];
  if (first >= last) return;
  float* st = state + (((size_t)seg_slot[seg] * H + h) * dv + cc) * N;
  float Bn[R], Cn[R], xn, zn;
  auto fetch = [&](int t) {
    const T* row = xbc + (size_t)t * at.stride;
    ss_rows<KS, R>(row + at.b_at + g * N, s, N, vec, Bn);
    ss_rows<KS, R>(row + at.c_at + g * N, s, N, vec, Cn);
    xn = to_f32(row[at.x_at + h * dv + cc]);
    zn = to_f32(z[(size_t)t * z_stride + h]);
  };
  fetch(first);
  float S[R];
  la_load_rows<KS, R>(st, s, N, seg_pos0[seg] > 0, S);
  const float bias = z_bias[h], rt = rate[h], sk = skip[h];
  for (int t = first; t < last; ++t) {
    float B[R], C[R];
#pragma unroll
    for (int r = 0; r < R; ++r) { B[r] = Bn[r]; C[r] = Cn[r]; }
    const float x = xn, dt = la_softplus(zn + bias);
    if (t + 1 < last) fetch(t + 1);
    const float a = expf(-rt * dt), u = dt * x;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < R; ++r) {
      S[r] = fmaf(a, S[r], B[r] * u);
      o[r % 4] = fmaf(S[r], C[r], o[r % 4]);
    }
    const float y = ks_sum<KS>((o[0] + o[1]) + (o[2] + o[3]));
    if (s == 0 && col_ok) out[((size_t)t * H + h) * dv + c] = fmaf(sk, x, y);
  }
  if (col_ok) la_store_rows<KS, R>(st, s, N, S);
}

template <typename T>
static int walk_launch(const T* xbc, ss_columns at, const T* z, int z_stride, const float* z_bias,
                       const float* rate, const float* skip, float* state, const int* seg_start,
                       const int* seg_pos0, const int* seg_slot, int S, int H, int G, int N,
                       int dv, float* out, hipStream_t stream) {
  const int r = N <= 64 * 8 ? 8 : 16;
  int ks = 1;
  while (ks * r < N) ks *= 2;
  const int vec = ((N | at.stride | at.b_at | at.c_at) % 4 == 0) && (uintptr_t)xbc % 8 == 0;
  const int per_block = (SS_THREADS / WAVE) * (WAVE / ks);
  const dim3 grid((dv + per_block - 1) / per_block, H, S);
#define SS_WALK(KS_, R_)                                                                         \
  case KS_ * 100 + R_:                                                                           \
    hipLaunchKernelGGL((state_space_walk_kernel<KS_, R_, T>), grid, dim3(SS_THREADS), 0, stream, \
                       xbc, at, z, z_stride, z_bias, rate, skip, state, seg_start, seg_pos0,     \
                       seg_slot, H, G, N, dv, vec, out);                                         \
    break;
  switch (ks * 100 + r) {
    SS_WALK(1, 8) SS_WALK(2, 8) SS_WALK(4, 8) SS_WALK(8, 8) SS_WALK(16, 8) SS_WALK(32, 8)
    SS_WALK(64, 8) SS_WALK(64, 16)
    default: return (int)hipErrorInvalidValue;
  }
#undef SS_WALK
  KAPPAI_RETURN_LAUNCH_STATUS();
}

// xbc [T, stride], z [T, >= H] with a row stride, state [slots, H, dv, N], out [T, H dv] float32.
extern "C" int kappai_state_space_walk(const void* xbc, int stride, int x_at, int b_at, int c_at,
                                       const void* z, int z_stride, const float* z_bias,
                                       const float* rate, const float* skip, float* state,
                                       const int* seg_start, const int* seg_pos0,
                                       const int* seg_slot, int T, int S, int H, int G, int N,
                                       int dv, float* out, int is_bf16, hipStream_t stream) {
  if (T <= 0 || S <= 0) return 0;
  if (H < 1 || G < 1 || H % G || H > 65535 || S > 65535 || N < 1 || N > 64 * 16 || dv < 1)
    return (int)hipErrorInvalidValue;
  const ss_columns at{stride, x_at, b_at, c_at};
  if (is_bf16)
    return walk_launch<bf16_t>((const bf16_t*)xbc, at, (const bf16_t*)z, z_stride, z_bias, rate,
                               skip, state, seg_start, seg_pos0, seg_slot, S, H, G, N, dv, out,
                               stream);
  return walk_launch<float>((const float*)xbc, at, (const float*)z, z_stride, z_bias, rate, skip,
                            state, seg_start, seg_pos0, seg_slot, S, H, G, N, dv, out, stream);
}

// ---------------------------------------------------------------------------------------
// Chunks.  With L_j the sum of -rate dt over the chunk's rows up to and with j, and S0 the state the
// chunk starts from,
//   y_i = sum_(j <= i) (C_i . B_j) exp(L_i - L_j) dt_j x_j + exp(L_i) S0 C_i + D x_i
//   S   = exp(L_(n-1)) S0 + sum_j exp(L_(n-1) - L_j) dt_j x_j B_j^T.
// Every exponent is <= 0 and nothing is divided by a decay.  The products run on the matrix cores
// (v_mfma_f32_16x16x32_bf16, float accumulators).  x, B and C are bfloat16 as they come; a float32
// operand (the weights between tokens, the weighted x, the state) goes in as three bfloat16 values
// whose sum is that float: three products in place of one keep all its bits.
//
// Fragments: lane l holds row (or column) l % 16 and eight values of the summed index, and of a
// result tile column l % 16 and rows 4 (l / 16) .. + 3.  Which eight is free as long as both operands
// agree: the weights between tokens leave the first product as rows j = 4 (l / 16) .. + 3 of two
// tiles, and go into the second as they are, with x read from LDS in that order.
// ---------------------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(8))) __bf16 ss_bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float ss_f32x4_t;

#define SS_L 128               // most rows of a chunk
#define SS_V 64                // value channels a block takes
#define SS_LS (SS_L + 4)       // row stride in LDS of what lies [channel][row] (8-byte pieces)

extern "C" int kappai_state_space_chunk_rows() { return SS_L; }

// three fragments whose sum is v
__device__ __forceinline__ void ss_split(const float (&v)[8], ss_bf16x8_t (&f)[3]) {
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const __bf16 a = (__bf16)v[i];
    const float r = v[i] - (float)a;
    const __bf16 b = (__bf16)r;
    f[0][i] = a;
    f[1][i] = b;
    f[2][i] = (__bf16)(r - (float)b);
  }
}

__device__ __forceinline__ ss_f32x4_t ss_mfma(ss_bf16x8_t a, ss_bf16x8_t b, ss_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// eight values from two 8-byte pieces of LDS
__device__ __forceinline__ ss_bf16x8_t ss_pieces(const bf16_t* p, const bf16_t* q) {
  const uint2 a = *reinterpret_cast<const uint2*>(p), b = *reinterpret_cast<const uint2*>(q);
  return __builtin_bit_cast(ss_bf16x8_t, make_uint4(a.x, a.y, b.x, b.y));
}

// By the first wave: Ls [SS_L] the sums of logarithms and dts [SS_L] the step sizes (zero behind row
// n); or, for the chunks' own sums, dts [SS_L] the step sizes times the decay up to the chunk's end and
// Ls [0] that of the whole chunk.
template <bool TO_END>
__device__ __forceinline__ void ss_decays(const bf16_t* __restrict__ z, int z_stride, int row0,
                                          int n, int h, float bias, float rate, float* Ls,
                                          float* dts) {
  if (threadIdx.x >= WAVE) return;
  const int lane = threadIdx.x;
  constexpr int PER = SS_L / WAVE;
  float l[PER], dt[PER], run = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int j = lane * PER + i;
    dt[i] = 0.f;
    if (j < n) dt[i] = la_softplus(bf16_to_f32(z[(size_t)(row0 + j) * z_stride + h]) + bias);
    run += -rate * dt[i];
    l[i] = run;
  }
  float before = run;                      // inclusive sum over the lanes, then without the own
#pragma unroll
  for (int m = 1; m < WAVE; m *= 2) {
    const float o = __shfl_up(before, m);
    if (lane >= m) before += o;
  }
  before = __shfl_up(before, 1);
  if (lane == 0) before = 0.f;
  if (TO_END) {
    const float end = __shfl(before + run, WAVE - 1);
#pragma unroll
    for (int i = 0; i < PER; ++i) dts[lane * PER + i] = dt[i] * expf(end - (before + l[i]));
    if (lane == 0) Ls[0] = end;
    return;
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    Ls[lane * PER + i] = before + l[i];
    dts[lane * PER + i] = dt[i];
  }
}

// `width` channels (a multiple of eight) of the chunk's rows from column `col`, to LDS as
// [channel][row]; zeros behind row n and behind channel `have`
__device__ __forceinline__ void ss_stage_turned(const bf16_t* __restrict__ xbc, int stride, int col,
                                                int row0, int n, int have, int width, bf16_t* dst) {
  const int oct = width / 8;
  for (int i = threadIdx.x; i < (oct + 7) / 8 * 8 * SS_L; i += blockDim.x) {
    // eight lanes take neighbouring pieces of a row, the next eight the next row
    const int o = (i % 8) + 8 * (i / (8 * SS_L)), j = (i / 8) % SS_L;
    if (o >= oct) continue;
    uint4 q = make_uint4(0u, 0u, 0u, 0u);
    if (j < n && 8 * o < have)
      q = *reinterpret_cast<const uint4*>(xbc + (size_t)(row0 + j) * stride + col + 8 * o);
    const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
    for (int e = 0; e < 8; ++e)
      dst[(8 * o + e) * SS_LS + j] = (bf16_t)(w[e / 2] >> (16 * (e % 2)));
  }
}

// The chunks' own sums: carry [n_chunks, H, dv, N] = sum_j exp(L_(n-1) - L_j) dt_j x_j B_j^T, total
// [n_chunks, H] = exp(L_(n-1)).  Grid (chunks, heads, pieces of SS_V value channels); a wave a tile
// of 16 value channels, all of N.
template <int NS>
__global__ __launch_bounds__(SS_THREADS) void state_space_sums_kernel(
    const bf16_t* __restrict__ xbc, ss_columns at, const bf16_t* __restrict__ z, int z_stride,
    const float* __restrict__ z_bias, const float* __restrict__ rate,
    const int* __restrict__ chunks, int H, int G, int N, int dv, float* __restrict__ carry,
    float* __restrict__ total) {
  extern __shared__ __attribute__((aligned(16))) bf16_t ss_lds[];
  __shared__ __attribute__((aligned(16))) float wt[SS_L];
  __shared__ float end[1];
  bf16_t* Xt = ss_lds;                           // [SS_V][SS_LS]
  bf16_t* Bt = ss_lds + SS_V * SS_LS;            // [32 NS][SS_LS]
  const int ch = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * SS_V;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int row0 = chunks[3 * ch + 1], n = min(chunks[3 * ch + 2], SS_L), g = h / (H / G);
  ss_decays<true>(z, z_stride, row0, n, h, z_bias[h], rate[h], end, wt);
  ss_stage_turned(xbc, at.stride, at.x_at + h * dv + v0, row0, n, dv - v0, SS_V, Xt);
  ss_stage_turned(xbc, at.stride, at.b_at + g * N, row0, n, N, 32 * NS, Bt);
  __syncthreads();
  if (blockIdx.z == 0 && threadIdx.x == 0) total[(size_t)ch * H + h] = expf(end[0]);
  const int lr = lane % 16, kg = lane / 16;
  const int v = v0 + 16 * wave + lr;
  if (v0 + 16 * wave >= dv) return;
  ss_f32x4_t acc[2 * NS];
#pragma unroll
  for (int i = 0; i < 2 * NS; ++i) acc[i] = ss_f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < n; k0 += 32) {
    const int j0 = k0 + 8 * kg;
    const bf16_t* xp = Xt + (16 * wave + lr) * SS_LS + j0;
    float w[8], f[8];
    const ss_bf16x8_t x8 = ss_pieces(xp, xp + 4);
    load8(wt + j0, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) w[e] = (float)x8[e] * f[e];
    ss_bf16x8_t xw[3];
    ss_split(w, xw);
#pragma unroll
    for (int i = 0; i < 2 * NS; ++i) {
      const bf16_t* bp = Bt + (16 * i + lr) * SS_LS + j0;
      const ss_bf16x8_t b = ss_pieces(bp, bp + 4);
#pragma unroll
      for (int t = 0; t < 3; ++t) acc[i] = ss_mfma(b, xw[t], acc[i]);
    }
  }
  if (v >= dv) return;
  float* dst = carry + (((size_t)ch * H + h) * dv + v) * N;
#pragma unroll
  for (int i = 0; i < 2 * NS; ++i) {
    const int at_n = 16 * i + 4 * kg;
    if (at_n < N)
      *reinterpret_cast<float4*>(dst + at_n) =
          make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
  }
}

// Over a segment's chunks in order: carry becomes the state every chunk starts from, the slot the
// state behind the last.  A thread four elements.
__global__ __launch_bounds__(SS_THREADS) void state_space_carry_kernel(
    const float* __restrict__ total, const int* __restrict__ seg_chunk0,
    const int* __restrict__ seg_pos0, const int* __restrict__ seg_slot, int H, int n_el,
    float* __restrict__ carry, float* __restrict__ state) {
  const int seg = blockIdx.x, h = blockIdx.y;
  const int e = (blockIdx.z * SS_THREADS + threadIdx.x) * 4;
  if (e >= n_el) return;
  const int ch0 = seg_chunk0[seg], ch1 = seg_chunk0[seg + 1];
  if (ch0 >= ch1) return;
  float* st = state + ((size_t)seg_slot[seg] * H + h) * n_el + e;
  float4 S = make_float4(0.f, 0.f, 0.f, 0.f);
  if (seg_pos0[seg] > 0) S = *reinterpret_cast<const float4*>(st);
  for (int c = ch0; c < ch1; c += 4) {
    float4 own[4];
    float f[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = min(c + i, ch1 - 1);
      own[i] = *reinterpret_cast<const float4*>(carry + ((size_t)k * H + h) * n_el + e);
      f[i] = total[(size_t)k * H + h];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (c + i >= ch1) break;
      *reinterpret_cast<float4*>(carry + ((size_t)(c + i) * H + h) * n_el + e) = S;
      S.x = fmaf(f[i], S.x, own[i].x);
      S.y = fmaf(f[i], S.y, own[i].y);
      S.z = fmaf(f[i], S.z, own[i].z);
      S.w = fmaf(f[i], S.w, own[i].w);
    }
  }
  *reinterpret_cast<float4*>(st) = S;
}

// The chunks' outputs.  Grid as for the sums; a wave takes two tiles of 16 rows of the chunk, one near
// its start and one near its end (a row meets as many of the chunk's rows as lie before it), and the
// block's value channels.
#define SS_TILES (SS_L / 16)
#define SS_OUT_THREADS (SS_TILES / 2 * WAVE)
template <int NS>
__global__ __launch_bounds__(SS_OUT_THREADS) void state_space_out_kernel(
    const bf16_t* __restrict__ xbc, ss_columns at, const bf16_t* __restrict__ z, int z_stride,
    const float* __restrict__ z_bias, const float* __restrict__ rate,
    const float* __restrict__ skip, const int* __restrict__ chunks, int H, int G, int N, int dv,
    const float* __restrict__ carry, float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) bf16_t ss_lds[];
  __shared__ __attribute__((aligned(16))) float Ls[SS_L];
  __shared__ __attribute__((aligned(16))) float dts[SS_L];
  constexpr int BS = 32 * NS + 8;                // row stride of B in LDS
  constexpr int VT = SS_V / 16;
  bf16_t* Xt = ss_lds;                           // [SS_V][SS_LS]
  bf16_t* Bs = ss_lds + SS_V * SS_LS;            // [SS_L][BS]
  const int ch = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * SS_V;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int row0 = chunks[3 * ch + 1], n = min(chunks[3 * ch + 2], SS_L), g = h / (H / G);
  const int lr = lane % 16, kg = lane / 16;
  const int first[2] = {16 * wave, 16 * (SS_TILES - 1 - wave)};
  // what only this wave reads is asked for first
  ss_bf16x8_t cf[2][NS];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      uint4 q = make_uint4(0u, 0u, 0u, 0u);
      const int i = first[u] + lr;
      if (i < n && 32 * s + 8 * kg < N)
        q = *reinterpret_cast<const uint4*>(xbc + (size_t)(row0 + i) * at.stride + at.c_at +
                                            g * N + 32 * s + 8 * kg);
      cf[u][s] = __builtin_bit_cast(ss_bf16x8_t, q);
    }
  ss_decays<false>(z, z_stride, row0, n, h, z_bias[h], rate[h], Ls, dts);
  ss_stage_turned(xbc, at.stride, at.x_at + h * dv + v0, row0, n, dv - v0, SS_V, Xt);
  for (int p = threadIdx.x; p < SS_L * 4 * NS; p += SS_OUT_THREADS) {
    const int j = p / (4 * NS), e = (p % (4 * NS)) * 8;
    uint4 q = make_uint4(0u, 0u, 0u, 0u);
    if (j < n && e < N)
      q = *reinterpret_cast<const uint4*>(xbc + (size_t)(row0 + j) * at.stride + at.b_at + g * N + e);
    *reinterpret_cast<uint4*>(Bs + j * BS + e) = q;
  }
  // the state the chunk starts from (before the barrier: it needs nothing that is staged)
  ss_f32x4_t acc[2][VT];
  const float* S0 = carry + (((size_t)ch * H + h) * dv + v0) * N;
#pragma unroll
  for (int vt = 0; vt < VT; ++vt) {
    acc[0][vt] = acc[1][vt] = ss_f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int v = 16 * vt + lr;
    if (v0 + 16 * vt >= dv || first[0] >= n) continue;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      float w[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = 0.f;
      if (v0 + v < dv && 32 * s + 8 * kg < N) load8(S0 + (size_t)v * N + 32 * s + 8 * kg, w);
      ss_bf16x8_t sf[3];
      ss_split(w, sf);
#pragma unroll
      for (int t = 0; t < 3; ++t) {
        acc[0][vt] = ss_mfma(sf[t], cf[0][s], acc[0][vt]);
        acc[1][vt] = ss_mfma(sf[t], cf[1][s], acc[1][vt]);
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int i0 = first[u], i = i0 + lr;
    if (i0 >= n) continue;
    // times the decay up to this row
    const float Li = Ls[i], fade = expf(Li);
#pragma unroll
    for (int vt = 0; vt < VT; ++vt)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[u][vt][r] *= fade;
    // the chunk's own rows, 32 at a time
    for (int jp = 0; jp <= i0; jp += 32) {
      float p[8];
#pragma unroll
      for (int jt = 0; jt < 2; ++jt) {
        ss_f32x4_t gt = ss_f32x4_t{0.f, 0.f, 0.f, 0.f};
        const bf16_t* bp = Bs + (jp + 16 * jt + lr) * BS + 8 * kg;
#pragma unroll
        for (int s = 0; s < NS; ++s)
          gt = ss_mfma(__builtin_bit_cast(ss_bf16x8_t, *reinterpret_cast<const uint4*>(bp + 32 * s)),
                       cf[u][s], gt);
        const int j = jp + 16 * jt + 4 * kg;
        const float4 l4 = *reinterpret_cast<const float4*>(Ls + j);
        const float4 d4 = *reinterpret_cast<const float4*>(dts + j);
        const float l[4] = {l4.x, l4.y, l4.z, l4.w}, d[4] = {d4.x, d4.y, d4.z, d4.w};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          p[4 * jt + r] = j + r <= i ? gt[r] * (expf(Li - l[r]) * d[r]) : 0.f;
      }
      ss_bf16x8_t pf[3];
      ss_split(p, pf);
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const bf16_t* xp = Xt + (16 * vt + lr) * SS_LS + jp + 4 * kg;
        const ss_bf16x8_t xf = ss_pieces(xp, xp + 16);
#pragma unroll
        for (int t = 0; t < 3; ++t) acc[u][vt] = ss_mfma(xf, pf[t], acc[u][vt]);
      }
    }
    if (i >= n) continue;
    const float sk = skip[h];
    const bf16_t* xr = xbc + (size_t)(row0 + i) * at.stride + at.x_at + h * dv;
    float* dst = out + ((size_t)(row0 + i) * H + h) * dv;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int v = v0 + 16 * vt + 4 * kg;
      if (v >= dv) continue;
      const uint2 q = *reinterpret_cast<const uint2*>(xr + v);
      *reinterpret_cast<float4*>(dst + v) =
          make_float4(fmaf(sk, __uint_as_float(q.x << 16), acc[u][vt][0]),
                      fmaf(sk, __uint_as_float(q.x & 0xffff0000u), acc[u][vt][1]),
                      fmaf(sk, __uint_as_float(q.y << 16), acc[u][vt][2]),
                      fmaf(sk, __uint_as_float(q.y & 0xffff0000u), acc[u][vt][3]));
    }
  }
}

// What the chunks take: sizes and columns in multiples of eight, N up to 256.
static bool chunks_fit(const void* xbc, int stride, int x_at, int b_at, int c_at, int N, int dv) {
  return ((stride | x_at | b_at | c_at | N | dv) % 8) == 0 && N <= 256 &&
         (uintptr_t)xbc % 16 == 0;
}

extern "C" int kappai_state_space_chunks_fit(const void* xbc, int stride, int x_at, int b_at,
                                             int c_at, int N, int dv) {
  return chunks_fit(xbc, stride, x_at, b_at, c_at, N, dv) ? 1 : 0;
}

// bfloat16 rows; chunks [n_chunks, 3] = (segment, first row, rows <= SS_L), seg_chunk0 [S + 1], carry
// [n_chunks, H, dv, N] and total [n_chunks, H] floats of scratch.
extern "C" int kappai_state_space_chunks(
    const void* xbc_v, int stride, int x_at, int b_at, int c_at, const void* z, int z_stride,
    const float* z_bias, const float* rate, const float* skip, float* state, const int* seg_pos0,
    const int* seg_slot, const int* chunks, const int* seg_chunk0, int n_chunks, int chunk_rows,
    int T, int S, int H, int G, int N, int dv, float* carry, float* total, float* out,
    hipStream_t stream) {
  if (T <= 0 || S <= 0) return 0;
  if (H < 1 || G < 1 || H % G || H > 65535 || N < 1 || dv < 1 || n_chunks < 1 || chunk_rows < 1 ||
      chunk_rows > SS_L || !chunks || !seg_chunk0 || !carry || !total ||
      !chunks_fit(xbc_v, stride, x_at, b_at, c_at, N, dv) ||
      ((uintptr_t)state | (uintptr_t)carry | (uintptr_t)out) % 16)
    return (int)hipErrorInvalidValue;
  const bf16_t* xbc = (const bf16_t*)xbc_v;
  const ss_columns at{stride, x_at, b_at, c_at};
  const dim3 grid(n_chunks, H, (dv + SS_V - 1) / SS_V);
  const int n_el = dv * N, el_blocks = (n_el / 4 + SS_THREADS - 1) / SS_THREADS;
  if (grid.z > 65535 || el_blocks > 65535) return (int)hipErrorInvalidValue;
#define SS_CHUNKS(NS_)                                                                           \
  hipLaunchKernelGGL(state_space_sums_kernel<NS_>, grid, dim3(SS_THREADS),                       \
                     (SS_V + 32 * NS_) * SS_LS * sizeof(bf16_t), stream, xbc, at,                \
                     (const bf16_t*)z, z_stride, z_bias, rate, chunks, H, G, N, dv, carry,       \
                     total);                                                                     \
  hipLaunchKernelGGL(state_space_carry_kernel, dim3(S, H, el_blocks), dim3(SS_THREADS), 0,       \
                     stream, total, seg_chunk0, seg_pos0, seg_slot, H, n_el, carry, state);      \
  hipLaunchKernelGGL(state_space_out_kernel<NS_>, grid, dim3(SS_OUT_THREADS),                    \
                     (SS_V * SS_LS + SS_L * (32 * NS_ + 8)) * sizeof(bf16_t), stream, xbc, at,   \
                     (const bf16_t*)z, z_stride, z_bias, rate, skip, chunks, H, G, N, dv, carry, \
                     out)
  if (N <= 32) { SS_CHUNKS(1); }
  else if (N <= 64) { SS_CHUNKS(2); }
  else if (N <= 128) { SS_CHUNKS(4); }
  else {
    static bool wide = false;            // (more than 64 KB of LDS a block)
    if (!wide) {
      (void)hipFuncSetAttribute((const void*)&state_space_sums_kernel<8>,
                                hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
      (void)hipFuncSetAttribute((const void*)&state_space_out_kernel<8>,
                                hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
      wide = true;
    }
    SS_CHUNKS(8);
  }
#undef SS_CHUNKS
  KAPPAI_RETURN_LAUNCH_STATUS();
}
