// What the recurrences that are worked in chunks of 64 tokens on the matrix cores share: fours of numbers in either storage
// type, running sums of log decays over a chunk, tiles of rows turned round in shared memory, numbers in two bfloat16 terms.
#pragma once
#include "attention_mfma.h"

#define SS_L 64                 // tokens of a chunk
#define SS_PAD 72               // a row of 64 tokens in shared memory: 16-byte pieces, rows four banks apart

static __device__ __forceinline__ void ss_store4(float* p, const float (&v)[4]) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
static __device__ __forceinline__ void ss_store4(bf16_t* p, const float (&v)[4]) {
  *(uint2*)p = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
}
static __device__ __forceinline__ void ss_load4(const float* p, float (&v)[4]) {
  const float4 x = *(const float4*)p;
  v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
}
static __device__ __forceinline__ void ss_load4(const bf16_t* p, float (&v)[4]) {
  const uint2 x = *(const uint2*)p;
  v[0] = __uint_as_float(x.x << 16); v[1] = __uint_as_float(x.x & 0xffff0000u);
  v[2] = __uint_as_float(x.y << 16); v[3] = __uint_as_float(x.y & 0xffff0000u);
}

// In the first wave, lane t: the running sum of the log decays up to token t of the chunk (tokens past its end add 0).
// Differences of two such sums are what counts, and one token may decay by thousands where its neighbours hardly do: the
// sums are 64-bit. A log decay below -128 counts as -128 (its exponential is 0 in 32-bit either way).
// `stride`: floats from a token's decays to the next token's (0: every token has the same).
static __device__ __forceinline__ double ss_running(const float* __restrict__ logs, int tok0, int len, int stride, int h) {
  const int t = threadIdx.x;
  double b = t < len ? (double)fmaxf(logs[(int64_t)(tok0 + t) * stride + h], -128.f) : 0.0;
#pragma unroll
  for (int off = 1; off < TS_WAVE; off <<= 1) {
    const double up = __shfl_up(b, off, TS_WAVE);
    if (t >= off) b += up;
  }
  return b;
}

static __device__ __forceinline__ uint4 ss_piece(const bf16_t* p, bool there) {
  return there ? *(const uint4*)p : make_uint4(0, 0, 0, 0);
}
static __device__ __forceinline__ float ss_half(const uint4& p, int k) {
  const uint32_t w = (&p.x)[k >> 1];
  return __uint_as_float(k & 1 ? w & 0xffff0000u : w << 16);
}
static __device__ __forceinline__ uint32_t ss_rest(uint32_t hi, float a, float b) {
  return pack_bf16(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

// A tile of 64 tokens by 64 columns of `src` (rows `row` apart, columns at `col`, those from `cols` on absent) turned
// round into dst[column][token]; as it is, or (WEIGHTED) times weight[token] in two terms.
template <bool WEIGHTED>
static __device__ __forceinline__ void ss_turn(bf16_t (*dst)[SS_PAD], bf16_t (*rest)[SS_PAD], const bf16_t* __restrict__ src, int row,
                                               int tok0, int len, int cols, const float* weight) {
  // a thread takes eight columns of two neighbouring tokens; neighbouring threads neighbouring pairs of tokens
  const int pair = threadIdx.x & 31, p = threadIdx.x >> 5;
  const int ta = 2 * pair, tb = ta + 1;
  const bf16_t* at = src + (int64_t)tok0 * row + 8 * p;
  const uint4 a = ss_piece(at + (int64_t)min(ta, len - 1) * row, ta < len && 8 * p < cols);
  const uint4 b = ss_piece(at + (int64_t)min(tb, len - 1) * row, tb < len && 8 * p < cols);
#pragma unroll
  for (int k = 0; k < 8; ++k) {
    float x = ss_half(a, k), y = ss_half(b, k);
    if constexpr (WEIGHTED) x *= weight[ta], y *= weight[tb];
    const uint32_t hi = pack_bf16(x, y);
    *(uint32_t*)&dst[8 * p + k][ta] = hi;
    if constexpr (WEIGHTED) *(uint32_t*)&rest[8 * p + k][ta] = ss_rest(hi, x, y);
  }
}
