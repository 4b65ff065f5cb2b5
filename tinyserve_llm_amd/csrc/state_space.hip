// A state-space mixer with one decay per head (the Mamba-2 recurrence). Per head a state S [vdim, state], 32-bit, zero
// at a request's start; head h shares its B and C rows with the heads of its group. For a token with x [vdim],
// B, C [state], a step size d > 0 and the log decay l = -exp(A_log) d <= 0:
//     S' = exp(l) S + d x B^T,   y = S' C + D x.
//   * `ts_ssd_prepare`: from a projected row [z | x | B | C | dt] (32-bit) to what the recurrence reads: x, B and C
//     through a causal convolution per channel with a bias and silu, in the activations' storage type and in a row of
//     their own where every head's x has `vp` places and every group's B and C `np` (multiples of 16 and 32; the places
//     behind a head's or a group's own numbers hold zeros, so that no kernel after this one asks for sizes); d and l in
//     32-bit. The rows ahead of a request's first token of the step come from its state slot.
//   * `ts_ssd_conv_keep`: leaves the convolution's last inputs in the slots (a step of single tokens does it in prepare).
//   * `ts_ssd_step`: walks each request's tokens of the step in order with the state in registers; a request's state is
//     read from its slot at the start and written back at the end. For decoded tokens, short portions, and 32-bit models.
//     Step sizes and decays may also be one number per head for all tokens (`token_stride` 0), the decays then given
//     themselves beside their logarithms (`keeps`), so that a long walk multiplies by exactly them.
//   * `ts_ssd_chunks`: long portions in bfloat16, in chunks of 64 tokens on the matrix cores. With b_t the sum of l from
//     the chunk's first token to t (every exponent below is <= 0) and S0 the state before the chunk,
//         y_t = exp(b_t) S0 C_t + sum_{j <= t} exp(b_t - b_j) d_j (C_t . B_j) x_j + D x_t,
//         S   = exp(b_L) S0 + sum_j exp(b_L - b_j) d_j x_j B_j^T:
//     what every chunk adds to the state (a workgroup per chunk and head), a scan over a request's chunks element by
//     element, and the read-outs. x, B and C are the operands as they are; what is 32-bit by nature (weighted x, the
//     weights of the second sum, S0) enters a product as two bfloat16 terms.
//   * `ts_gated_group_norm`: y silu(z), cut into equal parts, each divided by its own root mean square, times a weight.
#include "chunk_ops.h"

#define SS_THREADS 256
#define SS_WAVES (SS_THREADS / TS_WAVE)
#define SS_MAX_TAPS 16

struct SsSizes { int heads, vdim, vp, groups, state, np, taps; };

// A thread per four places of the mixed row (or per head, for d and l) and TT tokens. TAPS: 4 or 16, at least the taps.
// VEC: vdim and state are multiples of four and the projected rows 16-byte aligned.
template <typename TO, int TAPS, int TT, bool VEC>
__global__ void __launch_bounds__(SS_THREADS)
ssd_prepare_kernel(TO* __restrict__ mixed, float* __restrict__ steps, float* __restrict__ logs, const float* __restrict__ proj,
                   int64_t stride, const float* __restrict__ conv_w, const float* __restrict__ conv_b, float* __restrict__ kept,
                   int64_t kept_stride, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                   const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ seq_of_token,
                   const int32_t* __restrict__ state_slots, int num_tokens, SsSizes z, int moves) {
  const int inner = z.heads * z.vdim, row = z.heads * z.vp + 2 * z.groups * z.np;
  const int quad = blockIdx.x * blockDim.x + threadIdx.x;
  const int t0 = blockIdx.y * TT, t1 = min(t0 + TT, num_tokens);
  if (quad >= row / 4) {
    const int h = quad - row / 4;
    if (h >= z.heads) return;
    const float rate = -expf(a_log[h]), bias = dt_bias[h];
    const float* src = proj + 2 * inner + 2 * z.groups * z.state + h;
    for (int t = t0; t < t1; ++t) {
      const float s = src[(int64_t)t * stride] + bias;
      const float d = fmaxf(s, 0.f) + log1pf(expf(-fabsf(s)));          // softplus
      steps[(int64_t)t * z.heads + h] = d;
      logs[(int64_t)t * z.heads + h] = rate * d;
    }
    return;
  }
  const int place = 4 * quad;
  int col, count;                                            // the place's column of the projected row, how many of the four are there
  if (place < z.heads * z.vp) {
    const int h = place / z.vp, off = place - h * z.vp;
    col = inner + h * z.vdim + off;
    count = min(4, max(0, z.vdim - off));
  } else {
    const int at = place - z.heads * z.vp, half = z.groups * z.np;
    const int which = at / half, in = at - which * half;
    const int g = in / z.np, off = in - g * z.np;
    col = 2 * inner + (which * z.groups + g) * z.state + off;
    count = min(4, max(0, z.state - off));
  }
  float w[TAPS][4], b[4];
#pragma unroll
  for (int d = 0; d < TAPS; ++d)
#pragma unroll
    for (int k = 0; k < 4; ++k) w[d][k] = 0.f;
#pragma unroll
  for (int d = 0; d < TAPS; ++d)
    if (d < z.taps) ss_load4(conv_w + (int64_t)(z.taps - 1 - d) * row + place, w[d]);
  ss_load4(conv_b + place, b);
  auto input = [&](int t, float (&u)[4]) {
    const float* src = proj + (int64_t)t * stride + col;
    if constexpr (VEC) {
      if (count == 4) ss_load4(src, u);
      else u[0] = u[1] = u[2] = u[3] = 0.f;
    } else {
#pragma unroll
      for (int k = 0; k < 4; ++k) u[k] = k < count ? src[k] : 0.f;
    }
  };
  float past[TAPS][4];                                       // past[d]: the channel's input d tokens before the one at hand
#pragma unroll
  for (int d = 0; d < TAPS; ++d)
#pragma unroll
    for (int k = 0; k < 4; ++k) past[d][k] = 0.f;
  for (int t = t0; t < t1; ++t) {
    const int seq = seq_of_token[t], index = t - cu_seqlens[seq];
    float* slot = kept + (int64_t)state_slots[seq] * kept_stride + place;
    if (t == t0 || index == 0) {
#pragma unroll
      for (int d = 1; d < TAPS; ++d)
        if (d < z.taps) {
          if (index >= d) input(t - d, past[d]);
          else ss_load4(slot + (int64_t)(z.taps - 1 + index - d) * row, past[d]);
        }
    } else {
#pragma unroll
      for (int d = TAPS - 1; d > 0; --d)
#pragma unroll
        for (int k = 0; k < 4; ++k) past[d][k] = past[d - 1][k];
    }
    input(t, past[0]);
    float y[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      float s = b[k];
#pragma unroll
      for (int d = TAPS - 1; d >= 0; --d) s = fmaf(w[d][k], past[d][k], s);
      y[k] = s / (1.0f + expf(-s));
    }
    ss_store4(mixed + (int64_t)t * row + place, y);
    if (moves) {                                             // (the request's only token of the step: nobody else reads its slot)
#pragma unroll
      for (int d = 0; d < TAPS - 1; ++d)
        if (d < z.taps - 1) ss_store4(slot + (int64_t)(z.taps - 2 - d) * row, past[d]);
    }
  }
}

// kept: each slot's convolution inputs, float32 [taps - 1, row], `kept_stride` floats from slot to slot. conv_w float32
// [taps, row] (last: the current token's), conv_b float32 [row], zeros where a place holds no channel. moves: every
// request of the step feeds exactly one token.
extern "C" int ts_ssd_prepare(void* mixed, int out_dtype, float* steps, float* logs, const float* proj, int64_t stride,
                              const float* conv_w, const float* conv_b, float* kept, int64_t kept_stride, const float* dt_bias,
                              const float* a_log, const int32_t* cu_seqlens, const int32_t* seq_of_token,
                              const int32_t* state_slots, int num_tokens, int heads, int vdim, int vp, int groups, int state,
                              int np, int taps, int moves, hipStream_t stream) {
  if (num_tokens <= 0) return TS_OK;
  const int64_t row = (int64_t)heads * vp + 2 * (int64_t)groups * np;
  if (heads <= 0 || groups <= 0 || heads % groups || vdim <= 0 || state <= 0 || vp < vdim || np < state || vp % 16 || np % 32 ||
      taps < 1 || taps > SS_MAX_TAPS || row > (1 << 28) || stride < 2 * (int64_t)heads * vdim + 2 * (int64_t)groups * state + heads ||
      (taps > 1 && (!kept || kept_stride < (taps - 1) * row || kept_stride % 4 || ((uintptr_t)kept & 15))) ||
      (((uintptr_t)mixed | (uintptr_t)conv_w | (uintptr_t)conv_b) & 15))
    return TS_BAD_SHAPE;
  const SsSizes z = {heads, vdim, vp, groups, state, np, taps};
  const bool vec = vdim % 4 == 0 && state % 4 == 0 && stride % 4 == 0 && ((uintptr_t)proj & 15) == 0;
  const bool tiles = num_tokens > 256 && !moves;
  const int threads = tiles ? SS_THREADS : TS_WAVE;
  const int64_t items = row / 4 + heads;
  const int tt = tiles ? 8 : 1;
  dim3 grid((unsigned)((items + threads - 1) / threads), (num_tokens + tt - 1) / tt);
  if (grid.y > 65535) return TS_BAD_SHAPE;
#define SS_PREPARE(TO, TAPS, TT, VEC) \
  ssd_prepare_kernel<TO, TAPS, TT, VEC><<<grid, threads, 0, stream>>>((TO*)mixed, steps, logs, proj, stride, conv_w, conv_b, kept, \
      kept_stride, dt_bias, a_log, cu_seqlens, seq_of_token, state_slots, num_tokens, z, moves)
#define SS_PREPARE_V(TO, TAPS, TT) do { if (vec) SS_PREPARE(TO, TAPS, TT, true); else SS_PREPARE(TO, TAPS, TT, false); } while (0)
#define SS_PREPARE_T(TO, TAPS) do { if (tiles) SS_PREPARE_V(TO, TAPS, 8); else SS_PREPARE_V(TO, TAPS, 1); } while (0)
#define SS_PREPARE_O(TO) do { if (taps <= 4) SS_PREPARE_T(TO, 4); else SS_PREPARE_T(TO, SS_MAX_TAPS); } while (0)
  if (out_dtype == 0) SS_PREPARE_O(float);
  else if (out_dtype == 1) SS_PREPARE_O(bf16_t);
  else return TS_BAD_DTYPE;
#undef SS_PREPARE_O
#undef SS_PREPARE_T
#undef SS_PREPARE_V
#undef SS_PREPARE
  return ts_check_launch();
}

// A thread per (request, place): the last taps - 1 rows of (what the slot holds, the step's rows). Ascending i reads only
// rows not yet overwritten.
__global__ void __launch_bounds__(SS_THREADS)
ssd_conv_keep_kernel(float* __restrict__ kept, int64_t kept_stride, const float* __restrict__ proj, int64_t stride,
                     const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ state_slots, SsSizes z) {
  const int inner = z.heads * z.vdim, row = z.heads * z.vp + 2 * z.groups * z.np;
  const int place = blockIdx.x * SS_THREADS + threadIdx.x, seq = blockIdx.y;
  if (place >= row) return;
  const int first = cu_seqlens[seq], n = cu_seqlens[seq + 1] - first;
  if (n <= 0) return;
  int col;
  bool there;
  if (place < z.heads * z.vp) {
    const int h = place / z.vp, off = place - h * z.vp;
    col = inner + h * z.vdim + off;
    there = off < z.vdim;
  } else {
    const int at = place - z.heads * z.vp, half = z.groups * z.np;
    const int which = at / half, in = at - which * half;
    const int g = in / z.np, off = in - g * z.np;
    col = 2 * inner + (which * z.groups + g) * z.state + off;
    there = off < z.state;
  }
  float* slot = kept + (int64_t)state_slots[seq] * kept_stride + place;
  for (int i = 0; i < z.taps - 1; ++i) {
    const int src = n - (z.taps - 1) + i;                    // among the step's rows; below 0: still an old row
    slot[(int64_t)i * row] = src >= 0 ? (there ? proj[(int64_t)(first + src) * stride + col] : 0.f) : slot[(int64_t)(i + n) * row];
  }
}

extern "C" int ts_ssd_conv_keep(float* kept, int64_t kept_stride, const float* proj, int64_t stride, const int32_t* cu_seqlens,
                                const int32_t* state_slots, int num_seqs, int heads, int vdim, int vp, int groups, int state,
                                int np, int taps, hipStream_t stream) {
  if (num_seqs <= 0 || taps <= 1) return TS_OK;
  const int64_t row = (int64_t)heads * vp + 2 * (int64_t)groups * np;
  if (heads <= 0 || groups <= 0 || vdim <= 0 || state <= 0 || vp < vdim || np < state || taps > SS_MAX_TAPS || row > (1 << 28) ||
      kept_stride < (taps - 1) * row || stride < 2 * (int64_t)heads * vdim + 2 * (int64_t)groups * state || num_seqs > 65535)
    return TS_BAD_SHAPE;
  const SsSizes z = {heads, vdim, vp, groups, state, np, taps};
  ssd_conv_keep_kernel<<<dim3((unsigned)((row + SS_THREADS - 1) / SS_THREADS), num_seqs), SS_THREADS, 0, stream>>>(
      kept, kept_stride, proj, stride, cu_seqlens, state_slots, z);
  return ts_check_launch();
}

// A workgroup per (request, head, slice of 32 RV rows of the state). Eight lanes share a row, each with every eighth
// four of its numbers, so that a row is read and written in whole cache lines; NQ = np / 32 fours a lane. The next
// token's operands are fetched while one is worked on. Requests of more than `up_to` tokens are left out (0: none is).
template <typename T, int NQ, int RV>
__global__ void __launch_bounds__(SS_THREADS)
ssd_step_kernel(float* __restrict__ out, const T* __restrict__ mixed, const float* __restrict__ steps, const float* __restrict__ logs,
                const float* __restrict__ skip, const float* __restrict__ keeps, int token_stride, float* __restrict__ states,
                int64_t slot_stride, const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ state_slots, int heads,
                int vdim, int vp, int groups, int up_to) {
  constexpr int np = 32 * NQ;
  const int seq = blockIdx.x, h = blockIdx.y;
  const int t_begin = cu_seqlens[seq], t_end = cu_seqlens[seq + 1];
  if (t_begin >= t_end || (up_to > 0 && t_end - t_begin > up_to)) return;
  const int part = threadIdx.x & 7, v0 = blockIdx.z * 32 * RV + threadIdx.x / 8;
  const int row = heads * vp + 2 * groups * np, g = h / (heads / groups);
  const int b_at = heads * vp + g * np + 4 * part, c_at = b_at + groups * np;
  float* st = states + (int64_t)state_slots[seq] * slot_stride + (int64_t)h * vp * np + 4 * part;
  const float d_skip = skip ? skip[h] : 0.f, fixed_keep = keeps ? keeps[h] : 0.f;
  float S[RV][NQ][4];
#pragma unroll
  for (int rv = 0; rv < RV; ++rv)
#pragma unroll
    for (int i = 0; i < NQ; ++i) ss_load4(st + (int64_t)min(v0 + 32 * rv, vp - 1) * np + 32 * i, S[rv][i]);
  float Bn[NQ][4], Cn[NQ][4], xn[RV], dn, ln;
  auto fetch = [&](int t) {
    const T* m = mixed + (int64_t)t * row;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      ss_load4(m + b_at + 32 * i, Bn[i]);
      ss_load4(m + c_at + 32 * i, Cn[i]);
    }
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) xn[rv] = Num<T>::ld(m + h * vp + min(v0 + 32 * rv, vp - 1));
    dn = steps[(int64_t)t * token_stride + h];
    ln = logs[(int64_t)t * token_stride + h];
  };
  fetch(t_begin);
  for (int t = t_begin; t < t_end; ++t) {
    float B[NQ][4], C[NQ][4], x[RV];
#pragma unroll
    for (int i = 0; i < NQ; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k) B[i][k] = Bn[i][k], C[i][k] = Cn[i][k];
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) x[rv] = xn[rv];
    const float d = dn, keep = keeps ? fixed_keep : expf(ln);
    if (t + 1 < t_end) fetch(t + 1);
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) {
      const float dx = d * x[rv];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NQ; ++i)
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          S[rv][i][k] = fmaf(keep, S[rv][i][k], dx * B[i][k]);
          y = fmaf(S[rv][i][k], C[i][k], y);
        }
#pragma unroll
      for (int off = 1; off < 8; off <<= 1) y += __shfl_xor(y, off, TS_WAVE);
      const int v = v0 + 32 * rv;
      if (part == 0 && v < vdim) out[((int64_t)t * heads + h) * vdim + v] = fmaf(d_skip, x[rv], y);
    }
  }
#pragma unroll
  for (int rv = 0; rv < RV; ++rv)
    if (v0 + 32 * rv < vp) {
#pragma unroll
      for (int i = 0; i < NQ; ++i) ss_store4(st + (int64_t)(v0 + 32 * rv) * np + 32 * i, S[rv][i]);
    }
}

// states: each slot's S, float32 [heads, vp, np], `slot_stride` floats from slot to slot.
extern "C" int ts_ssd_step(float* out, const void* mixed, int dtype, const float* steps, const float* logs, const float* skip,
                           const float* keeps, int token_stride, float* states, int64_t slot_stride, const int32_t* cu_seqlens, const int32_t* state_slots, int num_seqs,
                           int heads, int vdim, int vp, int groups, int np, int up_to, hipStream_t stream) {
  if (num_seqs <= 0) return TS_OK;
  if (heads <= 0 || heads > 65535 || groups <= 0 || heads % groups || vdim <= 0 || vp < vdim || vp % 16 || np <= 0 || np % 32 || np > 512 ||
      slot_stride < (int64_t)heads * vp * np || slot_stride % 4 || (((uintptr_t)states | (uintptr_t)mixed) & 15) ||
      (token_stride != 0 && token_stride < heads))
    return TS_BAD_SHAPE;
  const int nq = np / 32;
  // (a slice of 64 rows where the step has workgroups enough and a lane's registers hold two rows' fours)
  const int rv = (vp > 32 && nq <= 4 && (int64_t)num_seqs * heads * ((vp + 63) / 64) >= 512) ? 2 : 1;
  const int slices = (vp + 32 * rv - 1) / (32 * rv);
  if (slices > 65535) return TS_BAD_SHAPE;
  dim3 grid(num_seqs, heads, slices);
#define SS_STEP(T, NQ, RV) \
  ssd_step_kernel<T, NQ, RV><<<grid, SS_THREADS, 0, stream>>>(out, (const T*)mixed, steps, logs, skip, keeps, token_stride, states, slot_stride, \
                                                              cu_seqlens, state_slots, heads, vdim, vp, groups, up_to)
#define SS_STEP_2(T, NQ) case NQ: if (rv == 2) SS_STEP(T, NQ, 2); else SS_STEP(T, NQ, 1); break;
#define SS_STEP_1(T, NQ) case NQ: SS_STEP(T, NQ, 1); break;
#define SS_STEP_N(T) \
  switch (nq) { \
    SS_STEP_2(T, 1) SS_STEP_2(T, 2) SS_STEP_2(T, 3) SS_STEP_2(T, 4) SS_STEP_1(T, 5) SS_STEP_1(T, 6) SS_STEP_1(T, 7) SS_STEP_1(T, 8) \
    SS_STEP_1(T, 9) SS_STEP_1(T, 10) SS_STEP_1(T, 11) SS_STEP_1(T, 12) SS_STEP_1(T, 13) SS_STEP_1(T, 14) SS_STEP_1(T, 15) SS_STEP_1(T, 16) \
  }
  if (dtype == 0) { SS_STEP_N(float) }
  else if (dtype == 1) { SS_STEP_N(bf16_t) }
  else return TS_BAD_DTYPE;
#undef SS_STEP_N
#undef SS_STEP_1
#undef SS_STEP_2
#undef SS_STEP
  return ts_check_launch();
}

// ---- chunks of 64 tokens on the matrix cores (bfloat16) ----------------------------------------------------------

// chunks: int32 [chunks, 4] (first token of the step, tokens 1 .. 64, request, whether the request's last). buf[chunk][head]
// [vp][np] gets what the chunk adds to the state, totals[chunk][head] the chunk's whole log decay.
__global__ void __launch_bounds__(SS_THREADS)
ssd_chunk_sums_kernel(float* __restrict__ buf, float* __restrict__ totals, const bf16_t* __restrict__ mixed,
                      const float* __restrict__ steps, const float* __restrict__ logs, int token_stride,
                      const int32_t* __restrict__ chunks, int heads, int vp, int groups, int np) {
  __shared__ __attribute__((aligned(16))) bf16_t x_s[64][SS_PAD], xr_s[64][SS_PAD];     // weighted x, turned: [channel][token]
  __shared__ __attribute__((aligned(16))) bf16_t b_s[128][SS_PAD];                     // B, turned: [state][token]
  __shared__ float weight_s[SS_L];
  const int chunk = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 64;
  const int tok0 = chunks[4 * chunk], len = chunks[4 * chunk + 1];
  const int row = heads * vp + 2 * groups * np, g = h / (heads / groups);
  const int wave = wave_index(), lane = threadIdx.x & (TS_WAVE - 1), r = lane & 15, q = lane >> 4;
  if (threadIdx.x < TS_WAVE) {
    const double b = ss_running(logs, tok0, len, token_stride, h);
    const double total = __shfl(b, TS_WAVE - 1, TS_WAVE);
    weight_s[lane] = lane < len ? expf((float)(total - b)) * steps[(int64_t)(tok0 + lane) * token_stride + h] : 0.f;
    if (lane == 0 && blockIdx.z == 0) totals[(int64_t)chunk * heads + h] = (float)total;
  }
  __syncthreads();
  ss_turn<true>(x_s, xr_s, mixed + h * vp + v0, row, tok0, len, vp - v0, weight_s);
  float* dst = buf + ((int64_t)chunk * heads + h) * vp * np;
  const int v = v0 + 16 * wave + r;
  for (int n0 = 0; n0 < np; n0 += 128) {
    if (n0) __syncthreads();                                 // (the stretch before has been read)
    const bf16_t* b_src = mixed + heads * vp + g * np + n0;
    ss_turn<false>(b_s, nullptr, b_src, row, tok0, len, np - n0, nullptr);
    ss_turn<false>(b_s + 64, nullptr, b_src + 64, row, tok0, len, np - n0 - 64, nullptr);
    __syncthreads();
    if (v0 + 16 * wave >= vp) continue;                      // (the whole wave)
    uint4 xf[2], xl[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      xf[k] = *(const uint4*)&x_s[16 * wave + r][32 * k + 8 * q];
      xl[k] = *(const uint4*)&xr_s[16 * wave + r][32 * k + 8 * q];
    }
#pragma unroll
    for (int nb = 0; nb < 8; ++nb) {
      if (n0 + 16 * nb >= np) break;
      float4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const uint4 bf = *(const uint4*)&b_s[16 * nb + r][32 * k + 8 * q];
        acc = mfma32(bf, xf[k], acc);
        acc = mfma32(bf, xl[k], acc);
      }
      *(float4_t*)(dst + (int64_t)v * np + n0 + 16 * nb + 4 * q) = acc;
    }
  }
}

// A thread per four numbers of a head's state: over a request's chunks in order, what the chunk adds makes room for the
// state before the chunk. chunk_cu: int32 [requests + 1]; requests without chunks keep their state as it is.
__global__ void __launch_bounds__(SS_THREADS)
ssd_chunk_scan_kernel(float* __restrict__ buf, const float* __restrict__ totals, float* __restrict__ states, int64_t slot_stride,
                      const int32_t* __restrict__ chunk_cu, const int32_t* __restrict__ state_slots, int heads, int per_head) {
  const int seq = blockIdx.x, h = blockIdx.y;
  const int begin = chunk_cu[seq], end = chunk_cu[seq + 1];
  const int e = 4 * (blockIdx.z * SS_THREADS + threadIdx.x);
  if (begin >= end || e >= per_head) return;
  float* st = states + (int64_t)state_slots[seq] * slot_stride + (int64_t)h * per_head + e;
  float4 S = *(const float4*)st;
  float* p = buf + ((int64_t)begin * heads + h) * per_head + e;
  const int64_t next = (int64_t)heads * per_head;
  constexpr int AHEAD = 4;                                   // chunks whose sums are on their way together
  for (int c = begin; c < end; c += AHEAD, p += AHEAD * next) {
    float4 add[AHEAD];
    float keep[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int k = min(i, end - 1 - c);
      add[i] = *(const float4*)(p + k * next);
      keep[i] = totals[(int64_t)(c + k) * heads + h];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i)
      if (c + i < end) {
        *(float4*)(p + i * next) = S;
        const float a = expf(keep[i]);
        S.x = fmaf(a, S.x, add[i].x);
        S.y = fmaf(a, S.y, add[i].y);
        S.z = fmaf(a, S.z, add[i].z);
        S.w = fmaf(a, S.w, add[i].w);
      }
  }
  *(float4*)st = S;
}

// One workgroup per (chunk, head, slice of 64 channels): first each wave makes the second sum's weights of its 16 tokens
// (keys as the product's rows, so that the weights come out in the order the next product reads), then each wave the
// outputs of its 16 channels for all tokens.
template <int NQ>
__global__ void __launch_bounds__(SS_THREADS)
ssd_chunk_out_kernel(float* __restrict__ out, const float* __restrict__ buf, const bf16_t* __restrict__ mixed,
                     const float* __restrict__ steps, const float* __restrict__ logs, const float* __restrict__ skip, int token_stride,
                     const int32_t* __restrict__ chunks, int heads, int vdim, int vp, int groups) {
  constexpr int np = 32 * NQ;
  __shared__ __attribute__((aligned(16))) bf16_t x_s[64][SS_PAD];                      // x, turned: [channel][token]
  __shared__ __attribute__((aligned(16))) bf16_t p_s[SS_L][SS_PAD], pr_s[SS_L][SS_PAD];  // weights: [token][key token], two terms
  __shared__ double b_s[SS_L];
  __shared__ float d_s[SS_L];
  const int chunk = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 64;
  const int tok0 = chunks[4 * chunk], len = chunks[4 * chunk + 1];
  const int row = heads * vp + 2 * groups * np, g = h / (heads / groups);
  const int wave = wave_index(), lane = threadIdx.x & (TS_WAVE - 1), r = lane & 15, q = lane >> 4;
  const bf16_t* rows = mixed + (int64_t)tok0 * row;
  const bf16_t* b_rows = rows + heads * vp + g * np + 8 * q;
  const bf16_t* c_rows = b_rows + groups * np;
  if (threadIdx.x < TS_WAVE) {
    b_s[lane] = ss_running(logs, tok0, len, token_stride, h);
    d_s[lane] = lane < len ? steps[(int64_t)(tok0 + lane) * token_stride + h] : 0.f;
  }
  ss_turn<false>(x_s, nullptr, mixed + h * vp + v0, row, tok0, len, vp - v0, nullptr);
  const int t = 16 * wave + r;                               // (this lane's token of the first product)
  float4_t st[2][2];
#pragma unroll
  for (int kk = 0; kk < 2; ++kk)
#pragma unroll
    for (int tau = 0; tau < 2; ++tau) st[kk][tau] = (float4_t){0.f, 0.f, 0.f, 0.f};
  if (16 * wave < len) {
    const bf16_t* c_row = c_rows + (int64_t)min(t, len - 1) * row;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      const uint4 cf = *(const uint4*)(c_row + 32 * i);
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        if (32 * kk <= 16 * wave + 15) {
#pragma unroll
          for (int tau = 0; tau < 2; ++tau) {
            const int key = 32 * kk + 8 * (r >> 2) + 4 * tau + (r & 3);
            st[kk][tau] = mfma32(*(const uint4*)(b_rows + (int64_t)min(key, len - 1) * row + 32 * i), cf, st[kk][tau]);
          }
        }
    }
  }
  __syncthreads();                                           // (b_s, d_s and x_s are there)
#pragma unroll
  for (int kk = 0; kk < 2; ++kk)
    if (32 * kk <= 16 * wave + 15) {
      uint4 hi, lo;
#pragma unroll
      for (int j = 0; j < 4; ++j) {                          // (two keys a word: 2 j and 2 j + 1 of the lane's eight)
        float p[2];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          const int e = 2 * j + k, key = 32 * kk + 8 * q + e;
          const float s = st[kk][e >> 2][e & 3];
          p[k] = (key <= t && t < len) ? s * expf((float)(b_s[t] - b_s[key])) * d_s[key] : 0.f;
        }
        (&hi.x)[j] = pack_bf16(p[0], p[1]);
        (&lo.x)[j] = ss_rest((&hi.x)[j], p[0], p[1]);
      }
      *(uint4*)&p_s[t][32 * kk + 8 * q] = hi;
      *(uint4*)&pr_s[t][32 * kk + 8 * q] = lo;
    }
  __syncthreads();
  if (v0 + 16 * wave >= vp) return;                          // (no barrier below)
  float4_t acc[4];
#pragma unroll
  for (int tb = 0; tb < 4; ++tb) acc[tb] = (float4_t){0.f, 0.f, 0.f, 0.f};
  const float* s_row = buf + ((int64_t)chunk * heads + h) * vp * np + (int64_t)(v0 + 16 * wave + r) * np + 8 * q;
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    float s[8];
    ss_load4(s_row + 32 * i, *(float (*)[4])&s[0]);
    ss_load4(s_row + 32 * i + 4, *(float (*)[4])&s[4]);
    uint4 hi, lo;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      (&hi.x)[j] = pack_bf16(s[2 * j], s[2 * j + 1]);
      (&lo.x)[j] = ss_rest((&hi.x)[j], s[2 * j], s[2 * j + 1]);
    }
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) {
      const uint4 cf = *(const uint4*)(c_rows + (int64_t)min(16 * tb + r, len - 1) * row + 32 * i);
      acc[tb] = mfma32(hi, cf, acc[tb]);
      acc[tb] = mfma32(lo, cf, acc[tb]);
    }
  }
  const float d_skip = skip ? skip[h] : 0.f;
  uint4 xf[2];
#pragma unroll
  for (int k = 0; k < 2; ++k) xf[k] = *(const uint4*)&x_s[16 * wave + r][32 * k + 8 * q];
#pragma unroll
  for (int tb = 0; tb < 4; ++tb) {
    const int tok = 16 * tb + r;
    const float decay = expf((float)b_s[tok]);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[tb][j] *= decay;
#pragma unroll
    for (int k = 0; k < 2; ++k)
      if (32 * k <= 16 * tb + 15) {
        acc[tb] = mfma32(xf[k], *(const uint4*)&p_s[tok][32 * k + 8 * q], acc[tb]);
        acc[tb] = mfma32(xf[k], *(const uint4*)&pr_s[tok][32 * k + 8 * q], acc[tb]);
      }
    if (tok < len) {
      const int v = v0 + 16 * wave + 4 * q;
      float y[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = fmaf(d_skip, bf2f(x_s[16 * wave + 4 * q + j][tok]), acc[tb][j]);
      float* dst = out + ((int64_t)(tok0 + tok) * heads + h) * vdim + v;
      if (vdim % 4 == 0) {
        if (v < vdim) ss_store4(dst, y);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (v + j < vdim) dst[j] = y[j];
      }
    }
  }
}

// buf float32 [chunks, heads, vp, np], totals float32 [chunks, heads].
extern "C" int ts_ssd_chunks(float* out, const void* mixed, const float* steps, const float* logs, const float* skip, int token_stride,
                             float* states, int64_t slot_stride, const int32_t* chunks, const int32_t* chunk_cu, const int32_t* state_slots,
                             float* buf, float* totals, int num_chunks, int num_seqs, int heads, int vdim, int vp, int groups, int np,
                             hipStream_t stream) {
  if (num_chunks <= 0 || num_seqs <= 0) return TS_OK;
  const int64_t per_head = (int64_t)vp * np;
  if (heads <= 0 || heads > 65535 || groups <= 0 || heads % groups || vdim <= 0 || vp < vdim || vp % 16 || np <= 0 || np % 32 || np > 512 ||
      per_head > (1 << 24) || slot_stride < heads * per_head || slot_stride % 4 ||
      (((uintptr_t)states | (uintptr_t)mixed | (uintptr_t)buf | (uintptr_t)out) & 15) || (token_stride != 0 && token_stride < heads))
    return TS_BAD_SHAPE;
  const int slices = (vp + 63) / 64;
  const int scan_blocks = (int)((per_head / 4 + SS_THREADS - 1) / SS_THREADS);
  const bf16_t* m = (const bf16_t*)mixed;
  ssd_chunk_sums_kernel<<<dim3(num_chunks, heads, slices), SS_THREADS, 0, stream>>>(buf, totals, m, steps, logs, token_stride, chunks, heads, vp,
                                                                                       groups, np);
  ssd_chunk_scan_kernel<<<dim3(num_seqs, heads, scan_blocks), SS_THREADS, 0, stream>>>(buf, totals, states, slot_stride, chunk_cu, state_slots,
                                                                                      heads, (int)per_head);
#define SS_OUT(NQ) case NQ: ssd_chunk_out_kernel<NQ><<<dim3(num_chunks, heads, slices), SS_THREADS, 0, stream>>>( \
    out, buf, m, steps, logs, skip, token_stride, chunks, heads, vdim, vp, groups); break;
  switch (np / 32) {
    SS_OUT(1) SS_OUT(2) SS_OUT(3) SS_OUT(4) SS_OUT(5) SS_OUT(6) SS_OUT(7) SS_OUT(8) SS_OUT(9) SS_OUT(10) SS_OUT(11) SS_OUT(12)
    SS_OUT(13) SS_OUT(14) SS_OUT(15) SS_OUT(16)
  }
#undef SS_OUT
  return ts_check_launch();
}

// ---- y silu(z), then a norm over equal parts of the row ----------------------------------------------------------

static __device__ __forceinline__ float ss_gate(float y, float z) { return y * z / (1.0f + expf(-z)); }

// WAVES waves a part (1: four parts a workgroup; 4: one), HELD fours of the part a lane.
template <typename TO, int WAVES, int HELD>
__global__ void __launch_bounds__(SS_THREADS)
gated_group_norm_kernel(TO* __restrict__ out, const float* __restrict__ y, const float* __restrict__ z, int64_t z_stride,
                        const float* __restrict__ weight, int width, int parts, float eps, int64_t items) {
  __shared__ float red[SS_WAVES];
  const int wave = threadIdx.x / TS_WAVE, lane = threadIdx.x & (TS_WAVE - 1);
  const int64_t item = WAVES == 1 ? (int64_t)blockIdx.x * SS_WAVES + wave : blockIdx.x;
  if (item >= items) return;                                 // (a whole wave; with WAVES == 4 no workgroup)
  const int size = width / parts;
  const int64_t t = item / parts;
  const int at = (int)(item - t * parts) * size, first = 4 * (WAVES == 1 ? lane : threadIdx.x);
  const float* y_row = y + t * width + at;
  const float* z_row = z + t * z_stride + at;
  float u[HELD][4];
  float squares = 0.f;
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int d = first + i * 4 * TS_WAVE * WAVES, dc = min(d, size - 4);
    float a[4], b[4];
    ss_load4(y_row + dc, a);
    ss_load4(z_row + dc, b);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      u[i][k] = ss_gate(a[k], b[k]);
      squares = d < size ? fmaf(u[i][k], u[i][k], squares) : squares;
    }
  }
  squares = wave_sum(squares);
  if constexpr (WAVES > 1) {
    if (lane == 0) red[wave] = squares;
    __syncthreads();
    squares = 0.f;
#pragma unroll
    for (int w = 0; w < SS_WAVES; ++w) squares += red[w];
  }
  const float inv = 1.0f / sqrtf(squares / (float)size + eps);
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int d = first + i * 4 * TS_WAVE * WAVES;
    if (d < size) {
      float w[4];
      ss_load4(weight + at + d, w);
#pragma unroll
      for (int k = 0; k < 4; ++k) w[k] *= u[i][k] * inv;
      ss_store4(out + t * width + at + d, w);
    }
  }
}

// Any size: a workgroup a part, the products made twice.
template <typename TO>
__global__ void __launch_bounds__(SS_THREADS)
gated_group_norm_any_kernel(TO* __restrict__ out, const float* __restrict__ y, const float* __restrict__ z, int64_t z_stride,
                            const float* __restrict__ weight, int width, int parts, float eps) {
  __shared__ float red[SS_WAVES];
  const int size = width / parts;
  const int64_t t = blockIdx.x / parts;
  const int at = (int)(blockIdx.x - t * parts) * size;
  const float* y_row = y + t * width + at;
  const float* z_row = z + t * z_stride + at;
  float squares = 0.f;
  for (int d = threadIdx.x; d < size; d += SS_THREADS) {
    const float u = ss_gate(y_row[d], z_row[d]);
    squares = fmaf(u, u, squares);
  }
  squares = wave_sum(squares);
  if ((threadIdx.x & (TS_WAVE - 1)) == 0) red[threadIdx.x / TS_WAVE] = squares;
  __syncthreads();
  squares = 0.f;
#pragma unroll
  for (int w = 0; w < SS_WAVES; ++w) squares += red[w];
  const float inv = 1.0f / sqrtf(squares / (float)size + eps);
  for (int d = threadIdx.x; d < size; d += SS_THREADS)
    Num<TO>::st(out + t * width + at + d, ss_gate(y_row[d], z_row[d]) * inv * weight[at + d]);
}

extern "C" int ts_gated_group_norm(void* out, int out_dtype, const float* y, const float* z, int64_t z_stride, const float* weight,
                                   int num_tokens, int width, int parts, float eps, hipStream_t stream) {
  if (num_tokens <= 0) return TS_OK;
  if (width <= 0 || parts <= 0 || width % parts || z_stride < width) return TS_BAD_SHAPE;
  if (out_dtype != 0 && out_dtype != 1) return TS_BAD_DTYPE;
  const int64_t items = (int64_t)num_tokens * parts;
  const int size = width / parts;
  if (items > 0x7fffffff) return TS_BAD_SHAPE;
  const bool fours = size % 4 == 0 && z_stride % 4 == 0 && size <= 8 * 4 * SS_THREADS &&
                     (((uintptr_t)out | (uintptr_t)y | (uintptr_t)z | (uintptr_t)weight) & 15) == 0;
#define SS_NORM(TO, WAVES, HELD) \
  gated_group_norm_kernel<TO, WAVES, HELD><<<(unsigned)(WAVES == 1 ? (items + SS_WAVES - 1) / SS_WAVES : items), SS_THREADS, 0, stream>>>( \
      (TO*)out, y, z, z_stride, weight, width, parts, eps, items)
#define SS_NORM_T(TO) \
  do { \
    if (!fours) gated_group_norm_any_kernel<TO><<<(unsigned)items, SS_THREADS, 0, stream>>>((TO*)out, y, z, z_stride, weight, width, parts, eps); \
    else if (size <= 256) SS_NORM(TO, 1, 1); \
    else if (size <= 512) SS_NORM(TO, 1, 2); \
    else if (size <= 1024) SS_NORM(TO, 4, 1); \
    else if (size <= 2048) SS_NORM(TO, 4, 2); \
    else if (size <= 4096) SS_NORM(TO, 4, 4); \
    else SS_NORM(TO, 4, 8); \
  } while (0)
  if (out_dtype == 0) SS_NORM_T(float);
  else SS_NORM_T(bf16_t);
#undef SS_NORM_T
#undef SS_NORM
  return ts_check_launch();
}
