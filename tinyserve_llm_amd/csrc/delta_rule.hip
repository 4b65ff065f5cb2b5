// The gated delta rule. Per head a state S [dim, vdim], 32-bit, zero at a request's start; head h shares its key and query
// with the heads of its group. For a token with unit vectors k, q [dim], v [vdim], a step 0 < beta < 1 and a log decay l <= 0:
//     S' = exp(l) S,   u = beta (v - S'^T k),   S = S' + k u^T,   o = S^T q.
//   * `ts_delta_prepare`: from a projected row [gate | v | k | q | a | b] (32-bit) to what the recurrence reads: v, k and q
//     through a causal convolution per channel and silu, in the activations' storage type and in a row of their own (every
//     head's v in `vp` places, every group's k and q in `np`, multiples of 16 and 32, zeros behind their own numbers); the
//     factors that make k and q unit vectors (q's also with dim^(-1/2)) beside them, 32-bit, a number per group: they scale
//     whole rows of the products below, so k and q themselves enter those as the convolution leaves them; beta = sigmoid(b)
//     and l = -exp(A_log) softplus(a + dt_bias), 32-bit. The rows ahead of a request's first token of the step come from
//     its state slot (`ts_ssd_conv_keep` leaves the last ones there; a step of single tokens does it here).
//   * `ts_delta_step`: walks each request's tokens of the step in order with the state in registers; a request's state is
//     read from its slot at the start and written back at the end. For decoded tokens, short portions, and 32-bit models.
//   * `ts_delta_chunks`: long portions in bfloat16, in chunks of 64 tokens on the matrix cores. With b_t the sum of l from
//     the chunk's first token to t (every exponent below is <= 0) and S0 the state before the chunk, the writes solve
//         u_t + sum_{j < t} A_tj u_j = beta_t v_t - beta_t exp(b_t) S0^T k_t,   A_tj = beta_t exp(b_t - b_j) (k_t . k_j),
//     so with T = (I + A)^(-1)
//         U = T (beta V - beta exp(b) K S0),   o_t = exp(b_t) S0^T q_t + sum_{j <= t} exp(b_t - b_j) (q_t . k_j) u_j,
//         S = exp(b_L) S0 + sum_j exp(b_L - b_j) k_j u_j^T.
//     One launch makes what does not depend on the state, every chunk and head by itself (T, the weights of the second sum,
//     k and v turned round); the other walks a request's chunks in order, a workgroup per head and 16 value columns.
//     Convolved k, q and v are operands as they are; what is 32-bit by nature (T, the weights, U, S) enters a product as two
//     bfloat16 terms.
#include "chunk_ops.h"

#define DL_THREADS 256
#define DL_WAVES (DL_THREADS / TS_WAVE)
#define DL_MAX_TAPS 16
#define DL_MAX_CHUNK_NP 256     // places of a key in the chunked form

struct DlSizes { int heads, vdim, vp, groups, dim, np, taps; };

// LP lanes side by side (a power of two) take one stretch of places: a group's k, a group's q (HELD fours a lane, so that
// LP HELD fours cover np), or LP fours of the heads' v, or LP heads' scalars; every lane TT tokens. TAPS: 4 or 16, at least
// the taps. VEC: sizes are multiples of four and the projected rows 16-byte aligned.
template <typename TO, int TAPS, int TT, bool VEC, int HELD>
__global__ void __launch_bounds__(DL_THREADS)
delta_prepare_kernel(TO* __restrict__ mixed, float* __restrict__ units, float* __restrict__ betas, float* __restrict__ logs,
                     const float* __restrict__ proj, int64_t stride, const float* __restrict__ conv_w, float* __restrict__ kept,
                     int64_t kept_stride, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                     const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ seq_of_token,
                     const int32_t* __restrict__ state_slots, int num_tokens, DlSizes z, int lp, float q_scale, int moves) {
  const int inner = z.heads * z.vdim, row = z.heads * z.vp + 2 * z.groups * z.np;
  const int sub = threadIdx.x & (lp - 1);
  const int stretch = (blockIdx.x * blockDim.x + threadIdx.x) / lp;
  const int t0 = blockIdx.y * TT, t1 = min(t0 + TT, num_tokens);
  const int v_fours = z.heads * z.vp / 4, v_stretches = (v_fours + lp - 1) / lp;
  const bool unit = stretch < 2 * z.groups;
  if (!unit && stretch >= 2 * z.groups + v_stretches) {        // (lanes of a wave that exchange sums never part ways here: see `sums`)
    const int h = (stretch - 2 * z.groups - v_stretches) * lp + sub;
    if (h < z.heads) {
      const float rate = -expf(a_log[h]), bias = dt_bias[h];
      const float* src = proj + 2 * inner + 2 * z.groups * z.dim + h;
      for (int t = t0; t < t1; ++t) {
        const float s = src[(int64_t)t * stride] + bias;
        logs[(int64_t)t * z.heads + h] = rate * (fmaxf(s, 0.f) + log1pf(expf(-fabsf(s))));      // softplus
        betas[(int64_t)t * z.heads + h] = 1.0f / (1.0f + expf(-src[(int64_t)t * stride + z.heads]));
      }
    }
  }
  int place[HELD], col[HELD], count[HELD];                     // a four's first place, its column of the projected row, how many of it are there
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    place[i] = 0; col[i] = inner; count[i] = -1;               // (-1: no four of this lane's)
    if (unit) {
      const int off = 4 * (sub + i * lp);
      if (off < z.np) {
        place[i] = z.heads * z.vp + stretch * z.np + off;
        col[i] = 2 * inner + stretch * z.dim + off;
        count[i] = min(4, max(0, z.dim - off));
      }
    } else if (i == 0) {
      const int four = (stretch - 2 * z.groups) * lp + sub;
      if (stretch < 2 * z.groups + v_stretches && four < v_fours) {
        const int h = 4 * four / z.vp, off = 4 * four - h * z.vp;
        place[i] = 4 * four;
        col[i] = inner + h * z.vdim + off;
        count[i] = min(4, max(0, z.vdim - off));
      }
    }
  }
  float w[HELD][TAPS][4];
#pragma unroll
  for (int i = 0; i < HELD; ++i)
#pragma unroll
    for (int d = 0; d < TAPS; ++d) {
#pragma unroll
      for (int k = 0; k < 4; ++k) w[i][d][k] = 0.f;
      if (d < z.taps) ss_load4(conv_w + (int64_t)(z.taps - 1 - d) * row + place[i], w[i][d]);
    }
  auto input = [&](int t, int i, float (&u)[4]) {
    const float* src = proj + (int64_t)t * stride + col[i];
    if constexpr (VEC) {
      if (count[i] == 4) ss_load4(src, u);
      else u[0] = u[1] = u[2] = u[3] = 0.f;
    } else {
#pragma unroll
      for (int k = 0; k < 4; ++k) u[k] = k < count[i] ? src[k] : 0.f;
    }
  };
  float past[HELD][TAPS][4];                                   // past[.][d]: the channel's input d tokens before the one at hand
#pragma unroll
  for (int i = 0; i < HELD; ++i)
#pragma unroll
    for (int d = 0; d < TAPS; ++d)
#pragma unroll
      for (int k = 0; k < 4; ++k) past[i][d][k] = 0.f;
  for (int t = t0; t < t1; ++t) {
    const int seq = seq_of_token[t], index = t - cu_seqlens[seq];
    float squares = 0.f;
#pragma unroll
    for (int i = 0; i < HELD; ++i) {
      float* slot = kept + (int64_t)state_slots[seq] * kept_stride + place[i];
      if (t == t0 || index == 0) {
#pragma unroll
        for (int d = 1; d < TAPS; ++d)
          if (d < z.taps) {
            if (index >= d) input(t - d, i, past[i][d]);
            else ss_load4(slot + (int64_t)(z.taps - 1 + index - d) * row, past[i][d]);
          }
      } else {
#pragma unroll
        for (int d = TAPS - 1; d > 0; --d)
#pragma unroll
          for (int k = 0; k < 4; ++k) past[i][d][k] = past[i][d - 1][k];
      }
      input(t, i, past[i][0]);
      float y[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        float s = 0.f;
#pragma unroll
        for (int d = TAPS - 1; d >= 0; --d) s = fmaf(w[i][d][k], past[i][d][k], s);
        y[k] = Num<TO>::round(s / (1.0f + expf(-s)));
        if (k < count[i]) squares = fmaf(y[k], y[k], squares);
        else y[k] = 0.f;
      }
      if (count[i] >= 0) {
        ss_store4(mixed + (int64_t)t * row + place[i], y);
        if (moves) {                                           // (the request's only token of the step: nobody else reads its slot)
#pragma unroll
          for (int d = 0; d < TAPS - 1; ++d)
            if (d < z.taps - 1) ss_store4(slot + (int64_t)(z.taps - 2 - d) * row, past[i][d]);
        }
      }
    }
    // sums: over the lanes of the stretch (all lanes of the wave walk the same tokens and come by here together)
    for (int off = lp / 2; off > 0; off >>= 1) squares += __shfl_xor(squares, off, TS_WAVE);
    if (unit && sub == 0)
      units[(int64_t)t * 2 * z.groups + stretch] = (stretch < z.groups ? 1.0f : q_scale) / sqrtf(squares + 1e-6f);
  }
}

// kept: each slot's convolution inputs, float32 [taps - 1, row], `kept_stride` floats from slot to slot. conv_w float32
// [taps, row] (last: the current token's), zeros where a place holds no channel. units [tokens, 2 groups]: k's factors,
// then q's. moves: every request of the step feeds exactly one token.
extern "C" int ts_delta_prepare(void* mixed, int out_dtype, float* units, float* betas, float* logs, const float* proj, int64_t stride,
                                const float* conv_w, float* kept, int64_t kept_stride, const float* dt_bias, const float* a_log,
                                const int32_t* cu_seqlens, const int32_t* seq_of_token, const int32_t* state_slots, int num_tokens,
                                int heads, int vdim, int vp, int groups, int dim, int np, int taps, float q_scale, int moves,
                                hipStream_t stream) {
  if (num_tokens <= 0) return TS_OK;
  const int64_t row = (int64_t)heads * vp + 2 * (int64_t)groups * np;
  if (heads <= 0 || groups <= 0 || heads % groups || vdim <= 0 || dim <= 0 || vp < vdim || np < dim || vp % 16 || np % 32 || np > 512 ||
      taps < 1 || taps > DL_MAX_TAPS || row > (1 << 28) || stride < 2 * (int64_t)heads * vdim + 2 * (int64_t)groups * dim + 2 * heads || !kept ||
      (taps > 1 && (kept_stride < (taps - 1) * row || kept_stride % 4 || ((uintptr_t)kept & 15))) ||
      (((uintptr_t)mixed | (uintptr_t)conv_w) & 15))
    return TS_BAD_SHAPE;
  const DlSizes z = {heads, vdim, vp, groups, dim, np, taps};
  const bool vec = vdim % 4 == 0 && dim % 4 == 0 && stride % 4 == 0 && ((uintptr_t)proj & 15) == 0;
  const bool tiles = num_tokens > 256 && !moves;
  const int threads = tiles ? DL_THREADS : TS_WAVE;
  int lp = 8;
  while (lp < TS_WAVE && 4 * lp < np) lp *= 2;
  const int64_t fours = (int64_t)heads * vp / 4;
  const int64_t stretches = 2 * (int64_t)groups + (fours + lp - 1) / lp + (heads + lp - 1) / lp;
  const int tt = tiles ? 8 : 1;
  dim3 grid((unsigned)((stretches * lp + threads - 1) / threads), (num_tokens + tt - 1) / tt);
  if (grid.y > 65535) return TS_BAD_SHAPE;
#define DL_PREPARE(TO, TAPS, TT, VEC, HELD) \
  delta_prepare_kernel<TO, TAPS, TT, VEC, HELD><<<grid, threads, 0, stream>>>((TO*)mixed, units, betas, logs, proj, stride, conv_w, kept, \
      kept_stride, dt_bias, a_log, cu_seqlens, seq_of_token, state_slots, num_tokens, z, lp, q_scale, moves)
#define DL_PREPARE_H(TO, TAPS, TT, VEC) do { if (np <= 256) DL_PREPARE(TO, TAPS, TT, VEC, 1); else DL_PREPARE(TO, TAPS, TT, VEC, 2); } while (0)
#define DL_PREPARE_V(TO, TAPS, TT) do { if (vec) DL_PREPARE_H(TO, TAPS, TT, true); else DL_PREPARE_H(TO, TAPS, TT, false); } while (0)
#define DL_PREPARE_T(TO, TAPS) do { if (tiles) DL_PREPARE_V(TO, TAPS, 8); else DL_PREPARE_V(TO, TAPS, 1); } while (0)
#define DL_PREPARE_O(TO) do { if (taps <= 4) DL_PREPARE_T(TO, 4); else DL_PREPARE_T(TO, DL_MAX_TAPS); } while (0)
  if (out_dtype == 0) DL_PREPARE_O(float);
  else if (out_dtype == 1) DL_PREPARE_O(bf16_t);
  else return TS_BAD_DTYPE;
#undef DL_PREPARE_O
#undef DL_PREPARE_T
#undef DL_PREPARE_V
#undef DL_PREPARE_H
#undef DL_PREPARE
  return ts_check_launch();
}

// A workgroup per (request, head, slice of 32 RV value columns; a state is kept as its columns, [vp][np]). Eight lanes share
// a column, each with every eighth four of its numbers, so that a column is read and written in whole cache lines; NQ =
// np / 32 fours a lane. The next token's operands are fetched while one is worked on. A token's three sums (S^T k, S^T q and
// k . q) are taken together from the state before it: o = exp(l) S^T q + (k . q) u. Requests of more than `up_to` tokens are
// left out (0: none is).
template <typename T, int NQ, int RV>
__global__ void __launch_bounds__(DL_THREADS)
delta_step_kernel(float* __restrict__ out, const T* __restrict__ mixed, const float* __restrict__ units, const float* __restrict__ betas,
                  const float* __restrict__ logs, float* __restrict__ states, int64_t slot_stride,
                  const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ state_slots, int heads, int vdim, int vp,
                  int groups, int up_to) {
  constexpr int np = 32 * NQ;
  const int seq = blockIdx.x, h = blockIdx.y;
  const int t_begin = cu_seqlens[seq], t_end = cu_seqlens[seq + 1];
  if (t_begin >= t_end || (up_to > 0 && t_end - t_begin > up_to)) return;
  const int part = threadIdx.x & 7, v0 = blockIdx.z * 32 * RV + threadIdx.x / 8;
  const int row = heads * vp + 2 * groups * np, g = h / (heads / groups);
  const int k_at = heads * vp + g * np + 4 * part, q_at = k_at + groups * np;
  float* st = states + (int64_t)state_slots[seq] * slot_stride + (int64_t)h * vp * np + 4 * part;
  float S[RV][NQ][4];
#pragma unroll
  for (int rv = 0; rv < RV; ++rv)
#pragma unroll
    for (int i = 0; i < NQ; ++i) ss_load4(st + (int64_t)min(v0 + 32 * rv, vp - 1) * np + 32 * i, S[rv][i]);
  float kn[NQ][4], qn[NQ][4], vn[RV], bn, ln, rkn, rqn;
  auto fetch = [&](int t) {
    const T* m = mixed + (int64_t)t * row;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      ss_load4(m + k_at + 32 * i, kn[i]);
      ss_load4(m + q_at + 32 * i, qn[i]);
    }
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) vn[rv] = Num<T>::ld(m + h * vp + min(v0 + 32 * rv, vp - 1));
    bn = betas[(int64_t)t * heads + h];
    ln = logs[(int64_t)t * heads + h];
    rkn = units[(int64_t)t * 2 * groups + g];
    rqn = units[(int64_t)t * 2 * groups + groups + g];
  };
  fetch(t_begin);
  for (int t = t_begin; t < t_end; ++t) {
    float k[NQ][4], q[NQ][4], v[RV];
    float kq = 0.f;
#pragma unroll
    for (int i = 0; i < NQ; ++i)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        k[i][c] = kn[i][c] * rkn;
        q[i][c] = qn[i][c] * rqn;
        kq = fmaf(k[i][c], q[i][c], kq);
      }
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) v[rv] = vn[rv];
    const float beta = bn, keep = expf(ln);
    if (t + 1 < t_end) fetch(t + 1);
    float sk[RV], sq[RV];
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) {
      sk[rv] = sq[rv] = 0.f;
#pragma unroll
      for (int i = 0; i < NQ; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          sk[rv] = fmaf(S[rv][i][c], k[i][c], sk[rv]);
          sq[rv] = fmaf(S[rv][i][c], q[i][c], sq[rv]);
        }
    }
#pragma unroll
    for (int off = 1; off < 8; off <<= 1) {
      kq += __shfl_xor(kq, off, TS_WAVE);
#pragma unroll
      for (int rv = 0; rv < RV; ++rv) {
        sk[rv] += __shfl_xor(sk[rv], off, TS_WAVE);
        sq[rv] += __shfl_xor(sq[rv], off, TS_WAVE);
      }
    }
#pragma unroll
    for (int rv = 0; rv < RV; ++rv) {
      const float u = beta * (v[rv] - keep * sk[rv]);
#pragma unroll
      for (int i = 0; i < NQ; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c) S[rv][i][c] = fmaf(k[i][c], u, keep * S[rv][i][c]);
      const int col = v0 + 32 * rv;
      if (part == 0 && col < vdim) out[((int64_t)t * heads + h) * vdim + col] = fmaf(kq, u, keep * sq[rv]);
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
extern "C" int ts_delta_step(float* out, const void* mixed, int dtype, const float* units, const float* betas, const float* logs,
                             float* states, int64_t slot_stride, const int32_t* cu_seqlens, const int32_t* state_slots, int num_seqs,
                             int heads, int vdim, int vp, int groups, int np, int up_to, hipStream_t stream) {
  if (num_seqs <= 0) return TS_OK;
  if (heads <= 0 || heads > 65535 || groups <= 0 || heads % groups || vdim <= 0 || vp < vdim || vp % 16 || np <= 0 || np % 32 || np > 512 ||
      slot_stride < (int64_t)heads * vp * np || slot_stride % 4 || (((uintptr_t)states | (uintptr_t)mixed) & 15))
    return TS_BAD_SHAPE;
  const int nq = np / 32;
  // (a slice of 64 columns where the step has workgroups enough and a lane's registers hold two columns' fours)
  const int rv = (vp > 32 && nq <= 4 && (int64_t)num_seqs * heads * ((vp + 63) / 64) >= 512) ? 2 : 1;
  const int slices = (vp + 32 * rv - 1) / (32 * rv);
  if (slices > 65535) return TS_BAD_SHAPE;
  dim3 grid(num_seqs, heads, slices);
#define DL_STEP(T, NQ, RV) \
  delta_step_kernel<T, NQ, RV><<<grid, DL_THREADS, 0, stream>>>(out, (const T*)mixed, units, betas, logs, states, slot_stride, cu_seqlens, \
                                                                state_slots, heads, vdim, vp, groups, up_to)
#define DL_STEP_2(T, NQ) case NQ: if (rv == 2) DL_STEP(T, NQ, 2); else DL_STEP(T, NQ, 1); break;
#define DL_STEP_1(T, NQ) case NQ: DL_STEP(T, NQ, 1); break;
#define DL_STEP_N(T) \
  switch (nq) { \
    DL_STEP_2(T, 1) DL_STEP_2(T, 2) DL_STEP_2(T, 3) DL_STEP_2(T, 4) DL_STEP_1(T, 5) DL_STEP_1(T, 6) DL_STEP_1(T, 7) DL_STEP_1(T, 8) \
    DL_STEP_1(T, 9) DL_STEP_1(T, 10) DL_STEP_1(T, 11) DL_STEP_1(T, 12) DL_STEP_1(T, 13) DL_STEP_1(T, 14) DL_STEP_1(T, 15) DL_STEP_1(T, 16) \
  }
  if (dtype == 0) { DL_STEP_N(float) }
  else if (dtype == 1) { DL_STEP_N(bf16_t) }
  else return TS_BAD_DTYPE;
#undef DL_STEP_N
#undef DL_STEP_1
#undef DL_STEP_2
#undef DL_STEP
  return ts_check_launch();
}

// ---- chunks of 64 tokens on the matrix cores (bfloat16) ----------------------------------------------------------

#define DL_TILE (SS_L * SS_L)   // a chunk's T or its weights, one bfloat16 term of them
#define DL_SCALES 5             // numbers of a chunk's token beside its rows
#define DL_F 68                 // a row of 64 numbers in shared memory, 32-bit

// D += A B over 4 k, 32-bit: lane (r, q) gives A[r][q] and B[q][r]; it gets D[4 q + i][r].
static __device__ __forceinline__ float4_t dl_mfma4(float a, float b, float4_t acc) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, acc, 0, 0, 0);
}

// acc += A M with A a 16 x 16 block in shared memory (rows DL_F apart) and M a product's result: lane (r, q) holds
// M[4 q + i][r], so step i takes row 4 q + i of M, and column 4 q + i of A, from every lane.
static __device__ __forceinline__ float4_t dl_times(const float* a, const float4_t& m, float4_t acc, int r, int q) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = dl_mfma4(a[r * DL_F + 4 * q + i], m[i], acc);
  return acc;
}
// acc += A B, both 16 x 16 blocks in shared memory
static __device__ __forceinline__ float4_t dl_blocks(const float* a, const float* b, float4_t acc, int r, int q) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = dl_mfma4(a[r * DL_F + 4 * q + i], b[(4 * q + i) * DL_F + r], acc);
  return acc;
}
static __device__ __forceinline__ void dl_put(float* dst, const float4_t& m, float sign, int r, int q) {
#pragma unroll
  for (int i = 0; i < 4; ++i) dst[(4 * q + i) * DL_F + r] = sign * m[i];
}

// What the walk reads lies in pieces: 16 rows by 32 of an operand as a wave takes them, lane after lane eight numbers of
// 2 bytes (lane (r, q): row r, columns 8 q .. 8 q + 7), a kilobyte side by side.
#define DL_PIECE (TS_WAVE * 8)

// One workgroup per (chunk, head). chunks: int32 [chunks, 4] (first token of the step, tokens 1 .. 64, request, whether the
// request's last). Per chunk and head: inv (T, rows tokens, as pieces [16 tokens][term][32 columns]), wts (the second sum's
// weights likewise; of both the pieces above the diagonal are never written nor read), vt (v, [16 value columns][16 tokens]
// [lane][4 tokens]), scales [5][64] (beta, beta exp(b) / |k|, exp(b) / |q| dim^(-1/2), exp(b_L - b) / |k|, zeros for tokens
// past the chunk's end; exp(b_L), 64 times); per chunk and group: keys (k and q as pieces [16 tokens][32 places], then k
// turned round as pieces [16 places][32 tokens]).
template <int NQ>
__global__ void __launch_bounds__(DL_THREADS, 4)
delta_chunk_solve_kernel(bf16_t* __restrict__ inv, bf16_t* __restrict__ wts, bf16_t* __restrict__ keys, bf16_t* __restrict__ vt,
                         float* __restrict__ scales, const bf16_t* __restrict__ mixed, const float* __restrict__ units, const float* __restrict__ betas, const float* __restrict__ logs,
                         const int32_t* __restrict__ chunks, int heads, int vp, int groups) {
  constexpr int np = 32 * NQ;
  __shared__ __attribute__((aligned(16))) float a_s[SS_L][DL_F], t_s[SS_L][DL_F];
  bf16_t (*turn_s)[SS_PAD] = (bf16_t (*)[SS_PAD])a_s;          // (at the end, where a_s has been read)
  __shared__ double b_s[SS_L];
  __shared__ float rk_s[SS_L], rq_s[SS_L], beta_s[SS_L];
  const int chunk = blockIdx.x, h = blockIdx.y;
  const int tok0 = chunks[4 * chunk], len = chunks[4 * chunk + 1];
  const int row = heads * vp + 2 * groups * np, per = heads / groups, g = h / per;
  const int wave = wave_index(), lane = threadIdx.x & (TS_WAVE - 1), r = lane & 15, q = lane >> 4;
  const int64_t ch = (int64_t)chunk * heads + h;
  const bf16_t* k_rows = mixed + (int64_t)tok0 * row + heads * vp + g * np + 8 * q;
  const bf16_t* q_rows = k_rows + groups * np;
  bf16_t* own_keys = keys + ((int64_t)chunk * groups + g) * 3 * np * SS_L;
  const int t = 16 * wave + r;                               // (this lane's token of the products)
  const int tc = min(t, len - 1);
  if (threadIdx.x < TS_WAVE) {
    const bool there = lane < len;
    const int64_t at = tok0 + min(lane, len - 1);
    const double b = ss_running(logs, tok0, len, heads, h);
    const double last = __shfl(b, TS_WAVE - 1, TS_WAVE);
    const float rk = units[at * 2 * groups + g], rq = units[at * 2 * groups + groups + g], beta = betas[at * heads + h];
    const float grown = expf((float)b);
    b_s[lane] = b;
    rk_s[lane] = rk;
    rq_s[lane] = rq;
    beta_s[lane] = beta;
    float* sc = scales + ch * DL_SCALES * SS_L + lane;
    sc[0] = there ? beta : 0.f;
    sc[SS_L] = there ? beta * grown * rk : 0.f;
    sc[2 * SS_L] = there ? grown * rq : 0.f;
    sc[3 * SS_L] = there ? expf((float)(last - b)) * rk : 0.f;
    sc[4 * SS_L] = expf((float)last);
  }
  // k_j . k_t and k_j . q_t, keys as the products' rows: lane (r, q) gets keys 16 jb + 4 q .. + 3 of token t
  float4_t kk[4], kq[4];
  {
    uint4 kf[NQ], qf[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      kf[i] = *(const uint4*)(k_rows + (int64_t)tc * row + 32 * i);
      qf[i] = *(const uint4*)(q_rows + (int64_t)tc * row + 32 * i);
    }
    if (h == g * per) {                                      // (the first head of a group leaves the group's pieces)
      bf16_t* piece = own_keys + (wave * NQ) * DL_PIECE + lane * 8;
#pragma unroll
      for (int i = 0; i < NQ; ++i) {
        *(uint4*)(piece + i * DL_PIECE) = kf[i];
        *(uint4*)(piece + i * DL_PIECE + np * SS_L) = qf[i];
      }
    }
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) {
      kk[jb] = kq[jb] = (float4_t){0.f, 0.f, 0.f, 0.f};
      if (jb > wave) continue;
      const bf16_t* key = k_rows + (int64_t)min(16 * jb + r, len - 1) * row;
#pragma unroll
      for (int i = 0; i < NQ; ++i) {
        const uint4 f = *(const uint4*)(key + 32 * i);
        kk[jb] = mfma32(f, kf[i], kk[jb]);
        kq[jb] = mfma32(f, qf[i], kq[jb]);
      }
    }
  }
  __syncthreads();
  {
    const double bt = b_s[t];
    const float kscale = beta_s[t] * rk_s[t], qscale = rq_s[t];
    // keys 16 jb + 4 q .. + 3 of a token are half of what lane (r, 2 (jb & 1) + q / 2) of piece jb / 2 holds
    bf16_t* w_piece = wts + ch * 2 * DL_TILE + wave * 4 * DL_PIECE + ((q >> 1) * 16 + r) * 8 + 4 * (q & 1);
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) {
      float a[4], p[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = 16 * jb + 4 * q + i;
        const bool before = j < t && t < len, upto = j <= t && t < len;
        const float fade = upto ? expf((float)(bt - b_s[j])) * rk_s[j] : 0.f;
        a[i] = before ? kscale * fade * kk[jb][i] : 0.f;
        p[i] = upto ? qscale * fade * kq[jb][i] : 0.f;
      }
      ss_store4(&a_s[t][16 * jb + 4 * q], a);
      if (jb <= (wave | 1)) {                                // (beyond the diagonal's piece: nobody reads)
        bf16_t* dst = w_piece + (jb >> 1) * DL_PIECE + (jb & 1) * 32 * 8;
        const uint32_t h0 = pack_bf16(p[0], p[1]), h1 = pack_bf16(p[2], p[3]);
        *(uint2*)dst = make_uint2(h0, h1);
        *(uint2*)(dst + 2 * DL_PIECE) = make_uint2(ss_rest(h0, p[0], p[1]), ss_rest(h1, p[2], p[3]));
      }
    }
  }
  __syncthreads();
  {
    // the diagonal blocks, a wave each: column r of the inverse by substitution, in registers (four lanes the same one)
    float x[16];
    const int d0 = 16 * wave;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == r ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < i; ++k) s = fmaf(-a_s[d0 + i][d0 + k], x[k], s);
      x[i] = s;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if ((i >> 2) == q) t_s[d0 + i][d0 + r] = x[i];
  }
  __syncthreads();
  const float4_t none = {0.f, 0.f, 0.f, 0.f};
  if (wave < 2) {                                            // blocks (1, 0) and (3, 2): -T_ii A_ij T_jj
    const int bi = 2 * wave + 1, bj = 2 * wave;
    const float4_t m = dl_blocks(&a_s[16 * bi][16 * bj], &t_s[16 * bj][16 * bj], none, r, q);
    dl_put(&t_s[16 * bi][16 * bj], dl_times(&t_s[16 * bi][16 * bi], m, none, r, q), -1.f, r, q);
  }
  __syncthreads();
  {                                                          // the lower left 32 x 32: -T_lower A T_upper, a block a wave
    const int bi = 2 + (wave >> 1), bj = wave & 1;
    float4_t sum = none;
#pragma unroll
    for (int k = 2; k < 4; ++k) {
      if (k > bi) continue;
      float4_t m = none;
      for (int u = bj; u < 2; ++u) m = dl_blocks(&a_s[16 * k][16 * u], &t_s[16 * u][16 * bj], m, r, q);
      sum = dl_times(&t_s[16 * bi][16 * k], m, sum, r, q);
    }
    dl_put(&t_s[16 * bi][16 * bj], sum, -1.f, r, q);
  }
  __syncthreads();
  {
    bf16_t* t_piece = inv + ch * 2 * DL_TILE + wave * 4 * DL_PIECE + lane * 8;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (kk == 1 && wave < 2) continue;
      float x[2][4];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int j = 32 * kk + 8 * q + 4 * half;
        if ((j >> 4) <= wave) ss_load4(&t_s[t][j], x[half]); // (the blocks above the diagonal were never written)
        else x[half][0] = x[half][1] = x[half][2] = x[half][3] = 0.f;
      }
      uint4 hi, lo;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float a = x[k >> 1][2 * (k & 1)], b = x[k >> 1][2 * (k & 1) + 1];
        (&hi.x)[k] = pack_bf16(a, b);
        (&lo.x)[k] = ss_rest((&hi.x)[k], a, b);
      }
      *(uint4*)(t_piece + kk * DL_PIECE) = hi;
      *(uint4*)(t_piece + (2 + kk) * DL_PIECE) = lo;
    }
  }
  // v and (by the first head of a group) k turned round, 64 columns at a time
  auto turn = [&](const bf16_t* src, int cols, auto leave) {
    for (int c0 = 0; c0 < cols; c0 += 64) {
      __syncthreads();                                       // (the tile before has been read)
      ss_turn<false>(turn_s, nullptr, src + c0, row, tok0, len, cols - c0, nullptr);
      __syncthreads();
      leave(c0);
    }
  };
  bf16_t* own_v = vt + ch * vp * SS_L;
  turn(mixed + h * vp, vp, [&](int c0) {
#pragma unroll
    for (int c = 0; c < 4; ++c)                              // (wave w: tokens 16 w .. + 15 of the tile's columns, 16 at a time)
      if (c0 + 16 * c < vp) *(uint2*)(own_v + ((c0 / 16 + c) * 4 + wave) * TS_WAVE * 4 + lane * 4) = *(const uint2*)&turn_s[16 * c + r][16 * wave + 4 * q];
  });
  if (h == g * per)
    turn(mixed + heads * vp + g * np, np, [&](int c0) {
      if (c0 + 16 * wave >= np) return;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        *(uint4*)(own_keys + 2 * np * SS_L + ((c0 / 16 + wave) * 2 + kk) * DL_PIECE + lane * 8) = *(const uint4*)&turn_s[16 * wave + r][32 * kk + 8 * q];
    });
}

// A number's two bfloat16 terms, four at a time.
static __device__ __forceinline__ void dl_split4(bf16_t* hi, bf16_t* lo, const float (&x)[4]) {
  const uint32_t h0 = pack_bf16(x[0], x[1]), h1 = pack_bf16(x[2], x[3]);
  *(uint2*)hi = make_uint2(h0, h1);
  *(uint2*)lo = make_uint2(ss_rest(h0, x[0], x[1]), ss_rest(h1, x[2], x[3]));
}

// One workgroup per (request and head, 16 value columns); it walks the request's chunks in order. Wave w has the chunk's
// tokens 16 w .. 16 w + 15 and of the state the blocks of 16 key places w, w + 4, ... (32-bit, in registers); what the next
// product needs whole goes through shared memory in two terms, laid out as that product's operand. The next chunk's
// operands are fetched while one is worked on. Between two barriers everything that lies in shared memory is asked for
// before the first of it is used, and a product's terms go into sums of their own, so that no product waits for another.
template <int NQ>
__global__ void __launch_bounds__(DL_THREADS, NQ <= 4 ? 2 : 1)
delta_chunk_walk_kernel(float* __restrict__ out, const bf16_t* __restrict__ inv, const bf16_t* __restrict__ wts,
                        const bf16_t* __restrict__ keys, const bf16_t* __restrict__ vt, const float* __restrict__ scales,
                        float* __restrict__ states, int64_t slot_stride, const int32_t* __restrict__ chunks,
                        const int32_t* __restrict__ chunk_cu, const int32_t* __restrict__ state_slots, int num_seqs, int heads, int vdim,
                        int vp, int groups) {
  constexpr int np = 32 * NQ, BLOCKS = (2 * NQ + 3) / 4, S_ROW = np + 8;
  __shared__ __attribute__((aligned(16))) bf16_t s_s[2][16][S_ROW];            // the state: [term][column][place]
  __shared__ __attribute__((aligned(16))) bf16_t r_s[2][16][SS_PAD];           // beta V - beta exp(b) K S0: [term][column][token]
  __shared__ __attribute__((aligned(16))) bf16_t u_s[2][16][SS_PAD], d_s[2][16][SS_PAD];     // U, and U fading to the chunk's end
  // the slices of one head run on one die (workgroup index mod 8), side by side, and share what they read in its cache
  const int slices = vp / 16, die = blockIdx.x % 8, turn = blockIdx.x / 8;
  const int pair = (turn / slices) * 8 + die, slice = turn % slices;
  if (pair >= num_seqs * heads) return;
  const int seq = pair / heads, h = pair - seq * heads, v0 = 16 * slice;
  const int begin = chunk_cu[seq], end = chunk_cu[seq + 1];
  if (begin >= end) return;
  const int g = h / (heads / groups);
  const int wave = wave_index(), lane = threadIdx.x & (TS_WAVE - 1), r = lane & 15, q = lane >> 4;
  float* st = states + (int64_t)state_slots[seq] * slot_stride + (int64_t)h * vp * np + (int64_t)(v0 + r) * np + 4 * q;
  const float4_t none = {0.f, 0.f, 0.f, 0.f};
  auto has = [&](int i) { return (2 * NQ) % 4 == 0 || wave + 4 * i < 2 * NQ; };              // whether this wave has an i-th block
  float4_t S[BLOCKS];
#pragma unroll
  for (int i = 0; i < BLOCKS; ++i) {
    S[i] = none;
    if (has(i)) {
      S[i] = *(const float4_t*)(st + 16 * (wave + 4 * i));
      const float x[4] = {S[i][0], S[i][1], S[i][2], S[i][3]};
      dl_split4(&s_s[0][r][16 * (wave + 4 * i) + 4 * q], &s_s[1][r][16 * (wave + 4 * i) + 4 * q], x);
    }
  }
  const bool second = wave >= 2;                             // whether this wave's tokens see the chunk's second half
  struct Operands {
    uint4 k[NQ], qq[NQ], t[2][2], w[2][2], kt[BLOCKS][2];
    uint2 v;
    float beta[4], bk[4], bq[4], dk[4], total;
  };
  // (a request's chunks lie side by side, all of 64 tokens but the last)
  const int first = chunks[4 * begin], stop = chunks[4 * end - 4] + chunks[4 * end - 3];
  auto fetch = [&](int c, Operands& o) {
    const int64_t ch = (int64_t)c * heads + h;
    const bf16_t* k_piece = keys + ((int64_t)c * groups + g) * 3 * np * SS_L + lane * 8;
    const bf16_t* t_piece = inv + ch * 2 * DL_TILE + wave * 4 * DL_PIECE + lane * 8;
    const bf16_t* w_piece = wts + ch * 2 * DL_TILE + wave * 4 * DL_PIECE + lane * 8;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      o.k[i] = *(const uint4*)(k_piece + (wave * NQ + i) * DL_PIECE);
      o.qq[i] = *(const uint4*)(k_piece + np * SS_L + (wave * NQ + i) * DL_PIECE);
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (kk == 1 && !second) continue;
#pragma unroll
      for (int term = 0; term < 2; ++term) {
        o.t[term][kk] = *(const uint4*)(t_piece + (2 * term + kk) * DL_PIECE);
        o.w[term][kk] = *(const uint4*)(w_piece + (2 * term + kk) * DL_PIECE);
      }
    }
    o.v = *(const uint2*)(vt + ch * vp * SS_L + (slice * 4 + wave) * TS_WAVE * 4 + lane * 4);
    const float* sc = scales + ch * DL_SCALES * SS_L + 16 * wave + 4 * q;
    ss_load4(sc, o.beta);
    ss_load4(sc + SS_L, o.bk);
    ss_load4(sc + 2 * SS_L, o.bq);
    ss_load4(sc + 3 * SS_L, o.dk);
    o.total = sc[4 * SS_L];
#pragma unroll
    for (int i = 0; i < BLOCKS; ++i) {
      const bf16_t* turned = k_piece + 2 * np * SS_L + min(wave + 4 * i, 2 * NQ - 1) * 2 * DL_PIECE;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) o.kt[i][kk] = *(const uint4*)(turned + kk * DL_PIECE);
    }
  };
  auto work = [&](int c, const Operands& now) {
    __syncthreads();                                         // (the state lies in s_s)
    float4_t x[2] = {none, none}, y[2] = {none, none};
    constexpr int AT_ONCE = NQ == 4 ? 2 : 4;                               // pieces of the state whose two terms are read together
#pragma unroll
    for (int i0 = 0; i0 < NQ; i0 += AT_ONCE) {
      uint4 s[AT_ONCE][2];
#pragma unroll
      for (int i = 0; i < AT_ONCE && i0 + i < NQ; ++i)
#pragma unroll
        for (int term = 0; term < 2; ++term) s[i][term] = *(const uint4*)&s_s[term][r][32 * (i0 + i) + 8 * q];
#pragma unroll
      for (int i = 0; i < AT_ONCE && i0 + i < NQ; ++i)
#pragma unroll
        for (int term = 0; term < 2; ++term) {
          x[term] = mfma32(now.k[i0 + i], s[i][term], x[term]);
          y[term] = mfma32(now.qq[i0 + i], s[i][term], y[term]);
        }
    }
    {
      const float v[4] = {__uint_as_float(now.v.x << 16), __uint_as_float(now.v.x & 0xffff0000u), __uint_as_float(now.v.y << 16),
                          __uint_as_float(now.v.y & 0xffff0000u)};
      float rest[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) rest[i] = fmaf(now.beta[i], v[i], -now.bk[i] * (x[0][i] + x[1][i]));
      dl_split4(&r_s[0][r][16 * wave + 4 * q], &r_s[1][r][16 * wave + 4 * q], rest);
    }
    __syncthreads();
    // rows of T and of the weights beyond this wave's tokens are zeros: the second half counts for waves 2 and 3 alone
    uint4 rest[2][2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int term = 0; term < 2; ++term) rest[kk][term] = *(const uint4*)&r_s[term][r][32 * kk + 8 * q];
    float4_t u0 = mfma32(now.t[0][0], rest[0][0], none), u1 = mfma32(now.t[0][0], rest[0][1], none), u2 = mfma32(now.t[1][0], rest[0][0], none);
    if (second) {
      u0 = mfma32(now.t[0][1], rest[1][0], u0);
      u1 = mfma32(now.t[0][1], rest[1][1], u1);
      u2 = mfma32(now.t[1][1], rest[1][0], u2);
    }
    {
      float w[4], fading[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        w[i] = u0[i] + (u1[i] + u2[i]);
        fading[i] = w[i] * now.dk[i];
      }
      dl_split4(&d_s[0][r][16 * wave + 4 * q], &d_s[1][r][16 * wave + 4 * q], fading);
      dl_split4(&u_s[0][r][16 * wave + 4 * q], &u_s[1][r][16 * wave + 4 * q], w);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {                            // (while the other waves come to the barrier)
      y[0][i] = now.bq[i] * (y[0][i] + y[1][i]);
#pragma unroll
      for (int b = 0; b < BLOCKS; ++b) S[b][i] *= now.total;
    }
    __syncthreads();
    uint4 d[2][2], w[2][2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int term = 0; term < 2; ++term) d[kk][term] = *(const uint4*)&d_s[term][r][32 * kk + 8 * q];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int term = 0; term < 2; ++term) w[kk][term] = *(const uint4*)&u_s[term][r][32 * kk + 8 * q];
    float4_t low[BLOCKS];
#pragma unroll
    for (int i = 0; i < BLOCKS; ++i) low[i] = none;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < BLOCKS; ++i) {
        S[i] = mfma32(now.kt[i][kk], d[kk][0], S[i]);
        low[i] = mfma32(now.kt[i][kk], d[kk][1], low[i]);
      }
    y[0] = mfma32(now.w[0][0], w[0][0], y[0]);
    y[1] = mfma32(now.w[0][0], w[0][1], none);
    float4_t y2 = mfma32(now.w[1][0], w[0][0], none);
    if (second) {
      y[0] = mfma32(now.w[0][1], w[1][0], y[0]);
      y[1] = mfma32(now.w[0][1], w[1][1], y[1]);
      y2 = mfma32(now.w[1][1], w[1][0], y2);
    }
#pragma unroll
    for (int i = 0; i < BLOCKS; ++i) {
#pragma unroll
      for (int j = 0; j < 4; ++j) S[i][j] += low[i][j];
      const float x4[4] = {S[i][0], S[i][1], S[i][2], S[i][3]};
      if (has(i)) dl_split4(&s_s[0][r][16 * (wave + 4 * i) + 4 * q], &s_s[1][r][16 * (wave + 4 * i) + 4 * q], x4);
    }
    if (v0 + r < vdim) {
      const int tok = first + SS_L * (c - begin) + 16 * wave + 4 * q;
      float* dst = out + ((int64_t)tok * heads + h) * vdim + v0 + r;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (tok + i < stop) dst[(int64_t)i * heads * vdim] = y[0][i] + (y[1][i] + y2[i]);
    }
  };
  Operands even, odd;                                        // (two sets in turn: nothing is copied from one to the other)
  fetch(begin, even);
  for (int c = begin; c < end; c += 2) {
    fetch(min(c + 1, end - 1), odd);
    work(c, even);
    if (c + 1 >= end) break;
    fetch(min(c + 2, end - 1), even);
    work(c + 1, odd);
  }
#pragma unroll
  for (int i = 0; i < BLOCKS; ++i)
    if (has(i)) *(float4_t*)(st + 16 * (wave + 4 * i)) = S[i];
}

// chunk_cu: int32 [requests + 1], each request's first chunk; requests without chunks keep their state as it is. inv and wts
// bfloat16 [chunks, heads, 2, 64, 64], keys [chunks, groups, 3, np, 64], vt [chunks, heads, vp, 64], scales float32 [chunks, heads,
// 5, 64]: scratch.
extern "C" int ts_delta_chunks(float* out, const void* mixed, const float* units, const float* betas, const float* logs, float* states,
                               int64_t slot_stride, const int32_t* chunks, const int32_t* chunk_cu, const int32_t* state_slots,
                               void* inv, void* wts, void* keys, void* vt, float* scales, int num_chunks, int num_seqs, int heads,
                               int vdim, int vp, int groups, int np, hipStream_t stream) {
  if (num_chunks <= 0 || num_seqs <= 0) return TS_OK;
  if (heads <= 0 || heads > 65535 || groups <= 0 || heads % groups || vdim <= 0 || vp < vdim || vp % 16 || np <= 0 || np % 32 ||
      np > DL_MAX_CHUNK_NP || slot_stride < (int64_t)heads * vp * np || slot_stride % 4 ||
      (((uintptr_t)states | (uintptr_t)mixed | (uintptr_t)inv | (uintptr_t)wts | (uintptr_t)keys | (uintptr_t)vt | (uintptr_t)scales) & 15))
    return TS_BAD_SHAPE;
  const bf16_t* m = (const bf16_t*)mixed;
  const int64_t walkers64 = ((int64_t)num_seqs * heads + 7) / 8 * 8 * (vp / 16);
  if (walkers64 > 0x7fffffff) return TS_BAD_SHAPE;
  const unsigned walkers = (unsigned)walkers64;
#define DL_CHUNKS(NQ) \
  case NQ: \
    delta_chunk_solve_kernel<NQ><<<dim3(num_chunks, heads), DL_THREADS, 0, stream>>>((bf16_t*)inv, (bf16_t*)wts, (bf16_t*)keys, (bf16_t*)vt, scales, \
                                                                                     m, units, betas, logs, chunks, heads, vp, groups); \
    delta_chunk_walk_kernel<NQ><<<walkers, DL_THREADS, 0, stream>>>(out, (const bf16_t*)inv, (const bf16_t*)wts, (const bf16_t*)keys, \
                                                                    (const bf16_t*)vt, scales, states, slot_stride, chunks, chunk_cu, state_slots, \
                                                                    num_seqs, heads, vdim, vp, groups); \
    break;
  switch (np / 32) { DL_CHUNKS(1) DL_CHUNKS(2) DL_CHUNKS(3) DL_CHUNKS(4) DL_CHUNKS(5) DL_CHUNKS(6) DL_CHUNKS(7) DL_CHUNKS(8) }
#undef DL_CHUNKS
  return ts_check_launch();
}
