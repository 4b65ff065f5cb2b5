// What lies between the projection and the recurrence of retention (a matrix state per head with a fixed decay, worked by
// the kernels of state_space.hip): from a projected 32-bit row v | k | q (then whatever else the fused projection makes) to
// the row those kernels read, in the activations' storage type: every head's v in `vp` places, every head's k and q in `np`
// (multiples of 16 and 32, zeros behind a head's own numbers), k and q turned by the token's position in pairs
// (i, i + rot/2) of their first `rot` dimensions, the angle position * f_i taken in 64-bit.
#include "chunk_ops.h"

#define RT_THREADS 256
#define RT_MAX_DIM 512

// A workgroup per token and slice of its row; it takes the token's sines and cosines once. VEC: sizes and halves are
// multiples of four and the rows 16-byte aligned.
template <typename TO, bool VEC>
__global__ void __launch_bounds__(RT_THREADS)
retention_prepare_kernel(TO* __restrict__ mixed, const float* __restrict__ proj, int64_t stride, const double* __restrict__ freqs,
                         const int32_t* __restrict__ positions, int heads, int vdim, int vp, int dim, int np, int rot) {
  __shared__ float cos_s[RT_MAX_DIM / 2], sin_s[RT_MAX_DIM / 2];
  const int t = blockIdx.x, half = rot / 2;
  const int pos = positions[t];
  for (int pair = threadIdx.x; pair < half; pair += RT_THREADS) {
    // the angle in 64-bit, brought to [-pi, pi] before the 32-bit sine and cosine
    const double angle = (double)pos * freqs[pair];
    const double turns = rint(angle * 0.15915494309189535);
    sincosf((float)fma(-turns, 6.283185307179586, angle), &sin_s[pair], &cos_s[pair]);
  }
  __syncthreads();
  const int row = heads * (vp + 2 * np);
  const float* src = proj + (int64_t)t * stride;
  TO* dst = mixed + (int64_t)t * row;
  for (int place = 4 * (blockIdx.y * RT_THREADS + threadIdx.x); place < row; place += 4 * RT_THREADS * gridDim.y) {
    float y[4];
    if (place < heads * vp) {
      const int h = place / vp, off = place - h * vp;
      const float* v = src + h * vdim + off;
      if (VEC && off < vdim) ss_load4(v, y);
      else {
#pragma unroll
        for (int k = 0; k < 4; ++k) y[k] = off + k < vdim ? v[k] : 0.f;
      }
    } else {
      const int at = place - heads * vp;
      const int which = at / (heads * np), in = at - which * heads * np;
      const int h = in / np, off = in - h * np;
      const float* x = src + heads * vdim + (which * heads + h) * dim;
      if (VEC) {
        float u[4] = {0.f, 0.f, 0.f, 0.f};
        if (off < dim) ss_load4(x + off, u);
        if (off < rot) {
          const bool first = off < half;
          const int pair = first ? off : off - half;
          float w[4];
          ss_load4(x + (first ? off + half : off - half), w);
#pragma unroll
          for (int k = 0; k < 4; ++k) y[k] = first ? u[k] * cos_s[pair + k] - w[k] * sin_s[pair + k] : u[k] * cos_s[pair + k] + w[k] * sin_s[pair + k];
        } else {
#pragma unroll
          for (int k = 0; k < 4; ++k) y[k] = u[k];
        }
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          const int d = off + k;
          float v = d < dim ? x[d] : 0.f;
          if (d < half) v = v * cos_s[d] - x[d + half] * sin_s[d];
          else if (d < rot) v = v * cos_s[d - half] + x[d - half] * sin_s[d - half];
          y[k] = v;
        }
      }
    }
    ss_store4(dst + place, y);
  }
}

extern "C" int ts_retention_prepare(void* mixed, int out_dtype, const float* proj, int64_t stride, const double* freqs,
                                    const int32_t* positions, int num_tokens, int heads, int vdim, int vp, int dim, int np, int rot,
                                    hipStream_t stream) {
  if (num_tokens <= 0) return TS_OK;
  const int64_t row = (int64_t)heads * (vp + 2 * (int64_t)np);
  if (heads <= 0 || vdim <= 0 || dim <= 0 || dim > RT_MAX_DIM || vp < vdim || np < dim || vp % 16 || np % 32 || rot < 0 || rot > dim || rot % 2 ||
      (rot && !freqs) || row > (1 << 28) || stride < (int64_t)heads * (vdim + 2 * (int64_t)dim) || ((uintptr_t)mixed & 15))
    return TS_BAD_SHAPE;
  const bool vec = vdim % 4 == 0 && dim % 4 == 0 && rot % 8 == 0 && stride % 4 == 0 && ((uintptr_t)proj & 15) == 0;
  // a thread takes one four of places in steps of few tokens, several (and so its workgroup's angles once for more) in long ones
  const int64_t fours = row / 4, all = (fours + RT_THREADS - 1) / RT_THREADS;
  const dim3 grid(num_tokens, (unsigned)(num_tokens >= 256 ? (all + 3) / 4 : all > 65535 ? 65535 : all));
#define RT_GO(TO, VEC) retention_prepare_kernel<TO, VEC><<<grid, RT_THREADS, 0, stream>>>((TO*)mixed, proj, stride, freqs, positions, heads, vdim, vp, dim, np, rot)
  if (out_dtype == 0) { if (vec) RT_GO(float, true); else RT_GO(float, false); }
  else if (out_dtype == 1) { if (vec) RT_GO(bf16_t, true); else RT_GO(bf16_t, false); }
  else return TS_BAD_DTYPE;
#undef RT_GO
  return ts_check_launch();
}
