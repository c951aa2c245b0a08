// Several residual streams per token (hyper-connections): one sublayer's write and the next sublayer's read.
//
//   y    = y1 * y_gate[t] + y3                          y1: activation row (float or bf16, row-strided); y3: fp32
//   x_t <- sum_s mix[s][t] x_s + w_out[t] y             all streams from the old ones (mix == nullptr: unchanged)
//   u    = sum_t w_in[t] x_t                            (w_in == nullptr: weights 1)
//   n    = u / sqrt(mean(u^2) + eps) * g                written as fp32 and / or as an activation tensor
//
// x is fp32 [T][S][W] and updated in place; `equal`: x is [T][W] and stands for S equal streams (a sequence's start), the
// streams then go to `xo` [T][S][W]. xo == nullptr: the new streams are not kept (nobody reads them again). dest !=
// nullptr: y3 holds the rows of a routed mixture in their sorted layout and what is added for token t is
// sum_j cw[t][j] * y3[dest[t][j]] over its `top` choices in order (cw == nullptr: weights 1).
//
// One workgroup per token. A thread takes four columns of every stream at a time (16-byte loads, all S streams in
// flight), keeps u in LDS until the row's root mean square is known, and never re-reads a stream.
#include "mixers_common.h"

#include <algorithm>

namespace xgm {

constexpr int kMaxStreams = 32;

// SM: streams held in registers; EXACT: S == SM (otherwise S <= SM, checked per stream)
template <typename TY, typename TO, int SM, bool EXACT>
__global__ __launch_bounds__(1024) void hyper_residual_kernel(
    const float* x, int equal, float* xo, int S_, const TY* __restrict__ y1, int64_t ld1,
    const float* __restrict__ y_gate, const float* __restrict__ y3, const int32_t* __restrict__ dest,
    const float* __restrict__ cw, int top, const float* __restrict__ w_out, const float* __restrict__ mix,
    const float* __restrict__ w_in, const float* __restrict__ g, float eps, float* __restrict__ n32,
    TO* __restrict__ nact, int W, int vec) {
  extern __shared__ __attribute__((aligned(16))) float ubuf[];   // [W] | [16] partial sums
  float* red = ubuf + ((W + 3) & ~3);
  const int S = EXACT ? SM : S_;
  const int t = blockIdx.x;
  const float* xr = x + (int64_t)t * (equal ? W : (int64_t)S * W);
  const int64_t lds = equal ? 0 : W;                             // distance of two streams of the token
  float* xw = xo ? xo + (int64_t)t * S * W : nullptr;
  const float gt = (y1 && y_gate) ? y_gate[t] : 1.f;
  float ss = 0.f;
  if (vec) {
    for (int c = 4 * threadIdx.x; c < W; c += 4 * blockDim.x) {
      float v[SM][4], y[4] = {0.f, 0.f, 0.f, 0.f}, u[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (EXACT || s < S) ld4(xr + s * lds + c, v[s]);
      if (mix) {
        if (y1) {
          ld4(y1 + (int64_t)t * ld1 + c, y);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[e] *= gt;
        }
        if (y3 && dest) {
          for (int j = 0; j < top; ++j) {
            float r[4];
            ld4(y3 + (int64_t)dest[(int64_t)t * top + j] * W + c, r);
            const float wj = cw ? cw[(int64_t)t * top + j] : 1.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) y[e] += wj * r[e];
          }
        } else if (y3) {
          float r[4];
          ld4(y3 + (int64_t)t * W + c, r);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[e] += r[e];
        }
#pragma unroll
        for (int o = 0; o < SM; ++o) {
          if (!EXACT && o >= S) break;
          const float wo = w_out[o], wi = w_in ? w_in[o] : 1.f;
          float z[4];
#pragma unroll
          for (int e = 0; e < 4; ++e) z[e] = wo * y[e];
#pragma unroll
          for (int s = 0; s < SM; ++s)
            if (EXACT || s < S) {
              const float ms = mix[s * S + o];
#pragma unroll
              for (int e = 0; e < 4; ++e) z[e] += ms * v[s][e];
            }
          if (xw) st4(xw + (int64_t)o * W + c, z);
#pragma unroll
          for (int e = 0; e < 4; ++e) u[e] += wi * z[e];
        }
      } else {
#pragma unroll
        for (int s = 0; s < SM; ++s)
          if (EXACT || s < S) {
            const float wi = w_in ? w_in[s] : 1.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) u[e] += wi * v[s][e];
          }
      }
      st4(ubuf + c, u);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += u[e] * u[e];
    }
  } else {
    for (int c = threadIdx.x; c < W; c += blockDim.x) {
      float v[SM], y = 0.f, u = 0.f;
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (EXACT || s < S) v[s] = xr[s * lds + c];
      if (mix) {
        if (y1) y = gt * ldf(y1 + (int64_t)t * ld1 + c);
        if (y3 && dest) {
          for (int j = 0; j < top; ++j)
            y += (cw ? cw[(int64_t)t * top + j] : 1.f) * y3[(int64_t)dest[(int64_t)t * top + j] * W + c];
        } else if (y3) {
          y += y3[(int64_t)t * W + c];
        }
#pragma unroll
        for (int o = 0; o < SM; ++o) {
          if (!EXACT && o >= S) break;
          float z = w_out[o] * y;
#pragma unroll
          for (int s = 0; s < SM; ++s)
            if (EXACT || s < S) z += mix[s * S + o] * v[s];
          if (xw) xw[(int64_t)o * W + c] = z;
          u += (w_in ? w_in[o] : 1.f) * z;
        }
      } else {
#pragma unroll
        for (int s = 0; s < SM; ++s)
          if (EXACT || s < S) u += (w_in ? w_in[s] : 1.f) * v[s];
      }
      ubuf[c] = u;
      ss += u * u;
    }
  }
  const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
  // each thread reads back only what it wrote itself
  if (vec) {
    for (int c = 4 * threadIdx.x; c < W; c += 4 * blockDim.x) {
      float u[4], gw[4];
      ld4(ubuf + c, u);
      ld4(g + c, gw);
#pragma unroll
      for (int e = 0; e < 4; ++e) u[e] = u[e] * r * gw[e];
      if (n32) st4(n32 + (int64_t)t * W + c, u);
      if (nact) st4(nact + (int64_t)t * W + c, u);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += blockDim.x) {
      const float v = ubuf[c] * r * g[c];
      if (n32) n32[(int64_t)t * W + c] = v;
      if (nact) stf(nact + (int64_t)t * W + c, v);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void soft_cap_kernel(T* __restrict__ x, float cap, float inv, int64_t n) {
  for (int64_t i = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x)
    stf(x + i, cap * tanhf(ldf(x + i) * inv));
}

// ================================================================== host launchers
int hyper_residual(const float* x, bool equal, float* xo, int S, const void* y1, int64_t ld1, bool y_f32,
                   const float* y_gate, const float* y3, const int32_t* dest, const float* cw, int top,
                   const float* w_out, const float* mix, const float* w_in, const float* g, float eps, float* n32,
                   void* nact, bool nact_f32, int T_, int W, hipStream_t st) {
  if (T_ <= 0) return 0;
  if (S < 1 || S > kMaxStreams || W < 1 || W > 16384 || !x || !g || (mix != nullptr) != (w_out != nullptr) ||
      (!mix && (xo || y1 || y3)) || (dest && (!y3 || top < 1)) || (xo && !equal && xo != x))
    return -1;
  const int ysz = y_f32 ? 4 : 2;
  const int vec = (W & 3) == 0 && (!y1 || ((ld1 & 3) == 0 && (uintptr_t)y1 % (4 * ysz) == 0));
  // few rows: a wider workgroup per row (one pass over the columns); many rows: four waves, several rows per CU
  const int quads = vec ? W / 4 : W;
  const int nth = T_ >= 1024 ? 256 : std::min(1024, std::max(64, (quads + 63) / 64 * 64));
  const size_t lds = (((size_t)W + 3) / 4 * 4 + 16) * sizeof(float);
#define XGM_HR2(TY, TO, SM, EX)                                                                                       \
  hyper_residual_kernel<TY, TO, SM, EX><<<T_, nth, lds, st>>>(x, equal ? 1 : 0, xo, S, (const TY*)y1, ld1, y_gate, y3, \
                                                              dest, cw, top, w_out, mix, w_in, g, eps, n32, (TO*)nact, \
                                                              W, vec);
#define XGM_HR1(SM, EX)                                                       \
  {                                                                           \
    if (y_f32) {                                                              \
      if (nact_f32) { XGM_HR2(float, float, SM, EX) } else { XGM_HR2(float, bf16, SM, EX) } \
    } else {                                                                  \
      if (nact_f32) { XGM_HR2(bf16, float, SM, EX) } else { XGM_HR2(bf16, bf16, SM, EX) }   \
    }                                                                         \
    return 0;                                                                 \
  }
  switch (S) {
    case 1: XGM_HR1(1, true)
    case 2: XGM_HR1(2, true)
    case 3: XGM_HR1(3, true)
    case 4: XGM_HR1(4, true)
    case 8: XGM_HR1(8, true)
    default: break;
  }
  if (S < 8) XGM_HR1(8, false)
  XGM_HR1(kMaxStreams, false)
#undef XGM_HR1
#undef XGM_HR2
}

void soft_cap(void* x, bool f32, float cap, int64_t n, hipStream_t st) {
  if (n <= 0) return;
  const int blocks = (int)std::min<int64_t>((n + 255) / 256, 1 << 16);
  XGM_DISPATCH_T(f32, soft_cap_kernel<T><<<blocks, 256, 0, st>>>((T*)x, cap, 1.f / cap, n);)
}

}  // namespace xgm
