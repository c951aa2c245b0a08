// Layer norm on a sublayer's output before it joins the residual stream:
//
//   layer_norm_residual   u  = s1 * y1 + s2 * y2                       (activation tensors; y2 may be nullptr)
//                         u  = sum_j cw[t][j] * y3[dest[t][j]]         (routed rows of a mixture, or plain fp32 rows)
//                         x <- x + L(u) * w          (ids != nullptr: u = y1[ids[t]] and x <- L(u) * w, an embedding)
//                         out = x, or L(x) * next_w, as an activation tensor (nullptr: not written)
//                       L(v) = (v - mean(v)) / sqrt(mean((v - mean(v))^2) + eps)
//
// x is the fp32 residual stream. One workgroup per row. Rows of up to 8192 aligned columns live in registers (every
// global load of the row is issued before the first reduction, deviations are squared after the mean is known); other
// rows in LDS.
#include "mixers_common.h"

namespace xgm {

struct LnArgs {
  float* x;
  const void *y1, *y2;
  int64_t ld1, ld2;
  float s1, s2;
  const int32_t* ids;
  int V;
  const float* y3;
  const int32_t* dest;
  const float* cw;
  int top;
  const float *w, *next_w;
  float eps;
  void* out;
  int W;
};

// columns c .. c + 3 of the sublayer's output for row t
template <typename TY>
__device__ __forceinline__ void ln_src4(const LnArgs& a, int t, int64_t row1, int c, float (&u)[4]) {
  u[0] = u[1] = u[2] = u[3] = 0.f;
  float r[4];
  if (a.y1) {
    if (row1 >= 0) ld4((const TY*)a.y1 + row1 * a.ld1 + c, u);
#pragma unroll
    for (int i = 0; i < 4; ++i) u[i] *= a.s1;
    if (a.y2) {
      ld4((const TY*)a.y2 + (int64_t)t * a.ld2 + c, r);
#pragma unroll
      for (int i = 0; i < 4; ++i) u[i] += a.s2 * r[i];
    }
  } else if (!a.dest) {
    ld4(a.y3 + (int64_t)t * a.W + c, u);
  } else {
    for (int j = 0; j < a.top; ++j) {
      const int64_t k = (int64_t)t * a.top + j;
      ld4(a.y3 + (int64_t)a.dest[k] * a.W + c, r);
      const float wj = a.cw ? a.cw[k] : 1.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) u[i] += wj * r[i];
    }
  }
}

template <typename TY>
__device__ __forceinline__ float ln_src1(const LnArgs& a, int t, int64_t row1, int c) {
  if (a.y1) {
    float u = row1 >= 0 ? a.s1 * ldf((const TY*)a.y1 + row1 * a.ld1 + c) : 0.f;
    if (a.y2) u += a.s2 * ldf((const TY*)a.y2 + (int64_t)t * a.ld2 + c);
    return u;
  }
  if (!a.dest) return a.y3[(int64_t)t * a.W + c];
  float u = 0.f;
  for (int j = 0; j < a.top; ++j) {
    const int64_t k = (int64_t)t * a.top + j;
    u += (a.cw ? a.cw[k] : 1.f) * a.y3[(int64_t)a.dest[k] * a.W + c];
  }
  return u;
}

template <typename TY, typename TO, int NV, int NTH>
__global__ __launch_bounds__(NTH) void layer_norm_residual_vec_kernel(const LnArgs a) {
  __shared__ float red[NTH / 64];
  const int t = blockIdx.x, W = a.W;
  float* xr = a.x + (int64_t)t * W;
  const float inv_w = 1.f / (float)W;
  int64_t row1 = t;
  if (a.ids) {
    row1 = a.ids[t];
    if (row1 >= a.V) row1 = -1;
  }
  float xv[NV][4], u[NV][4], g[NV][4], g2[NV][4];
  float s = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NTH * j);
#pragma unroll
    for (int i = 0; i < 4; ++i) xv[j][i] = u[j][i] = g[j][i] = g2[j][i] = 0.f;
    if (c < W) {
      if (!a.ids) ld4(xr + c, xv[j]);
      ld4(a.w + c, g[j]);
      if (a.next_w) ld4(a.next_w + c, g2[j]);
      ln_src4<TY>(a, t, row1, c, u[j]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) s += u[j][i];
  }
  const float mean = block_sum(s, red) * inv_w;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    if (4 * (threadIdx.x + NTH * j) < W) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        u[j][i] -= mean;
        ss += u[j][i] * u[j][i];
      }
    }
  }
  const float r = 1.f / sqrtf(block_sum(ss, red) * inv_w + a.eps);
  float sx = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NTH * j);
    if (c < W) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        xv[j][i] += u[j][i] * r * g[j][i];
        sx += xv[j][i];
      }
      st4(xr + c, xv[j]);
      if (a.out && !a.next_w) st4((TO*)a.out + (int64_t)t * W + c, xv[j]);
    }
  }
  if (!a.next_w) return;
  const float mx = block_sum(sx, red) * inv_w;
  float sxx = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    if (4 * (threadIdx.x + NTH * j) < W) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        xv[j][i] -= mx;
        sxx += xv[j][i] * xv[j][i];
      }
    }
  }
  const float rx = 1.f / sqrtf(block_sum(sxx, red) * inv_w + a.eps);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NTH * j);
    if (c < W) {
#pragma unroll
      for (int i = 0; i < 4; ++i) xv[j][i] *= rx * g2[j][i];
      st4((TO*)a.out + (int64_t)t * W + c, xv[j]);
    }
  }
}

template <typename TY, typename TO>
__global__ __launch_bounds__(256) void layer_norm_residual_kernel(const LnArgs a) {
  extern __shared__ float row[];   // [W], every thread touches only the columns it owns
  __shared__ float red[4];
  const int t = blockIdx.x, W = a.W;
  float* xr = a.x + (int64_t)t * W;
  const float inv_w = 1.f / (float)W;
  int64_t row1 = t;
  if (a.ids) {
    row1 = a.ids[t];
    if (row1 >= a.V) row1 = -1;
  }
  float s = 0.f;
  for (int c = threadIdx.x; c < W; c += 256) {
    const float u = ln_src1<TY>(a, t, row1, c);
    row[c] = u;
    s += u;
  }
  const float mean = block_sum(s, red) * inv_w;
  float ss = 0.f;
  for (int c = threadIdx.x; c < W; c += 256) ss += (row[c] - mean) * (row[c] - mean);
  const float r = 1.f / sqrtf(block_sum(ss, red) * inv_w + a.eps);
  float sx = 0.f;
  for (int c = threadIdx.x; c < W; c += 256) {
    const float v = (a.ids ? 0.f : xr[c]) + (row[c] - mean) * r * a.w[c];
    xr[c] = v;
    row[c] = v;
    sx += v;
    if (a.out && !a.next_w) stf((TO*)a.out + (int64_t)t * W + c, v);
  }
  if (!a.next_w) return;
  const float mx = block_sum(sx, red) * inv_w;
  float sxx = 0.f;
  for (int c = threadIdx.x; c < W; c += 256) sxx += (row[c] - mx) * (row[c] - mx);
  const float rx = 1.f / sqrtf(block_sum(sxx, red) * inv_w + a.eps);
  for (int c = threadIdx.x; c < W; c += 256) stf((TO*)a.out + (int64_t)t * W + c, (row[c] - mx) * rx * a.next_w[c]);
}

int layer_norm_residual(float* x, const void* y1, int64_t ld1, float s1, const void* y2, int64_t ld2, float s2, bool y_f32,
                        const int32_t* ids, int V, const float* y3, const int32_t* dest, const float* cw, int top,
                        const float* w, const float* next_w, float eps, void* out, bool out_f32, int T_, int W,
                        hipStream_t st) {
  if (T_ <= 0) return 0;
  if (W < 1 || W > 16000 || !w || (!y1) == (!y3) || (y2 && !y1) || (ids && (!y1 || y2 || V < 1)) || (dest && top < 1) ||
      (next_w && !out))
    return -1;
  const LnArgs a = {x, y1, y2, ld1, ld2, s1, s2, ids, V, y3, dest, cw, top, w, next_w, eps, out, W};
  const int ysz = y_f32 ? 4 : 2;
  const bool vec = (W & 3) == 0 && W <= 8192 && (!y1 || ((ld1 & 3) == 0 && (uintptr_t)y1 % (4 * ysz) == 0)) &&
                   (!y2 || ((ld2 & 3) == 0 && (uintptr_t)y2 % (4 * ysz) == 0));
#define XGM_LV(TY, TO, NV, NTH) layer_norm_residual_vec_kernel<TY, TO, NV, NTH><<<T_, NTH, 0, st>>>(a);
#define XGM_LN(TY, TO)                                                                                  \
  if (vec && W <= 1024) {                                                                               \
    XGM_LV(TY, TO, 1, 256)                                                                              \
  } else if (vec && W <= 2048) {                                                                        \
    XGM_LV(TY, TO, 2, 256)                                                                              \
  } else if (vec && W <= 4096) {                                                                        \
    XGM_LV(TY, TO, 2, 512)                                                                              \
  } else if (vec) {                                                                                     \
    XGM_LV(TY, TO, 4, 512)                                                                              \
  } else {                                                                                              \
    layer_norm_residual_kernel<TY, TO><<<T_, 256, (size_t)W * sizeof(float), st>>>(a);                  \
  }
  if (y_f32) {
    if (out_f32) { XGM_LN(float, float) } else { XGM_LN(float, bf16) }
  } else {
    if (out_f32) { XGM_LN(bf16, float) } else { XGM_LN(bf16, bf16) }
  }
#undef XGM_LN
#undef XGM_LV
  return 0;
}

}  // namespace xgm
