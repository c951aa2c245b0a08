// Constants and small helpers of the grouped-query attention kernels (chunk_attention.hip, single_attention.hip).
#pragma once

#include "mixers_common.h"

namespace xgm {

constexpr int kMaskCausal = 0, kMaskWindow = 1, kMaskChunk = 2;
constexpr int kValuesOwn = -1, kValuesAll = -2;
constexpr int kWeightsSoftmax = 0, kWeightsSigmoid = 1;
// matrix-core forms of the bounded softmax: kWeightsBounded needs no running maximum (|score| <= softcap, so every
// exponential and every sum of them stays in range without a reference), kWeightsCapped keeps one (large bounds, sinks)
constexpr int kWeightsBounded = 2, kWeightsCapped = 3;
constexpr float kBoundedMaxLog2 = 90.f;   // largest bound in units of ln 2: 2^90 x 2^20 keys x values stays far from 2^127
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ int first_visible(int mask, int size, int pos) {
  if (mask == kMaskWindow) return max(0, pos - size + 1);
  if (mask == kMaskChunk) return (pos / size) * size;
  return 0;
}

__device__ __forceinline__ float exp2_fast(float x) {
#if defined(__HIP_DEVICE_COMPILE__)
  return __builtin_amdgcn_exp2f(x);
#else
  return exp2f(x);
#endif
}

__device__ __forceinline__ float rcp_fast(float x) {
#if defined(__HIP_DEVICE_COMPILE__)
  return __builtin_amdgcn_rcpf(x);
#else
  return 1.f / x;
#endif
}

// arguments of one attention launch (see the comment of chunk_attention.hip)
struct AttnArgs {
  const bf16 *q, *kcache, *vcache;
  const int32_t* block_tables;
  int bt_width, bs;
  const int32_t *qsl, *seq_lens, *slots;
  const float *temp, *sink;
  bf16* out;
  int T, ns, H, G, dk, dv_head, mask, size;
  float scale;
  const bf16* gate;
  int64_t ld_gate;
  const float *r1, *r2;
  int vmode, gate_elem;
  const float* hbias;
  float softcap;
  int keep;
};

constexpr int kSingleMaxRep = 16;   // query heads per key / value head the single-token kernel takes

// single_attention.hip: steps of single tokens (dk <= 128, dv <= 128 value columns, H / G <= kSingleMaxRep). nsplit > 1:
// unnormalised shares go to part_o / part_ml. Returns false when the sizes are not served.
bool single_attention(const AttnArgs& a, int wfn, int nsplit, float* part_o, float* part_ml, hipStream_t st);

// prompt_attention.hip: portions of more than kPromptMinRows rows (dk and dv 64 or 128, block sizes a multiple of 16).
// Returns false when the sizes are not served.
constexpr int kPromptMinRows = 32;
bool prompt_attention(const AttnArgs& a, int max_q, int wfn, hipStream_t st);

}  // namespace xgm
