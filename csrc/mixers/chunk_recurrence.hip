// Outer-product recurrences over prompt portions on the matrix cores, bf16 activations and an fp32 state:
//
//   retention    S_t = a_h S_(t-1) + k_t v_t^T,          o_t = S_t^T q_t           (q, k rotated, k scaled)
//   time mixing  S_t = diag(w_t) S_(t-1) + k_t v_t^T,    o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,  w = exp(-exp(z + w0))
//
// followed by the head norm and the gate, out = o / rms(o) * weight * silu(g), when one workgroup holds the whole head
// (else o goes out as fp32).
//
// A portion is walked in chunks of 32 tokens. With L the running sum of log-decays inside a chunk and R its value after 16
// tokens, q' = q 2^(L_i - R) and k' = k 2^(R - L_j) (time mixing: L_(i-1) in q') make the chunk's weights one product,
//   P = mask(q' k'^T),   o = P v + q' (2^R S),   S <- 2^E S + 2^(E - R) k'^T v        (E = L after the chunk)
// so no decay is ever applied twice and the exponents stay within half a chunk of zero. fp32 accuracy on bf16 matrix
// cores: q', k', P and S enter as two bf16 terms each (value and rounding error; products of two error terms are left
// out), v is bf16 already. Time mixing decays by data: a chunk in which some channel decays by more than 2^-100 in one of
// its halves (the factors would leave the fp32 range) is run token by token in plain fp32 instead, chosen per workgroup.
//
// One workgroup = (sequence, head, 16 NW value columns), NW = 4 or 8 waves. A wave owns 16 columns of the state for all dk
// rows in accumulator layout; two 16-row accumulator tiles, converted in registers, are the operand of the next product (the
// contraction index runs (tile, row quad) on both sides). The score tiles are split over the waves and meet in LDS;
// k' and v are read transposed from LDS. The next chunk's global loads are in flight during the current chunk's products.
//
// Long portions of few sequences are cut into segments that run side by side: pass 1 sums every segment up from a zero
// state (and sets the incoming state aside), pass 2 folds the segments before its own and runs with outputs. Segment slot
// of (sequence s, segment z): q0_s / seg + s + z, distinct for all segments of a step.
#include "attention_common.h"

namespace xgm {

using xgk::as_frag;
using xgk::bf16x4_t;
using xgk::bf16x8_t;
using xgk::f32x4_t;
using xgk::ld16;
using xgk::lds_read_tr16;
using xgk::mfma16x16x32;
using xgk::pack2;
using xgk::unpack8;

constexpr int kRetention = 0, kTimeMix = 1;
constexpr int kChunkTok = 32;
constexpr float kMaxHalfDecay = 100.f;   // log2 of the largest decay over half a chunk that the scaled form takes

struct ChunkArgs {
  const bf16 *q, *k, *v, *g, *z;
  int64_t ld_q, ld_k, ld_v, ld_g, ld_z;
  const float *decay, *w0, *bonus, *rot;
  int rot_rows, rot_dims;
  float k_scale;
  const float* norm_w;
  float eps;
  float* state;
  const int32_t *qsl, *seq_lens, *slots;
  bf16* out;     // normed and gated rows [T][H dv], or
  float* o32;    // o itself
  int H, dv;
  int pass, nc, seg;
  float *chA, *chB, *s_in;
};

// value and rounding error of four floats as packed bf16 pairs
__device__ __forceinline__ void split4(const float (&f)[4], uint2& hi, uint2& lo) {
  hi = make_uint2(pack2(f[0], f[1]), pack2(f[2], f[3]));
  lo = make_uint2(pack2(f[0] - __uint_as_float(hi.x << 16), f[1] - __uint_as_float(hi.x & 0xFFFF0000u)),
                  pack2(f[2] - __uint_as_float(hi.y << 16), f[3] - __uint_as_float(hi.y & 0xFFFF0000u)));
}

__device__ __forceinline__ bf16x8_t frag2(uint2 a, uint2 b) { return as_frag(make_uint4(a.x, a.y, b.x, b.y)); }

__device__ __forceinline__ bf16x8_t tr_frag(const bf16* p, int row16) {   // rows .. + 3 and row16 elements further on
  const bf16x4_t a = lds_read_tr16(p), b = lds_read_tr16(p + row16);
  return bf16x8_t{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// waves per SIMD that the registers must allow
constexpr int chunk_occ(int mode, int dk) { return dk > 128 ? 2 : mode == kTimeMix ? (dk > 64 ? 2 : 3) : 4; }

__device__ __forceinline__ void sched_fence() {
#if defined(__HIP_DEVICE_COMPILE__)
  __builtin_amdgcn_sched_barrier(0);
#endif
}

// the same value, unknown to the compiler: lane offsets derived from it are formed where they are used instead of being
// kept (and spilled: a reload would wait for every load in flight) across the chunk loop
__device__ __forceinline__ int opaque(int x) {
  asm volatile("" : "+v"(x));
  return x;
}

template <int MODE, int DK, int NW>
__global__ __launch_bounds__(64 * NW, chunk_occ(MODE, DK)) void chunk_recurrence_kernel(const ChunkArgs a) {
  constexpr int C = kChunkTok, MT = DK / 16, KK = DK / 32, COLS = 16 * NW, NTH = 64 * NW;
  constexpr int QE = DK + 8, VE = COLS + 8, PE = C + 8;    // LDS row strides (elements)
  constexpr bool TM = MODE == kTimeMix;
  __shared__ __attribute__((aligned(16))) bf16 qs[2][C * QE], ks[2][C * QE], vs[C * VE], ps[2][C * PE];
  __shared__ __attribute__((aligned(16))) float wraw[TM ? C * DK : 4];    // decays of a chunk that is run token by token
  // row factors of the state: 2^R, 2^E, 2^(E - R); time mixing only. gsum: log-decays per token group
  constexpr int CP = DK / 2, TGN = NTH / CP, TT = C / TGN;   // channel pairs, token groups, tokens per thread
  __shared__ __attribute__((aligned(16))) float rowf[3][TM ? DK : 4], gsum[TM ? TGN * DK : 4], ltot[TM ? DK : 4];
  __shared__ float diag[2][C], rsum[NW][C];

  const int s = blockIdx.x / a.nc, z = blockIdx.x % a.nc, h = blockIdx.y;
  const int q0 = a.qsl[s], qn = a.qsl[s + 1] - q0, slot = a.slots[s];
  const int c0 = z * a.seg, c1 = min(qn, c0 + a.seg);
  if (slot < 0 || c0 >= qn) return;
  const int pass = a.pass;
  const int ctx = a.seq_lens[s] - qn;
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g4 = lane >> 4, l16 = lane & 15;
  const int dv = a.dv, p0 = blockIdx.z * COLS;
  float* Sg = a.state + (((int64_t)slot * a.H + h) * DK) * dv;
  const int64_t cs0 = q0 / a.seg + s;
  const float la = TM ? 0.f : log2f(a.decay[h]);
  const bool last_seg = c1 == qn;

  // ---- incoming state: rows 16 m + 4 g4 + r, column col
  const int col = p0 + 16 * w + l16;
  float S[MT][4];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) S[m][r] = 0.f;
  // element (m, r) of a [DK][dv] block: uniform row pointer + one lane offset
  const uint32_t lofs = (uint32_t)(4 * g4) * dv + col;
  const bool cok = col < dv;
  float* s_in = a.s_in + ((int64_t)s * a.H + h) * DK * dv;
  const float* first = pass == 2 ? s_in : Sg;
  if (cok && (pass == 2 || ctx > 0)) {
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[m][r] = (first + (int64_t)(16 * m + r) * dv)[lofs];
  }
  if (pass == 1) {   // segments are summed up from zero; the incoming state is set aside
    if (z == 0 && cok) {
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) (s_in + (int64_t)(16 * m + r) * dv)[lofs] = S[m][r];
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[m][r] = 0.f;
  }
  if (pass == 1 && last_seg) return;   // nobody reads its sum
  if (pass == 2) {
    for (int zc = 0; zc < z; ++zc) {
      const float fa = TM ? 0.f : exp2f(la * (float)a.seg);
      const int64_t cr = ((cs0 + zc) * a.H + h) * DK;
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        float f[4] = {fa, fa, fa, fa};
        if constexpr (TM) ld4(a.chA + cr + 16 * m + 4 * g4, f);
        if (cok) {
#pragma unroll
          for (int r = 0; r < 4; ++r) S[m][r] = f[r] * S[m][r] + (a.chB + (cr + 16 * m + r) * dv)[lofs];
        }
      }
    }
  }
  for (int i = tid; i < C * PE; i += NTH) ps[0][i] = ps[1][i] = 0;   // (the tile above the diagonal stays zero)
  if (TM)
    for (int i = tid; i < DK; i += NTH) ltot[i] = 0.f;

  // ---- global loads of a chunk, one chunk ahead of their use
  // retention: a unit is (q or k, token, 8 + 8 channels)
  constexpr int UNITS = C * DK / 16, UPT = (2 * UNITS + NTH - 1) / NTH;
  constexpr int TT2 = TM ? TT : 1, UP2 = TM ? 1 : UPT;
  uint4 fx[UP2][2], fv;
  float4 fc[UP2][4];                    // (cos, sin) of 8 channel pairs
  uint32_t mr[TT2], mk[TT2], mz[TT2];   // time mixing: a channel pair of TT tokens
  uint2 gt2[2];                         // gate of the current chunk: tokens 16 it + l16, columns 16 w + 4 g4 .. + 3
  const int half = a.rot_dims / 2;
  auto unit_ch = [&](int u, bool& is_k, int& tok, int& ca, int& cb, bool& turned) {
    is_k = u >= UNITS;
    u -= is_k ? UNITS : 0;
    tok = u / (DK / 16);
    const int p = u % (DK / 16);
    turned = 8 * p < half;
    ca = turned ? 8 * p : a.rot_dims + 16 * (p - half / 8);
    cb = turned ? half + 8 * p : ca + 8;
  };
  auto fetch = [&](int t0) {
    const int n = min(C, c1 - t0), tid = opaque(threadIdx.x);
    const int64_t row0 = q0 + t0;   // uniform bases, 32-bit lane offsets
    const bf16 *qb = a.q + row0 * a.ld_q + h * DK, *kb = a.k + row0 * a.ld_k + h * DK;
    const bf16 *zb = TM ? a.z + row0 * a.ld_z + h * DK : nullptr;
    if constexpr (!TM) {
#pragma unroll
      for (int j = 0; j < UPT; ++j) {
        const int u = tid + NTH * j;
        int tok, ca, cb;
        bool turned, is_k;
        unit_ch(u, is_k, tok, ca, cb, turned);
        fx[j][0] = fx[j][1] = make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 4; ++i) fc[j][i] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (u < 2 * UNITS && tok < n && (is_k || pass != 1)) {
          if (is_k) {
            const uint32_t o = (uint32_t)tok * (uint32_t)a.ld_k;
            fx[j][0] = ld16(kb + (o + ca)), fx[j][1] = ld16(kb + (o + cb));
          } else {
            const uint32_t o = (uint32_t)tok * (uint32_t)a.ld_q;
            fx[j][0] = ld16(qb + (o + ca)), fx[j][1] = ld16(qb + (o + cb));
          }
          if (turned) {
            const uint32_t o = ((uint32_t)min(ctx + t0 + tok, a.rot_rows - 1) * half + ca) * 2;
#pragma unroll
            for (int i = 0; i < 4; ++i) fc[j][i] = *reinterpret_cast<const float4*>(a.rot + (o + 4 * i));
          }
        }
      }
    } else {
      const int d = 2 * (tid % CP), tg = tid / CP;
#pragma unroll
      for (int i = 0; i < TT; ++i) {
        const int tok = tg * TT + i;
        mr[i] = mk[i] = mz[i] = 0;
        if (tok < n) {
          mr[i] = *reinterpret_cast<const uint32_t*>(qb + ((uint32_t)tok * (uint32_t)a.ld_q + d));
          mk[i] = *reinterpret_cast<const uint32_t*>(kb + ((uint32_t)tok * (uint32_t)a.ld_k + d));
          mz[i] = *reinterpret_cast<const uint32_t*>(zb + ((uint32_t)tok * (uint32_t)a.ld_z + d));
        }
      }
    }
    {   // (32 tokens x 2 NW chunks of 8 columns: one per thread)
      const int tok = tid / (2 * NW), c = p0 + 8 * (tid % (2 * NW));
      fv = make_uint4(0, 0, 0, 0);
      if (tok < n && c < dv) fv = ld16(a.v + row0 * a.ld_v + h * dv + ((uint32_t)tok * (uint32_t)a.ld_v + c));
    }
  };
  auto fetch_gate = [&](int t0, int n) {
    if (pass == 1 || !a.out) return;
    const int lane = opaque(threadIdx.x) & 63, g4 = lane >> 4, l16 = lane & 15;
    const bf16* gb = a.g + (int64_t)(q0 + t0) * a.ld_g + h * dv;
    const int c = 16 * w + 4 * g4;
#pragma unroll
    for (int it = 0; it < 2; ++it) {
      const int tok = 16 * it + l16;
      gt2[it] = make_uint2(0, 0);
      if (tok < n && c < dv) gt2[it] = *reinterpret_cast<const uint2*>(gb + ((uint32_t)tok * (uint32_t)a.ld_g + c));
    }
  };

  // ---- a chunk's operands into LDS; true: the chunk must run token by token
  auto put8 = [&](bf16* hi, bf16* lo, const float (&f)[8]) {
    uint2 h0, l0, h1, l1;
    const float f0[4] = {f[0], f[1], f[2], f[3]}, f1[4] = {f[4], f[5], f[6], f[7]};
    split4(f0, h0, l0);
    split4(f1, h1, l1);
    *reinterpret_cast<uint4*>(hi) = make_uint4(h0.x, h0.y, h1.x, h1.y);
    *reinterpret_cast<uint4*>(lo) = make_uint4(l0.x, l0.y, l1.x, l1.y);
  };
  auto stage = [&](int n) -> bool {
    const int tid = opaque(threadIdx.x), lane = tid & 63;
    *reinterpret_cast<uint4*>(vs + (tid / (2 * NW)) * VE + 8 * (tid % (2 * NW))) = fv;
    if constexpr (!TM) {
#pragma unroll
      for (int j = 0; j < UPT; ++j) {
        const int u = tid + NTH * j;
        int tok, ca, cb;
        bool turned, is_k;
        unit_ch(u, is_k, tok, ca, cb, turned);
        if (u >= 2 * UNITS || (pass == 1 && !is_k)) continue;
        const float f = exp2_fast(la * (float)(is_k ? 15 - tok : tok - 15)) * (is_k ? a.k_scale : 1.f);
        float x[8], y[8], xo[8], yo[8];
        unpack8(fx[j][0], x);
        unpack8(fx[j][1], y);
        if (turned) {
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const float4 c4 = fc[j][i / 2];
            const float cs = ((i & 1) ? c4.z : c4.x) * f, sn = ((i & 1) ? c4.w : c4.y) * f;
            xo[i] = x[i] * cs - y[i] * sn;
            yo[i] = y[i] * cs + x[i] * sn;
          }
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i) xo[i] = x[i] * f, yo[i] = y[i] * f;
        }
        bf16* hi = is_k ? ks[0] : qs[0];
        bf16* lo = is_k ? ks[1] : qs[1];
        put8(hi + tok * QE + ca, lo + tok * QE + ca, xo);
        put8(hi + tok * QE + cb, lo + tok * QE + cb, yo);
      }
      return false;
    } else {
      const int d = 2 * (tid % CP), tg = tid / CP;
      float lw[TT][2], run[2] = {0.f, 0.f};
      const float b0 = a.w0[h * DK + d], b1 = a.w0[h * DK + d + 1];
      const float u0 = a.bonus[h * DK + d], u1 = a.bonus[h * DK + d + 1];
#pragma unroll
      for (int i = 0; i < TT; ++i) {
        const bool on = tg * TT + i < n;
        run[0] -= on ? exp2_fast((__uint_as_float(mz[i] << 16) + b0) * kLog2e) * kLog2e : 0.f;
        run[1] -= on ? exp2_fast((__uint_as_float(mz[i] & 0xFFFF0000u) + b1) * kLog2e) * kLog2e : 0.f;
        lw[i][0] = run[0], lw[i][1] = run[1];
        if (pass != 1) {   // the current token's own weight, sum_d r u k
          float b = __uint_as_float(mr[i] << 16) * u0 * __uint_as_float(mk[i] << 16) +
                    __uint_as_float(mr[i] & 0xFFFF0000u) * u1 * __uint_as_float(mk[i] & 0xFFFF0000u);
#pragma unroll
          for (int o = 1; o < (CP < 64 ? CP : 64); o <<= 1) b += __shfl_xor(b, o, 64);
          if (CP >= 64 ? lane == 0 : lane % CP == 0) diag[CP > 64 ? (tid % CP) / 64 : 0][tg * TT + i] = b;
        }
      }
      *reinterpret_cast<float2*>(gsum + tg * DK + d) = make_float2(run[0], run[1]);
      __syncthreads();
      float off[2] = {0.f, 0.f}, R[2] = {0.f, 0.f}, E[2] = {0.f, 0.f};
#pragma unroll
      for (int gg = 0; gg < TGN; ++gg) {
        const float2 v = *reinterpret_cast<const float2*>(gsum + gg * DK + d);
        if (gg < tg) off[0] += v.x, off[1] += v.y;
        if (gg < TGN / 2) R[0] += v.x, R[1] += v.y;
        E[0] += v.x, E[1] += v.y;
      }
      const bool bad = R[0] < -kMaxHalfDecay || R[1] < -kMaxHalfDecay || E[0] - R[0] < -kMaxHalfDecay ||
                       E[1] - R[1] < -kMaxHalfDecay;
      const bool slow = __syncthreads_or(bad);
      if (slow) {
        float* rf = reinterpret_cast<float*>(qs[0]);   // [C][DK] fp32, over both terms' rows
        float* kf = reinterpret_cast<float*>(ks[0]);
#pragma unroll
        for (int i = 0; i < TT; ++i) {
          const int at = (tg * TT + i) * DK + d;
          *reinterpret_cast<float2*>(rf + at) = make_float2(__uint_as_float(mr[i] << 16), __uint_as_float(mr[i] & 0xFFFF0000u));
          *reinterpret_cast<float2*>(kf + at) = make_float2(__uint_as_float(mk[i] << 16), __uint_as_float(mk[i] & 0xFFFF0000u));
          const float2 lp = i ? make_float2(lw[i - 1][0], lw[i - 1][1]) : make_float2(0.f, 0.f);
          *reinterpret_cast<float2*>(wraw + at) = make_float2(exp2f(lw[i][0] - lp.x), exp2f(lw[i][1] - lp.y));
        }
        if (tg == 0) ltot[d] += E[0], ltot[d + 1] += E[1];
        return true;
      }
      if (tg == 0) {
        rowf[0][d] = exp2f(R[0]), rowf[0][d + 1] = exp2f(R[1]);
        rowf[1][d] = exp2f(E[0]), rowf[1][d + 1] = exp2f(E[1]);
        rowf[2][d] = exp2f(E[0] - R[0]), rowf[2][d + 1] = exp2f(E[1] - R[1]);
        ltot[d] += E[0], ltot[d + 1] += E[1];
      }
#pragma unroll
      for (int i = 0; i < TT; ++i) {
        const int at = (tg * TT + i) * QE + d;
        if (pass != 1) {
          const float x0 = (i ? lw[i - 1][0] : 0.f) + off[0] - R[0], x1 = (i ? lw[i - 1][1] : 0.f) + off[1] - R[1];
          const float r0 = __uint_as_float(mr[i] << 16) * exp2_fast(x0), r1 = __uint_as_float(mr[i] & 0xFFFF0000u) * exp2_fast(x1);
          const uint32_t hi = pack2(r0, r1);
          *reinterpret_cast<uint32_t*>(qs[0] + at) = hi;
          *reinterpret_cast<uint32_t*>(qs[1] + at) = pack2(r0 - __uint_as_float(hi << 16), r1 - __uint_as_float(hi & 0xFFFF0000u));
        }
        const float k0 = __uint_as_float(mk[i] << 16) * exp2_fast(R[0] - lw[i][0] - off[0]);
        const float k1 = __uint_as_float(mk[i] & 0xFFFF0000u) * exp2_fast(R[1] - lw[i][1] - off[1]);
        const uint32_t hi = pack2(k0, k1);
        *reinterpret_cast<uint32_t*>(ks[0] + at) = hi;
        *reinterpret_cast<uint32_t*>(ks[1] + at) = pack2(k0 - __uint_as_float(hi << 16), k1 - __uint_as_float(hi & 0xFFFF0000u));
      }
      return false;
    }
  };

  // fragment of rows (token base + l16), contraction slots (g4, 0..3) = channels 32 kk + 4 g4 .., (g4, 4..7) = 16 further
  auto rowfrag = [&](const bf16* x, int base, int kk, int rl) {   // rl = l16 QE + 4 g4
    const bf16* p = x + base * QE + 32 * kk + rl;
    return frag2(*reinterpret_cast<const uint2*>(p), *reinterpret_cast<const uint2*>(p + 16));
  };

  float nw[4] = {1.f, 1.f, 1.f, 1.f};
  if (TM && a.norm_w && a.out && 16 * w + 4 * g4 < dv) ld4(a.norm_w + h * dv + 16 * w + 4 * g4, nw);
  const float inv_dv = 1.f / (float)dv;
  fetch(c0);
  for (int t0 = c0; t0 < c1; t0 += C) {
    const int n = min(C, c1 - t0);
    __syncthreads();   // (the previous chunk's LDS reads are done)
    const bool slow = stage(n);
    fetch_gate(t0, n);   // (before the next chunk's loads: they stay in flight when the gate is waited for)
    if (t0 + C < c1) fetch(t0 + C);
    __syncthreads();
    // o^T: columns 16 w + 4 g4 + r, token 16 it + l16
    f32x4_t oacc[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
    if (TM && slow) {
      const float* rf = reinterpret_cast<const float*>(qs[0]);
      const float* kf = reinterpret_cast<const float*>(ks[0]);
      for (int t = 0; t < n; ++t) {
        const float vv = bf2f(vs[t * VE + 16 * w + l16]);
        float acc = 0.f;
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          float rr[4], kr[4], wr[4];
          ld4(rf + t * DK + 16 * m + 4 * g4, rr);
          ld4(kf + t * DK + 16 * m + 4 * g4, kr);
          ld4(wraw + t * DK + 16 * m + 4 * g4, wr);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            acc = fmaf(S[m][r], rr[r], acc);
            S[m][r] = fmaf(wr[r], S[m][r], kr[r] * vv);
          }
        }
        if (pass == 1) continue;
        acc += __shfl_xor(acc, 16, 64);
        acc += __shfl_xor(acc, 32, 64);
        acc = fmaf(CP > 64 ? diag[0][t] + diag[1][t] : diag[0][t], vv, acc);
        // lane (g4, l16) of the output layout wants columns 4 g4 .. + 3 of token t
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float o = __shfl(acc, 4 * g4 + r, 64);
          if (l16 == (t & 15)) {
            if (t < 16) oacc[0][r] = o;
            else oacc[1][r] = o;
          }
        }
      }
    } else {
      if (pass != 1) {
        if (w < 3) {   // score tiles (token tile, key tile): (0, 0), (1, 0), (1, 1)
          const int it = w > 0, jt = w > 1;
          f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
          const int lane = opaque(threadIdx.x) & 63, g4 = lane >> 4, l16 = lane & 15, rl = l16 * QE + 4 * g4;
#pragma unroll
          for (int kk = 0; kk < KK; ++kk) {
            const bf16x8_t qh = rowfrag(qs[0], 16 * it, kk, rl), ql = rowfrag(qs[1], 16 * it, kk, rl);
            const bf16x8_t kh = rowfrag(ks[0], 16 * jt, kk, rl), kl = rowfrag(ks[1], 16 * jt, kk, rl);
            acc = mfma16x16x32(kh, qh, acc);
            acc = mfma16x16x32(kh, ql, acc);
            acc = mfma16x16x32(kl, qh, acc);
          }
          const int i = 16 * it + l16;
          float p[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = 16 * jt + 4 * g4 + r;
            if constexpr (TM) p[r] = j < i ? acc[r] : j == i ? (CP > 64 ? diag[0][i] + diag[1][i] : diag[0][i]) : 0.f;
            else p[r] = j <= i ? acc[r] : 0.f;
          }
          uint2 hi, lo;
          split4(p, hi, lo);
          *reinterpret_cast<uint2*>(ps[0] + i * PE + 16 * jt + 4 * g4) = hi;
          *reinterpret_cast<uint2*>(ps[1] + i * PE + 16 * jt + 4 * g4) = lo;
        }
        // o = q' (2^R S)
        const float sr = TM ? 0.f : exp2_fast(la * 16.f);
        const int lane = opaque(threadIdx.x) & 63, g4 = lane >> 4, rl = (lane & 15) * QE + 4 * g4;
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
          float f0[4], f1[4];
          if constexpr (TM) {
            ld4(rowf[0] + 32 * kk + 4 * g4, f0);
            ld4(rowf[0] + 32 * kk + 16 + 4 * g4, f1);
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) f0[r] = f1[r] = sr;
          }
          const bf16x8_t qh0 = rowfrag(qs[0], 0, kk, rl), ql0 = rowfrag(qs[1], 0, kk, rl);
          const bf16x8_t qh1 = rowfrag(qs[0], 16, kk, rl), ql1 = rowfrag(qs[1], 16, kk, rl);
          float e0[4], e1[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) e0[r] = S[2 * kk][r] * f0[r], e1[r] = S[2 * kk + 1][r] * f1[r];
          uint2 h0, l0, h1, l1;
          split4(e0, h0, l0);
          split4(e1, h1, l1);
          const bf16x8_t sh = frag2(h0, h1), sl = frag2(l0, l1);
          oacc[0] = mfma16x16x32(sh, qh0, oacc[0]);
          oacc[1] = mfma16x16x32(sh, qh1, oacc[1]);
          oacc[0] = mfma16x16x32(sh, ql0, oacc[0]);
          oacc[1] = mfma16x16x32(sh, ql1, oacc[1]);
          oacc[0] = mfma16x16x32(sl, qh0, oacc[0]);
          oacc[1] = mfma16x16x32(sl, qh1, oacc[1]);
          sched_fence();   // bounds the fragment reads in flight (registers)
        }
        __syncthreads();
      }
      // tokens (g4, 0..3) = 4 g4 .., (g4, 4..7) = 16 further, on both sides
      const int lane = opaque(threadIdx.x) & 63, g4 = lane >> 4, l16 = lane & 15, tq = l16 >> 2, tp = l16 & 3;
      const bf16x8_t vf = tr_frag(vs + (4 * g4 + tq) * VE + 16 * w + 4 * tp, 16 * VE);
      if (pass != 1) {
#pragma unroll
        for (int it = 0; it < 2; ++it)
#pragma unroll
          for (int e = 0; e < 2; ++e) {
            const bf16* p = ps[e] + (16 * it + l16) * PE + 4 * g4;
            const bf16x8_t pf = frag2(*reinterpret_cast<const uint2*>(p), *reinterpret_cast<const uint2*>(p + 16));
            oacc[it] = mfma16x16x32(vf, pf, oacc[it]);
          }
      }
      const float fe = TM ? 0.f : exp2_fast(la * (float)n), fr = TM ? 0.f : exp2_fast(la * (float)(n - 16));
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        float f1[4], f2[4];
        if constexpr (TM) {
          ld4(rowf[1] + 16 * m + 4 * g4, f1);
          ld4(rowf[2] + 16 * m + 4 * g4, f2);
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r) f1[r] = fe, f2[r] = fr;
        }
        const int at = (4 * g4 + tq) * QE + 16 * m + 4 * tp;
        const bf16x8_t kh = tr_frag(ks[0] + at, 16 * QE), kl = tr_frag(ks[1] + at, 16 * QE);
        f32x4_t u = {0.f, 0.f, 0.f, 0.f};
        u = mfma16x16x32(kh, vf, u);
        u = mfma16x16x32(kl, vf, u);
#pragma unroll
        for (int r = 0; r < 4; ++r) S[m][r] = fmaf(f1[r], S[m][r], f2[r] * u[r]);
        sched_fence();
      }
    }
    if (pass == 1) continue;
    const int lane = opaque(threadIdx.x) & 63, g4 = lane >> 4, l16 = lane & 15, c = 16 * w + 4 * g4;
    if (a.o32) {
#pragma unroll
      for (int it = 0; it < 2; ++it) {
        const int tok = 16 * it + l16;
        const float y[4] = {oacc[it][0], oacc[it][1], oacc[it][2], oacc[it][3]};
        if (tok < n && p0 + c < dv) st4(a.o32 + ((int64_t)(q0 + t0) * a.H + h) * dv + ((uint32_t)(tok * a.H) * dv + p0 + c), y);
      }
      continue;
    }
    // head norm, gate (columns past dv hold zeros)
#pragma unroll
    for (int it = 0; it < 2; ++it) {
      float ss = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) ss = fmaf(oacc[it][r], oacc[it][r], ss);
      ss += __shfl_xor(ss, 16, 64);
      ss += __shfl_xor(ss, 32, 64);
      if (g4 == 0) rsum[w][16 * it + l16] = ss;
    }
    __syncthreads();
#pragma unroll
    for (int it = 0; it < 2; ++it) {
      const int tok = 16 * it + l16;
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NW; ++i) ss += rsum[i][tok];
      const float inv = 1.f / sqrtf(ss * inv_dv + a.eps);
      if (tok < n && c < dv) {
        const float gt[4] = {__uint_as_float(gt2[it].x << 16), __uint_as_float(gt2[it].x & 0xFFFF0000u),
                             __uint_as_float(gt2[it].y << 16), __uint_as_float(gt2[it].y & 0xFFFF0000u)};
        float y[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] = oacc[it][r] * inv * nw[r] * gt[r] * rcp_fast(1.f + exp2_fast(-kLog2e * gt[r]));
        st4(a.out + ((int64_t)(q0 + t0) * a.H + h) * dv + ((uint32_t)(tok * a.H) * dv + c), y);
      }
    }
  }
  // ---- outgoing state, or the segment's sum
  if (pass == 1) __syncthreads();   // (ltot)
  float* last = pass == 1 ? a.chB + ((cs0 + z) * a.H + h) * DK * (int64_t)dv : Sg;
  if (cok && (pass == 1 || last_seg)) {
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) (last + (int64_t)(16 * m + r) * dv)[lofs] = S[m][r];
  }
  if (TM && pass == 1 && blockIdx.z == 0)
    for (int i = tid; i < DK; i += NTH) a.chA[((cs0 + z) * a.H + h) * DK + i] = exp2f(ltot[i]);
}

int64_t chunk_recurrence_scratch_floats(int T_, int ns, int H, int dk, int dv, int seg) {
  const int64_t cslots = T_ / seg + ns + 1;
  return (cslots * (dv + 1) + (int64_t)ns * dv) * H * dk;
}

// bf16 rows; nc > 1: scratch of chunk_recurrence_scratch_floats, segments of `seg` tokens (a multiple of 32)
int chunk_recurrence(const void* q, int64_t ld_q, const void* k, int64_t ld_k, const void* v, int64_t ld_v, const void* g,
                     int64_t ld_g, const void* z, int64_t ld_z, const float* decay, const float* w0, const float* bonus,
                     const float* rot, int rot_rows, int rot_dims, float k_scale, const float* norm_w, float eps,
                     float* state, const int32_t* qsl, const int32_t* seq_lens, const int32_t* slots, void* out, float* o32,
                     int ns, int max_q, int T_, int H, int dk, int dv, int seg, float* scratch, hipStream_t st) {
  if (ns <= 0 || max_q <= 0) return 0;
  const int nw = dv <= 64 ? 4 : 8, cols = 16 * nw, nz = (dv + cols - 1) / cols;
  auto al = [](const void* p, int64_t ld, int n) { return (uintptr_t)p % (2 * n) == 0 && ld % n == 0; };
  if (H < 1 || dv < 8 || dv % 8 || !al(v, ld_v, 8) || (out && (!g || !al(g, ld_g, 4) || nz > 1)) || (!out) == (!o32)) return -1;
  if (!decay && (dv != dk || dk == 96)) return -1;
  if (decay ? (!al(q, ld_q, 8) || !al(k, ld_k, 8) || rot_dims % 16 || rot_dims > dk || (rot_dims && (!rot || rot_rows < 1)))
            : (!z || !w0 || !bonus || !al(q, ld_q, 2) || !al(k, ld_k, 2) || !al(z, ld_z, 2)))
    return -1;
  if (scratch ? (seg < kChunkTok || seg % kChunkTok) : false) return -1;
  if (!scratch) seg = (max_q + kChunkTok - 1) / kChunkTok * kChunkTok;
  const int nc = (max_q + seg - 1) / seg;
  const int64_t cslots = T_ / seg + ns + 1;
  ChunkArgs a = {(const bf16*)q, (const bf16*)k, (const bf16*)v, (const bf16*)g, (const bf16*)z, ld_q, ld_k, ld_v, ld_g, ld_z,
                 decay, w0, bonus, rot, rot_rows, rot_dims, k_scale, norm_w, eps, state, qsl, seq_lens, slots, (bf16*)out,
                 o32, H, dv, 0, nc, seg, scratch, scratch ? scratch + cslots * H * dk : nullptr,
                 scratch ? scratch + cslots * H * dk * (1 + dv) : nullptr};
  dim3 grid(ns * nc, H, nz);
#define XGM_CR3(MODE, DK, NW)                                          \
  if (nc > 1) {                                                        \
    a.pass = 1;                                                        \
    chunk_recurrence_kernel<MODE, DK, NW><<<grid, 64 * NW, 0, st>>>(a); \
    a.pass = 2;                                                        \
    chunk_recurrence_kernel<MODE, DK, NW><<<grid, 64 * NW, 0, st>>>(a); \
  } else {                                                             \
    chunk_recurrence_kernel<MODE, DK, NW><<<grid, 64 * NW, 0, st>>>(a); \
  }                                                                    \
  return 0;
#define XGM_CR(DK, NWT)              /* (time mixing: dv = dk, NWT waves) */ \
  if (!decay) {                                                      \
    XGM_CR3(kTimeMix, DK, NWT)                                       \
  } else if (nw == 4) {                                              \
    XGM_CR3(kRetention, DK, 4)                                       \
  }                                                                  \
  XGM_CR3(kRetention, DK, 8)
  switch (dk) {
    case 32: XGM_CR(32, 4)
    case 64: XGM_CR(64, 4)
    case 128: XGM_CR(128, 8)
    case 256: XGM_CR(256, 8)
    case 96:
      if (nw == 4) { XGM_CR3(kRetention, 96, 4) }
      XGM_CR3(kRetention, 96, 8)
    default: return -1;
  }
#undef XGM_CR
#undef XGM_CR3
}

}  // namespace xgm
