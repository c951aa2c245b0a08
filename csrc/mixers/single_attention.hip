// Attention of a step of single tokens (one query per sequence) on the matrix cores, bf16.
//
// One workgroup = one sequence x one key/value head (x one share of its keys): the head group's queries (<= 16) are the
// columns of the 16 x 16 x 32 products. Every wave walks 32-key tiles of its own (w, w + NW, ..): K rows go straight from
// global memory into the A fragments of S^T = K Q^T, V rows through a piece of LDS that belongs to the wave alone
// (the A operand of O^T += V^T P^T is a transposed LDS read), so no barrier stands between two tiles and every wave's
// loads run ahead on their own; the next tile's rows are loaded while this one's weights are formed, and its cache rows
// are looked up one tile earlier still. The waves' sums meet once, at the end.
//
// Visibility, scores, weights, gates: as described in chunk_attention.hip (keys are numbered without the gap between kept
// first keys and the window).
#include "attention_common.h"

#include <algorithm>

namespace xgm {

constexpr int kST = 32;   // keys per wave tile

template <int NKK, int NMT, int NW, int WFN>
__global__ __launch_bounds__(64 * NW) void single_attention_kernel(const AttnArgs a, int nsplit, float* __restrict__ part_o,
                                                               float* __restrict__ part_ml) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  constexpr bool sig = WFN == kWeightsSigmoid, capped = WFN == kWeightsBounded || WFN == kWeightsCapped;
  constexpr bool bounded = WFN == kWeightsBounded;
  constexpr int CPR = 2 * NMT;             // 16-byte chunks of a value row (guarded by dv)
  // block b runs on XCD b % 8: an XCD takes a contiguous run of (sequence, share, head group) with the head groups
  // fastest, so the groups' neighbouring pieces of one cache row are read through one L2 (and all of its channels)
  const int nb = gridDim.x, q8 = nb >> 3, r8 = nb & 7, xcd = blockIdx.x & 7;
  const int v = (xcd < r8 ? xcd * (q8 + 1) : r8 * (q8 + 1) + (xcd - r8) * q8) + (blockIdx.x >> 3);
  const int g = v % a.G, share = v / a.G % nsplit, s = v / a.G / nsplit;
  const int H = a.H, G = a.G, dk = a.dk, rep = H / G;
  const int dv = a.vmode == kValuesAll ? G * a.dv_head : a.dv_head;
  const int voff = a.vmode == kValuesAll ? 0 : (a.vmode >= 0 ? a.vmode : g) * a.dv_head;
  const int LDV = dv + 8;
  const int t = a.qsl[s];                  // the sequence's one row
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  if (a.slots[s] < 0) {                    // padding row: a defined output
    for (int d = tid; d < rep * dv; d += blockDim.x) a.out[((int64_t)t * H + g * rep) * dv + d] = 0;
    return;
  }
  const int li = lane & 15, kg = lane >> 4;
  const bool valid = li < rep;
  const int head = g * rep + min(li, rep - 1);
  const int pos = a.seq_lens[s] - 1;
  const int lo = first_visible(a.mask, a.size, pos);
  const int kept = min(a.keep, lo), gap = lo - kept;
  const int nkeys = pos + 1 - gap;
  // this share's keys [k_beg, k_end)
  const int tiles = (nkeys + kST - 1) / kST, per = (tiles + nsplit - 1) / nsplit;
  const int k_beg = share * per * kST, k_end = min(nkeys, k_beg + per * kST);
  const int32_t* bt = a.block_tables + (int64_t)s * a.bt_width;
  uint16_t* vt = lds + wave * kST * LDV;

  const float cap2 = capped ? a.softcap * kLog2e : 0.f;
  const float sc_h = a.scale * (a.temp ? a.temp[head] : 1.f) * (capped ? 2.f / a.softcap : 1.f) * kLog2e;
  const float pen1 = a.r1 ? a.r1[head] : 0.f, pen2 = a.r1 ? a.r2[head] : 0.f;
  const float sbias = (sig && a.hbias) ? a.hbias[head] * kLog2e : 0.f;
  const bool with_sink = a.sink && share == 0 && wave == 0;   // one key share's running sums start with it
  float m = bounded ? 0.f : with_sink ? a.sink[head] * kLog2e : -INFINITY, l = 0.f;
  if (with_sink && kg == 0) l = 1.f;       // (lanes sum their own keys; the four lanes of a column meet at the end)

  xgk::bf16x8_t qf[NKK];
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk) {
    uint4 v = make_uint4(0, 0, 0, 0);
    if (valid && kk * 32 < dk) v = xgk::ld16(a.q + ((int64_t)t * H + head) * dk + kk * 32 + kg * 8);
    qf[kk] = xgk::as_frag(v);
  }
  xgk::f32x4_t o[NMT];
#pragma unroll
  for (int mt = 0; mt < NMT; ++mt) o[mt] = xgk::f32x4_t{0.f, 0.f, 0.f, 0.f};

  // lane L looks up the cache row of key k0 + (L & 31) (-1: outside the share)
  auto lookup = [&](int k0) -> int {
    const int kv = k0 + (lane & 31);
    if (kv >= k_end) return -1;
    const int key = kv < kept ? kv : kv + gap;
    return bt[key / a.bs] * a.bs + key % a.bs;
  };
  uint4 kr[2][NKK], vr[NMT];
  auto fetch = [&](int row) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int r = __shfl(row, n * 16 + li, 64);
      const bf16* ks = a.kcache + ((int64_t)max(r, 0) * G + g) * dk + kg * 8;
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        kr[n][kk] = (r >= 0 && kk * 32 < dk) ? xgk::ld16(ks + kk * 32) : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < NMT; ++i) {
      const int c = lane + 64 * i, vrow = c / CPR, ch = c % CPR;
      const int r = __shfl(row, vrow, 64);
      vr[i] = (r >= 0 && ch * 8 < dv) ? xgk::ld16(a.vcache + (int64_t)r * G * a.dv_head + voff + ch * 8)
                                      : make_uint4(0, 0, 0, 0);
    }
  };
  int k0 = k_beg + wave * kST;
  int row_next = -1;
  if (k0 < k_end) {
    fetch(lookup(k0));
    if (k0 + NW * kST < k_end) row_next = lookup(k0 + NW * kST);
  }
  for (; k0 < k_end; k0 += NW * kST) {
    // V rows of this tile into the wave's LDS (its reads of the previous tile precede these writes in the LDS queue)
#pragma unroll
    for (int i = 0; i < NMT; ++i) {
      const int c = lane + 64 * i, vrow = c / CPR, ch = c % CPR;
      if (ch * 8 < dv) xgk::st16(vt + vrow * LDV + ch * 8, vr[i]);
    }
    xgk::f32x4_t sacc[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      sacc[n] = xgk::f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        if (kk * 32 < dk) sacc[n] = xgk::mfma16x16x32(xgk::as_frag(kr[n][kk]), qf[kk], sacc[n]);
    }
    if (k0 + NW * kST < k_end) {
      fetch(row_next);
      row_next = lookup(k0 + 2 * NW * kST);
    }
    const bool full = k0 + kST <= k_end;   // every key of the share is visible to the one query
    float mx = -INFINITY;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kv = k0 + n * 16 + kg * 4 + r;
        float v = sacc[n][r] * sc_h;
        if constexpr (capped) v = cap2 - 2.f * cap2 * rcp_fast(1.f + exp2_fast(v));
        if (a.r1) v -= pen1 * __log2f(1.f + pen2 * (float)(pos - (kv < kept ? kv : kv + gap)));
        if (!full && kv >= k_end) v = -INFINITY;
        sacc[n][r] = v;
        mx = fmaxf(mx, v);
      }
    if constexpr (sig) {
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) sacc[n][r] = rcp_fast(1.f + exp2_fast(-(sacc[n][r] + sbias)));
    } else {
      if constexpr (!bounded) {
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m, mx);    // finite: a tile holds at least one key of the share
        const float alpha = m == -INFINITY ? 0.f : exp2_fast(m - m_new);
        l *= alpha;
        m = m_new;
#pragma unroll
        for (int mt = 0; mt < NMT; ++mt)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[mt][r] *= alpha;
      }
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = exp2_fast(bounded ? sacc[n][r] : sacc[n][r] - m);
          sacc[n][r] = p;
          l += p;
        }
    }
    uint4 pb;
    pb.x = xgk::pack2(sacc[0][0], sacc[0][1]);
    pb.y = xgk::pack2(sacc[0][2], sacc[0][3]);
    pb.z = xgk::pack2(sacc[1][0], sacc[1][1]);
    pb.w = xgk::pack2(sacc[1][2], sacc[1][3]);
    const xgk::bf16x8_t pfrag = xgk::as_frag(pb);
    __builtin_amdgcn_wave_barrier();         // the V writes above stay ahead of the transposed reads
    asm volatile("" ::: "memory");
    const int qq = li >> 2, pp = li & 3, ra = 4 * kg + qq, rb = ra + 16;
#pragma unroll
    for (int mt = 0; mt < NMT; ++mt)
      if (mt * 16 < dv) {
        const xgk::bf16x4_t a0 = xgk::lds_read_tr16(vt + ra * LDV + mt * 16 + 4 * pp);
        const xgk::bf16x4_t a1 = xgk::lds_read_tr16(vt + rb * LDV + mt * 16 + 4 * pp);
        const xgk::bf16x8_t vfrag = {a0[0], a0[1], a0[2], a0[3], a1[0], a1[1], a1[2], a1[3]};
        o[mt] = xgk::mfma16x16x32(vfrag, pfrag, o[mt]);
      }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  // ---- the waves' sums: m, l and O rows [wave][column][dv]
  __shared__ float ms[NW][16], ls[NW][16];
  float* os = reinterpret_cast<float*>(lds);
  if (kg == 0) ms[wave][li] = m, ls[wave][li] = l;
  __syncthreads();                           // (also: every wave is done with its V tiles)
  float M = bounded ? 0.f : -INFINITY;
  if (!sig && !bounded)
    for (int w = 0; w < NW; ++w) M = fmaxf(M, ms[w][li]);
  const float f = (sig || bounded) ? 1.f : (m == -INFINITY ? 0.f : exp2_fast(m - M));
  if (valid) {
#pragma unroll
    for (int mt = 0; mt < NMT; ++mt)
      if (mt * 16 < dv)
        *reinterpret_cast<float4*>(os + (wave * 16 + li) * dv + mt * 16 + 4 * kg) =
            make_float4(o[mt][0] * f, o[mt][1] * f, o[mt][2] * f, o[mt][3] * f);
  }
  __syncthreads();
  for (int e = tid; e < rep * dv; e += blockDim.x) {
    const int c = e / dv, d = e % dv, hh = g * rep + c;
    float acc = 0.f, L = 0.f, Mc = bounded ? 0.f : -INFINITY;
#pragma unroll
    for (int w = 0; w < NW; ++w) acc += os[(w * 16 + c) * dv + d];
    if (!sig) {
      if (!bounded)
        for (int w = 0; w < NW; ++w) Mc = fmaxf(Mc, ms[w][c]);
      for (int w = 0; w < NW; ++w)
        if (ms[w][c] != -INFINITY) L += (bounded ? 1.f : exp2_fast(ms[w][c] - Mc)) * ls[w][c];
    }
    if (nsplit > 1) {
      const int64_t row = ((int64_t)share * a.T + t) * H + hh;
      if (d == 0) {
        part_ml[2 * row] = Mc;
        part_ml[2 * row + 1] = L;
      }
      part_o[row * dv + d] = acc;
    } else {
      float inv = sig ? 1.f : (L > 0.f ? 1.f / L : 0.f);
      if (a.gate && !a.gate_elem) inv *= sigmoidf(bf2f(a.gate[(int64_t)t * a.ld_gate + hh]));
      acc *= inv;
      if (a.gate && a.gate_elem) acc *= sigmoidf(bf2f(a.gate[(int64_t)t * a.ld_gate + (int64_t)hh * dv + d]));
      a.out[((int64_t)t * H + hh) * dv + d] = f2bf(acc);
    }
  }
}

bool single_attention(const AttnArgs& a, int wfn, int nsplit, float* part_o, float* part_ml, hipStream_t st) {
  const int dv = a.vmode == kValuesAll ? a.G * a.dv_head : a.dv_head;
  if (a.H / a.G > kSingleMaxRep || a.dk > 128 || a.dk % 32 != 0 || dv > 128 || dv % 16 != 0) return false;
  const int grid = nsplit * a.G * a.ns;
  const int nw = (a.dk <= 64 && dv <= 64) ? 8 : 4;   // (registers: 16 / 8 waves per compute unit)
  // the waves' V tiles, then (the same bytes) their sums
  const size_t lds = std::max((size_t)nw * kST * (dv + 8) * sizeof(uint16_t), (size_t)nw * 16 * dv * sizeof(float));
#define XGM_SA2(NKK, NMT, NW, WFN) single_attention_kernel<NKK, NMT, NW, WFN><<<grid, 64 * NW, lds, st>>>(a, nsplit, part_o, part_ml);
#define XGM_SA(NKK, NMT, NW)                        \
  switch (wfn) {                                    \
    case kWeightsSigmoid:                           \
      XGM_SA2(NKK, NMT, NW, kWeightsSigmoid) break; \
    case kWeightsBounded:                           \
      XGM_SA2(NKK, NMT, NW, kWeightsBounded) break; \
    case kWeightsCapped:                            \
      XGM_SA2(NKK, NMT, NW, kWeightsCapped) break;  \
    default:                                        \
      XGM_SA2(NKK, NMT, NW, kWeightsSoftmax) break; \
  }
  if (nw == 8) {
    XGM_SA(2, 4, 8)
  } else {
    XGM_SA(4, 8, 4)
  }
#undef XGM_SA
#undef XGM_SA2
  return true;
}

}  // namespace xgm
