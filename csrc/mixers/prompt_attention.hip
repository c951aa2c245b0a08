// Attention of prompt portions on the matrix cores, bf16: 32 query rows per wave on v_mfma_f32_32x32x16_bf16.
//
// A workgroup of 8 waves = GH query heads of one key/value head x 8 / GH blocks of 32 rows, over 64-key tiles of K and V
// that LDS-DMA brings into a ring NSLOT - 1 tiles ahead (no staging registers, counted vmcnt waits, one raw barrier per
// tile). S^T = K Q^T leaves a lane with 32 scores of ONE query row; packed to bf16 they are the B operand of
// O^T += V^T P^T, whose A operand is a transposed LDS read. A row of DK = 64 / 128 entries is 8 / 16 chunks of 16 bytes;
// chunk c of row r lies at chunk c ^ xsw(r), applied to the DMA's source address, so that both the row reads of K and the
// transposed reads of V touch every bank once.
//
// Visibility, scores, weights and gates are those of chunk_attention.hip. Keys are walked in whole tiles: first the tiles
// that hold kept first keys (when the window starts behind them), then from the window's first key, rounded down to 16, to
// the last row's own; a tile (or a wave's part of it) that lies wholly inside every row's view skips the per-key tests, one
// that no row of the wave sees is passed over. 16 keys in a row share a page (block sizes are multiples of 16), so the page
// index of a wave's DMA rows is one scalar load.
#include "attention_common.h"
#include "glds.h"

namespace xgm {

constexpr int kPT = 64;   // keys per tile

typedef xgk::f32x16_t f32x16_t;

__device__ __forceinline__ f32x16_t mfma32x32x16(xgk::bf16x8_t a, xgk::bf16x8_t b, f32x16_t c) {
#if defined(__HIP_DEVICE_COMPILE__)
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
#else
  return c;
#endif
}

__device__ __forceinline__ float xor32_max(float x) {
#if defined(__HIP_DEVICE_COMPILE__)
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
#else
  return x;
#endif
}

__device__ __forceinline__ void sched_fence() {
#if defined(__HIP_DEVICE_COMPILE__)
  __builtin_amdgcn_sched_barrier(0);
#endif
}

// chunk permutation of a row: 16 consecutive rows hit all 16-byte slots of the banks for one chunk, and 4 rows x 4
// neighbouring chunks do too
template <int D>
__device__ __forceinline__ int xsw(int r) {
  return D == 128 ? ((r & 3) << 2) | ((r >> 2) & 3) : (((r >> 1) & 1) << 2) | ((r >> 2) & 3);
}

template <int DK, int DV, int GH, int NSLOT, int WFN>
__global__ __launch_bounds__(512, (DK == 64 && DV == 64) ? 4 : 2) void prompt_attention_kernel(
    const AttnArgs a, const int32_t* __restrict__ block_tables, const bf16* __restrict__ kcache,
    const bf16* __restrict__ vcache, int tiles_per_seq, int n_hg) {
  constexpr bool sig = WFN == kWeightsSigmoid, capped = WFN == kWeightsBounded || WFN == kWeightsCapped;
  constexpr bool bounded = WFN == kWeightsBounded;
  constexpr int NW = 8, RBLK = NW / GH, BM = 32 * RBLK;
  constexpr int KROW = DK * 2, VROW = DV * 2;            // bytes of a row
  constexpr int KT = kPT * KROW, SLOT = KT + kPT * VROW;  // bytes of a K tile, of a ring slot [K | V]
  constexpr int KD = DK / 64, VD = DV / 64;               // DMA instructions per wave and tile (8 rows per wave)
  __shared__ __attribute__((aligned(1024))) char lds[NSLOT * SLOT];

  const int bid = blockIdx.x;
  const int hg = bid % n_hg, rest = bid / n_hg;           // head groups fastest: an XCD streams few key/value heads
  const int s = rest % a.ns;
  const int qt = tiles_per_seq - 1 - rest / a.ns;         // late row tiles see the most keys: first
  const int q0 = a.qsl[s], qn = a.qsl[s + 1] - q0;
  const int i0 = qt * BM;
  if (a.slots[s] < 0 || i0 >= qn) return;
  const int rep = a.H / a.G, hb = rep / GH;
  const int g = hg / hb;
  const int lane = threadIdx.x & 63;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int head = g * rep + (hg % hb) * GH + w % GH;
  const int rb = w / GH;
  const int r = lane & 31, hf = lane >> 5;
  const int voff = a.vmode == kValuesAll ? 0 : (a.vmode >= 0 ? a.vmode : g) * a.dv_head;
  const int64_t krow = (int64_t)a.G * DK, vrow = (int64_t)a.G * a.dv_head;   // elements between two cached rows
  const int ctx = a.seq_lens[s] - qn;
  const int my_row = i0 + rb * 32 + r;
  const int pos_q = ctx + my_row;
  const int lo_q = first_visible(a.mask, a.size, pos_q);
  const int pos_lo = ctx + i0 + rb * 32, pos_hi = ctx + min(qn, i0 + rb * 32 + 32) - 1;   // the wave's rows (uniform)
  const int lo_lo = first_visible(a.mask, a.size, pos_lo), lo_hi = first_visible(a.mask, a.size, pos_hi);
  // tiles of the workgroup: `kt` tiles from key 0 on, then from key `kfirst` on (kt = 0: no kept keys behind a gap)
  const int last = ctx + min(qn, i0 + BM) - 1;
  int kfirst = first_visible(a.mask, a.size, ctx + i0) & ~15;
  int kt = (a.keep + kPT - 1) / kPT;
  if (kfirst <= kt * kPT) kfirst = a.keep > 0 ? 0 : kfirst, kt = 0;
  const int ntiles = kt + (last - kfirst + kPT) / kPT;
  const int32_t* bt = block_tables + (int64_t)s * a.bt_width;
  auto tile_key = [&](int t) { return t < kt ? t * kPT : kfirst + (t - kt) * kPT; };

  auto issue = [&](int t) {
    char* dst = lds + (t % NSLOT) * SLOT;
    const int key0 = min(tile_key(t) + 8 * w, last);      // the wave's 8 rows: inside one aligned run of 16 keys
    const int pidx = key0 / a.bs;
    const int64_t prow = (int64_t)bt[pidx] * a.bs - (int64_t)pidx * a.bs;
    const int k1 = tile_key(t) + 8 * w;
#pragma unroll
    for (int i = 0; i < KD; ++i) {
      const int rr = KD == 2 ? 4 * i + (lane >> 4) : lane >> 3;
      const int ch = (KD == 2 ? lane & 15 : lane & 7) ^ xsw<DK>(8 * w + rr);
      const int64_t row = prow + min(k1 + rr, last);
      xgk::glds16(kcache + row * krow + g * DK + ch * 8, dst + (8 * w) * KROW + i * 1024);
    }
#pragma unroll
    for (int i = 0; i < VD; ++i) {
      const int rr = VD == 2 ? 4 * i + (lane >> 4) : lane >> 3;
      const int ch = (VD == 2 ? lane & 15 : lane & 7) ^ xsw<DV>(8 * w + rr);
      const int64_t row = prow + min(k1 + rr, last);
      xgk::glds16(vcache + row * vrow + voff + ch * 8, dst + KT + (8 * w) * VROW + i * 1024);
    }
  };

  // Q^T (B operand): lane holds Q[row r][16 ks + 8 hf + 0..7]
  xgk::bf16x8_t qf[DK / 16];
  {
    const bf16* qp = a.q + ((int64_t)(q0 + min(my_row, qn - 1)) * a.H + head) * DK + 8 * hf;
#pragma unroll
    for (int ks = 0; ks < DK / 16; ++ks) qf[ks] = xgk::as_frag(xgk::ld16(qp + 16 * ks));
  }
  const float cap2 = capped ? a.softcap * kLog2e : 0.f;
  float sc_h = a.scale * (a.temp ? a.temp[head] : 1.f) * (capped ? 2.f / a.softcap : 1.f) * kLog2e;
  float pen1 = a.r1 ? a.r1[head] : 0.f, pen2 = a.r1 ? a.r2[head] : 0.f;
  float sbias = (sig && a.hbias) ? a.hbias[head] * kLog2e : 0.f;
  float m = bounded ? 0.f : a.sink ? a.sink[head] * kLog2e : -INFINITY;
  float l = (a.sink && hf == 0) ? 1.f : 0.f;   // each half of a row's two lanes sums its own keys
  f32x16_t o[DV / 32];
#pragma unroll
  for (int db = 0; db < DV / 32; ++db)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[db][e] = 0.f;
  // everything loaded so far is complete before the first DMA: from here on vmcnt counts the DMAs alone
#pragma unroll
  for (int ks = 0; ks < DK / 16; ++ks) asm volatile("" : "+v"(qf[ks]));
  asm volatile("" : "+v"(sc_h), "+v"(pen1), "+v"(pen2), "+v"(sbias), "+v"(m));
  xgk::wait_vmcnt<0>();
#pragma unroll
  for (int p = 0; p < NSLOT - 1; ++p)
    if (p < ntiles) issue(p);

  const int tg = lane >> 4, tq = (lane & 15) >> 2, tp = lane & 3;
  const bool wave_on = pos_lo <= pos_hi;
  for (int j = 0; j < ntiles; ++j) {
    if constexpr (NSLOT == 3) {
      if (j + 1 < ntiles) xgk::wait_vmcnt<KD + VD>();
      else xgk::wait_vmcnt<0>();
    } else {
      xgk::wait_vmcnt<0>();
    }
    xgk::raw_barrier();
    if (j + NSLOT - 1 < ntiles) issue(j + NSLOT - 1);
    const int base = tile_key(j);
    // (wave-uniform) nothing of this tile is visible to the wave's rows
    if (!wave_on || base > pos_hi || (base + kPT - 1 < lo_lo && base >= a.keep)) continue;
    const uint32_t slot = (j % NSLOT) * SLOT;
    const uint32_t k_lane = (slot + r * KROW) ^ ((uint32_t)(hf ^ xsw<DK>(r)) << 4);
    const uint32_t v_row = slot + KT + (4 * hf + tq) * VROW + 8 * (tp & 1);
    const uint32_t v_hi = (uint32_t)(DV == 128 ? tq : tq >> 1) << 6, v_lo = 2 * (tg & 1) + (tp >> 1);
    const uint32_t v_lane0 = (v_row + ((v_lo ^ hf) << 4)) | v_hi;
    const uint32_t v_lane1 = (v_row + 8 * VROW + ((v_lo ^ (hf + 2)) << 4)) | v_hi;

    f32x16_t sacc[2];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
      for (int e = 0; e < 16; ++e) sacc[kb][e] = 0.f;
#pragma unroll
      for (int ks = 0; ks < DK / 16; ++ks)
        sacc[kb] = mfma32x32x16(xgk::as_frag(xgk::ld16(lds + ((k_lane ^ (ks << 5)) + kb * 32 * KROW))), qf[ks], sacc[kb]);
      sched_fence();   // bound the hoisted fragment reads
    }
    // scores in units of ln 2; register e of block kb is key base + 32 kb + 4 hf + (e & 3) + 8 (e >> 2)
    const bool full = base + kPT - 1 <= pos_lo && (base >= lo_hi || base + kPT <= a.keep);
    const int vis_hi = pos_q - base - 4 * hf, vis_lo = lo_q - base - 4 * hf, vis_keep = a.keep - base - 4 * hf;
    float mx = -INFINITY;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        float v = sacc[kb][e] * sc_h;
        if constexpr (capped) v = cap2 - 2.f * cap2 * rcp_fast(1.f + exp2_fast(v));
        sacc[kb][e] = v;
      }
    if (a.r1) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 16; ++e)
          sacc[kb][e] -= pen1 * __log2f(1.f + pen2 * (float)max(vis_hi - (kb * 32 + (e & 3) + 8 * (e >> 2)), 0));
    }
    if (!full) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          const int c = kb * 32 + (e & 3) + 8 * (e >> 2);
          if (c > vis_hi || (c < vis_lo && c >= vis_keep)) sacc[kb][e] = -INFINITY;
        }
    }
    if constexpr (sig) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 16; ++e) sacc[kb][e] = rcp_fast(1.f + exp2_fast(-(sacc[kb][e] + sbias)));
    } else {
      float nm = 0.f;
      if constexpr (!bounded) {
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int e = 0; e < 16; ++e) mx = fmaxf(mx, sacc[kb][e]);
        mx = xor32_max(mx);
        const float m_new = fmaxf(m, mx);
        nm = m_new == -INFINITY ? 0.f : -m_new;
        // no row of the wave raised its maximum: nothing to rescale
        if (__builtin_amdgcn_ballot_w64(m_new > m) != 0) {
          const float alpha = m == -INFINITY ? 0.f : exp2_fast(m + nm);
          l *= alpha;
#pragma unroll
          for (int db = 0; db < DV / 32; ++db)
#pragma unroll
            for (int e = 0; e < 16; ++e) o[db][e] *= alpha;
          m = m_new;
        }
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          const float p = exp2_fast(bounded ? sacc[kb][e] : sacc[kb][e] + nm);
          sacc[kb][e] = p;
          l += p;
        }
    }
    // O^T += V^T P^T: step (kb, ss) takes score registers 8 ss .. 8 ss + 7 (keys 32 kb + 16 ss + ..)
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int ss = 0; ss < 2; ++ss) {
        uint4 pb;
        pb.x = xgk::pack2(sacc[kb][8 * ss + 0], sacc[kb][8 * ss + 1]);
        pb.y = xgk::pack2(sacc[kb][8 * ss + 2], sacc[kb][8 * ss + 3]);
        pb.z = xgk::pack2(sacc[kb][8 * ss + 4], sacc[kb][8 * ss + 5]);
        pb.w = xgk::pack2(sacc[kb][8 * ss + 6], sacc[kb][8 * ss + 7]);
        const xgk::bf16x8_t pf = xgk::as_frag(pb);
        const uint32_t ro = (kb * 32 + 16 * ss) * VROW;
#pragma unroll
        for (int db = 0; db < DV / 32; ++db) {
          const xgk::bf16x4_t a0 = xgk::lds_read_tr16(reinterpret_cast<const uint16_t*>(lds + ((v_lane0 ^ (db << 6)) + ro)));
          const xgk::bf16x4_t a1 = xgk::lds_read_tr16(reinterpret_cast<const uint16_t*>(lds + ((v_lane1 ^ (db << 6)) + ro)));
          const xgk::bf16x8_t vf = {a0[0], a0[1], a0[2], a0[3], a1[0], a1[1], a1[2], a1[3]};
          o[db] = mfma32x32x16(vf, pf, o[db]);
        }
        sched_fence();
      }
  }
  l += __shfl_xor(l, 32, 64);
  // lane holds O[row r][32 db + 8 t + 4 hf + 0..3] in registers 4 t .. 4 t + 3
  if (my_row < qn) {
    const int64_t row = q0 + my_row;
    float inv = sig ? 1.f : (l > 0.f ? 1.f / l : 0.f);
    if (a.gate && !a.gate_elem) inv *= sigmoidf(bf2f(a.gate[row * a.ld_gate + head]));
    bf16* op = a.out + (row * a.H + head) * DV + 4 * hf;
    const bf16* ge = (a.gate && a.gate_elem) ? a.gate + row * a.ld_gate + (int64_t)head * DV + 4 * hf : nullptr;
#pragma unroll
    for (int db = 0; db < DV / 32; ++db)
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        float e[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          e[i] = o[db][4 * t + i] * inv;
          if (ge) e[i] *= sigmoidf(bf2f(ge[32 * db + 8 * t + i]));
        }
        *reinterpret_cast<uint2*>(op + 32 * db + 8 * t) = make_uint2(xgk::pack2(e[0], e[1]), xgk::pack2(e[2], e[3]));
      }
  }
}

bool prompt_attention(const AttnArgs& a, int max_q, int wfn, hipStream_t st) {
  const int dv = a.vmode == kValuesAll ? a.G * a.dv_head : a.dv_head;
  const int rep = a.H / a.G;
  if (a.bs % 16 != 0 || (a.dk != 64 && a.dk != 128) || (dv != 64 && dv != 128) || (uintptr_t)a.kcache % 16 != 0 ||
      (uintptr_t)a.vcache % 16 != 0 || (a.G * a.dv_head) % 8 != 0 || a.dv_head % 8 != 0)
    return false;
  const int gh = rep % 4 == 0 ? 4 : rep % 2 == 0 ? 2 : 1, bm = 32 * 8 / gh;
  const int tps = (max_q + bm - 1) / bm, n_hg = a.G * rep / gh;
  const int grid = n_hg * a.ns * tps;
#define XGM_PA3(DK, DV, GH, WFN)                                                                                      \
  prompt_attention_kernel<DK, DV, GH, 3, WFN><<<grid, 512, 0, st>>>(a, a.block_tables, a.kcache, a.vcache, tps, n_hg)
#define XGM_PA2(DK, DV, GH)                                  \
  switch (wfn) {                                             \
    case kWeightsSigmoid:                                    \
      XGM_PA3(DK, DV, GH, kWeightsSigmoid);                  \
      break;                                                 \
    case kWeightsBounded:                                    \
      XGM_PA3(DK, DV, GH, kWeightsBounded);                  \
      break;                                                 \
    case kWeightsCapped:                                     \
      XGM_PA3(DK, DV, GH, kWeightsCapped);                   \
      break;                                                 \
    default:                                                 \
      XGM_PA3(DK, DV, GH, kWeightsSoftmax);                  \
      break;                                                 \
  }
#define XGM_PA1(DK, DV)        \
  if (gh == 4) {               \
    XGM_PA2(DK, DV, 4)         \
  } else if (gh == 2) {        \
    XGM_PA2(DK, DV, 2)         \
  } else {                     \
    XGM_PA2(DK, DV, 1)         \
  }
  if (a.dk == 64 && dv == 64) {
    XGM_PA1(64, 64)
  } else if (a.dk == 128 && dv == 128) {
    XGM_PA1(128, 128)
  } else if (a.dk == 64) {
    XGM_PA1(64, 128)
  } else {
    XGM_PA1(128, 64)
  }
#undef XGM_PA1
#undef XGM_PA2
#undef XGM_PA3
  return true;
}

}  // namespace xgm
