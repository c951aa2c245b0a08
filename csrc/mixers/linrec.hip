// Outer-product recurrences with a fixed decay per head (retention) or a data-dependent decay per key channel and a bonus
// for the current token (time mixing): what surrounds the scans, and their single-token steps.
//
//   rotate_qk        q and k of a fused projection row, the first rot_dims entries of each head rotated in pairs
//                    (i, i + rot_dims / 2) by the token's position, k times a constant; fp32 tensors
//   token_shift_mix  n mixes x_t + (x_(t-1) - x_t) mu_s of each row with the previous token's, as activation tensors
//                    [n][T rounded up to whole tiles][W]; x_(-1) comes from the slot's carried row (zeros at a sequence's start), which takes the
//                    portion's last row
//   time_mix_gates   r, k as fp32 and the decay f = exp(-exp(z + w0))
//   recurrent_step   steps of single tokens, one workgroup per (sequence, head): rotation or decay, the state update
//                      S <- diag(f) S + k v^T,   o = S^T q  (after the update)  or  o = (S_old + diag(u) k v^T)^T q,
//                    the head's output divided by its root mean square, times a weight, times silu(gate). Every state
//                    element is read and written once, in whole 256-byte rows.
//
// chunk_recurrence.hip holds the matrix-core form for prompt portions, gla.hip the general scan.
#include "mixers_common.h"

namespace xgm {

template <typename T>
__global__ __launch_bounds__(256) void rotate_qk_kernel(const T* __restrict__ proj, int64_t ld, int off_q, int off_k, int H,
                                                        int dk, const float* __restrict__ rot, int rot_rows, int rot_dims,
                                                        float k_scale, const int32_t* __restrict__ positions,
                                                        float* __restrict__ q, float* __restrict__ k, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int n = H * dk, half = rot_dims / 2;
  const int64_t t = i / n;
  const int c = (int)(i % n), d = c % dk;
  const T* row = proj + t * ld;
  float a = ldf(row + off_q + c), b = ldf(row + off_k + c);
  if (d < rot_dims) {
    const int p = min(max(positions[t], 0), rot_rows - 1), j = d % half;
    const float cs = rot[((int64_t)p * half + j) * 2], sn = rot[((int64_t)p * half + j) * 2 + 1];
    const int o = d < half ? half : -half;
    const float a2 = ldf(row + off_q + c + o), b2 = ldf(row + off_k + c + o);
    const float sg = d < half ? -sn : sn;
    a = a * cs + a2 * sg;
    b = b * cs + b2 * sg;
  }
  q[i] = a;
  k[i] = b * k_scale;
}

constexpr int kMaxMixes = 8;

template <typename TO>
__global__ __launch_bounds__(256) void token_shift_mix_kernel(const float* __restrict__ x, const float* __restrict__ mu, int n,
                                                              float* __restrict__ state, const int32_t* __restrict__ qsl,
                                                              const int32_t* __restrict__ seq_lens,
                                                              const int32_t* __restrict__ slots,
                                                              const int32_t* __restrict__ token_seq, TO* __restrict__ out,
                                                              int64_t pitch, int W) {
  const int t = blockIdx.x;
  const int c = 4 * (blockIdx.y * 256 + threadIdx.x);
  if (c >= W) return;
  const int s = token_seq[t];
  const int slot = s < 0 ? -1 : slots[s];
  const bool quad = c + 4 <= W && (W & 3) == 0;
  const int m = quad ? 4 : min(4, W - c);
  float v[4] = {0.f, 0.f, 0.f, 0.f}, p[4] = {0.f, 0.f, 0.f, 0.f};
  if (slot >= 0) {
    auto get = [&](const float* r, float (&f)[4]) {
      if (quad) ld4(r + c, f);
      else
        for (int i = 0; i < m; ++i) f[i] = r[c + i];
    };
    const int q0 = qsl[s], q1 = qsl[s + 1];
    get(x + (int64_t)t * W, v);
    if (t > q0) {
      get(x + (int64_t)(t - 1) * W, p);
    } else {   // the portion's first row: the carried row, which this workgroup alone reads and then replaces
      float* sr = state + (int64_t)slot * W;
      if (seq_lens[s] > q1 - q0) get(sr, p);
      float l[4];
      get(x + (int64_t)(q1 - 1) * W, l);
      for (int i = 0; i < m; ++i) sr[c + i] = l[i];
    }
  }
  for (int j = 0; j < n; ++j) {
    float o[4];
    const float* mj = mu + (int64_t)j * W + c;
    TO* oj = out + (j * pitch + t) * W + c;
    if (quad) {
      float g[4];
      ld4(mj, g);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] = v[i] + (p[i] - v[i]) * g[i];
      st4(oj, o);
    } else {
      for (int i = 0; i < m; ++i) stf(oj + i, v[i] + (p[i] - v[i]) * mj[i]);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void time_mix_gates_kernel(const T* __restrict__ r, int64_t ld_r, const T* __restrict__ k,
                                                             int64_t ld_k, const T* __restrict__ z, int64_t ld_z,
                                                             const float* __restrict__ w0, int n, float* __restrict__ ro,
                                                             float* __restrict__ fo, float* __restrict__ ko, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / n;
  const int c = (int)(i % n);
  ro[i] = ldf(r + t * ld_r + c);
  ko[i] = ldf(k + t * ld_k + c);
  fo[i] = expf(-expf(ldf(z + t * ld_z + c) + w0[c]));
}

// ------------------------------------------------------------------ single tokens
struct StepArgs {
  const void *q, *k, *v, *g, *z;   // head h of token t at row t: columns h dk .. / h dv ..
  int64_t ld_q, ld_k, ld_v, ld_g, ld_z;
  int z_f32;
  const float *decay, *w0, *bonus;   // decay [H]: retention; else w0 [H dk] beside z, bonus [H dk]
  const float* rot;
  int rot_rows, rot_dims;
  float k_scale;
  const float* norm_w;
  float eps;
  float* state;
  const int32_t *seq_lens, *slots, *positions;
  void* out;
  int H, dk, dv;
};

constexpr int kStepThreads = 256, kStepMaxDk = 256;

template <typename T, typename TO, int CV>
__global__ __launch_bounds__(kStepThreads) void recurrent_step_kernel(const StepArgs a) {
  extern __shared__ float opart[];   // [row groups][dv]
  __shared__ float qs[kStepMaxDk], ks[kStepMaxDk], fs[kStepMaxDk];
  __shared__ float red[kStepThreads / 64];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int dk = a.dk, dv = a.dv, slot = a.slots[s];
  TO* out = (TO*)a.out + ((int64_t)s * a.H + h) * dv;
  if (slot < 0) {   // padding row
    for (int c = tid; c < dv; c += kStepThreads) stf(out + c, 0.f);
    return;
  }
  const bool fresh = a.seq_lens[s] <= 1;
  const T* qr = (const T*)a.q + s * a.ld_q + h * dk;
  const T* kr = (const T*)a.k + s * a.ld_k + h * dk;
  const T* vr = (const T*)a.v + s * a.ld_v + h * dv;
  const T* gr = (const T*)a.g + s * a.ld_g + h * dv;
  float ruk = 0.f;
  if (tid < dk) {
    const int d = tid;
    float q = ldf(qr + d), k = ldf(kr + d), f;
    if (a.decay) {
      f = a.decay[h];
      const int half = a.rot_dims / 2;
      if (d < a.rot_dims) {
        const int p = min(max(a.positions[s], 0), a.rot_rows - 1), j = d < half ? d : d - half;
        const float cs = a.rot[((int64_t)p * half + j) * 2], sn = a.rot[((int64_t)p * half + j) * 2 + 1];
        const int o = d < half ? half : -half;
        const float sg = d < half ? -sn : sn;
        const float q2 = ldf(qr + d + o), k2 = ldf(kr + d + o);
        q = q * cs + q2 * sg;
        k = k * cs + k2 * sg;
      }
      k *= a.k_scale;
    } else {
      const int64_t zi = s * a.ld_z + h * dk + d;
      f = expf(-expf((a.z_f32 ? ((const float*)a.z)[zi] : bf2f(((const bf16*)a.z)[zi])) + a.w0[h * dk + d]));
      ruk = q * a.bonus[h * dk + d] * k;
    }
    qs[d] = q, ks[d] = k, fs[d] = f;
  }
  // the bonus term (sum_d r u k) v; for retention the output reads the updated state, adding (sum_d q k) v to f S q
  ruk = block_sum(a.decay ? (tid < dk ? qs[tid] * ks[tid] : 0.f) : ruk, red);
  const int ct = (dv + CV - 1) / CV;                               // threads per state row
  const int rg = ct < kStepThreads ? kStepThreads / ct : 1;        // row groups
  float* Sg = a.state + (((int64_t)slot * a.H + h) * dk) * dv;
  const int r0 = ct < kStepThreads ? tid / ct : 0;
  for (int cc = ct < kStepThreads ? tid % ct : tid; cc < ct && r0 < rg; cc += kStepThreads) {
    const int c = CV * cc;
    float acc[CV], vv[CV];
#pragma unroll
    for (int i = 0; i < CV; ++i) acc[i] = 0.f, vv[i] = ldf(vr + c + i);
    constexpr int U = 4;
    for (int n0 = r0; n0 < dk; n0 += U * rg) {
      float S[U][CV];
#pragma unroll
      for (int j = 0; j < U; ++j) {
        const int n = n0 + j * rg;
#pragma unroll
        for (int i = 0; i < CV; ++i) S[j][i] = 0.f;
        if (n < dk && !fresh) {
          if constexpr (CV == 4) ld4(Sg + (int64_t)n * dv + c, S[j]);
          else S[j][0] = Sg[(int64_t)n * dv + c];
        }
      }
#pragma unroll
      for (int j = 0; j < U; ++j) {
        const int n = n0 + j * rg;
        if (n < dk) {
          const float f = fs[n], k = ks[n], qo = a.decay ? qs[n] * f : qs[n];
#pragma unroll
          for (int i = 0; i < CV; ++i) {
            acc[i] = fmaf(S[j][i], qo, acc[i]);
            S[j][i] = fmaf(f, S[j][i], k * vv[i]);
          }
          if constexpr (CV == 4) st4(Sg + (int64_t)n * dv + c, S[j]);
          else Sg[(int64_t)n * dv + c] = S[j][0];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < CV; ++i) opart[r0 * dv + c + i] = acc[i];
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < dv; c += kStepThreads) {
    float o = ruk * ldf(vr + c);
    for (int r = 0; r < rg; ++r) o += opart[r * dv + c];
    opart[c] = o;   // (row group 0, column c: read and written by this thread alone)
    ss += o * o;
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)dv + a.eps);
  for (int c = tid; c < dv; c += kStepThreads) {
    const float w = a.norm_w ? a.norm_w[h * dv + c] : 1.f;
    stf(out + c, opart[c] * inv * w * siluf(ldf(gr + c)));
  }
}

// ================================================================== host launchers
void rotate_qk(const void* proj, bool f32, int64_t ld, int off_q, int off_k, int H, int dk, const float* rot, int rot_rows,
               int rot_dims, float k_scale, const int32_t* positions, float* q, float* k, int T_, hipStream_t st) {
  if (T_ <= 0) return;
  const int64_t total = (int64_t)T_ * H * dk;
  XGM_DISPATCH_T(f32, rotate_qk_kernel<T><<<(unsigned)((total + 255) / 256), 256, 0, st>>>(
                          (const T*)proj, ld, off_q, off_k, H, dk, rot, rot_rows, rot_dims, k_scale, positions, q, k, total);)
}

void token_shift_mix(const float* x, const float* mu, int n, float* state, const int32_t* qsl, const int32_t* seq_lens,
                     const int32_t* slots, const int32_t* token_seq, void* out, bool out_f32, int T_, int pitch, int W,
                     hipStream_t st) {
  if (T_ <= 0 || n <= 0) return;
  dim3 grid(T_, (W + 1023) / 1024);
  XGM_DISPATCH_T(out_f32, token_shift_mix_kernel<T><<<grid, 256, 0, st>>>(x, mu, n, state, qsl, seq_lens, slots, token_seq,
                                                                          (T*)out, pitch, W);)
}

void time_mix_gates(const void* r, int64_t ld_r, const void* k, int64_t ld_k, const void* z, int64_t ld_z, bool f32,
                    const float* w0, int n, float* ro, float* fo, float* ko, int T_, hipStream_t st) {
  if (T_ <= 0) return;
  const int64_t total = (int64_t)T_ * n;
  XGM_DISPATCH_T(f32, time_mix_gates_kernel<T><<<(unsigned)((total + 255) / 256), 256, 0, st>>>(
                          (const T*)r, ld_r, (const T*)k, ld_k, (const T*)z, ld_z, w0, n, ro, fo, ko, total);)
}

int recurrent_step(const void* q, int64_t ld_q, const void* k, int64_t ld_k, const void* v, int64_t ld_v, const void* g,
                   int64_t ld_g, const void* z, int64_t ld_z, bool z_f32, bool f32, bool out_f32, const float* decay, const float* w0,
                   const float* bonus, const float* rot, int rot_rows, int rot_dims, float k_scale, const float* norm_w,
                   float eps, float* state, const int32_t* seq_lens, const int32_t* slots, const int32_t* positions,
                   void* out, int ns, int H, int dk, int dv, hipStream_t st) {
  if (ns <= 0) return 0;
  if (H < 1 || dk < 1 || dk > kStepMaxDk || dv < 1 || dv > 8192 || (!decay && (!z || !w0 || !bonus)) || rot_dims % 2 ||
      rot_dims > dk || (rot_dims && !rot))
    return -1;
  const StepArgs a = {q, k, v, g, z, ld_q, ld_k, ld_v, ld_g, ld_z, z_f32, decay, w0, bonus, rot, rot_rows, rot_dims, k_scale,
                      norm_w, eps, state, seq_lens, slots, positions, out, H, dk, dv};
  const int cv = dv % 4 == 0 ? 4 : 1, ct = (dv + cv - 1) / cv, rg = ct < kStepThreads ? kStepThreads / ct : 1;
  const size_t lds = (size_t)rg * dv * sizeof(float);
  dim3 grid(ns, H);
  if (!f32 && out_f32) return -1;
#define XGM_RS(TI, TO)                                                          \
  if (cv == 4) {                                                                \
    recurrent_step_kernel<TI, TO, 4><<<grid, kStepThreads, lds, st>>>(a);       \
  } else {                                                                      \
    recurrent_step_kernel<TI, TO, 1><<<grid, kStepThreads, lds, st>>>(a);       \
  }
  if (!f32) {
    XGM_RS(bf16, bf16)
  } else if (out_f32) {
    XGM_RS(float, float)
  } else {
    XGM_RS(float, bf16)
  }
#undef XGM_RS
  return 0;
}

}  // namespace xgm
