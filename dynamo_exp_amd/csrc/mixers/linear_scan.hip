// Linear recurrences over a running matrix for gfx950: per (sequence, head) a
// matrix S [dk, dv], without softmax and without a denominator,
//     S_t = D_t S_(t-1) + (k_scale k_t) (u_t v_t)^T,   o_t = S_t^T (q_scale q_t) + skip_h v_t
// in three forms of the decay D_t and the step u_t (kMode):
//   kFixed    D_t = decay_h, u_t = 1                                         (retention)
//   kStep     u_t = softplus(g_t,h + bias_h), D_t = exp(-rate_h u_t)         (state-space duality)
//   kChannel  D_t = diag(sigmoid(g_t,h,i + bias_h,i)^(1 / tau)), u_t = 1     (gated linear attention)
// Query head h reads the q / k head h / qk_rep (state-space groups share them).
//
// Columns of S are independent: R neighbouring lanes share a column (up to
// kRows rows each, in registers) and join their partial q^T S by DPP lane
// exchanges; a workgroup owns blockDim / R columns of one (sequence, head).
// Tokens are staged through LDS kTok at a time.  State layout [slots, H, dv,
// dk]: a column's rows are contiguous.  This file scans token by token (any
// sizes, decode steps, fp32); chunk_scan.hip has the matrix-core form for prompt
// portions in bf16.  Slots, seq_rows and the reset at position 0 as in
// recurrent.hip.  Decays, step sizes, the state and all sums
// are fp32 whatever the activation element is.
#include "linear_scan.h"

namespace {

// step size and decay of one (row, head)
template <typename T> __device__ __forceinline__ float2 step_terms(const ScanArgs& g, int64_t row, int h) {
  const float u = step_size<T>(g, row, h);
  return float2{u, expf(-g.rate[h] * u)};
}

constexpr int kMaxKey = 512;

// Any sizes: rows and columns beyond dk / dv are guarded one by one.  Lane r of a column's group owns
// rows r, r + R, ...
template <typename T, int R, int MODE, int ROWS = kRows>
__global__ void __launch_bounds__(256) scan_kernel(ScanArgs g) {
  extern __shared__ float scan_lds[];
  const int s = blockIdx.x, h = blockIdx.y, hq = h / g.qk_rep;
  const int tid = threadIdx.x, cols = blockDim.x / R;
  const int cl = tid / R, r = tid % R;
  const int col0 = blockIdx.z * cols, j = col0 + cl;
  const int r0 = g.seq_rows ? g.seq_rows[s] : s, r1 = g.seq_rows ? g.seq_rows[s + 1] : s + 1;
  if (r1 <= r0 || r0 < 0 || r1 > g.T || r1 - r0 > g.max_rows) return;
  const bool colok = j < g.dv;
  const int slot = g.slots[s];
  const int64_t ow = (int64_t)g.H * g.dv;
  if (slot < 0 || slot >= g.n_slots) {  // a padding row: zeros out, no state touched
    for (int t = r0; t < r1; ++t)
      if (r == 0 && colok) g.out[(int64_t)t * ow + h * g.dv + j] = 0.f;
    return;
  }
  float* qs_ = scan_lds;
  float* ks_ = qs_ + kTok * g.dk;
  float* vs_ = ks_ + kTok * g.dk;
  float* gs_ = vs_ + kTok * cols;  // kStep: (step, decay) per token; kChannel: [kTok][dk] decays
  float* sp = g.state + (((int64_t)slot * g.H + h) * g.dv + (colok ? j : 0)) * g.dk;
  const bool fresh = g.pos[r0] == 0;
  float S[ROWS];
#pragma unroll
  for (int ii = 0; ii < ROWS; ++ii) {
    const int i = r + R * ii;
    S[ii] = (!fresh && colok && i < g.dk) ? sp[i] : 0.f;
  }
  const float fixed = MODE == kFixed ? g.decay[h] : 0.f, skip = g.skip ? g.skip[h] : 0.f;
  const T* q = (const T*)g.q;
  const T* k = (const T*)g.k;
  const T* v = (const T*)g.v;
  for (int t0 = r0; t0 < r1; t0 += kTok) {
    const int nt = r1 - t0 < kTok ? r1 - t0 : kTok;
    __syncthreads();  // the previous block's reads are done
    for (int e = tid; e < nt * g.dk; e += blockDim.x) {
      const int tt = e / g.dk, i = e - tt * g.dk;
      qs_[e] = ldf<T>(q, (int64_t)(t0 + tt) * g.qs + hq * g.dk + i) * g.q_scale;
      ks_[e] = ldf<T>(k, (int64_t)(t0 + tt) * g.ks + hq * g.dk + i) * g.k_scale;
      if constexpr (MODE == kChannel)
        gs_[e] = channel_decay(ldf<T>((const T*)g.g, (int64_t)(t0 + tt) * g.gs + h * g.dk + i) +
                                   (g.g_bias ? g.g_bias[h * g.dk + i] : 0.f), g.inv_tau);
    }
    for (int e = tid; e < nt * cols; e += blockDim.x) {
      const int tt = e / cols, c = e - tt * cols;
      vs_[e] = col0 + c < g.dv ? ldf<T>(v, (int64_t)(t0 + tt) * g.vs + h * g.dv + col0 + c) : 0.f;
    }
    if constexpr (MODE == kStep) {
      if (tid < nt) {
        const float2 st = step_terms<T>(g, t0 + tid, h);
        gs_[2 * tid] = st.x;
        gs_[2 * tid + 1] = st.y;
      }
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      const float vj = vs_[tt * cols + cl];
      const float uv = MODE == kStep ? vj * gs_[2 * tt] : vj;
      const float dec = MODE == kStep ? gs_[2 * tt + 1] : fixed;
      const float* qt = qs_ + tt * g.dk;
      const float* kt = ks_ + tt * g.dk;
      const float* gt = gs_ + tt * g.dk;
      float acc = 0.f;
#pragma unroll
      for (int ii = 0; ii < ROWS; ++ii) {
        const int i = r + R * ii;
        if (i < g.dk) {
          S[ii] = (MODE == kChannel ? gt[i] : dec) * S[ii] + kt[i] * uv;
          acc += qt[i] * S[ii];
        }
      }
      acc = group_sum<R>(acc);
      if (r == 0 && colok) g.out[(int64_t)(t0 + tt) * ow + h * g.dv + j] = acc + skip * vj;
    }
  }
  if (colok) {
#pragma unroll
    for (int ii = 0; ii < ROWS; ++ii) {
      const int i = r + R * ii;
      if (i < g.dk) sp[i] = S[ii];
    }
  }
}

// The same for key widths dk = 16 R and 16-byte aligned operands: nothing in the token loop is
// conditional.  Lane r of a column's group owns the four row quads 4 (r + R qd) .. + 3, qd < 4, so
// a group's 128-bit LDS reads of a row vector are neighbouring chunks and the state is read and
// written as 16-byte runs.  The next block's eight tokens (q, k, decay logits of the head, v of the
// workgroup's columns) are fetched into registers as 16-byte chunks while the current block's chain runs.
template <typename T, int R, int MODE>
__global__ void __launch_bounds__(256) scan_fast_kernel(ScanArgs g) {
  constexpr int dk = 16 * R, cols = 256 / R, VEC = 16 / (int)sizeof(T);
  constexpr int QC = dk / VEC, VC = cols / VEC;  // chunks per token row
  constexpr int QK_CH = kTok * QC, V_CH = kTok * VC;
  constexpr int N_ROWS = MODE == kChannel ? 3 : 2;  // row vectors of dk staged per token
  constexpr int N_CH = N_ROWS * QK_CH + V_CH;
  constexpr int PER = (N_CH + 255) / 256;
  __shared__ __attribute__((aligned(16))) float qs_[kTok * dk];
  __shared__ __attribute__((aligned(16))) float ks_[kTok * dk];
  __shared__ __attribute__((aligned(16))) float as_[MODE == kChannel ? kTok * dk : 4];
  __shared__ __attribute__((aligned(16))) float vs_[kTok * cols];
  __shared__ float2 us_[kTok];
  const int s = blockIdx.x, h = blockIdx.y, hq = h / g.qk_rep;
  const int tid = threadIdx.x, cl = tid / R, r = tid % R;
  const int col0 = blockIdx.z * cols, j = col0 + cl;
  const int r0 = g.seq_rows ? g.seq_rows[s] : s, r1 = g.seq_rows ? g.seq_rows[s + 1] : s + 1;
  if (r1 <= r0 || r0 < 0 || r1 > g.T || r1 - r0 > g.max_rows) return;
  const int slot = g.slots[s];
  const int64_t ow = (int64_t)g.H * g.dv;
  if (slot < 0 || slot >= g.n_slots) {  // a padding row: zeros out, no state touched
    for (int t = r0; t < r1; ++t)
      if (r == 0) g.out[(int64_t)t * ow + h * g.dv + j] = 0.f;
    return;
  }
  float* sp = g.state + (((int64_t)slot * g.H + h) * g.dv + j) * dk;
  const bool fresh = g.pos[r0] == 0;
  float S[16];
#pragma unroll
  for (int qd = 0; qd < 4; ++qd) {
    const f32x4 v4 = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(sp + 4 * (r + R * qd));
#pragma unroll
    for (int e = 0; e < 4; ++e) S[4 * qd + e] = v4[e];
  }
  const float fixed = MODE == kFixed ? g.decay[h] : 0.f, skip = g.skip ? g.skip[h] : 0.f;
  const T* q = (const T*)g.q + (int64_t)hq * dk;
  const T* k = (const T*)g.k + (int64_t)hq * dk;
  const T* gl = (const T*)g.g + (int64_t)h * dk;
  const T* v = (const T*)g.v + (int64_t)h * g.dv + col0;
  raw_u32x4 pf[PER];
  float2 step{0.f, 1.f};
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = tid + i * 256;
      const T* src = nullptr;
      if (c < QK_CH) {
        const int tt = c / QC;
        if (t0 + tt < r1) src = q + (int64_t)(t0 + tt) * g.qs + (c % QC) * VEC;
      } else if (c < 2 * QK_CH) {
        const int c2 = c - QK_CH, tt = c2 / QC;
        if (t0 + tt < r1) src = k + (int64_t)(t0 + tt) * g.ks + (c2 % QC) * VEC;
      } else if (MODE == kChannel && c < 3 * QK_CH) {
        const int c2 = c - 2 * QK_CH, tt = c2 / QC;
        if (t0 + tt < r1) src = gl + (int64_t)(t0 + tt) * g.gs + (c2 % QC) * VEC;
      } else if (c < N_CH) {
        const int c2 = c - N_ROWS * QK_CH, tt = c2 / VC;
        if (t0 + tt < r1) src = v + (int64_t)(t0 + tt) * g.vs + (c2 % VC) * VEC;
      }
      pf[i] = src ? *reinterpret_cast<const raw_u32x4*>(src) : raw_u32x4{0u, 0u, 0u, 0u};
    }
    if constexpr (MODE == kStep) {
      if (tid < kTok && t0 + tid < r1) step = step_terms<T>(g, t0 + tid, h);
    }
  };
  auto commit = [&]() {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = tid + i * 256;
      float f[VEC];
      chunk_to_f32<T>(pf[i], f);
      float* dst = nullptr;
      if (c < QK_CH) {
        dst = qs_ + c * VEC;
#pragma unroll
        for (int e = 0; e < VEC; ++e) f[e] *= g.q_scale;
      } else if (c < 2 * QK_CH) {
        dst = ks_ + (c - QK_CH) * VEC;
#pragma unroll
        for (int e = 0; e < VEC; ++e) f[e] *= g.k_scale;
      } else if (MODE == kChannel && c < 3 * QK_CH) {
        const int e0 = (c - 2 * QK_CH) * VEC, ch = h * dk + e0 % dk;
        dst = as_ + e0;
#pragma unroll
        for (int e = 0; e < VEC; ++e) f[e] = channel_decay(f[e] + (g.g_bias ? g.g_bias[ch + e] : 0.f), g.inv_tau);
      } else if (c < N_CH) {
        dst = vs_ + (c - N_ROWS * QK_CH) * VEC;
      }
      if (dst) {
#pragma unroll
        for (int e = 0; e < VEC; e += 4) *reinterpret_cast<f32x4*>(dst + e) = f32x4{f[e], f[e + 1], f[e + 2], f[e + 3]};
      }
    }
    if constexpr (MODE == kStep) {
      if (tid < kTok) us_[tid] = step;
    }
  };
  fetch(r0);
  for (int t0 = r0; t0 < r1; t0 += kTok) {
    const int nt = r1 - t0 < kTok ? r1 - t0 : kTok;
    __syncthreads();  // the previous block's reads are done
    commit();
    __syncthreads();
    if (t0 + kTok < r1) fetch(t0 + kTok);
    for (int tt = 0; tt < nt; ++tt) {
      const float vj = vs_[tt * cols + cl];
      float uv = vj, dec = fixed;
      if constexpr (MODE == kStep) {
        const float2 u = us_[tt];
        uv = vj * u.x;
        dec = u.y;
      }
      float acc = 0.f;
#pragma unroll
      for (int qd = 0; qd < 4; ++qd) {
        const f32x4 kk = *reinterpret_cast<const f32x4*>(ks_ + tt * dk + 4 * (r + R * qd));
        const f32x4 qq = *reinterpret_cast<const f32x4*>(qs_ + tt * dk + 4 * (r + R * qd));
        f32x4 aa;
        if constexpr (MODE == kChannel) aa = *reinterpret_cast<const f32x4*>(as_ + tt * dk + 4 * (r + R * qd));
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[4 * qd + e] = (MODE == kChannel ? aa[e] : dec) * S[4 * qd + e] + kk[e] * uv;
          acc += qq[e] * S[4 * qd + e];
        }
      }
      acc = group_sum<R>(acc);
      if (r == 0) g.out[(int64_t)(t0 + tt) * ow + h * g.dv + j] = acc + skip * vj;
    }
  }
#pragma unroll
  for (int qd = 0; qd < 4; ++qd)
    *reinterpret_cast<f32x4*>(sp + 4 * (r + R * qd)) = f32x4{S[4 * qd], S[4 * qd + 1], S[4 * qd + 2], S[4 * qd + 3]};
}

// whether the unconditional kernel serves the launch: dk = 16 R exactly, whole column blocks,
// 16-byte aligned rows and sections
template <typename T, int R, int MODE>
bool scan_fast_ok(const ScanArgs& g) {
  constexpr int VEC = 16 / (int)sizeof(T), cols = 256 / R;
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  return g.dk == 16 * R && g.dv % cols == 0 && cols % VEC == 0 && g.qs % VEC == 0 && g.ks % VEC == 0 &&
         g.vs % VEC == 0 && al(g.q) && al(g.k) && al(g.v) && al(g.state) &&
         (MODE != kChannel || (g.gs % VEC == 0 && al(g.g)));
}

template <typename T, int R, int MODE, int ROWS = kRows>
void launch_scan(const ScanArgs& g, int n_seq, hipStream_t st) {
  if constexpr (ROWS == kRows) {
    if (scan_fast_ok<T, R, MODE>(g)) {
      hipLaunchKernelGGL((scan_fast_kernel<T, R, MODE>), dim3(n_seq, g.H, g.dv / (256 / R)), dim3(256), 0, st, g);
      return;
    }
  }
  int nt = (R * g.dv + 63) / 64 * 64;
  nt = nt > 256 ? 256 : nt;
  const int cols = nt / R;
  const size_t lds = (size_t)((MODE == kChannel ? 3 : 2) * kTok * g.dk + kTok * cols + 2 * kTok) * sizeof(float);
  hipLaunchKernelGGL((scan_kernel<T, R, MODE, ROWS>), dim3(n_seq, g.H, (g.dv + cols - 1) / cols), dim3(nt), lds, st, g);
}

template <typename T, int MODE>
void dispatch_rows(const ScanArgs& g, int n_seq, hipStream_t st) {
  const int need = (g.dk + kRows - 1) / kRows;
  if (need <= 1) launch_scan<T, 1, MODE>(g, n_seq, st);
  else if (need <= 2) launch_scan<T, 2, MODE>(g, n_seq, st);
  else if (need <= 4) launch_scan<T, 4, MODE>(g, n_seq, st);
  else if (need <= 8) launch_scan<T, 8, MODE>(g, n_seq, st);
  else if (need <= 16) launch_scan<T, 16, MODE>(g, n_seq, st);
  else launch_scan<T, 16, MODE, kMaxKey / 16>(g, n_seq, st);
}

}  // namespace

extern "C" int dxm_linear_scan(int mode, float* out, float* state, int n_slots, const void* q, int64_t qs, const void* k,
                               int64_t ks, const void* v, int64_t vs, float q_scale, float k_scale, int qk_rep,
                               const float* decay, const void* gate, int64_t gs, const float* g_bias, const float* rate,
                               const float* skip, float inv_tau, const int64_t* pos, const int* seq_rows,
                               const int* slots, int n_seq, int T_, int H, int dk, int dv, int f32, hipStream_t st) {
  if (n_seq <= 0 || T_ <= 0) return 0;
  if (H < 1 || dk < 1 || dv < 1 || n_slots < 1 || H > 65535 || (int64_t)T_ * H * dv > 0x7fffffffffffLL) return 1;
  if (dk > kMaxKey) return 2;  // wider keys need more rows per lane than instantiated
  if (!out || !state || !pos || !slots || !q || !k || !v) return 3;
  if (!seq_rows && n_seq != T_) return 4;
  if (qk_rep < 1 || H % qk_rep) return 5;
  ScanArgs g{out, state, q, k, v, qs, ks, vs, q_scale, k_scale, qk_rep, decay, gate, gs, g_bias, rate, skip, inv_tau,
             pos, seq_rows, slots, n_slots, T_, H, dk, dv, 1, 0x7fffffff};
  // prompt portions in bf16: matrix-core chunks where the sizes fit; shorter runs of a sequence
  // (decode tokens among them) stay with the token scan
  if (!f32 && seq_rows && n_seq <= 65535 && T_ >= kChunkMinRows + n_seq - 1 && chunk_scan_ok(mode, g)) {
    if ((mode == kFixed && !decay) || (mode == kStep && (!gate || !rate)) || (mode == kChannel && !gate)) return 6;
    g.min_rows = kChunkMinRows;
    launch_chunk_scan(mode, g, n_seq, st);
    if (n_seq == 1) {
      DX_CHECK_LAUNCH();
      return 0;
    }
    g.max_rows = kChunkMinRows - 1;
  }
  if (mode == kFixed) {
    if (!decay) return 6;
    DISPATCH_T(f32, (dispatch_rows<T, kFixed>(g, n_seq, st)));
  } else if (mode == kStep) {
    if (!gate || !rate) return 6;
    DISPATCH_T(f32, (dispatch_rows<T, kStep>(g, n_seq, st)));
  } else if (mode == kChannel) {
    if (!gate) return 6;
    DISPATCH_T(f32, (dispatch_rows<T, kChannel>(g, n_seq, st)));
  } else {
    return 7;
  }
  DX_CHECK_LAUNCH();
  return 0;
}
