// Kernels with per-sequence state for gfx950: the generalized delta rule (a
// running matrix per head), short causal convolutions over time (bias and
// activation optional) fused with rotary positions and the paged cache write,
// the convolution tail update, and the norms + gates that follow a recurrent
// mixer.  (Linear recurrences without a removal term: linear_scan.hip.)
//
// State lives in slots ([slots, ...] tensors); a step names the slot of each of
// its sequences (state_slots [n_seq], -1: a padding row that touches nothing)
// and the first row of each (seq_rows [n_seq + 1]; null: row i is sequence i).
// Rows of a sequence are consecutive positions.  A sequence whose first row of
// the step is at position 0 starts from zero state, whatever its slot held.
//
// Every kernel is a template over the activation element (bf16 bits or float);
// decays, removal rates, unit keys, the running matrix, angles and all sums are
// fp32 whatever the element is.  Sizes are run-time arguments.
#include "recurrent.h"

namespace {

// ---------------------------------------------------------------------------
// Generalized delta rule.  Per (sequence, head) a matrix S [dk, dv]:
//     S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T,   o_t = S_t^T r_t
// with w_t = exp(-decay_scale * sigmoid(wl_t + w_bias)), a_t = sigmoid(al_t + a_bias),
// u_t = k_t / sqrt(sum(k_t^2) + key_eps).  Columns of S are independent, so a
// thread owns a tile of kRows consecutive rows x CT consecutive columns in
// registers (every row vector it reads from LDS serves CT columns), R
// neighbouring lanes share the columns and join their partial dot products by
// DPP lane exchanges (no LDS traffic), and a workgroup of NT threads owns
// NT / R * CT columns of one (sequence, head).  CT is 4 where the launch has
// waves to fill the chip twice over, else 2 or 1 (a few long prompts): a
// token's dependent chain leaves a lone wave on a SIMD waiting most of the
// time, so the launch wants at least two waves on every SIMD.  The
// state tensor is stored column-major per head ([slots, H, dv, dk]) so that a
// wave's state traffic is contiguous runs.  What the recurrence needs per
// token and key channel beside r and k -- the unit key u, the decay w and
// a * u -- is computed for all rows at once by delta_prep_kernel (fp32, [T, H,
// 3, dk]): it is elementwise work and would otherwise sit in the sequential
// chain.  Tokens are staged through LDS kTok at a time, fetched into registers
// one block ahead (the latency hides behind the current block's recurrence).

struct DeltaArgs {
  float* out;    // [T, H * dv]
  float* state;  // [slots, H, dv, dk]
  const void *r, *k, *v;
  int64_t rs, ks, vs;  // row strides (elements)
  const float* prep;   // [T, H, 3, dk]: unit key, decay, removal rate * unit key
  const int64_t* pos;
  const int* seq_rows;  // null: row i is sequence i
  const int* slots;
  int n_slots, T, H, dk, dv;
};

// one wave per (row, head): u = k / sqrt(sum k^2 + key_eps), w = exp(-decay_scale sigmoid(wl + w_bias)),
// a u with a = sigmoid(al + a_bias)
template <typename T>
__global__ void __launch_bounds__(64) delta_prep_kernel(float* __restrict__ prep, const T* __restrict__ k, int64_t ks,
                                                        const T* __restrict__ a, int64_t as, const T* __restrict__ w,
                                                        int64_t ws, const float* __restrict__ a_bias,
                                                        const float* __restrict__ w_bias, float decay_scale,
                                                        float key_eps, int H, int dk) {
  const int64_t v = blockIdx.x, row = v / H;
  const int h = (int)(v - row * H), lane = threadIdx.x;
  const T* kp = k + row * ks + (int64_t)h * dk;
  float ss = 0.f;
  for (int ch = lane; ch < dk; ch += 64) {
    const float x = ldf<T>(kp, ch);
    ss += x * x;
  }
  const float inv = rsqrtf(wave_reduce_sum(ss) + key_eps);
  float* o = prep + v * 3 * dk;
  for (int ch = lane; ch < dk; ch += 64) {
    const float u = ldf<T>(kp, ch) * inv;
    const float ab = a_bias ? a_bias[h * dk + ch] : 0.f, wb = w_bias ? w_bias[h * dk + ch] : 0.f;
    o[ch] = u;
    o[dk + ch] = expf(-decay_scale * sigmoidf_(ldf<T>(w, row * ws + (int64_t)h * dk + ch) + wb));
    o[2 * dk + ch] = sigmoidf_(ldf<T>(a, row * as + (int64_t)h * dk + ch) + ab) * u;
  }
}

template <typename T, int R, int NT, int CT>
__global__ void __launch_bounds__(NT) delta_rule_kernel(DeltaArgs g) {
  constexpr int kCols = CT;
  constexpr int kGroups = NT / R;            // column tiles per workgroup
  constexpr int kWgCols = kGroups * kCols;   // columns per workgroup
  constexpr int kDkp = kRows * R;            // padded key width
  constexpr int kE = (kTok * kDkp + NT - 1) / NT;  // staged elements per thread and array
  constexpr int kEv = (kTok * kWgCols + NT - 1) / NT;
  __shared__ __attribute__((aligned(16))) float sr[kTok][kDkp];
  __shared__ __attribute__((aligned(16))) float sk[kTok][kDkp];
  __shared__ __attribute__((aligned(16))) float su[kTok][kDkp];
  __shared__ __attribute__((aligned(16))) float sw[kTok][kDkp];
  __shared__ __attribute__((aligned(16))) float sa[kTok][kDkp];
  __shared__ __attribute__((aligned(16))) float sv[kTok][kWgCols];
  const int tid = threadIdx.x, part = tid % R, grp = tid / R;
  const int s = blockIdx.x, h = blockIdx.y, j0 = blockIdx.z * kWgCols + grp * kCols;
  const int r0 = g.seq_rows ? g.seq_rows[s] : s;
  const int r1 = g.seq_rows ? g.seq_rows[s + 1] : s + 1;
  const int slot = g.slots[s];
  const int n = r1 - r0;
  if (n <= 0 || r0 < 0 || r1 > g.T) return;
  if (slot < 0 || slot >= g.n_slots) {  // padding rows: a defined result, no state
    if (part == 0)
      for (int t = r0; t < r1; ++t)
        for (int c = 0; c < kCols; ++c)
          if (j0 + c < g.dv) g.out[(int64_t)t * g.H * g.dv + h * g.dv + j0 + c] = 0.f;
    return;
  }
  // The thread's 16 rows are four quads, quad m at row (m * R + part) * 4: for one m the R lanes of a
  // group read R consecutive 16-byte pieces of a row vector, so a wave's LDS read touches every bank once
  // (16 consecutive rows per lane would put lanes 0, 2, 4, .. on the same banks).
  float* sp = g.state + (((int64_t)slot * g.H + h) * g.dv) * g.dk;  // + column * dk + row
  const bool fresh = g.pos[r0] == 0;
  int rq[kRows / 4];
#pragma unroll
  for (int m = 0; m < kRows / 4; ++m) rq[m] = (m * R + part) * 4;
  float S[kCols][kRows];
#pragma unroll
  for (int c = 0; c < kCols; ++c) {
#pragma unroll
    for (int q = 0; q < kRows; ++q) S[c][q] = 0.f;
    if (fresh || j0 + c >= g.dv) continue;
    const float* spc = sp + (int64_t)(j0 + c) * g.dk;
#pragma unroll
    for (int m = 0; m < kRows / 4; ++m) {
      if (g.dk % 4 == 0 && rq[m] + 4 <= g.dk) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(spc + rq[m]);
        S[c][4 * m] = x[0], S[c][4 * m + 1] = x[1], S[c][4 * m + 2] = x[2], S[c][4 * m + 3] = x[3];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (rq[m] + e < g.dk) S[c][4 * m + e] = spc[rq[m] + e];
      }
    }
  }
  const T* pr = (const T*)g.r + (int64_t)h * g.dk;
  const T* pk = (const T*)g.k + (int64_t)h * g.dk;
  const float* pp = g.prep + (int64_t)h * 3 * g.dk;
  const T* pv = (const T*)g.v + (int64_t)h * g.dv + blockIdx.z * kWgCols;
  float fr[kE], fk[kE], fu[kE], fa[kE], fw[kE], fv[kEv];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int e = 0; e < kE; ++e) {
      const int idx = tid + e * NT, tt = idx / kDkp, ch = idx % kDkp;
      const bool ok = idx < kTok * kDkp && t0 + tt < n && ch < g.dk;
      const int64_t row = r0 + t0 + tt;
      const float* pq = pp + row * g.H * 3 * g.dk + ch;
      fr[e] = ok ? ldf<T>(pr, row * g.rs + ch) : 0.f;
      fk[e] = ok ? ldf<T>(pk, row * g.ks + ch) : 0.f;
      fu[e] = ok ? pq[0] : 0.f;
      fw[e] = ok ? pq[g.dk] : 0.f;
      fa[e] = ok ? pq[2 * g.dk] : 0.f;
    }
#pragma unroll
    for (int e = 0; e < kEv; ++e) {
      const int idx = tid + e * NT, tt = idx / kWgCols, cc = idx % kWgCols;
      const bool ok = idx < kTok * kWgCols && t0 + tt < n && blockIdx.z * kWgCols + cc < g.dv;
      fv[e] = ok ? ldf<T>(pv, (int64_t)(r0 + t0 + tt) * g.vs + cc) : 0.f;
    }
  };
  fetch(0);
  float* outp = g.out + (int64_t)r0 * g.H * g.dv + h * g.dv + j0;
  const bool out4 = g.dv % 4 == 0 && j0 + kCols <= g.dv;
  for (int t0 = 0; t0 < n; t0 += kTok) {
    __syncthreads();  // the previous block's tokens are consumed
#pragma unroll
    for (int e = 0; e < kE; ++e) {
      const int idx = tid + e * NT, tt = idx / kDkp, ch = idx % kDkp;
      if (idx < kTok * kDkp) {
        sr[tt][ch] = fr[e];
        sk[tt][ch] = fk[e];
        su[tt][ch] = fu[e];
        sw[tt][ch] = fw[e];
        sa[tt][ch] = fa[e];
      }
    }
#pragma unroll
    for (int e = 0; e < kEv; ++e) {
      const int idx = tid + e * NT;
      if (idx < kTok * kWgCols) sv[idx / kWgCols][idx % kWgCols] = fv[e];
    }
    __syncthreads();
    if (t0 + kTok < n) fetch(t0 + kTok);
    const int nt = n - t0 < kTok ? n - t0 : kTok;
    // the five row vectors of a token (unit key, decay, removal, key, read-out) and its values
    auto load = [&](int tt, float (*b)[kRows], float* vj) {
#pragma unroll
      for (int q = 0; q < kRows; q += 4) {
        *reinterpret_cast<f32x4*>(b[0] + q) = *reinterpret_cast<const f32x4*>(&su[tt][rq[q / 4]]);
        *reinterpret_cast<f32x4*>(b[1] + q) = *reinterpret_cast<const f32x4*>(&sw[tt][rq[q / 4]]);
        *reinterpret_cast<f32x4*>(b[2] + q) = *reinterpret_cast<const f32x4*>(&sa[tt][rq[q / 4]]);
        *reinterpret_cast<f32x4*>(b[3] + q) = *reinterpret_cast<const f32x4*>(&sk[tt][rq[q / 4]]);
        *reinterpret_cast<f32x4*>(b[4] + q) = *reinterpret_cast<const f32x4*>(&sr[tt][rq[q / 4]]);
      }
#pragma unroll
      for (int c = 0; c < kCols; ++c) vj[c] = sv[tt][grp * kCols + c];
    };
    auto step = [&](const float (*b)[kRows], const float* vj, float* o_) {
      float us[kCols];
#pragma unroll
      for (int c = 0; c < kCols; ++c) {
        float a_ = 0.f;
#pragma unroll
        for (int q = 0; q < kRows; ++q) a_ += b[0][q] * S[c][q];
        us[c] = group_sum<R>(a_);
      }
#pragma unroll
      for (int c = 0; c < kCols; ++c) {
        float a_ = 0.f;
#pragma unroll
        for (int q = 0; q < kRows; ++q) {
          S[c][q] = S[c][q] * b[1][q] - b[2][q] * us[c] + b[3][q] * vj[c];
          a_ += b[4][q] * S[c][q];
        }
        o_[c] = group_sum<R>(a_);
      }
    };
    auto store = [&](int tt, const float* o_) {
      float* op = outp + (int64_t)(t0 + tt) * g.H * g.dv;
      if constexpr (kCols == 4) {
        if (out4) *reinterpret_cast<f32x4*>(op) = f32x4{o_[0], o_[1], o_[2], o_[3]};
      }
      if (kCols != 4 || !out4) {
#pragma unroll
        for (int c = 0; c < kCols; ++c)
          if (j0 + c < g.dv) op[c] = o_[c];
      }
    };
    if (kCols <= 2 && nt == kTok) {
      // a whole block of the narrow tile (the wide one has no registers to spare), unrolled in one basic
      // block: the next token's vectors are read from LDS while the current token's chain runs, and the
      // outputs are stored once at the end
      float b0[5][kRows], b1[5][kRows], v0[kCols], v1[kCols], ob[kTok][kCols];
      load(0, b0, v0);
#pragma unroll
      for (int tt = 0; tt < kTok; tt += 2) {
        load(tt + 1, b1, v1);
        step(b0, v0, ob[tt]);
        if (tt + 2 < kTok) load(tt + 2, b0, v0);
        step(b1, v1, ob[tt + 1]);
      }
      if (part == 0) {
#pragma unroll
        for (int tt = 0; tt < kTok; ++tt) store(tt, ob[tt]);
      }
    } else {
      for (int tt = 0; tt < nt; ++tt) {
        float b0[5][kRows], v0[kCols], o_[kCols];
        load(tt, b0, v0);
        step(b0, v0, o_);
        if (part == 0) store(tt, o_);
      }
    }
  }
#pragma unroll
  for (int c = 0; c < kCols; ++c) {
    if (j0 + c >= g.dv) continue;
    float* spc = sp + (int64_t)(j0 + c) * g.dk;
#pragma unroll
    for (int m = 0; m < kRows / 4; ++m) {
      if (g.dk % 4 == 0 && rq[m] + 4 <= g.dk) {
        *reinterpret_cast<f32x4*>(spc + rq[m]) = f32x4{S[c][4 * m], S[c][4 * m + 1], S[c][4 * m + 2], S[c][4 * m + 3]};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (rq[m] + e < g.dk) spc[rq[m] + e] = S[c][4 * m + e];
      }
    }
  }
}

// NT threads per workgroup: 64 where that covers all columns of a head, else 256.  Columns per
// thread: the widest tile that still gives the launch two waves per SIMD (2048 on the chip) -- a
// token's chain leaves a lone wave waiting most of the time -- down to one column for a few long prompts.
template <typename T, int R, int CT>
void launch_delta_ct(const DeltaArgs& g, int n_seq, hipStream_t st) {
  const int need = R * ((g.dv + CT - 1) / CT);
  if constexpr (R < 16) {  // (a single wave staging 256 key channels would spill its registers)
    if (need <= 64) {
      hipLaunchKernelGGL((delta_rule_kernel<T, R, 64, CT>), dim3(n_seq, g.H, 1), dim3(64), 0, st, g);
      return;
    }
  }
  {
    const int cols = 256 / R * CT;
    hipLaunchKernelGGL((delta_rule_kernel<T, R, 256, CT>), dim3(n_seq, g.H, (g.dv + cols - 1) / cols), dim3(256), 0,
                       st, g);
  }
}
template <typename T, int R>
void launch_delta(const DeltaArgs& g, int n_seq, hipStream_t st) {
  const int64_t waves4 = (int64_t)n_seq * g.H * ((R * ((g.dv + 3) / 4) + 63) / 64);
  if (waves4 >= 2048) launch_delta_ct<T, R, 4>(g, n_seq, st);
  else if (waves4 >= 1024) launch_delta_ct<T, R, 2>(g, n_seq, st);
  else launch_delta_ct<T, R, 1>(g, n_seq, st);
}

// ---------------------------------------------------------------------------
// Short causal convolution over time on the leading C = n_q d + n_k (d + dv)
// columns of a fused projection (plus a bias and silu where given), then rotary positions on the first 2 * half
// columns of every q and k head (column i paired with i + half), q to its own
// tensor, k and v into the paged caches.  y_t = sum_j cw[j][c] u_(t - taps + 1 + j);
// u at positions before the step's first row of the sequence comes from the
// sequence's tail state [taps - 1, C], and is zero before position 0.
struct ConvArgs {
  void* q_out;  // [T, n_q * d]
  const void* x;
  int64_t xs;
  const float* cw;  // [taps, C] (tap-major: a run of channels shares a load)
  const float* cb;  // [C] bias or null
  int silu;         // silu after the convolution (in front of the rotation)
  int taps;
  const void* tail;  // [slots, taps - 1, C]
  int n_slots;
  const int64_t* pos;
  const int64_t* kv_slots;
  const int* row_seq;   // null (with seq_rows null): row i is sequence i
  const int* seq_rows;
  const int* slots;
  int n_seq, T, n_q, n_k, d, dv;
  const float* inv_freq;  // [half]
  int half;
  void* kc;
  void* vc;
};

template <typename T>
__global__ void __launch_bounds__(256) conv_rope_cache_kernel(ConvArgs g) {
  const int t = blockIdx.x;
  const int C = g.n_q * g.d + g.n_k * (g.d + g.dv);
  const int s = g.row_seq ? g.row_seq[t] : t;
  const bool seq_ok = s >= 0 && s < g.n_seq;
  const int r0 = !seq_ok ? t : (g.seq_rows ? g.seq_rows[s] : t);
  const int slot = seq_ok ? g.slots[s] : -1;
  const bool live = slot >= 0 && slot < g.n_slots && r0 >= 0 && r0 <= t;
  const int64_t p = g.pos[t];
  const int64_t p0 = p - (t - r0);  // position of the step's first row of this sequence
  const int m = g.taps - 1;
  const T* x = (const T*)g.x;
  const T* tail = (const T*)g.tail + (int64_t)(live ? slot : 0) * m * C;
  auto conv = [&](int c) -> float {
    float y = g.cb ? g.cb[c] : 0.f;
    for (int jj = 0; jj < g.taps; ++jj) {
      const int64_t qp = p - m + jj;
      float u = 0.f;
      if (qp >= p0) u = ldf<T>(x, (int64_t)(r0 + (qp - p0)) * g.xs + c);
      else if (qp >= 0) u = ldf<T>(tail, (qp - p0 + m) * C + c);
      y += g.cw[(int64_t)jj * C + c] * u;
    }
    return g.silu ? y * sigmoidf_(y) : y;
  };
  // the row's angles: one cosine and sine per rotated pair, shared by all heads
  extern __shared__ float cs_sn[];  // [half] cosines, [half] sines
  for (int i = threadIdx.x; i < g.half; i += blockDim.x) sincosf((float)p * g.inv_freq[i], &cs_sn[g.half + i], &cs_sn[i]);
  __syncthreads();
  const int qk = (g.n_q + g.n_k) * g.d;
  const int64_t kvs = g.kv_slots[t];
  for (int c = threadIdx.x; c < C; c += blockDim.x) {
    float y = live ? conv(c) : 0.f;
    if (c < qk) {
      const int e = c % g.d;
      if (live && e < 2 * g.half) {
        const int i = e < g.half ? e : e - g.half;
        const float other = conv(e < g.half ? c + g.half : c - g.half);
        const float cs = cs_sn[i], sn = cs_sn[g.half + i];
        y = e < g.half ? y * cs - other * sn : y * cs + other * sn;
      }
      if (c < g.n_q * g.d) stf<T>((T*)g.q_out, (int64_t)t * g.n_q * g.d + c, y);
      else if (kvs >= 0 && live) stf<T>((T*)g.kc, kvs * (g.n_k * g.d) + (c - g.n_q * g.d), y);
    } else if (kvs >= 0 && live) {
      stf<T>((T*)g.vc, kvs * (g.n_k * g.dv) + (c - qk), y);
    }
  }
}

// The same on V consecutive channels per thread with 16-byte loads and stores (V = 8 bf16 or
// 4 fp32): a thread takes a run of the low rotary half together with its partner run of the
// high half, so every channel is convolved once and every angle evaluated once.  Needs d, dv,
// half, the row stride and the cache widths to be multiples of V, and 16-byte aligned bases.
// A workgroup takes kConvRows consecutive rows of the step (they may belong to different
// sequences); the taps loop is outermost, so a thread loads a tap's weights once for all its rows.
constexpr int kConvRows = 4;
template <typename T, int V>
__global__ void __launch_bounds__(128) conv_rope_cache_vec_kernel(ConvArgs g) {
  const int t0 = blockIdx.x * kConvRows;
  const int C = g.n_q * g.d + g.n_k * (g.d + g.dv);
  const int m = g.taps - 1;
  const T* x = (const T*)g.x;
  // per row: liveness, position, first position of its sequence in the step, first row, tail, cache slot
  bool live[kConvRows];
  int64_t p[kConvRows], p0[kConvRows], kvs[kConvRows];
  int r0[kConvRows];
  const T* tail[kConvRows];
#pragma unroll
  for (int r = 0; r < kConvRows; ++r) {
    const int t = t0 + r < g.T ? t0 + r : g.T - 1;
    const int s = g.row_seq ? g.row_seq[t] : t;
    const bool seq_ok = s >= 0 && s < g.n_seq;
    r0[r] = !seq_ok ? t : (g.seq_rows ? g.seq_rows[s] : t);
    const int slot = seq_ok ? g.slots[s] : -1;
    live[r] = t0 + r < g.T && slot >= 0 && slot < g.n_slots && r0[r] >= 0 && r0[r] <= t;
    p[r] = g.pos[t];
    p0[r] = p[r] - (t - r0[r]);
    tail[r] = (const T*)g.tail + (int64_t)(live[r] ? slot : 0) * m * C;
    kvs[r] = live[r] ? g.kv_slots[t] : -1;
  }
  extern __shared__ float cs_sn[];  // per row [half] cosines, [half] sines of its angles
  for (int i = threadIdx.x; i < kConvRows * g.half; i += blockDim.x) {
    const int r = i / g.half, e = i - r * g.half;
    sincosf((float)p[r] * g.inv_freq[e], &cs_sn[(2 * r + 1) * g.half + e], &cs_sn[2 * r * g.half + e]);
  }
  __syncthreads();
  const int qk = (g.n_q + g.n_k) * g.d, nq = g.n_q * g.d;
  auto put = [&](int r, int c, const float* y) {
    if (t0 + r >= g.T) return;
    if (c < nq) VecIO<T, V>::st((T*)g.q_out + (int64_t)(t0 + r) * nq + c, y);
    else if (kvs[r] < 0) return;
    else if (c < qk) VecIO<T, V>::st((T*)g.kc + kvs[r] * (g.n_k * g.d) + (c - nq), y);
    else VecIO<T, V>::st((T*)g.vc + kvs[r] * (g.n_k * g.dv) + (c - qk), y);
  };
  // work items: per q / k head its rotated pairs of runs (a run of the low half with its partner of
  // the high half), then its runs that are not rotated; then the runs of v
  const int n_pair = g.half / V, per_head = n_pair + (g.d - 2 * g.half) / V;
  const int n_head_items = (g.n_q + g.n_k) * per_head, n_items = n_head_items + (C - qk) / V;
  for (int it = threadIdx.x; it < n_items; it += blockDim.x) {
    int c, e;
    bool pair = false;
    if (it < n_head_items) {
      const int hd = it / per_head, j = it - hd * per_head;
      pair = j < n_pair;
      e = pair ? j * V : 2 * g.half + (j - n_pair) * V;
      c = hd * g.d + e;
    } else {
      e = 0;
      c = qk + (it - n_head_items) * V;
    }
    float y[kConvRows][V], z[kConvRows][V];
#pragma unroll
    for (int i = 0; i < V; ++i) {
      const float b = g.cb ? g.cb[c + i] : 0.f, b2 = g.cb && pair ? g.cb[c + g.half + i] : 0.f;
#pragma unroll
      for (int r = 0; r < kConvRows; ++r) y[r][i] = live[r] ? b : 0.f, z[r][i] = live[r] ? b2 : 0.f;
    }
    for (int jj = 0; jj < g.taps; ++jj) {
      float w[V], w2[V];
      const float* wp = g.cw + (int64_t)jj * C + c;
#pragma unroll
      for (int i = 0; i < V; i += 4) *reinterpret_cast<f32x4*>(w + i) = *reinterpret_cast<const f32x4*>(wp + i);
      if (pair) {
#pragma unroll
        for (int i = 0; i < V; i += 4)
          *reinterpret_cast<f32x4*>(w2 + i) = *reinterpret_cast<const f32x4*>(wp + g.half + i);
      }
#pragma unroll
      for (int r = 0; r < kConvRows; ++r) {
        const int64_t qp = p[r] - m + jj;
        if (!live[r] || qp < 0) continue;
        const T* src = qp >= p0[r] ? x + (int64_t)(r0[r] + (qp - p0[r])) * g.xs + c : tail[r] + (qp - p0[r] + m) * C + c;
        float u[V];
        VecIO<T, V>::ld(src, u);
#pragma unroll
        for (int i = 0; i < V; ++i) y[r][i] += w[i] * u[i];
        if (pair) {
          VecIO<T, V>::ld(src + g.half, u);
#pragma unroll
          for (int i = 0; i < V; ++i) z[r][i] += w2[i] * u[i];
        }
      }
    }
#pragma unroll
    for (int r = 0; r < kConvRows; ++r) {
      if (g.silu) {
#pragma unroll
        for (int i = 0; i < V; ++i) {
          y[r][i] *= sigmoidf_(y[r][i]);
          if (pair) z[r][i] *= sigmoidf_(z[r][i]);
        }
      }
      if (pair) {
        float lo[V], hi[V];
        const float* cs = cs_sn + 2 * r * g.half + e;
        const float* sn = cs + g.half;
#pragma unroll
        for (int i = 0; i < V; ++i) {
          lo[i] = y[r][i] * cs[i] - z[r][i] * sn[i];
          hi[i] = z[r][i] * cs[i] + y[r][i] * sn[i];
        }
        put(r, c, lo);
        put(r, c + g.half, hi);
      } else {
        put(r, c, y[r]);
      }
    }
  }
}

// The convolution alone (no heads, no rotation, no cache) with the taps known at compile time: a thread
// walks V neighbouring channels down R consecutive rows of the step with the last TAPS - 1 inputs in
// registers, so an input row is read once (and its TAPS - 1 predecessors at the start of a run).  The inputs
// before a run's or a sequence's first row come from the step's earlier rows or from the tail state.
// R = 1 with one row per sequence (a decode step) also writes the new tail: the thread holds all of it.
template <typename T, int V, int TAPS, int R>
__global__ void __launch_bounds__(128) conv_run_kernel(ConvArgs g, T* __restrict__ new_tail) {
  constexpr int M = TAPS - 1;
  const int C = g.d, c = (blockIdx.x * 128 + threadIdx.x) * V, t0 = blockIdx.y * R;
  if (c >= C) return;
  const T* x = (const T*)g.x + c;
  raw_u32x4 in[R];
  float h[M > 0 ? M : 1][V], w[TAPS][V], b[V];
#pragma unroll
  for (int i = 0; i < R; ++i)
    if (t0 + i < g.T) in[i] = *reinterpret_cast<const raw_u32x4*>(x + (int64_t)(t0 + i) * g.xs);
#pragma unroll
  for (int j = 0; j < TAPS; ++j)
#pragma unroll
    for (int e = 0; e < V; e += 4) VecIO<float, 4>::ld(g.cw + (int64_t)j * C + c + e, w[j] + e);
#pragma unroll
  for (int e = 0; e < V; ++e) b[e] = g.cb ? g.cb[c + e] : 0.f;
  auto seq_of = [&](int t) { return g.row_seq ? g.row_seq[t] : t; };
  int s = seq_of(t0), slot = -1;
  const bool one = R == 1 || (t0 + R <= g.T && seq_of(t0 + R - 1) == s);  // the run lies in one sequence
  bool live = false;
  auto enter = [&](int t) {  // row t begins a run of sequence s: its slot, and the inputs in front of it
    const bool seq_ok = s >= 0 && s < g.n_seq;
    slot = seq_ok ? g.slots[s] : -1;
    const int r0 = seq_ok ? (g.seq_rows ? g.seq_rows[s] : t) : t;
    live = slot >= 0 && slot < g.n_slots && r0 >= 0 && r0 <= t;
    if (M == 0 || !live) return;
    const T* tl = (const T*)g.tail + (int64_t)slot * M * C + c;
    const int64_t p = g.pos[t];
#pragma unroll
    for (int m = 0; m < M; ++m) {  // h[m]: the input at position p - M + m
      const int back = M - m, rel = t - r0 - back;  // its row in this step's run of the sequence
#pragma unroll
      for (int e = 0; e < V; ++e) h[m][e] = 0.f;
      if (p >= back) VecIO<T, V>::ld(rel >= 0 ? x + (int64_t)(r0 + rel) * g.xs : tl + (int64_t)(rel + M) * C, h[m]);
    }
  };
  enter(t0);
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int t = t0 + i;
    if (t >= g.T) break;
    if (i > 0 && !one) {
      const int s2 = seq_of(t);
      if (s2 != s) {
        s = s2;
        enter(t);
      }
    }
    float xi[V], y[V];
    chunk_to_f32<T>(in[i], xi);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      float a = b[e];
#pragma unroll
      for (int m = 0; m < M; ++m) a += w[m][e] * h[m][e];
      a += w[M][e] * xi[e];
      if (g.silu) a *= fast_sigmoid(a);
      y[e] = live ? a : 0.f;
    }
    VecIO<T, V>::st((T*)g.q_out + (int64_t)t * C + c, y);
    if constexpr (M > 0) {
#pragma unroll
      for (int m = 0; m + 1 < M; ++m)
#pragma unroll
        for (int e = 0; e < V; ++e) h[m][e] = h[m + 1][e];
#pragma unroll
      for (int e = 0; e < V; ++e) h[M - 1][e] = xi[e];
      if (R == 1 && new_tail && live) {
#pragma unroll
        for (int m = 0; m < M; ++m) VecIO<T, V>::st(new_tail + ((int64_t)slot * M + m) * C + c, h[m]);
      }
    }
  }
}

template <typename T, int V, int TAPS> void launch_conv_run(const ConvArgs& g, hipStream_t st) {
  const int gx = (g.d / V + 127) / 128;
  if (!g.row_seq)
    hipLaunchKernelGGL((conv_run_kernel<T, V, TAPS, 1>), dim3(gx, g.T), dim3(128), 0, st, g, (T*)g.tail);
  else
    hipLaunchKernelGGL((conv_run_kernel<T, V, TAPS, 8>), dim3(gx, (g.T + 7) / 8), dim3(128), 0, st, g, (T*)nullptr);
}

// tail [slots, m, C] <- the last m projected rows of every sequence of the step
template <typename T>
__global__ void __launch_bounds__(256) conv_state_update_kernel(T* __restrict__ tail, int n_slots,
                                                                const T* __restrict__ x, int64_t xs,
                                                                const int64_t* __restrict__ pos,
                                                                const int* __restrict__ seq_rows,
                                                                const int* __restrict__ slots, int T_, int C, int m) {
  const int s = blockIdx.x;
  const int r0 = seq_rows ? seq_rows[s] : s, r1 = seq_rows ? seq_rows[s + 1] : s + 1;
  const int slot = slots[s];
  const int n = r1 - r0;
  if (slot < 0 || slot >= n_slots || n <= 0 || r0 < 0 || r1 > T_) return;
  const int64_t p0 = pos[r0];
  T* ts = tail + (int64_t)slot * m * C;
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < C; c += gridDim.y * blockDim.x) {
    // new[i] is the step-relative row n - m + i: a row of x, or an old entry shifted down.
    // Ascending i reads old entries at i + n > i only, so a thread may overwrite as it goes.
    for (int i = 0; i < m; ++i) {
      const int rel = n - m + i;
      T val;
      if (rel >= 0) val = x[(int64_t)(r0 + rel) * xs + c];
      else if (p0 + rel >= 0) val = ts[(int64_t)(i + n) * C + c];
      else val = (T)0;
      ts[(int64_t)i * C + c] = val;
    }
  }
}

// out = o / sqrt(mean_head(o^2) + eps) * w * sigmoid(gate) (or * silu(gate)): one wave per (row, head), four per workgroup;
// a lane keeps its elements (V neighbours at a time, up to kHnKeep times) in registers between the mean
// square and the result.  V = 2 needs an even dv and gate stride and 8-byte aligned o and w.
constexpr int kHnKeep = 4;
template <typename T, int V>
__global__ void __launch_bounds__(256) head_norm_gate_kernel(T* __restrict__ out, const float* __restrict__ o,
                                                             const float* __restrict__ w, const T* __restrict__ gate,
                                                             int64_t gs, int64_t n_vec, int H, int dv, float eps,
                                                             int gate_act) {
  const int lane = threadIdx.x & 63;
  const int64_t v = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (v >= n_vec) return;
  const int64_t row = v / H;
  const int h = (int)(v - row * H);
  const float* op = o + v * dv;
  auto ldo = [&](int e, float* x) {
    if constexpr (V == 2) {
      const float2 t = *reinterpret_cast<const float2*>(op + e);
      x[0] = t.x, x[1] = t.y;
    } else {
      x[0] = op[e];
    }
  };
  float x[kHnKeep][V], ss = 0.f;
#pragma unroll
  for (int k = 0; k < kHnKeep; ++k) {
    const int e = (lane + 64 * k) * V;
#pragma unroll
    for (int i = 0; i < V; ++i) x[k][i] = 0.f;
    if (e < dv) ldo(e, x[k]);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += x[k][i] * x[k][i];
  }
  for (int e = (lane + 64 * kHnKeep) * V; e < dv; e += 64 * V) {
    float t[V];
    ldo(e, t);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += t[i] * t[i];
  }
  const float inv = rsqrtf(wave_reduce_sum(ss) / (float)dv + eps);
  auto put = [&](int e, const float* xv) {
    float y[V];
#pragma unroll
    for (int i = 0; i < V; ++i) {
      y[i] = xv[i] * inv;
      if (w) y[i] *= w[h * dv + e + i];
      if (gate) {  // gate_act 0: sigmoid(z); 1: silu, z sigmoid(z)
        const float z = ldf<T>(gate, row * gs + h * dv + e + i);
        y[i] *= gate_act ? z * fast_sigmoid(z) : fast_sigmoid(z);
      }
    }
    if constexpr (V == 2 && sizeof(T) == 2) {
      *reinterpret_cast<uint32_t*>((bf16_t*)out + v * dv + e) = pack_bf16x2(y[0], y[1]);
    } else {
#pragma unroll
      for (int i = 0; i < V; ++i) stf<T>(out, v * dv + e + i, y[i]);
    }
  };
#pragma unroll
  for (int k = 0; k < kHnKeep; ++k)
    if ((lane + 64 * k) * V < dv) put((lane + 64 * k) * V, x[k]);
  for (int e = (lane + 64 * kHnKeep) * V; e < dv; e += 64 * V) {
    float t[V];
    ldo(e, t);
    put(e, t);
  }
}

// The same for heads of up to 256 elements in whole runs of four: LPH neighbouring lanes (a power of two)
// share a head, four elements each, so a wave works on 64 / LPH heads with 16-byte accesses.
template <typename T, int LPH>
__global__ void __launch_bounds__(256) head_norm_gate_vec_kernel(T* __restrict__ out, const float* __restrict__ o,
                                                                 const float* __restrict__ w, const T* __restrict__ gate,
                                                                 int64_t gs, int64_t n_vec, int H, int dv, float eps,
                                                                 int gate_act) {
  const int64_t v = (int64_t)blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const int e = (threadIdx.x % LPH) * 4;
  if (v >= n_vec) return;  // (whole lane groups)
  const bool on = e < dv;
  const int64_t row = v / H;
  const int c = (int)(v - row * H) * dv + e;  // column of the row
  f32x4 x{0.f, 0.f, 0.f, 0.f};
  float z[4] = {0.f, 0.f, 0.f, 0.f};
  if (on) {
    x = *reinterpret_cast<const f32x4*>(o + v * dv + e);
    if (gate) {
      if constexpr (sizeof(T) == 2) {
        const uint2 t = *reinterpret_cast<const uint2*>((const bf16_t*)gate + row * gs + c);
        z[0] = bf16lo(t.x), z[1] = bf16hi(t.x), z[2] = bf16lo(t.y), z[3] = bf16hi(t.y);
      } else {
        VecIO<float, 4>::ld((const float*)gate + row * gs + c, z);
      }
    }
  }
  float ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
#pragma unroll
  for (int m = LPH / 2; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
  const float inv = rsqrtf(ss / (float)dv + eps);
  if (!on) return;
  float y[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    y[i] = x[i] * inv;
    if (w) y[i] *= w[c + i];
    if (gate) y[i] *= gate_act ? z[i] * fast_sigmoid(z[i]) : fast_sigmoid(z[i]);
  }
  if constexpr (sizeof(T) == 2)
    *reinterpret_cast<uint2*>((bf16_t*)out + v * dv + e) = uint2{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
  else
    VecIO<float, 4>::st((float*)out + v * dv + e, y);
}

template <typename T, int LPH>
void launch_head_norm_vec(void* out, const float* o, const float* w, const void* gate, int64_t gs, int64_t n_vec, int H,
                          int dv, float eps, int gate_act, hipStream_t st) {
  const int per = 256 / LPH;
  hipLaunchKernelGGL((head_norm_gate_vec_kernel<T, LPH>), dim3((unsigned)((n_vec + per - 1) / per)), dim3(256), 0, st,
                     (T*)out, o, w, (const T*)gate, gs, n_vec, H, dv, eps, gate_act);
}

// out = y silu(z), divided by the root mean square of its group (n equal groups of the row, eps inside the
// root), times w: the gate enters in front of the norm.  One workgroup per (row, group); a thread keeps its
// elements (V neighbours at a time, up to kGnKeep times) in registers between the mean square and the result.
// GATE 1, 2: the gate enters behind the norm instead (sigmoid(z) or silu(z); no z: none), for head norms whose
// heads are wider than a wave's registers.
constexpr int kGnKeep = 4;
template <typename T, int V, int NT, int GATE>
__global__ void __launch_bounds__(NT) gate_group_norm_kernel(T* __restrict__ out, int64_t os,
                                                             const float* __restrict__ y, const T* __restrict__ z,
                                                             int64_t zs, const float* __restrict__ w, int n_groups,
                                                             int n, float eps) {
  __shared__ float red[16];
  const int64_t row = blockIdx.x / n_groups;
  const int c0 = (int)(blockIdx.x - row * n_groups) * n;
  const float* yp = y + row * (int64_t)n_groups * n + c0;
  const T* zp = z + row * zs + c0;
  auto load = [&](int e, float* x) {
    if constexpr (V == 1) {
      x[0] = yp[e];
    } else {
#pragma unroll
      for (int i = 0; i < V; i += 4) VecIO<float, 4>::ld(yp + e + i, x + i);
    }
    if constexpr (GATE == 0) {
      float b[V];
      if constexpr (V == 1) b[0] = ldf<T>(zp, e);
      else VecIO<T, V>::ld(zp + e, b);
#pragma unroll
      for (int i = 0; i < V; ++i) x[i] *= b[i] * fast_sigmoid(b[i]);
    }
  };
  float x[kGnKeep][V], ss = 0.f;
#pragma unroll
  for (int k = 0; k < kGnKeep; ++k) {
    const int e = (threadIdx.x + NT * k) * V;
#pragma unroll
    for (int i = 0; i < V; ++i) x[k][i] = 0.f;
    if (e < n) load(e, x[k]);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += x[k][i] * x[k][i];
  }
  for (int e = (threadIdx.x + NT * kGnKeep) * V; e < n; e += NT * V) {
    float t[V];
    load(e, t);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += t[i] * t[i];
  }
  const float inv = rsqrtf(block_reduce_sum(ss, red) / (float)n + eps);
  auto put = [&](int e, const float* xv) {
    float o[V];
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] = xv[i] * inv * (w ? w[c0 + e + i] : 1.f);
    if constexpr (GATE != 0) {
      if (z) {
        float b[V];
        if constexpr (V == 1) b[0] = ldf<T>(zp, e);
        else VecIO<T, V>::ld(zp + e, b);
#pragma unroll
        for (int i = 0; i < V; ++i) o[i] *= GATE == 2 ? b[i] * fast_sigmoid(b[i]) : fast_sigmoid(b[i]);
      }
    }
    if constexpr (V == 1) stf<T>(out, row * os + c0 + e, o[0]);
    else VecIO<T, V>::st(out + row * os + c0 + e, o);
  };
#pragma unroll
  for (int k = 0; k < kGnKeep; ++k)
    if ((int)(threadIdx.x + NT * k) * V < n) put((threadIdx.x + NT * k) * V, x[k]);
  for (int e = (threadIdx.x + NT * kGnKeep) * V; e < n; e += NT * V) {
    float t[V];
    load(e, t);
    put(e, t);
  }
}

template <typename T, int V, int GATE = 0>
void launch_gate_group_norm(void* out, int64_t os, const float* y, const void* z, int64_t zs, const float* w, int rows,
                            int n_groups, int n, float eps, hipStream_t st) {
  const dim3 grid((unsigned)((int64_t)rows * n_groups));
  if (n > 64 * V)
    hipLaunchKernelGGL((gate_group_norm_kernel<T, V, 256, GATE>), grid, dim3(256), 0, st, (T*)out, os, y, (const T*)z, zs, w,
                       n_groups, n, eps);
  else
    hipLaunchKernelGGL((gate_group_norm_kernel<T, V, 64, GATE>), grid, dim3(64), 0, st, (T*)out, os, y, (const T*)z, zs, w,
                       n_groups, n, eps);
}

}  // namespace

extern "C" {

int dxm_delta_rule(float* out, float* state, int n_slots, float* prep, const void* r, int64_t rs, const void* k,
                   int64_t ks, const void* v, int64_t vs, const void* a, int64_t as, const void* w, int64_t ws,
                   const float* a_bias, const float* w_bias, float decay_scale, float key_eps, const int64_t* pos,
                   const int* seq_rows, const int* slots, int n_seq, int T_, int H, int dk, int dv, int f32,
                   hipStream_t st) {
  if (n_seq <= 0 || T_ <= 0) return 0;
  if (H < 1 || dk < 1 || dv < 1 || n_slots < 1 || H > 65535 || n_seq > 0x7fffffff || (int64_t)T_ * H > 0x7fffffff)
    return 1;
  if (dk > kRows * 16) return 2;  // wider keys need more lanes per column than instantiated
  if (!out || !state || !pos || !slots || !prep) return 3;
  if (!seq_rows && n_seq != T_) return 4;
  DISPATCH_T(f32, hipLaunchKernelGGL(delta_prep_kernel<T>, dim3((unsigned)(T_ * H)), dim3(64), 0, st, prep, (const T*)k,
                                     ks, (const T*)a, as, (const T*)w, ws, a_bias, w_bias, decay_scale, key_eps, H, dk));
  DeltaArgs g{out, state, r, k, v, rs, ks, vs, prep, pos, seq_rows, slots, n_slots, T_, H, dk, dv};
  const int need = (dk + kRows - 1) / kRows;
  if (need <= 4) { DISPATCH_T(f32, (launch_delta<T, 4>(g, n_seq, st))); }
  else if (need <= 8) { DISPATCH_T(f32, (launch_delta<T, 8>(g, n_seq, st))); }
  else { DISPATCH_T(f32, (launch_delta<T, 16>(g, n_seq, st))); }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_conv_rope_cache(void* q_out, const void* x, int64_t xs, const float* cw, const float* cb, int silu, int taps,
                        const void* tail,
                        int n_slots, const int64_t* pos, const int64_t* kv_slots, const int* row_seq,
                        const int* seq_rows, const int* slots, int n_seq, int T_, int n_q, int n_k, int d, int dv,
                        const float* inv_freq, int half, void* kc, void* vc, int f32, hipStream_t st) {
  if (T_ <= 0) return 0;
  if (taps < 1 || n_q < 0 || n_k < 0 || d < 1 || dv < 0 || half < 0 || 2 * half > d || half > 4096) return 1;
  if ((half && !inv_freq) || (n_k && (!kc || !vc)) || (taps > 1 && !tail) || !cw || !pos || !kv_slots || !slots)
    return 2;
  if ((row_seq == nullptr) != (seq_rows == nullptr) || (!row_seq && n_seq != T_)) return 3;
  ConvArgs g{q_out, x, xs, cw, cb, silu, taps, tail, n_slots, pos, kv_slots, row_seq, seq_rows, slots, n_seq, T_,
             n_q, n_k, d, dv, inv_freq, half, kc, vc};
  const int V = f32 ? 4 : 8, esz = f32 ? 4 : 2;
  auto al = [&](const void* ptr) { return (uintptr_t)ptr % 16 == 0; };
  const bool vec = d % V == 0 && dv % V == 0 && half % V == 0 && xs % V == 0 && al(x) && al(q_out) && al(tail) &&
                   al(kc) && al(vc) && al(cw) && ((n_q * d + n_k * (d + dv)) * esz) % 16 == 0;
  const size_t lds = (size_t)2 * half * sizeof(float);
  const dim3 vgrid((T_ + kConvRows - 1) / kConvRows);
  if (vec && f32) hipLaunchKernelGGL((conv_rope_cache_vec_kernel<float, 4>), vgrid, dim3(128), kConvRows * lds, st, g);
  else if (vec) hipLaunchKernelGGL((conv_rope_cache_vec_kernel<bf16_t, 8>), vgrid, dim3(128), kConvRows * lds, st, g);
  else { DISPATCH_T(f32, hipLaunchKernelGGL(conv_rope_cache_kernel<T>, dim3(T_), dim3(256), lds, st, g)); }
  DX_CHECK_LAUNCH();
  return 0;
}

// The convolution alone, for 1 to 4 taps and channels in whole 16-byte runs (any other: returns 1 and does
// nothing; dxm_conv_rope_cache takes every size).  A step of one row per sequence (row_seq null) also leaves the
// new tail in `tail`; a step of longer runs leaves it to dxm_conv_state_update.
int dxm_conv_run_ok(int64_t xs, int C, int taps, int T_, uint64_t ptrs, int f32) {
  const int V = f32 ? 4 : 8;
  return taps >= 1 && taps <= 4 && C > 0 && C % V == 0 && xs % V == 0 && ptrs % 16 == 0 && T_ < 65535;
}

int dxm_conv_run(void* out, const void* x, int64_t xs, const float* cw, const float* cb, int silu, int taps, void* tail,
                 int n_slots, const int64_t* pos, const int* row_seq, const int* seq_rows, const int* slots, int n_seq,
                 int T_, int C, int f32, hipStream_t st) {
  if (T_ <= 0) return 0;
  const uint64_t ptrs = (uint64_t)out | (uint64_t)x | (uint64_t)cw | (uint64_t)tail;
  if (!dxm_conv_run_ok(xs, C, taps, T_, ptrs, f32)) return 1;
  if (!out || !x || !cw || !pos || !slots || (taps > 1 && !tail)) return 2;
  if ((row_seq == nullptr) != (seq_rows == nullptr) || (!row_seq && n_seq != T_)) return 3;
  ConvArgs g{out, x, xs, cw, cb, silu, taps, tail, n_slots, pos, nullptr, row_seq, seq_rows, slots, n_seq, T_,
             1, 0, C, 0, nullptr, 0, nullptr, nullptr};
#define CONV_RUN(TAPS) \
  if (f32) launch_conv_run<float, 4, TAPS>(g, st); \
  else launch_conv_run<bf16_t, 8, TAPS>(g, st);
  if (taps == 1) { CONV_RUN(1) }
  else if (taps == 2) { CONV_RUN(2) }
  else if (taps == 3) { CONV_RUN(3) }
  else { CONV_RUN(4) }
#undef CONV_RUN
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_conv_state_update(void* tail, int n_slots, const void* x, int64_t xs, const int64_t* pos, const int* seq_rows,
                          const int* slots, int n_seq, int T_, int C, int taps, int f32, hipStream_t st) {
  if (n_seq <= 0 || taps <= 1 || C <= 0) return 0;
  if (!tail || !x || !pos || !slots || (!seq_rows && n_seq != T_)) return 1;
  const int gy = (C + 255) / 256 < 64 ? (C + 255) / 256 : 64;
  DISPATCH_T(f32, hipLaunchKernelGGL(conv_state_update_kernel<T>, dim3(n_seq, gy), dim3(256), 0, st, (T*)tail, n_slots,
                                     (const T*)x, xs, pos, seq_rows, slots, T_, C, taps - 1));
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_head_norm_gate(void* out, const float* o, const float* w, const void* gate, int64_t gs, int rows, int H,
                       int dv, float eps, int gate_act, int f32, hipStream_t st) {
  if (rows <= 0) return 0;
  if (H < 1 || dv < 1 || (int64_t)rows * H > 0x7fffffff || gate_act < 0 || gate_act > 1) return 1;
  const int64_t n_vec = (int64_t)rows * H;
  const dim3 grid((unsigned)((n_vec + 3) / 4));
  const int esz = f32 ? 4 : 2;
  if (dv % 4 == 0 && dv <= 256 && gs % 4 == 0 && (uintptr_t)o % 16 == 0 && (uintptr_t)out % (4 * esz) == 0 &&
      (uintptr_t)gate % (4 * esz) == 0) {
    DISPATCH_T(f32, {
      if (dv <= 32) launch_head_norm_vec<T, 8>(out, o, w, gate, gs, n_vec, H, dv, eps, gate_act, st);
      else if (dv <= 64) launch_head_norm_vec<T, 16>(out, o, w, gate, gs, n_vec, H, dv, eps, gate_act, st);
      else if (dv <= 128) launch_head_norm_vec<T, 32>(out, o, w, gate, gs, n_vec, H, dv, eps, gate_act, st);
      else launch_head_norm_vec<T, 64>(out, o, w, gate, gs, n_vec, H, dv, eps, gate_act, st);
    });
    DX_CHECK_LAUNCH();
    return 0;
  }
  const int V = f32 ? 4 : 8;
  if (dv > 512 && dv % V == 0 && gs % V == 0 && (uintptr_t)o % 16 == 0 && (uintptr_t)out % 16 == 0 &&
      (uintptr_t)gate % 16 == 0) {  // a workgroup per head
    const int64_t os = (int64_t)H * dv;
    if (f32 && gate_act) launch_gate_group_norm<float, 4, 2>(out, os, o, gate, gs, w, rows, H, dv, eps, st);
    else if (f32) launch_gate_group_norm<float, 4, 1>(out, os, o, gate, gs, w, rows, H, dv, eps, st);
    else if (gate_act) launch_gate_group_norm<bf16_t, 8, 2>(out, os, o, gate, gs, w, rows, H, dv, eps, st);
    else launch_gate_group_norm<bf16_t, 8, 1>(out, os, o, gate, gs, w, rows, H, dv, eps, st);
    DX_CHECK_LAUNCH();
    return 0;
  }
  const bool v2 = dv % 2 == 0 && gs % 2 == 0 && (uintptr_t)o % 8 == 0 && (uintptr_t)out % 4 == 0;
  if (v2) {
    DISPATCH_T(f32, hipLaunchKernelGGL((head_norm_gate_kernel<T, 2>), grid, dim3(256), 0, st, (T*)out, o, w,
                                       (const T*)gate, gs, n_vec, H, dv, eps, gate_act));
  } else {
    DISPATCH_T(f32, hipLaunchKernelGGL((head_norm_gate_kernel<T, 1>), grid, dim3(256), 0, st, (T*)out, o, w,
                                       (const T*)gate, gs, n_vec, H, dv, eps, gate_act));
  }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_gate_group_norm(void* out, int64_t os, const float* y, const void* z, int64_t zs, const float* w, int rows,
                        int n_groups, int n, float eps, int f32, hipStream_t st) {
  if (rows <= 0) return 0;
  if (n_groups < 1 || n < 1 || (int64_t)rows * n_groups > 0x7fffffff) return 1;
  if (!out || !y || !z || !w) return 2;
  const int V = f32 ? 4 : 8;
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = n % V == 0 && os % V == 0 && zs % V == 0 && al(out) && al(y) && al(z);
  if (vec && f32) launch_gate_group_norm<float, 4>(out, os, y, z, zs, w, rows, n_groups, n, eps, st);
  else if (vec) launch_gate_group_norm<bf16_t, 8>(out, os, y, z, zs, w, rows, n_groups, n, eps, st);
  else if (f32) launch_gate_group_norm<float, 1>(out, os, y, z, zs, w, rows, n_groups, n, eps, st);
  else launch_gate_group_norm<bf16_t, 1>(out, os, y, z, zs, w, rows, n_groups, n, eps, st);
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
