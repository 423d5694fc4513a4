// Mixture-of-experts kernels for gfx950: expert choice from router logits, the
// per-step plan (slots sorted by expert, on the device), grouped GEMMs over
// each expert's rows on the matrix cores, and the weighted combine.
//
// A step of T tokens with `top` experts each has R = T * top slots; slot
// t * top + k is token t's k-th choice.  Nothing here needs the host to know
// how many rows an expert got: the grouped GEMM is launched with an upper
// bound of row tiles and every workgroup finds its (expert, tile) from the
// offsets, so a step can be captured in a HIP graph.
//
// Router arithmetic (sigmoid, correction, group sums, comparisons) is fp32.
// GEMMs take bf16 (v_mfma_f32_16x16x16_bf16) or fp32 (v_mfma_f32_16x16x4_f32,
// true fp32 products) operands and accumulate in fp32.
#include "../kernels/common.h"

namespace {

// (value, index) argmax over a wave; ties go to the lower index
__device__ __forceinline__ void wave_argmax(float& v, int& i) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(i, o, 64);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}

// Expert choice of one token by one wave.  c[e] = s[e] + corr[e] are the choice scores, s = sigmoid(z)
// or softmax(z) over all experts; with n_groups > 1 only the experts of the `keep` groups with the
// largest group score (the sum of their two best choice scores, or with group_max their best)
// compete; the `top` best are written with weight s (no correction), with renorm divided by the sum of
// the chosen s (+ 1e-20), times scale.  zt [E] (global or LDS), c [E] and gs [n_groups] LDS of the wave.
// Every wave of the workgroup calls this together (it holds barriers); `on`: the token exists.
struct RouteArgs {
  const float* corr;
  int E, top, n_groups, keep, score, group_max, renorm;
  float scale;
};
__device__ __forceinline__ void route_token(const RouteArgs& g, const float* zt, float* c, float* gs, bool on,
                                            int* __restrict__ idx, float* __restrict__ w, int lane) {
  const int E = g.E;
  // score 0: s = sigmoid(z); 1: s = softmax(z) over all experts (zmax, zinv: its maximum and 1 / sum)
  float zmax = 0.f, zinv = 1.f;
  if (g.score == 1) {
    float mxv = -INFINITY;
    for (int e = lane; e < E; e += 64) mxv = fmaxf(mxv, zt[e]);
    zmax = wave_reduce_max(mxv);
    float sm_ = 0.f;
    for (int e = lane; e < E; e += 64) sm_ += expf(zt[e] - zmax);
    zinv = 1.f / wave_reduce_sum(sm_);
  }
  auto score = [&](int e) { return g.score == 1 ? expf(zt[e] - zmax) * zinv : 1.f / (1.f + expf(-zt[e])); };
  for (int e = lane; e < E; e += 64) c[e] = score(e) + (g.corr ? g.corr[e] : 0.f);
  __syncthreads();
  if (g.n_groups > 1) {
    const int per = E / g.n_groups;
    for (int q = lane; q < g.n_groups; q += 64) {
      float a = -INFINITY, b = -INFINITY;  // two largest
      for (int e = q * per; e < (q + 1) * per; ++e) {
        const float v = c[e];
        if (v > a) {
          b = a;
          a = v;
        } else if (v > b) {
          b = v;
        }
      }
      gs[q] = per > 1 && !g.group_max ? a + b : a;
    }
    __syncthreads();
    for (int k = 0; k < g.keep; ++k) {  // kept groups are marked +inf
      float bv = -INFINITY;
      int bi = 0x7fffffff;
      for (int q = lane; q < g.n_groups; q += 64) {
        const float v = gs[q];
        if (v != INFINITY && (v > bv || (v == bv && q < bi))) {
          bv = v;
          bi = q;
        }
      }
      wave_argmax(bv, bi);
      __syncthreads();
      if (lane == 0 && bi < g.n_groups) gs[bi] = INFINITY;
      __syncthreads();
    }
    for (int e = lane; e < E; e += 64)
      if (gs[e / per] != INFINITY) c[e] = -INFINITY;
    __syncthreads();
  }
  float mine = 0.f, sum = 0.f;  // renorm: lane k's chosen score (top <= 64)
  for (int k = 0; k < g.top; ++k) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = c[e];
      if (v > bv || (v == bv && e < bi && v != -INFINITY)) {
        bv = v;
        bi = e;
      }
    }
    wave_argmax(bv, bi);
    if (bi >= E) bi = 0;  // nothing left to choose (rejected on the host)
    __syncthreads();
    if (lane == 0) c[bi] = -INFINITY;
    const float s = score(bi);
    if (g.renorm) {
      sum += s;
      if (lane == k) mine = s;
    }
    if (lane == 0 && on) {
      idx[k] = bi;
      if (!g.renorm) w[k] = s * g.scale;
    }
    __syncthreads();
  }
  if (g.renorm && on && lane < g.top) w[lane] = mine / (sum + 1e-20f) * g.scale;
}

// router logits z [T, E] given: one wave per token
constexpr int kRouteWaves = 4;
__global__ void __launch_bounds__(64 * kRouteWaves) moe_route_kernel(int* __restrict__ idx, float* __restrict__ w,
                                                                     const float* __restrict__ z, int T, RouteArgs g) {
  extern __shared__ float sm[];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int64_t t = (int64_t)blockIdx.x * kRouteWaves + wv;
  const bool on = t < T;
  float* c = sm + wv * (g.E + g.n_groups);
  const int64_t tc = on ? t : 0;
  route_token(g, z + tc * g.E, c, c + g.E, on, idx + tc * g.top, w + tc * g.top, lane);
}

// The same result for few tokens: a workgroup per token whose waves share the width, kOut outputs at a time --
// wide rows get many waves, so that a thread has one piece of the row and all its loads are in flight together.
template <typename T, int V, int NW>
__global__ void __launch_bounds__(64 * NW) moe_router_rows_kernel(int* __restrict__ idx, float* __restrict__ wgt,
                                                                  float* __restrict__ gates, const T* __restrict__ h,
                                                                  int64_t hs, const float* __restrict__ w, int n_out, int W,
                                                                  RouteArgs g) {
  constexpr int kOut = 12;
  extern __shared__ float rsm[];
  float* part = rsm;              // [NW waves][n_out]
  float* z = part + NW * n_out;   // [n_out]
  float* scratch = z + n_out;     // [NW][E + n_groups]
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int64_t t = blockIdx.x;
  const T* hp = h + t * hs;
  auto load_h = [&](int e, float* x) {
    if constexpr (V == 1) {
      if constexpr (sizeof(T) == 2) x[0] = bf16_to_f32(hp[e]); else x[0] = hp[e];
    } else if constexpr (sizeof(T) == 2) {
      const uint2 q = *reinterpret_cast<const uint2*>(hp + e);
      x[0] = bf16lo(q.x), x[1] = bf16hi(q.x), x[2] = bf16lo(q.y), x[3] = bf16hi(q.y);
    } else {
      const f32x4 q = *reinterpret_cast<const f32x4*>(hp + e);
      x[0] = q[0], x[1] = q[1], x[2] = q[2], x[3] = q[3];
    }
  };
  for (int o0 = 0; o0 < n_out; o0 += kOut) {
    float acc[kOut];
#pragma unroll
    for (int j = 0; j < kOut; ++j) acc[j] = 0.f;
    for (int e = tid * V; e < W; e += 64 * NW * V) {
      float x[V];
      load_h(e, x);
      float q[kOut][V];
#pragma unroll
      for (int j = 0; j < kOut; ++j) {
        const float* wp = w + (int64_t)min(o0 + j, n_out - 1) * W + e;  // (past the last: not used)
        if constexpr (V == 1) {
          q[j][0] = wp[0];
        } else {
          const f32x4 u = *reinterpret_cast<const f32x4*>(wp);
          q[j][0] = u[0], q[j][1] = u[1], q[j][2] = u[2], q[j][3] = u[3];
        }
      }
#pragma unroll
      for (int j = 0; j < kOut; ++j)
#pragma unroll
        for (int i = 0; i < V; ++i) acc[j] += x[i] * q[j][i];
    }
#pragma unroll
    for (int j = 0; j < kOut; ++j) {
      const float s = wave_reduce_sum(acc[j]);
      if (lane == 0 && o0 + j < n_out) part[wv * n_out + o0 + j] = s;
    }
  }
  __syncthreads();
  for (int o = tid; o < n_out; o += 64 * NW) {
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < NW; ++k) s += part[k * n_out + o];
    z[o] = s;
  }
  __syncthreads();
  for (int j = tid; j < n_out - g.E; j += 64 * NW) gates[t * (n_out - g.E) + j] = 1.f / (1.f + expf(-z[g.E + j]));
  // (every wave takes part in the choice's barriers; wave 0 writes it)
  float* c = scratch + wv * (g.E + g.n_groups);
  route_token(g, z, c, c + g.E, wv == 0, idx + t * g.top, wgt + t * g.top, lane);
}

// order [R]: slots sorted by expert, stable; offsets [E + 1].  One workgroup:
// counts by LDS atomics (the counts do not depend on their order), a serial
// scan over the experts, then every wave places the slots of its experts in
// slot order with ballots.  Choices that are no expert (identity outputs, >= E)
// get no place: order holds offsets[E] slots.  STAGE: the choices are first
// copied into LDS as bytes (E <= 255, R <= kPlanStage), so the placement passes
// read no global memory.
constexpr int kPlanThreads = 1024;
constexpr int kPlanStage = 48 * 1024;
template <bool STAGE>
__global__ void __launch_bounds__(kPlanThreads) moe_plan_kernel(int* __restrict__ order, int* __restrict__ offsets,
                                                                const int* __restrict__ idx, int R, int E) {
  extern __shared__ int ism[];
  int* cnt = ism;
  int* base = ism + E;
  unsigned char* mine = reinterpret_cast<unsigned char*>(ism + 2 * E + 1);
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  for (int e = tid; e < E; e += kPlanThreads) cnt[e] = 0;
  __syncthreads();
  for (int r = tid; r < R; r += kPlanThreads) {
    const int e = idx[r];
    const bool ok = e >= 0 && e < E;
    if (ok) atomicAdd(&cnt[e], 1);
    if constexpr (STAGE) mine[r] = ok ? (unsigned char)e : 255;
  }
  __syncthreads();
  if (tid == 0) {
    int acc = 0;
    for (int e = 0; e < E; ++e) {
      base[e] = acc;
      acc += cnt[e];
    }
    base[E] = acc;
  }
  __syncthreads();
  for (int e = tid; e <= E; e += kPlanThreads) offsets[e] = base[e];
  for (int e = wv; e < E; e += kPlanThreads / 64) {
    int at = base[e];
    for (int r0 = 0; r0 < R; r0 += 64) {
      const int r = r0 + lane;
      bool hit;
      if constexpr (STAGE) hit = r < R && mine[r] == e;
      else hit = r < R && idx[r] == e;
      const unsigned long long m = __builtin_amdgcn_ballot_w64(hit);
      if (hit) order[at + __builtin_popcountll(m & ((1ull << lane) - 1ull))] = r;
      at += __builtin_popcountll(m);
    }
  }
}

// ---------------------------------------------------------------------------
// Grouped GEMM.  For expert e, rows r in [offsets[e], offsets[e + 1]):
//     out[dst(r), :] = a[src(r), :] @ w[e]^T        w [E, N, K]
// src(r) = order[r] / top (gather: a has one row per token) or r; dst(r) =
// order[r] (scatter: slot order) or r.  A workgroup (4 waves) computes a
// 64-row x 64-column tile; K runs in steps of 32 through LDS, the next step's
// global loads in flight during the products.  The products are swapped,
// C^T = W A^T, so a lane ends up with four neighbouring columns of one row.
constexpr int kTM = 64, kTN = 64, kTK = 32;

template <typename T> struct Frag;
template <> struct Frag<bf16_t> {
  static constexpr int kPad = 8;
  __device__ static __forceinline__ f32x4 mma(const bf16_t* wp, const bf16_t* ap, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(*reinterpret_cast<const i16x4*>(wp),
                                                     *reinterpret_cast<const i16x4*>(ap), c, 0, 0, 0);
  }
  __device__ static __forceinline__ void store4(bf16_t* o, f32x4 v, int n) {
    if (n >= 4 && (uintptr_t)o % 8 == 0) {
      uint2 p;
      p.x = pack_bf16x2(v[0], v[1]);
      p.y = pack_bf16x2(v[2], v[3]);
      *reinterpret_cast<uint2*>(o) = p;
    } else {
      for (int i = 0; i < n && i < 4; ++i) o[i] = f32_to_bf16(v[i]);
    }
  }
};
template <> struct Frag<float> {
  static constexpr int kPad = 4;
  // the four lane groups supply k = 4 g + s in step s: every k of the 16 once
  __device__ static __forceinline__ f32x4 mma(const float* wp, const float* ap, f32x4 c) {
#pragma unroll
    for (int s = 0; s < 4; ++s) c = __builtin_amdgcn_mfma_f32_16x16x4f32(wp[s], ap[s], c, 0, 0, 0);
    return c;
  }
  __device__ static __forceinline__ void store4(float* o, f32x4 v, int n) {
    if (n >= 4 && (uintptr_t)o % 16 == 0) {
      *reinterpret_cast<f32x4*>(o) = v;
    } else {
      for (int i = 0; i < n && i < 4; ++i) o[i] = v[i];
    }
  }
};

// eight consecutive elements of a row, zeros past `left` (elements left in the row)
template <typename T> struct Oct {
  T v[8];
  __device__ __forceinline__ void load(const T* p, int left, bool on) {
    if (on && left >= 8 && (uintptr_t)p % 16 == 0) {
      typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
      u32x4* d = reinterpret_cast<u32x4*>(v);
      const u32x4* s = reinterpret_cast<const u32x4*>(p);
      d[0] = s[0];
      if constexpr (sizeof(T) == 4) d[1] = s[1];
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = (on && i < left) ? p[i] : (T)0;
    }
  }
  __device__ __forceinline__ void store(T* p) const {
    typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
    const u32x4* s = reinterpret_cast<const u32x4*>(v);
    u32x4* d = reinterpret_cast<u32x4*>(p);
    d[0] = s[0];
    if constexpr (sizeof(T) == 4) d[1] = s[1];
  }
};

// Router in one pass over the normed rows h [T, W]: logits z = h w^T with w [n_out, W] fp32 (the E router rows,
// then n_out - E rows of gates), true fp32 products of h as it is and w on the fp32 matrix cores
// (v_mfma_f32_16x16x4_f32), then the choice of every token (route_token); gates[t, j] = sigmoid(z[t, E + j]).
// A workgroup takes 16 tokens; its NW waves share the width in pieces of 32, 32 outputs per pass, and their partial
// sums are added in LDS in wave order.
template <typename T, int NW>
__global__ void __launch_bounds__(64 * NW) moe_router_kernel(int* __restrict__ idx, float* __restrict__ wgt,
                                                             float* __restrict__ gates, const T* __restrict__ h,
                                                             int64_t hs, const float* __restrict__ w, int n_out, int T_,
                                                             int W, RouteArgs g) {
  extern __shared__ float rsm[];
  float* part = rsm;                 // [NW][32 outputs][16 rows + 1]
  float* z = part + NW * 32 * 17;    // [16 rows][n_out]
  float* scratch = z + 16 * n_out;   // [NW][E + n_groups]
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int64_t t0 = (int64_t)blockIdx.x * 16;
  const bool row_on = t0 + c16 < T_;
  const T* hp = h + (row_on ? t0 + c16 : t0) * hs;
  auto f = [](T v) -> float {
    if constexpr (sizeof(T) == 2) return bf16_to_f32(v);
    else return v;
  };
  for (int o0 = 0; o0 < n_out; o0 += 32) {
    f32x4 C[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    bool on[2];
    const float* wp[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      on[i] = o0 + 16 * i + c16 < n_out;
      wp[i] = w + (int64_t)(on[i] ? o0 + 16 * i + c16 : 0) * W;
    }
    for (int k0 = wv * 32 + 8 * g4; k0 - 8 * g4 < W; k0 += NW * 32) {
      Oct<T> a;
      Oct<float> b[2];
      a.load(hp + k0, W - k0, row_on);
      b[0].load(wp[0] + k0, W - k0, on[0]);
      b[1].load(wp[1] + k0, W - k0, on[1]);
#pragma unroll
      for (int s = 0; s < 8; ++s) {  // the four lane groups supply k = 8 g4 + s
        const float x = f(a.v[s]);
        C[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(b[0].v[s], x, C[0], 0, 0, 0);
        C[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(b[1].v[s], x, C[1], 0, 0, 0);
      }
    }
    __syncthreads();  // (the previous pass's sums are read)
    // C[i]: outputs o0 + 16 i + 4 g4 + r of row c16
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) part[(wv * 32 + 16 * i + 4 * g4 + r) * 17 + c16] = C[i][r];
    __syncthreads();
    for (int it = tid; it < 32 * 16; it += 64 * NW) {
      const int o = it >> 4, r = it & 15;
      float acc = 0.f;
#pragma unroll
      for (int k = 0; k < NW; ++k) acc += part[(k * 32 + o) * 17 + r];
      if (o0 + o < n_out) z[r * n_out + o0 + o] = acc;
    }
  }
  __syncthreads();
  const int n_gate = n_out - g.E;
  for (int it = tid; it < 16 * n_gate; it += 64 * NW) {
    const int r = it / n_gate, j = it - r * n_gate;
    if (t0 + r < T_) gates[(t0 + r) * n_gate + j] = 1.f / (1.f + expf(-z[r * n_out + g.E + j]));
  }
  float* c = scratch + wv * (g.E + g.n_groups);
  for (int r = wv; r < 16; r += NW) {
    const bool on = t0 + r < T_;
    const int64_t t = on ? t0 + r : t0;
    route_token(g, z + r * n_out, c, c + g.E, on, idx + t * g.top, wgt + t * g.top, lane);
  }
}

template <typename T>
__global__ void __launch_bounds__(256) grouped_gemm_kernel(T* __restrict__ out, const T* __restrict__ a,
                                                           int64_t a_stride, const T* __restrict__ w,
                                                           const int* __restrict__ order,
                                                           const int* __restrict__ offsets, int E, int N, int K,
                                                           int top, int gather, int scatter) {
  constexpr int kStride = kTK + Frag<T>::kPad;
  __shared__ __attribute__((aligned(16))) T As[kTM * kStride];
  __shared__ __attribute__((aligned(16))) T Ws[kTN * kStride];
  // this workgroup's expert and row tile
  int tile = blockIdx.x, e = 0, lo = 0, hi = 0;
  for (; e < E; ++e) {
    lo = offsets[e];
    hi = offsets[e + 1];
    const int nt = (hi - lo + kTM - 1) / kTM;
    if (tile < nt) break;
    tile -= nt;
  }
  if (e >= E) return;
  const int row0 = lo + tile * kTM;
  const int rows = hi - row0 < kTM ? hi - row0 : kTM;
  const int n0 = blockIdx.y * kTN;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int c16 = lane & 15, g4 = lane >> 4;
  // staging: thread t moves eight k-elements (t % 4) of row t / 4 of both tiles
  const int sr = tid >> 2, sk = (tid & 3) * 8;
  const bool a_on = sr < rows;
  const int ar = row0 + (a_on ? sr : 0);
  const int64_t src = gather ? order[ar] / top : ar;
  const T* ap = a + src * a_stride + sk;
  const bool w_on = n0 + sr < N;
  const T* wp = w + ((int64_t)e * N + (w_on ? n0 + sr : 0)) * K + sk;
  const int wm = wv >> 1, wn = wv & 1;  // this wave: rows 32 wm .., columns 32 wn ..
  f32x4 C[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) C[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  Oct<T> ra, rw;
  ra.load(ap, K - sk, a_on);
  rw.load(wp, K - sk, w_on);
  for (int k0 = 0; k0 < K; k0 += kTK) {
    ra.store(As + sr * kStride + sk);
    rw.store(Ws + sr * kStride + sk);
    __syncthreads();
    if (k0 + kTK < K) {
      ra.load(ap + k0 + kTK, K - (k0 + kTK + sk), a_on);
      rw.load(wp + k0 + kTK, K - (k0 + kTK + sk), w_on);
    }
#pragma unroll
    for (int kk = 0; kk < kTK; kk += 16) {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const T* wf = Ws + (32 * wn + 16 * j + c16) * kStride + kk + 4 * g4;
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          const T* af = As + (32 * wm + 16 * i + c16) * kStride + kk + 4 * g4;
          C[i][j] = Frag<T>::mma(wf, af, C[i][j]);
        }
      }
    }
    __syncthreads();
  }
  // C[i][j]: row 32 wm + 16 i + c16, columns n0 + 32 wn + 16 j + 4 g4 .. + 3
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int m = 32 * wm + 16 * i + c16;
    if (m >= rows) continue;
    const int64_t dst = scatter ? order[row0 + m] : row0 + m;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + 32 * wn + 16 * j + 4 * g4;
      if (n < N) Frag<T>::store4(out + dst * N + n, C[i][j], N - n);
    }
  }
}

// out[t, :] = sum_k wgt[t, k] * y[t * top + k, :] (+ shared[t, :]), fp32 sum in the order of k;
// V elements (16 bytes) per thread and access, V = 1 for unaligned widths
template <typename T, int V>
__global__ void __launch_bounds__(256) moe_combine_kernel(T* __restrict__ out, const T* __restrict__ y,
                                                          const float* __restrict__ wgt, const T* __restrict__ shared,
                                                          int64_t sh_stride, int top, int W) {
  const int64_t t = blockIdx.x;
  auto load = [](const T* p, float* f) {
    if constexpr (V == 1) {
      if constexpr (sizeof(T) == 2) f[0] = bf16_to_f32(p[0]); else f[0] = p[0];
    } else if constexpr (sizeof(T) == 2) {
      const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
      for (int i = 0; i < 4; ++i) f[2 * i] = bf16lo(a.w[i]), f[2 * i + 1] = bf16hi(a.w[i]);
    } else {
      const f32x4 a = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
      for (int i = 0; i < 4; ++i) f[i] = a[i];
    }
  };
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float acc[V], f[V];
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] = 0.f;
    for (int k = 0; k < top; ++k) {
      load(y + (t * top + k) * (int64_t)W + c, f);
      const float g = wgt[t * top + k];
#pragma unroll
      for (int i = 0; i < V; ++i) acc[i] += g * f[i];
    }
    if (shared) {
      load(shared + t * sh_stride + c, f);
#pragma unroll
      for (int i = 0; i < V; ++i) acc[i] += f[i];
    }
    T* o = out + t * (int64_t)W + c;
    if constexpr (V == 1) {
      if constexpr (sizeof(T) == 2) o[0] = f32_to_bf16(acc[0]); else o[0] = acc[0];
    } else if constexpr (sizeof(T) == 2) {
      u16x8 r;
#pragma unroll
      for (int i = 0; i < 4; ++i) r.w[i] = pack_bf16x2(acc[2 * i], acc[2 * i + 1]);
      *reinterpret_cast<u16x8*>(o) = r;
    } else {
      *reinterpret_cast<f32x4*>(o) = f32x4{acc[0], acc[1], acc[2], acc[3]};
    }
  }
}

}  // namespace

extern "C" {

static int route_args_bad(const RouteArgs& g) {
  if (g.score < 0 || g.score > 1) return 3;
  if (g.E < 1 || g.n_groups < 1 || g.E % g.n_groups || g.keep < 1 || g.keep > g.n_groups || g.top < 1 ||
      g.top > g.keep * (g.E / g.n_groups))
    return 1;
  if (g.renorm && g.top > 64) return 4;
  return 0;
}

int dxm_moe_route(int* idx, float* w, const float* z, const float* corr, int T, int E, int top, int n_groups,
                  int keep, int score, int group_max, int renorm, float scale, hipStream_t st) {
  if (T <= 0) return 0;
  const RouteArgs g{corr, E, top, n_groups, keep, score, group_max, renorm, scale};
  if (const int bad = route_args_bad(g)) return bad;
  const size_t lds = (size_t)kRouteWaves * (E + n_groups) * sizeof(float);
  if (lds > 48 * 1024) return 2;
  hipLaunchKernelGGL(moe_route_kernel, dim3((T + kRouteWaves - 1) / kRouteWaves), dim3(64 * kRouteWaves), lds, st, idx,
                     w, z, T, g);
  DX_CHECK_LAUNCH();
  return 0;
}

// LDS of moe_router with nw waves (bytes); the launcher takes what fits 64 KB
static size_t router_lds(int nw, int n_out, int E, int n_groups) {
  return ((size_t)nw * 32 * 17 + 16 * (size_t)n_out + (size_t)nw * (E + n_groups)) * sizeof(float);
}

// 1 when moe_router takes this many outputs (else: logits by a GEMM, then moe_route)
int dxm_moe_router_ok(int n_out, int E, int n_groups) {
  return E >= 1 && n_out >= E && router_lds(8, n_out, E, n_groups) <= 60 * 1024;
}

int dxm_moe_router(int* idx, float* w, float* gates, const void* h, int64_t h_stride, const float* rw, int n_out, int T,
                   int W, const float* corr, int E, int top, int n_groups, int keep, int score, int group_max, int renorm,
                   float scale, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  const RouteArgs g{corr, E, top, n_groups, keep, score, group_max, renorm, scale};
  if (const int bad = route_args_bad(g)) return bad;
  if (!dxm_moe_router_ok(n_out, E, n_groups) || W < 1) return 2;
  if (!idx || !w || !h || !rw || (n_out > E && !gates)) return 5;
  const int esz = f32 ? 4 : 2;
  if (T <= 256) {
    const bool vec = W % 4 == 0 && h_stride % 4 == 0 && (uintptr_t)h % (4 * esz) == 0 && (uintptr_t)rw % 16 == 0;
    auto lds = [&](int nw) { return ((nw + 1) * (size_t)n_out + nw * (size_t)(E + n_groups)) * sizeof(float); };
    const bool wide = vec && W >= 2048 && lds(16) <= 60 * 1024;
#define ROUTER_ROWS(TY, V, NW)                                                                                        \
  hipLaunchKernelGGL((moe_router_rows_kernel<TY, V, NW>), dim3(T), dim3(64 * NW), lds(NW), st, idx, w, gates,          \
                     (const TY*)h, h_stride, rw, n_out, W, g);
    if (f32 && wide) { ROUTER_ROWS(float, 4, 16) }
    else if (f32 && vec) { ROUTER_ROWS(float, 4, 4) }
    else if (f32) { ROUTER_ROWS(float, 1, 4) }
    else if (wide) { ROUTER_ROWS(bf16_t, 4, 16) }
    else if (vec) { ROUTER_ROWS(bf16_t, 4, 4) }
    else { ROUTER_ROWS(bf16_t, 1, 4) }
#undef ROUTER_ROWS
    DX_CHECK_LAUNCH();
    return 0;
  }
  const dim3 grid((unsigned)((T + 15) / 16));
  // few tokens: more waves share the width
  const bool many = T <= 1024 && router_lds(16, n_out, E, n_groups) <= 60 * 1024;
#define ROUTER(TY, NW)                                                                                               \
  hipLaunchKernelGGL((moe_router_kernel<TY, NW>), grid, dim3(64 * NW), router_lds(NW, n_out, E, n_groups), st, idx, w, \
                     gates, (const TY*)h, h_stride, rw, n_out, T, W, g);
  if (f32 && many) { ROUTER(float, 16) }
  else if (f32) { ROUTER(float, 8) }
  else if (many) { ROUTER(bf16_t, 16) }
  else { ROUTER(bf16_t, 8) }
#undef ROUTER
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_moe_plan(int* order, int* offsets, const int* idx, int R, int E, hipStream_t st) {
  if (E < 1 || R < 0) return 1;
  const size_t lds = (size_t)(2 * E + 1) * sizeof(int);
  if (lds > 12 * 1024) return 2;
  if (E <= 255 && R <= kPlanStage)
    hipLaunchKernelGGL(moe_plan_kernel<true>, dim3(1), dim3(kPlanThreads), lds + R, st, order, offsets, idx, R, E);
  else
    hipLaunchKernelGGL(moe_plan_kernel<false>, dim3(1), dim3(kPlanThreads), lds, st, order, offsets, idx, R, E);
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_grouped_gemm(void* out, const void* a, int64_t a_stride, const void* w, const int* order, const int* offsets,
                     int R, int E, int N, int K, int top, int gather, int scatter, int f32, hipStream_t st) {
  if (R <= 0) return 0;
  if (E < 1 || N < 1 || K < 1 || top < 1) return 1;
  const unsigned tiles = (unsigned)((R + kTM - 1) / kTM + E);  // at most this many row tiles over all experts
  const unsigned ny = (unsigned)((N + kTN - 1) / kTN);
  if (ny > 65535) return 2;
  if (f32)
    hipLaunchKernelGGL(grouped_gemm_kernel<float>, dim3(tiles, ny), dim3(256), 0, st, (float*)out, (const float*)a,
                       a_stride, (const float*)w, order, offsets, E, N, K, top, gather, scatter);
  else
    hipLaunchKernelGGL(grouped_gemm_kernel<bf16_t>, dim3(tiles, ny), dim3(256), 0, st, (bf16_t*)out, (const bf16_t*)a,
                       a_stride, (const bf16_t*)w, order, offsets, E, N, K, top, gather, scatter);
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_moe_combine(void* out, const void* y, const float* wgt, const void* shared, int64_t sh_stride, int T, int top,
                    int W, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (top < 1 || W < 1) return 1;
  const int per = f32 ? 4 : 8;  // elements per 16 bytes
  const bool vec = W % per == 0 && sh_stride % per == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)y % 16 == 0 &&
                   (uintptr_t)shared % 16 == 0;
  if (f32) {
    if (vec)
      hipLaunchKernelGGL((moe_combine_kernel<float, 4>), dim3(T), dim3(256), 0, st, (float*)out, (const float*)y, wgt,
                         (const float*)shared, sh_stride, top, W);
    else
      hipLaunchKernelGGL((moe_combine_kernel<float, 1>), dim3(T), dim3(256), 0, st, (float*)out, (const float*)y, wgt,
                         (const float*)shared, sh_stride, top, W);
  } else {
    if (vec)
      hipLaunchKernelGGL((moe_combine_kernel<bf16_t, 8>), dim3(T), dim3(256), 0, st, (bf16_t*)out, (const bf16_t*)y,
                         wgt, (const bf16_t*)shared, sh_stride, top, W);
    else
      hipLaunchKernelGGL((moe_combine_kernel<bf16_t, 1>), dim3(T), dim3(256), 0, st, (bf16_t*)out, (const bf16_t*)y,
                         wgt, (const bf16_t*)shared, sh_stride, top, W);
  }
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
