// Query / key preparation with one norm over all heads, for gfx950: per token
// row of a fused projection x = [q (n_q d) | k (n_k d) | v (v_w) | ...]
//   * q and k are each RMS-normed over their whole section (all heads together)
//     with a weight per column, when weights are given;
//   * every q and k head is then rotated: columns (2i, 2i + 1), i < half, by the
//     angle position * inv_freq[i] (interleaved pairs); the rest pass unchanged;
//   * q is written back in place, k and v go to the paged cache rows of the
//     token's slot (slot < 0: nothing is cached);
//   * another section of the row (the query, key and value of a second, recurrent
//     mixer that reads the same input) takes silu in place, when one is given.
// Norm sums, angles and the rotation are fp32 whatever the element type is.
#include "recurrent.h"

namespace {

template <typename T> struct VecIO<T, 1> {
  __device__ static __forceinline__ void ld(const T* p, float* o) { o[0] = ldf<T>(p, 0); }
  __device__ static __forceinline__ void st(T* p, const float* v) { stf<T>(p, 0, v[0]); }
};
// pairs of neighbours: what the narrow path works on (a pair never straddles two items)
template <> struct VecIO<bf16_t, 2> {
  __device__ static __forceinline__ void ld(const bf16_t* p, float* o) { o[0] = bf16_to_f32(p[0]), o[1] = bf16_to_f32(p[1]); }
  __device__ static __forceinline__ void st(bf16_t* p, const float* v) { p[0] = f32_to_bf16(v[0]), p[1] = f32_to_bf16(v[1]); }
};
template <> struct VecIO<float, 2> {
  __device__ static __forceinline__ void ld(const float* p, float* o) { o[0] = p[0], o[1] = p[1]; }
  __device__ static __forceinline__ void st(float* p, const float* v) { p[0] = v[0], p[1] = v[1]; }
};

struct NormRopeArgs {
  void* x;
  int64_t xs;
  const int64_t* pos;
  const int64_t* slots;
  int n_q, n_k, d, v_w;
  const float *qw, *kw;  // [n_q * d], [n_k * d] or null
  float eps;
  const float* inv_freq;  // [half]
  int half;
  void *kc, *vc;
  int act_off, act_n;  // columns act_off .. + act_n of the row: z <- z sigmoid(z) (act_n 0: none)
};

// V: elements per work item -- 16-byte chunks where the sizes allow, pairs for even head widths, single
// elements (no pair to rotate is lost: an odd head's last column is never rotated, and V = 1 reads its
// partner from memory) otherwise.  A thread keeps up to kKeep items in registers between sum and result.
constexpr int kKeep = 4;
template <typename T, int V>
__global__ void __launch_bounds__(256) norm_rope_cache_kernel(NormRopeArgs g) {
  extern __shared__ float cs_sn[];  // [half] cosines, [half] sines
  __shared__ float red[8];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  const int nq = g.n_q * g.d, nk = g.n_k * g.d;
  T* row = (T*)g.x + t * g.xs;
  const float p = (float)g.pos[t];
  const int64_t slot = g.slots[t];
  for (int i = tid; i < g.half; i += 256) sincosf(p * g.inv_freq[i], &cs_sn[g.half + i], &cs_sn[i]);
  const int iq = nq / V, items = iq + nk / V;
  float a[kKeep][V], sq = 0.f, sk = 0.f;
  auto sum = [&](int it, const float* v) {
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < V; ++e) s += v[e] * v[e];
    if (it < iq) sq += s;
    else sk += s;
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int it = tid + 256 * k;
    if (it < items) {
      VecIO<T, V>::ld(row + it * V, a[k]);
      sum(it, a[k]);
    }
  }
  if (g.qw || g.kw)
    for (int it = tid + 256 * kKeep; it < items; it += 256) {
      float v[V];
      VecIO<T, V>::ld(row + it * V, v);
      sum(it, v);
    }
  sq = wave_reduce_sum(sq);
  sk = wave_reduce_sum(sk);
  if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sk;
  __syncthreads();  // (also orders the angles)
  const float rq = g.qw ? rsqrtf((red[0] + red[1] + red[2] + red[3]) / (float)nq + g.eps) : 1.f;
  const float rk = g.kw ? rsqrtf((red[4] + red[5] + red[6] + red[7]) / (float)nk + g.eps) : 1.f;
  auto finish = [&](int it, float* v) {
    const bool is_q = it < iq;
    const int c = is_q ? it * V : it * V - nq, e0 = c % g.d;  // column of the section, of the head
    const float r = is_q ? rq : rk;
    const float* w = is_q ? g.qw : g.kw;
    if (w) {
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] *= r * w[c + e];
    }
#pragma unroll
    for (int e = 0; e + 1 < V; e += 2) {
      const int i = (e0 + e) >> 1;
      if (i < g.half) {
        const float cs = cs_sn[i], sn = cs_sn[g.half + i], u = v[e];
        v[e] = u * cs - v[e + 1] * sn;
        v[e + 1] = v[e + 1] * cs + u * sn;
      }
    }
    if (is_q) VecIO<T, V>::st(row + c, v);
    else if (slot >= 0) VecIO<T, V>::st((T*)g.kc + slot * nk + c, v);
  };
  if constexpr (V > 1) {
#pragma unroll
    for (int k = 0; k < kKeep; ++k)
      if (tid + 256 * k < items) finish(tid + 256 * k, a[k]);
    for (int it = tid + 256 * kKeep; it < items; it += 256) {
      float v[V];
      VecIO<T, V>::ld(row + it * V, v);
      finish(it, v);
    }
  } else {
    // odd head widths: an item is a pair of columns of one head, or its last single column
    const int per = (g.d + 1) / 2;
    for (int it = tid; it < (g.n_q + g.n_k) * per; it += 256) {
      const int hd = it / per, e = (it - hd * per) * 2;
      const bool is_q = hd < g.n_q, two = e + 1 < g.d;
      const int c = (is_q ? hd : hd - g.n_q) * g.d + e;  // column of the section
      const float r = is_q ? rq : rk;
      const float* w = is_q ? g.qw : g.kw;
      const T* src = row + (is_q ? 0 : nq) + c;
      float u = ldf<T>(src, 0) * (w ? r * w[c] : 1.f);
      float v = two ? ldf<T>(src, 1) * (w ? r * w[c + 1] : 1.f) : 0.f;
      if (e / 2 < g.half) {
        const float cs = cs_sn[e / 2], sn = cs_sn[g.half + e / 2], u0 = u;
        u = u0 * cs - v * sn;
        v = v * cs + u0 * sn;
      }
      T* dst = is_q ? row + c : (slot >= 0 ? (T*)g.kc + slot * nk + c : nullptr);
      if (dst) {
        stf<T>(dst, 0, u);
        if (two) stf<T>(dst, 1, v);
      }
    }
  }
  for (int c = tid * V; c < g.act_n; c += 256 * V) {
    float z[V];
    VecIO<T, V>::ld(row + g.act_off + c, z);
#pragma unroll
    for (int e = 0; e < V; ++e) z[e] *= fast_sigmoid(z[e]);
    VecIO<T, V>::st(row + g.act_off + c, z);
  }
  if (slot >= 0 && g.vc) {
    const T* v = row + nq + nk;
    T* dst = (T*)g.vc + slot * g.v_w;
    if constexpr (V * sizeof(T) == 16) {
      typedef uint32_t raw4 __attribute__((ext_vector_type(4)));
      for (int c = tid * V; c < g.v_w; c += 256 * V) *reinterpret_cast<raw4*>(dst + c) = *reinterpret_cast<const raw4*>(v + c);
    } else {
      for (int c = tid; c < g.v_w; c += 256) dst[c] = v[c];
    }
  }
}

template <typename T, int V> void launch_norm_rope(const NormRopeArgs& g, int rows, hipStream_t st) {
  hipLaunchKernelGGL((norm_rope_cache_kernel<T, V>), dim3(rows), dim3(256), (size_t)2 * g.half * sizeof(float), st, g);
}

}  // namespace

extern "C" int dxm_norm_rope_cache(void* x, int64_t xs, const int64_t* pos, const int64_t* slots, int rows, int n_q,
                                   int n_k, int d, int v_w, const float* qw, const float* kw, float eps,
                                   const float* inv_freq, int half, void* kc, void* vc, int act_off, int act_n,
                                   int f32, hipStream_t st) {
  if (rows <= 0) return 0;
  if (n_q < 1 || n_k < 1 || d < 1 || v_w < 0 || half < 0 || 2 * half > d || half > 4096) return 1;
  if (!x || !pos || !slots || !kc || (v_w && !vc) || (half && !inv_freq)) return 2;
  if (act_n < 0 || (act_n && act_off < n_q * d + n_k * d + v_w)) return 3;
  NormRopeArgs g{x, xs, pos, slots, n_q, n_k, d, v_w, qw, kw, eps, inv_freq, half, kc, v_w ? vc : nullptr,
                 act_off, act_n};
  const int V = f32 ? 4 : 8;
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = d % V == 0 && v_w % V == 0 && act_off % V == 0 && act_n % V == 0 && xs % V == 0 && al(x) && al(kc) && al(vc);
  if (vec && f32) launch_norm_rope<float, 4>(g, rows, st);
  else if (vec) launch_norm_rope<bf16_t, 8>(g, rows, st);
  else if (d % 2 == 0 && act_n % 2 == 0) { DISPATCH_T(f32, (launch_norm_rope<T, 2>(g, rows, st))); }
  else { DISPATCH_T(f32, (launch_norm_rope<T, 1>(g, rows, st))); }
  DX_CHECK_LAUNCH();
  return 0;
}
