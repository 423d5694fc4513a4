// Attention of many query heads over ONE shared cache row per key, [latent | key part] (D columns are the
// key, the first DV of them the value), over pages of whole 64-key tiles, for gfx950: latent attention with
// the key up-projection folded into the queries.  bf16; softmax weights, causal, window or chunk mask, an
// optional sink; scores and sums are fp32.  A tile is read from memory once and laid out twice in LDS on its
// way through registers: rows (the keys) and, transposed, the value columns in the order the weights'
// fragments have them (stream_attention.h).
//
// latent_decode: a workgroup (4 waves) per (decode row, 16 QB heads, key part).  The waves share the tile:
// each scores 16 of its keys against all heads, they agree on the maxima through LDS and exchange the
// weights there (as the sum of two bf16 numbers), and each forms DV / 4 columns of the result.  Partition and
// workspace as in group_decode (merge_parts joins the parts).
// latent_prefill: eight waves per (32 RT prompt rows, HPW heads), 32 rows of one head each, sharing every
// tile, which are double-buffered; RT = 8 / HPW.
#include "stream_attention.h"

namespace {

// the tile's 16-byte pieces in groups of 4 keys x 8 columns, NT threads
template <int D, int DV, int NT> struct LatentStage {
  static constexpr int CH = D / 8, kItems = 16 * CH, NI = (kItems + NT - 1) / NT;
  raw_u32x4 st[NI][4];
  __device__ __forceinline__ void fetch(const bf16_t* base, int stride, int tid) {  // base: the tile's first row
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = tid + NT * i;
      if (kItems % NT == 0 || it < kItems) {
        const bf16_t* src = base + (int64_t)(4 * (it / CH)) * stride + 8 * (it % CH);
#pragma unroll
        for (int k = 0; k < 4; ++k) st[i][k] = *reinterpret_cast<const raw_u32x4*>(src + (int64_t)k * stride);
      }
    }
  }
  // left: keys of the tile that exist; the rows behind them hold stale values, which must not meet a zero weight
  __device__ __forceinline__ void commit(bf16_t* K, bf16_t* V, int left, int tid) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = tid + NT * i;
      if (kItems % NT == 0 || it < kItems) {
        const int kg = it / CH, ch = it % CH;
        if (left < 64) {
#pragma unroll
          for (int k = 0; k < 4; ++k)
            if (4 * kg + k >= left) st[i][k] = raw_u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) *reinterpret_cast<raw_u32x4*>(K + kimg<D>(4 * kg + k, ch)) = st[i][k];
        if (DV == D || ch < DV / 8) put_v(V, st[i], kg, ch);
      }
    }
  }
};

struct LatentArgs {
  void* out;  // prefill: bf16 [T, n_qh, dv]; decode: workspace float [rows, n_qh, parts, 2 + dv]
  const bf16_t* q;
  int64_t q_stride;
  const bf16_t* cache;
  int stride;  // elements per cache row
  const int64_t* pos;
  const int* seq;  // decode: null: row i is sequence i
  const int* bt;
  int bt_stride, bs_shift;
  const int* tiles;  // prefill: [n, 2]: first row, rows (up to 128) of one sequence
  int subs;          // prefill: workgroups per tile entry
  int n_qh;
  float scale_log2;
  int mask, size, parts;
  const float* sink;  // prefill: [n_qh] or null
};

// ---------------------------------------------------------------- decode rows
template <int D, int DV, int QB>
__global__ void __launch_bounds__(256, 2) latent_decode_kernel(LatentArgs a) {
  constexpr int NK = D / 32, NCW = DV / 64;  // key fragments, 16-column blocks of the result per wave
  static_assert(D % 32 == 0 && DV % 64 == 0, "whole fragments, equal column shares");
  extern __shared__ __attribute__((aligned(16))) bf16_t lsm[];
  bf16_t *K = lsm, *V = K + 64 * D;
  uint2* P = reinterpret_cast<uint2*>(V + 64 * DV);               // [hi, lo][QB][2 halves of 32 keys][64 lanes][2]
  float* M = reinterpret_cast<float*>(P + 2 * QB * 2 * 64 * 2);   // [4 waves][QB][16]
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int row = blockIdx.y, part = blockIdx.z, h0 = blockIdx.x * 16 * QB;
  const int p = __builtin_amdgcn_readfirstlane((int)a.pos[row]);
  const int lo = first_key(p, a.mask, a.size);
  const int first = lo >> 6, n_tiles = (p >> 6) - first + 1;
  const int tpp = (n_tiles + a.parts - 1) / a.parts;
  const int t0 = first + part * tpp, t1 = min(t0 + tpp, first + n_tiles);
  const int* bt = a.bt + (int64_t)__builtin_amdgcn_readfirstlane(a.seq ? a.seq[row] : row) * a.bt_stride;
  bf16x8_t qf[QB][NK];
  bool okh[QB];
#pragma unroll
  for (int qb = 0; qb < QB; ++qb) {
    okh[qb] = h0 + 16 * qb + c16 < a.n_qh;
    const bf16_t* q = a.q + (int64_t)row * a.q_stride + (int64_t)(okh[qb] ? h0 + 16 * qb + c16 : 0) * D + 8 * g4;
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
      const raw_u32x4 zero{0u, 0u, 0u, 0u};
      qf[qb][ks] = __builtin_bit_cast(bf16x8_t, okh[qb] ? *reinterpret_cast<const raw_u32x4*>(q + 32 * ks) : zero);
    }
  }
  float mx[QB], lsum[QB];  // log2 units; the sum over this wave's keys
  f32x4 O[QB][NCW];
#pragma unroll
  for (int qb = 0; qb < QB; ++qb) {
    mx[qb] = -INFINITY;
    lsum[qb] = 0.f;
#pragma unroll
    for (int cb = 0; cb < NCW; ++cb) O[qb][cb] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  LatentStage<D, DV, 256> stage;
  if (t0 < t1) stage.fetch(a.cache + tile_slot(bt, a.bs_shift, t0) * a.stride, a.stride, tid);
  for (int t = t0; t < t1; ++t) {
    stage.commit(K, V, p + 1 - (t << 6), tid);
    __syncthreads();
    if (t + 1 < t1) stage.fetch(a.cache + tile_slot(bt, a.bs_shift, t + 1) * a.stride, a.stride, tid);
    // scores of keys 16 w .. + 15: lane column = head, rows = keys 4 g4 + r
    f32x4 S[QB];
#pragma unroll
    for (int qb = 0; qb < QB; ++qb) S[qb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
      const bf16x8_t kf = frag16(K + kimg<D>(16 * w + c16, 4 * ks + g4));
#pragma unroll
      for (int qb = 0; qb < QB; ++qb) S[qb] = mma(kf, qf[qb][ks], S[qb]);
    }
    const bool edge = t == first || t == (p >> 6);
#pragma unroll
    for (int qb = 0; qb < QB; ++qb) {
      float m = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        S[qb][r] *= a.scale_log2;
        const int j = (t << 6) + 16 * w + 4 * g4 + r;
        if (edge && (j < lo || j > p)) S[qb][r] = -INFINITY;
        m = fmaxf(m, S[qb][r]);
      }
      m = fmaxf(m, __shfl_xor(m, 16, 64));
      m = fmaxf(m, __shfl_xor(m, 32, 64));
      if (g4 == 0) M[(w * QB + qb) * 16 + c16] = m;
    }
    __syncthreads();
#pragma unroll
    for (int qb = 0; qb < QB; ++qb) {
      float mn = mx[qb];  // finite from here on: every visited tile holds a visible key
#pragma unroll
      for (int v = 0; v < 4; ++v) mn = fmaxf(mn, M[(v * QB + qb) * 16 + c16]);
      if (__any(mn > mx[qb])) {
        const float alpha = fast_exp2(mx[qb] - mn);
        lsum[qb] *= alpha;
#pragma unroll
        for (int cb = 0; cb < NCW; ++cb)
#pragma unroll
          for (int r = 0; r < 4; ++r) O[qb][cb][r] *= alpha;
        mx[qb] = mn;
      }
      float w4[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        w4[r] = fast_exp2(S[qb][r] - mn);
        lsum[qb] += w4[r];
      }
      const uint2 hi{pack_bf16x2(w4[0], w4[1]), pack_bf16x2(w4[2], w4[3])};
      const uint2 lw{pack_bf16x2(w4[0] - bf16lo(hi.x), w4[1] - bf16hi(hi.x)),
                     pack_bf16x2(w4[2] - bf16lo(hi.y), w4[3] - bf16hi(hi.y))};
      // keys 16 w .. of half w / 2 are the first or second four slots of every lane group
      P[((0 * QB + qb) * 2 + (w >> 1)) * 128 + 2 * lane + (w & 1)] = hi;
      P[((1 * QB + qb) * 2 + (w >> 1)) * 128 + 2 * lane + (w & 1)] = lw;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8_t Pf[2][QB];
#pragma unroll
      for (int x = 0; x < 2; ++x)
#pragma unroll
        for (int qb = 0; qb < QB; ++qb)
          Pf[x][qb] = frag16(reinterpret_cast<const bf16_t*>(P + ((x * QB + qb) * 2 + kk) * 128 + 2 * lane));
#pragma unroll
      for (int cb = 0; cb < NCW; ++cb) {
        const bf16x8_t vf = frag16(V + voff(16 * (w * NCW + cb) + c16, 4 * kk + g4));
#pragma unroll
        for (int qb = 0; qb < QB; ++qb) {
          O[qb][cb] = mma(vf, Pf[0][qb], O[qb][cb]);
          O[qb][cb] = mma(vf, Pf[1][qb], O[qb][cb]);
        }
      }
    }
    __syncthreads();  // the images are free again
  }
  // sums over all waves' keys
#pragma unroll
  for (int qb = 0; qb < QB; ++qb) {
    float l = lsum[qb];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g4 == 0) M[(w * QB + qb) * 16 + c16] = l;
  }
  __syncthreads();
#pragma unroll
  for (int qb = 0; qb < QB; ++qb) {
    if (!okh[qb]) continue;
    float* o = (float*)a.out + (((int64_t)row * a.n_qh + h0 + 16 * qb + c16) * a.parts + part) * (2 + DV);
    if (w == 0 && g4 == 0) {
      float l = 0.f;
#pragma unroll
      for (int v = 0; v < 4; ++v) l += M[(v * QB + qb) * 16 + c16];
      o[0] = mx[qb] * 0.6931471805599453f;
      o[1] = l;
    }
#pragma unroll
    for (int cb = 0; cb < NCW; ++cb)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[2 + 16 * (w * NCW + cb) + 4 * g4 + r] = O[qb][cb][r];
  }
}

// ---------------------------------------------------------------- prompt rows
template <int D, int DV, int HPW>
__global__ void __launch_bounds__(512, 2) latent_prefill_kernel(LatentArgs a) {
  constexpr int NK = D / 32, NC = DV / 16, RT = 8 / HPW, ROWS = 32 * RT;
  extern __shared__ __attribute__((aligned(16))) bf16_t lsm[];
  bf16_t *Ks = lsm, *Vs = lsm + 2 * 64 * D;  // two tiles each
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int yi = gridDim.y - 1 - blockIdx.y;  // later rows see more keys: hand them out first
  const int ti = yi / a.subs, off = (yi - ti * a.subs) * ROWS;
  const int n = a.tiles[2 * ti + 1] - off;
  if (n <= 0) return;
  const int row0 = a.tiles[2 * ti] + off;
  const int p0 = __builtin_amdgcn_readfirstlane((int)a.pos[row0]);
  const int* bt = a.bt + (int64_t)__builtin_amdgcn_readfirstlane(a.seq[row0]) * a.bt_stride;
  const int qh = blockIdx.x * HPW + wave / RT;
  const int rw = 32 * (wave % RT);  // the wave's first row
  const int hi = p0 + min(n, ROWS) - 1;
  const int first = first_key(p0, a.mask, a.size) >> 6, last = hi >> 6;
  // the wave's rows: 16 qb + c16; rows beyond n repeat the last one and are not stored
  bf16x8_t qf[2][NK];
  int prow[2], lrow[2];  // position and first visible key of the lane's rows
#pragma unroll
  for (int qb = 0; qb < 2; ++qb) {
    const int r = min(rw + 16 * qb + c16, n - 1);
    prow[qb] = p0 + r;
    lrow[qb] = first_key(p0 + r, a.mask, a.size);
#pragma unroll
    for (int ks = 0; ks < NK; ++ks)
      qf[qb][ks] = frag16(a.q + (int64_t)(row0 + r) * a.q_stride + (int64_t)qh * D + 32 * ks + 8 * g4);
  }
  const int wlo = p0 + min(rw, n - 1), whi = p0 + min(rw + 31, n - 1);  // first and last row position of the wave
  const int wfirst = first_key(wlo, a.mask, a.size), wlast = first_key(whi, a.mask, a.size);
  LatentStage<D, DV, 512> stage;
  auto fetch = [&](int t) { stage.fetch(a.cache + tile_slot(bt, a.bs_shift, t) * a.stride, a.stride, tid); };
  auto commit = [&](int buf, int t) { stage.commit(Ks + buf * 64 * D, Vs + buf * 64 * DV, hi + 1 - (t << 6), tid); };
  float mx[2] = {-INFINITY, -INFINITY}, lsum[2] = {0.f, 0.f};  // log2 units
  f32x4 O[2][NC];
#pragma unroll
  for (int qb = 0; qb < 2; ++qb)
#pragma unroll
    for (int cb = 0; cb < NC; ++cb) O[qb][cb] = f32x4{0.f, 0.f, 0.f, 0.f};
  fetch(first);
  commit(0, first);
  if (first < last) fetch(first + 1);
  for (int t = first, cur = 0; t <= last; ++t, cur ^= 1) {
    __syncthreads();  // tile t is in LDS; the other half is consumed
    if (t < last) {
      commit(cur ^ 1, t + 1);
      if (t + 1 < last) fetch(t + 2);
    }
    const int kt = t << 6;
    if (rw >= n || kt > whi || kt + 63 < wfirst) continue;  // nothing the wave's rows see
    const bf16_t *K = Ks + cur * 64 * D, *V = Vs + cur * 64 * DV;
    f32x4 S[2][4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      S[0][kb] = S[1][kb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        const bf16x8_t kf = frag16(K + kimg<D>(16 * kb + c16, 4 * ks + g4));
        S[0][kb] = mma(kf, qf[0][ks], S[0][kb]);
        S[1][kb] = mma(kf, qf[1][ks], S[1][kb]);
      }
    }
    if (kt + 63 > wlo || kt < wlast) {  // some key is not seen by some row
#pragma unroll
      for (int qb = 0; qb < 2; ++qb)
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = kt + 16 * kb + 4 * g4 + r;
            if (j > prow[qb] || j < lrow[qb]) S[qb][kb][r] = -INFINITY;
          }
    }
    bf16x8_t P[2][2];
#pragma unroll
    for (int qb = 0; qb < 2; ++qb) {
      float m = S[qb][0][0];
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) m = fmaxf(m, S[qb][kb][r]);
      m = fmaxf(m, __shfl_xor(m, 16, 64));
      m = fmaxf(m, __shfl_xor(m, 32, 64));
      const float mn = fmaxf(mx[qb], m * a.scale_log2);
      const float mu = mn == -INFINITY ? 0.f : mn;  // a row that has seen nothing yet
      if (__any(mn > mx[qb])) {
        const float alpha = fast_exp2(mx[qb] - mu);
        lsum[qb] *= alpha;
#pragma unroll
        for (int cb = 0; cb < NC; ++cb)
#pragma unroll
          for (int r = 0; r < 4; ++r) O[qb][cb][r] *= alpha;
      }
      mx[qb] = mn;
      float add = 0.f;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        raw_u32x4 pk;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float w0 = fast_exp2(fmaf(S[qb][2 * kk + e / 2][2 * (e % 2)], a.scale_log2, -mu));
          const float w1 = fast_exp2(fmaf(S[qb][2 * kk + e / 2][2 * (e % 2) + 1], a.scale_log2, -mu));
          add += w0 + w1;
          pk[e] = pack_bf16x2(w0, w1);
        }
        P[qb][kk] = __builtin_bit_cast(bf16x8_t, pk);
      }
      lsum[qb] += add;
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int cb = 0; cb < NC; ++cb) {
        const bf16x8_t vf = frag16(V + voff(16 * cb + c16, 4 * kk + g4));
        O[0][cb] = mma(vf, P[0][kk], O[0][cb]);
        O[1][cb] = mma(vf, P[1][kk], O[1][cb]);
      }
  }
#pragma unroll
  for (int qb = 0; qb < 2; ++qb) {
    float l = lsum[qb];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    const int r = rw + 16 * qb + c16;
    if (r >= n) continue;
    if (a.sink) l += fast_exp2(a.sink[qh] * 1.4426950408889634f - mx[qb]);  // (finite: a row sees itself)
    const float inv = 1.f / l;
    bf16_t* o = (bf16_t*)a.out + ((int64_t)(row0 + r) * a.n_qh + qh) * DV + 4 * g4;
#pragma unroll
    for (int cb = 0; cb < NC; ++cb)
      *reinterpret_cast<uint2*>(o + 16 * cb) = uint2{pack_bf16x2(O[qb][cb][0] * inv, O[qb][cb][1] * inv),
                                                     pack_bf16x2(O[qb][cb][2] * inv, O[qb][cb][3] * inv)};
  }
}

template <typename Kern> int raise_lds(Kern kern, size_t bytes, bool& raised) {  // once per instance
  if (bytes > 48 * 1024 && !raised) {
    if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess)
      return 7;
    raised = true;
  }
  return 0;
}

template <int D, int DV, int HPW> int launch_prefill(const LatentArgs& a0, int n_tiles, hipStream_t st) {
  LatentArgs a = a0;
  a.subs = 128 / (32 * (8 / HPW));
  const size_t lds = (size_t)2 * 64 * (D + DV) * sizeof(bf16_t);
  auto kern = latent_prefill_kernel<D, DV, HPW>;
  static bool raised = false;
  if (raise_lds(kern, lds, raised)) return 7;
  const int step = 65535 / a.subs;
  for (int t0 = 0; t0 < n_tiles; t0 += step) {
    a.tiles = a0.tiles + 2 * t0;
    const int nt = n_tiles - t0 < step ? n_tiles - t0 : step;
    hipLaunchKernelGGL(kern, dim3(a.n_qh / HPW, nt * a.subs), dim3(512), lds, st, a);
  }
  DX_CHECK_LAUNCH();
  return 0;
}
template <int D, int DV> int prefill_heads(const LatentArgs& a, int n_tiles, hipStream_t st) {
  if (a.n_qh % 8 == 0) return launch_prefill<D, DV, 8>(a, n_tiles, st);
  if (a.n_qh % 4 == 0) return launch_prefill<D, DV, 4>(a, n_tiles, st);
  return launch_prefill<D, DV, 2>(a, n_tiles, st);
}

template <int D, int DV, int QB> int launch_decode(const LatentArgs& a, int rows, hipStream_t st) {
  const size_t lds = (size_t)64 * (D + DV) * sizeof(bf16_t) + (size_t)2 * QB * 2 * 128 * sizeof(uint2) + 4 * QB * 16 * sizeof(float);
  auto kern = latent_decode_kernel<D, DV, QB>;
  static bool raised = false;
  if (raise_lds(kern, lds, raised)) return 7;
  hipLaunchKernelGGL(kern, dim3((a.n_qh + 16 * QB - 1) / (16 * QB), rows, a.parts), dim3(256), lds, st, a);
  DX_CHECK_LAUNCH();
  return 0;
}
template <int D, int DV> int decode_heads(const LatentArgs& a, int rows, hipStream_t st) {
  return a.n_qh <= 16 ? launch_decode<D, DV, 1>(a, rows, st) : launch_decode<D, DV, 2>(a, rows, st);
}

}  // namespace

#define LATENT_CASES(FN, ...)                                \
  if (d == 96 && dv == 64) return FN<96, 64>(__VA_ARGS__);   \
  if (d == 160 && dv == 128) return FN<160, 128>(__VA_ARGS__); \
  if (d == 192 && dv == 128) return FN<192, 128>(__VA_ARGS__); \
  if (d == 256 && dv == 192) return FN<256, 192>(__VA_ARGS__);

extern "C" {

// 1 when the kernels take these heads: one shared row that is key and value, widths they are instantiated for,
// pages of whole 64-key tiles; prompt rows: an even number of heads
int dxm_latent_attention_ok(int d, int dv, int n_qh, int maps, int group, int bs, int prefill) {
  const bool width = (d == 96 && dv == 64) || (d == 160 && dv == 128) || (d == 192 && dv == 128) || (d == 256 && dv == 192);
  return width && maps == 1 && group == n_qh && bs >= 64 && (bs & (bs - 1)) == 0 && (!prefill || n_qh % 2 == 0);
}

int dxm_latent_prefill(void* out, const void* q, int64_t q_stride, const void* cache, int stride, const int64_t* pos,
                       const int* seq, const int* bt, int bt_stride, int bs, const int* tiles, int n_tiles, int n_qh, int d,
                       int dv, float scale, int mask, int size, const float* sink, hipStream_t st) {
  if (n_tiles <= 0) return 0;
  if (!dxm_latent_attention_ok(d, dv, n_qh, 1, n_qh, bs, 1) || n_qh < 1) return 2;
  if (mask < 0 || mask > 2 || (mask && size < 1) || !(scale > 0.f)) return 3;
  if (!out || !seq || !tiles || stride % 8 || q_stride % 8 || (uintptr_t)q % 16 || (uintptr_t)cache % 16 || (uintptr_t)out % 8)
    return 4;
  LatentArgs a{out, (const bf16_t*)q, q_stride, (const bf16_t*)cache, stride, pos, seq, bt, bt_stride,
               __builtin_ctz((unsigned)bs), tiles, 1, n_qh, scale * 1.4426950408889634f, mask, size, 1, sink};
  LATENT_CASES(prefill_heads, a, n_tiles, st)
  return 2;
}

int dxm_latent_decode(float* ws, const void* q, int64_t q_stride, const void* cache, int stride, const int64_t* pos,
                      const int* seq, const int* bt, int bt_stride, int bs, int rows, int n_qh, int d, int dv, float scale,
                      int mask, int size, int parts, hipStream_t st) {
  if (rows <= 0) return 0;
  if (!dxm_latent_attention_ok(d, dv, n_qh, 1, n_qh, bs, 0) || n_qh < 1 || rows > 65535) return 2;
  if (mask < 0 || mask > 2 || (mask && size < 1) || parts < 1 || parts > 65535 || !(scale > 0.f)) return 3;
  if (!ws || stride % 8 || q_stride % 8 || (uintptr_t)q % 16 || (uintptr_t)cache % 16) return 4;
  LatentArgs a{ws, (const bf16_t*)q, q_stride, (const bf16_t*)cache, stride, pos, seq, bt, bt_stride,
               __builtin_ctz((unsigned)bs), nullptr, 1, n_qh, scale * 1.4426950408889634f, mask, size, parts, nullptr};
  LATENT_CASES(decode_heads, a, rows, st)
  return 2;
}

}  // extern "C"
