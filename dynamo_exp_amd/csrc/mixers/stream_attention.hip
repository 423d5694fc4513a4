// Attention of plain grouped-query heads (softmax weights, causal, window or chunk
// mask, no score terms) over pages of whole 64-key tiles, for gfx950: the general
// kernels of tile_attention.hip with the key loop laid out for this case.
//   * tiles are the 64-key pieces of the pages (pages are multiples of 64 keys),
//     so a tile's rows are one scalar base plus lane constants;
//   * V is transposed on its way through registers into a swizzled LDS image
//     whose keys lie in the order the weights' fragments have them;
//   * masks apply to the first and the last tiles only; scores and sums are fp32.
// stream_decode: one wave per (decode row, K head, key part), up to 16 heads;
// partition and workspace as in group_decode (merge_parts joins the parts).  K
// goes from memory straight into MFMA A fragments (a lane reads 16 bytes of its
// key); each half's registers are refilled with the next tile as soon as they are
// free.  Weights enter the value product as the sum of two bf16 numbers.
// stream_prefill: eight waves per (64 or 128 prompt rows, 4 or 2 heads of a
// group), 32 rows of one head each, sharing every key tile; tiles are
// double-buffered in LDS.  Weights enter the value product as bf16, or (FINE) as
// the sum of two.
#include "stream_attention.h"

namespace {

struct StreamArgs {
  const bf16_t* q;
  int64_t q_stride;
  const bf16_t* kc;
  const bf16_t* vc;
  float* ws;  // [rows, n_qh, parts, 2 + dv]
  const int64_t* pos;
  const int* seq;  // null: row i is sequence i
  const int* bt;
  int bt_stride, bs_shift;
  int n_qh, maps, group;
  int Wk, Wv;
  float scale_log2;
  int mask, size;
  int parts;
};

template <int D, int DV>
__global__ void __launch_bounds__(64, 2) stream_decode_kernel(StreamArgs a) {
  constexpr int NK = D / 32, NC = DV / 16, CH = DV / 8, VI = 16 * CH / 64;  // VI: V items (4 keys x 8 columns) per lane
  static_assert(D % 32 == 0 && 16 * CH % 64 == 0, "whole fragments, whole V items");
  __shared__ __attribute__((aligned(16))) bf16_t Vt[DV * 64];
  const int lane = threadIdx.x, c16 = lane & 15, g4 = lane >> 4;
  const int gm = blockIdx.x, row = blockIdx.y, part = blockIdx.z;
  const int g = gm / a.maps, m = gm - g * a.maps;
  const int p = __builtin_amdgcn_readfirstlane((int)a.pos[row]);
  const int lo = first_key(p, a.mask, a.size);
  const int first = lo >> 6, n_tiles = (p >> 6) - first + 1;
  const int tpp = (n_tiles + a.parts - 1) / a.parts;
  const int t0 = first + part * tpp, t1 = min(t0 + tpp, first + n_tiles);
  const int* bt = a.bt + (int64_t)__builtin_amdgcn_readfirstlane(a.seq ? a.seq[row] : row) * a.bt_stride;
  const bool okh = c16 < a.group;
  const int qh = (g * a.group + (okh ? c16 : 0)) * a.maps + m;
  bf16x8_t qf[NK];
#pragma unroll
  for (int ks = 0; ks < NK; ++ks) {
    const raw_u32x4 zero{0u, 0u, 0u, 0u};
    qf[ks] = __builtin_bit_cast(bf16x8_t, okh ? *reinterpret_cast<const raw_u32x4*>(
        a.q + (int64_t)row * a.q_stride + (int64_t)qh * D + 32 * ks + 8 * g4) : zero);
  }
  // lane constants inside a tile: the K fragment of key c16, the V item (keys 4 vk .. + 3, columns 8 vc8 .. + 7)
  const int vk = lane / CH, vc8 = lane % CH;
  const bf16_t* kl = a.kc + (int64_t)gm * D + (int64_t)c16 * a.Wk + 8 * g4;
  const bf16_t* vl = a.vc + (int64_t)g * DV + (int64_t)(4 * vk) * a.Wv + 8 * vc8;
  raw_u32x4 kr[4][NK], vr[VI][4];
  auto fetch_k = [&](int64_t base) {
    const bf16_t* src = kl + base * a.Wk;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int ks = 0; ks < NK; ++ks)
        kr[kb][ks] = __builtin_nontemporal_load(reinterpret_cast<const raw_u32x4*>(src + (int64_t)kb * 16 * a.Wk + 32 * ks));
  };
  auto fetch_v = [&](int64_t base) {
    const bf16_t* src = vl + base * a.Wv;
#pragma unroll
    for (int i = 0; i < VI; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k)
        vr[i][k] = __builtin_nontemporal_load(
            reinterpret_cast<const raw_u32x4*>(src + (int64_t)(4 * (64 / CH) * i + k) * a.Wv));
  };
  float mx = -INFINITY, lsum = 0.f;  // log2 units
  f32x4 O[NC];
#pragma unroll
  for (int cb = 0; cb < NC; ++cb) O[cb] = f32x4{0.f, 0.f, 0.f, 0.f};
  int64_t next = 0;
  if (t0 < t1) {
    const int64_t base = tile_slot(bt, a.bs_shift, t0);
    fetch_k(base);
    fetch_v(base);
    next = tile_slot(bt, a.bs_shift, min(t0 + 1, t1 - 1));
  }
  for (int t = t0; t < t1; ++t) {
    const bool more = t + 1 < t1;
    f32x4 S[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      S[kb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks)
        S[kb] = mma(__builtin_bit_cast(bf16x8_t, kr[kb][ks]), qf[ks], S[kb]);
    }
    if (more) fetch_k(next);
    if (t == (p >> 6)) {  // the page's rows behind the query: stale values must not meet a zero weight
#pragma unroll
      for (int i = 0; i < VI; ++i)
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if ((t << 6) + 4 * (vk + 64 / CH * i) + k > p) vr[i][k] = raw_u32x4{0u, 0u, 0u, 0u};
    }
    __syncthreads();  // (one wave: orders the image's reads and writes)
#pragma unroll
    for (int i = 0; i < VI; ++i) put_v(Vt, vr[i], vk + 64 / CH * i, vc8);
    if (more) {
      fetch_v(next);
      next = tile_slot(bt, a.bs_shift, min(t + 2, t1 - 1));
    }
    // scores in log2 units: lane column = head, rows = keys 16 kb + 4 g4 + r
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[kb][r] *= a.scale_log2;
    if (t == first || t == (p >> 6)) {
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = (t << 6) + 16 * kb + 4 * g4 + r;
          if (j < lo || j > p) S[kb][r] = -INFINITY;
        }
    }
    float mloc = S[0][0];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int r = 0; r < 4; ++r) mloc = fmaxf(mloc, S[kb][r]);
    mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float mn = fmaxf(mx, mloc);  // finite: every visited tile holds a visible key
    if (__any(mn > mx)) {
      const float alpha = fast_exp2(mx - mn);
      mx = mn;
      lsum *= alpha;
#pragma unroll
      for (int cb = 0; cb < NC; ++cb)
#pragma unroll
        for (int r = 0; r < 4; ++r) O[cb][r] *= alpha;
    }
    bf16x8_t Ph[2], Pl[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      float w8[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        w8[e] = fast_exp2(S[2 * kk + e / 4][e % 4] - mn);
        lsum += w8[e];
      }
      raw_u32x4 hi, lw;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        hi[e] = pack_bf16x2(w8[2 * e], w8[2 * e + 1]);
        lw[e] = pack_bf16x2(w8[2 * e] - bf16lo(hi[e]), w8[2 * e + 1] - bf16hi(hi[e]));
      }
      Ph[kk] = __builtin_bit_cast(bf16x8_t, hi);
      Pl[kk] = __builtin_bit_cast(bf16x8_t, lw);
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int cb = 0; cb < NC; ++cb) {
        const bf16x8_t vf = frag16(Vt + voff(16 * cb + c16, 4 * kk + g4));
        O[cb] = mma(vf, Ph[kk], O[cb]);
        O[cb] = mma(vf, Pl[kk], O[cb]);
      }
  }
  lsum += __shfl_xor(lsum, 16, 64);
  lsum += __shfl_xor(lsum, 32, 64);
  if (!okh) return;
  float* w = a.ws + (((int64_t)row * a.n_qh + qh) * a.parts + part) * (2 + DV);
  if (g4 == 0) {
    w[0] = mx * 0.6931471805599453f;
    w[1] = lsum;
  }
#pragma unroll
  for (int cb = 0; cb < NC; ++cb)
#pragma unroll
    for (int r = 0; r < 4; ++r) w[2 + cb * 16 + 4 * g4 + r] = O[cb][r];
}

struct StreamTileArgs {
  bf16_t* out;  // [T, n_qh, dv]
  const bf16_t* q;
  int64_t q_stride;
  const bf16_t* kc;
  const bf16_t* vc;
  const int64_t* pos;
  const int* seq;
  const int* bt;
  int bt_stride, bs_shift;
  const int* tiles;  // [n, 2]: first row, rows (up to 128) of one sequence
  int subs;          // workgroups per tile entry
  int n_qh, group;
  int Wk, Wv;
  float scale_log2;
  int mask, size;
};

template <int D, int DV, int HPW, bool FINE>
__global__ void __launch_bounds__(512, 2) stream_prefill_kernel(StreamTileArgs a) {
  constexpr int NK = D / 32, NC = DV / 16, RT = 8 / HPW, ROWS = 32 * RT;  // waves along the rows, rows per workgroup
  constexpr int KCH = D / 8, KI = 64 * KCH / 256;  // K items (16 bytes) per thread of the upper waves
  constexpr int VCH = DV / 8, VT = 16 * VCH;        // V items (4 keys x 8 columns), one per thread of the lower waves
  static_assert(VT <= 256 && 64 * KCH % 256 == 0, "one V item, whole K items per thread");
  __shared__ __attribute__((aligned(16))) bf16_t Ks[2][64 * D];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[2][DV * 64];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int yi = gridDim.y - 1 - blockIdx.y;  // later rows see more keys: hand them out first
  const int ti = yi / a.subs, off = (yi - ti * a.subs) * ROWS;
  const int n = a.tiles[2 * ti + 1] - off;
  if (n <= 0) return;
  const int row0 = a.tiles[2 * ti] + off;
  const int p0 = __builtin_amdgcn_readfirstlane((int)a.pos[row0]);
  const int* bt = a.bt + (int64_t)__builtin_amdgcn_readfirstlane(a.seq[row0]) * a.bt_stride;
  const int per = a.group / HPW;  // head blocks of a group
  const int g = blockIdx.x / per, qh = g * a.group + (blockIdx.x - g * per) * HPW + wave / RT;
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
  const bool upper = tid >= 256;
  const int ht = tid & 255;
  const bf16_t* kl = a.kc + (int64_t)g * D + (int64_t)(ht / KCH) * a.Wk + 8 * (ht % KCH);
  const bf16_t* vl = a.vc + (int64_t)g * DV + (int64_t)(4 * (ht / VCH)) * a.Wv + 8 * (ht % VCH);
  constexpr int SI = KI > 4 ? KI : 4;
  raw_u32x4 st[SI];
  auto fetch = [&](int t) {
    const int64_t base = tile_slot(bt, a.bs_shift, t);
    if (upper) {
#pragma unroll
      for (int i = 0; i < KI; ++i)
        st[i] = *reinterpret_cast<const raw_u32x4*>(kl + base * a.Wk + (int64_t)i * (256 / KCH) * a.Wk);
    } else if (VT == 256 || ht < VT) {
#pragma unroll
      for (int k = 0; k < 4; ++k) st[k] = *reinterpret_cast<const raw_u32x4*>(vl + base * a.Wv + (int64_t)k * a.Wv);
    }
  };
  auto commit = [&](int buf, int t) {
    if (upper) {
#pragma unroll
      for (int i = 0; i < KI; ++i)
        *reinterpret_cast<raw_u32x4*>(Ks[buf] + kimg<D>(ht / KCH + i * (256 / KCH), ht % KCH)) = st[i];
    } else if (VT == 256 || ht < VT) {
      if (t == last) {  // rows of the page behind the last query: stale values must not meet a zero weight
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if ((t << 6) + 4 * (ht / VCH) + k > hi) st[k] = raw_u32x4{0u, 0u, 0u, 0u};
      }
      put_v(Vt[buf], st, ht / VCH, ht % VCH);
    }
  };
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
    const bf16_t *K = Ks[cur], *V = Vt[cur];
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
    bf16x8_t P[2][2], Pl[2][2];  // weights (FINE: hi and lo)
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
        raw_u32x4 pk, pl;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float w0 = fast_exp2(fmaf(S[qb][2 * kk + e / 2][2 * (e % 2)], a.scale_log2, -mu));
          const float w1 = fast_exp2(fmaf(S[qb][2 * kk + e / 2][2 * (e % 2) + 1], a.scale_log2, -mu));
          add += w0 + w1;
          pk[e] = pack_bf16x2(w0, w1);
          if constexpr (FINE) pl[e] = pack_bf16x2(w0 - bf16lo(pk[e]), w1 - bf16hi(pk[e]));
        }
        P[qb][kk] = __builtin_bit_cast(bf16x8_t, pk);
        if constexpr (FINE) Pl[qb][kk] = __builtin_bit_cast(bf16x8_t, pl);
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
        if constexpr (FINE) {
          O[0][cb] = mma(vf, Pl[0][kk], O[0][cb]);
          O[1][cb] = mma(vf, Pl[1][kk], O[1][cb]);
        }
      }
  }
#pragma unroll
  for (int qb = 0; qb < 2; ++qb) {
    float l = lsum[qb];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    const int r = rw + 16 * qb + c16;
    if (r >= n) continue;
    const float inv = 1.f / l;
    bf16_t* o = a.out + ((int64_t)(row0 + r) * a.n_qh + qh) * DV + 4 * g4;
#pragma unroll
    for (int cb = 0; cb < NC; ++cb)
      *reinterpret_cast<uint2*>(o + 16 * cb) = uint2{pack_bf16x2(O[qb][cb][0] * inv, O[qb][cb][1] * inv),
                                                     pack_bf16x2(O[qb][cb][2] * inv, O[qb][cb][3] * inv)};
  }
}

template <int D, int HPW, bool FINE> void launch_stream_prefill(const StreamTileArgs& a0, int n_tiles, hipStream_t st) {
  StreamTileArgs a = a0;
  a.subs = 128 / (32 * (8 / HPW));
  const int step = 65535 / a.subs;
  for (int t0 = 0; t0 < n_tiles; t0 += step) {
    a.tiles = a0.tiles + 2 * t0;
    const int nt = n_tiles - t0 < step ? n_tiles - t0 : step;
    hipLaunchKernelGGL((stream_prefill_kernel<D, D, HPW, FINE>), dim3(a.n_qh / HPW, nt * a.subs), dim3(512), 0, st, a);
  }
}

}  // namespace

extern "C" {

// 1 when the prompt kernel takes these heads: one map, an even number of heads per key/value head
int dxm_stream_prefill_ok(int d, int dv, int maps, int group, int bs, int mask) {
  return ((d == 128 && dv == 128) || (d == 64 && dv == 64)) && maps == 1 && group % 2 == 0 && bs >= 64 &&
         (bs & (bs - 1)) == 0 && mask >= 0 && mask <= 2;
}

int dxm_stream_prefill(void* out, const void* q, int64_t q_stride, const void* kc, const void* vc, const int64_t* pos,
                       const int* seq, const int* bt, int bt_stride, int bs, const int* tiles, int n_tiles, int n_qh,
                       int group, int d, int dv, int Wk, int Wv, float scale, int mask, int size, int fine,
                       hipStream_t st) {
  if (n_tiles <= 0) return 0;
  if (!dxm_stream_prefill_ok(d, dv, 1, group, bs, mask)) return 2;
  if (n_qh < 1 || n_qh % group) return 1;
  if ((mask && size < 1) || !(scale > 0.f)) return 3;
  if (!out || !seq || !tiles || Wk % 8 || Wv % 8 || q_stride % 8 || (uintptr_t)q % 16 || (uintptr_t)kc % 16 ||
      (uintptr_t)vc % 16 || (uintptr_t)out % 8)
    return 4;
  StreamTileArgs a{(bf16_t*)out, (const bf16_t*)q, q_stride, (const bf16_t*)kc, (const bf16_t*)vc, pos, seq, bt, bt_stride,
                   __builtin_ctz((unsigned)bs), tiles, 1, n_qh, group, Wk, Wv, scale * 1.4426950408889634f,
                   mask, size};
#define STREAM_PREFILL(D, HPW)                                  \
  if (fine) launch_stream_prefill<D, HPW, true>(a, n_tiles, st); \
  else launch_stream_prefill<D, HPW, false>(a, n_tiles, st);
  if (d == 128 && group % 4 == 0) { STREAM_PREFILL(128, 4) }
  else if (d == 128) { STREAM_PREFILL(128, 2) }
  else if (group % 4 == 0) { STREAM_PREFILL(64, 4) }
  else { STREAM_PREFILL(64, 2) }
#undef STREAM_PREFILL
  DX_CHECK_LAUNCH();
  return 0;
}

// 1 when the decode kernel takes these heads: widths it is instantiated for, pages of whole 64-key tiles
int dxm_stream_decode_ok(int d, int dv, int group, int bs, int mask) {
  return ((d == 128 && dv == 128) || (d == 64 && dv == 64)) && group >= 1 && group <= 16 && bs >= 64 &&
         (bs & (bs - 1)) == 0 && mask >= 0 && mask <= 2;
}

int dxm_stream_decode(float* ws, const void* q, int64_t q_stride, const void* kc, const void* vc, const int64_t* pos,
                      const int* seq, const int* bt, int bt_stride, int bs, int rows, int n_qh, int maps, int group, int d,
                      int dv, int Wk, int Wv, float scale, int mask, int size, int parts, hipStream_t st) {
  if (rows <= 0) return 0;
  if (!dxm_stream_decode_ok(d, dv, group, bs, mask)) return 2;
  if (n_qh < 1 || maps < 1 || n_qh % maps || (n_qh / maps) % group || rows > 65535) return 1;
  if ((mask && size < 1) || parts < 1 || parts > 65535 || !(scale > 0.f)) return 3;
  if (!ws || Wk % 8 || Wv % 8 || q_stride % 8 || (uintptr_t)q % 16 || (uintptr_t)kc % 16 || (uintptr_t)vc % 16) return 4;
  StreamArgs a{(const bf16_t*)q, q_stride, (const bf16_t*)kc, (const bf16_t*)vc, ws, pos, seq, bt, bt_stride,
               __builtin_ctz((unsigned)bs), n_qh, maps, group, Wk, Wv, scale * 1.4426950408889634f, mask, size, parts};
  const dim3 grid(n_qh / group, rows, parts);
  if (d == 128) hipLaunchKernelGGL((stream_decode_kernel<128, 128>), grid, dim3(64), 0, st, a);
  else hipLaunchKernelGGL((stream_decode_kernel<64, 64>), grid, dim3(64), 0, st, a);
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
