// Differential attention: every head holds two softmax maps over the same
// values, combined as a_1 - lambda a_2 and RMS-normed per head. Queries, keys
// and values pass a short causal convolution on the way in. The kernels:
//   conv_qkv_store   convolution of a fused q | k | v projection, k and v into
//                    the paged caches, q times the query temperature (one launch)
//   attn_diff_paged  both maps, the combination and the norm over the paged
//                    cache, plain causal
//     - a plain kernel (any size, bf16 or fp32; the exact-mode path)
//     - MFMA kernels (bf16): query tiles of prompt portions, and a form for
//       single rows whose keys are shared out over the chip.
// Cache layout: keys [NB, G, BS, 2 D] = [map 1 | map 2] per head and token,
// values [NB, G, BS, V]. Scores, softmax weights, running sums, the
// combination and its norm are fp32 everywhere.

#include "seq_common.h"

#define DISPATCH_T(is_f32, ...)                                  \
  if (is_f32) { typedef float T; __VA_ARGS__ } else { typedef bfraw T; __VA_ARGS__ }

template <int VEC, typename T>
__device__ __forceinline__ void ldv(const T* p, float v[VEC]) {
  if constexpr (VEC == 8) ld8(p, v); else v[0] = ldf(p);
}
template <int VEC, typename T>
__device__ __forceinline__ void stv(T* p, const float v[VEC]) {
  if constexpr (VEC == 8) st8(p, v); else stf(p, v[0]);
}

// ---- step input: short convolution, query temperature, paged store -----------------
// A thread owns VEC columns of `run` consecutive rows. KT > 0: up to KT taps with
// the taps and the last KT rows in registers (missing leading taps are zero);
// KT == 0: any number of taps, rows re-read. Rows before a segment come from
// hist [slot, K-1, C] (oldest first), zeros for a fresh sequence. Columns
// [qo, qo + qn) go to q_out times 1 + coef ln(floor((p + 1) / every) + 1);
// [ko, ko + kn) and [vo, vo + vn) to the caches; the rest are alignment gaps.
// single: every segment is one row, and the thread moves its columns' history on.
template <typename T, int VEC, int KT>
__global__ void __launch_bounds__(256) conv_qkv_store_kernel(
    T* __restrict__ q_out, const T* __restrict__ y, const float* __restrict__ w, T* __restrict__ hist_,
    const int* __restrict__ slots, const int* __restrict__ cu, const int* __restrict__ seg_start,
    const int* __restrict__ token_seg, const int64_t* __restrict__ positions, T* __restrict__ kc, T* __restrict__ vc,
    const int64_t* __restrict__ slot_map, int T_, int C, int K, int y_stride, int qo, int qn, int ko, int kn, int vo,
    int vn, int D2, int V, int G, int BS, float coef, int every, int run, int single) {
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (c >= C) return;
  const bool isq = c >= qo && c < qo + qn, isk = kn > 0 && c >= ko && c < ko + kn, isv = vn > 0 && c >= vo && c < vo + vn;
  if (!isq && !isk && !isv) return;
  T* cache = isk ? kc : vc;
  const int hw = isk ? D2 : V;                        // row width of one cached head
  const int cc = isk ? c - ko : c - vo;
  const int g = (isk || isv) ? cc / hw : 0, ce = cc - g * hw;
  constexpr int KW = KT > 0 ? KT : 1;
  float wt[KW][VEC], win[KW][VEC];
  if (KT > 0) {
#pragma unroll
    for (int j = 0; j < KW; ++j) {
      const int src = j - (KW - K);                   // tap index, aligned to the last one
#pragma unroll
      for (int e = 0; e < VEC; ++e) wt[j][e] = 0.f;
      if (src >= 0) ldv<VEC>(w + (int64_t)src * C + c, wt[j]);
    }
  }
  const int t0 = blockIdx.y * run, t1 = min(T_, t0 + run);
  for (int t = t0; t < t1; ++t) {
    const int b = token_seg[t];
    const int i = t - cu[b];
    const bool fresh = seg_start[b] == 0;
    T* hist = hist_ + (int64_t)slots[b] * (K - 1) * C + c;
    float acc[VEC];
    if (KT > 0) {
      if (t == t0 || i == 0) {                        // the window anew
#pragma unroll
        for (int j = 0; j < KW - 1; ++j) {
          const int back = KW - 1 - j;                // rows before t
#pragma unroll
          for (int e = 0; e < VEC; ++e) win[j][e] = 0.f;
          if (back <= K - 1) {
            if (i - back >= 0) ldv<VEC>(y + (int64_t)(t - back) * y_stride + c, win[j]);
            else if (!fresh) ldv<VEC>(hist + (int64_t)(K - 1 + i - back) * C, win[j]);
          }
        }
      } else {
#pragma unroll
        for (int j = 0; j < KW - 1; ++j)
#pragma unroll
          for (int e = 0; e < VEC; ++e) win[j][e] = win[j + 1][e];
      }
      ldv<VEC>(y + (int64_t)t * y_stride + c, win[KW - 1]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
#pragma unroll
      for (int j = 0; j < KW; ++j)
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] += wt[j][e] * win[j][e];
      if (single) {
#pragma unroll
        for (int j = 1; j < KW; ++j)
          if (j - (KW - K) >= 1) stv<VEC>(hist + (int64_t)(j - (KW - K) - 1) * C, win[j]);
      }
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
      for (int j = 0; j < K; ++j) {
        const int src = i - (K - 1 - j);
        float xv[VEC], wv[VEC];
        if (src >= 0) ldv<VEC>(y + (int64_t)(t - (K - 1 - j)) * y_stride + c, xv);
        else if (!fresh) ldv<VEC>(hist + (int64_t)(K - 1 + src) * C, xv);
        else continue;
        ldv<VEC>(w + (int64_t)j * C + c, wv);
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] += wv[e] * xv[e];
      }
      if (single) {                                   // oldest first: every row is read before it is overwritten
        float xv[VEC];
        for (int j = 0; j < K - 1; ++j) {
          if (j == K - 2) ldv<VEC>(y + (int64_t)t * y_stride + c, xv);
          else if (!fresh) ldv<VEC>(hist + (int64_t)(j + 1) * C, xv);
          else {
#pragma unroll
            for (int e = 0; e < VEC; ++e) xv[e] = 0.f;
          }
          stv<VEC>(hist + (int64_t)j * C, xv);
        }
      }
    }
    if (isq) {
      if (coef != 0.f) {
        const float temp = 1.0f + coef * logf((float)((positions[t] + 1) / every + 1));
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] *= temp;
      }
      stv<VEC>(q_out + (int64_t)t * qn + (c - qo), acc);
    } else {
      const int64_t s = slot_map[t], blk = s / BS, off = s - blk * BS;
      stv<VEC>(cache + ((blk * G + g) * BS + off) * hw + ce, acc);
    }
  }
}

// ---- plain attention kernel ----------------------------------------------------------
// grid (T, H), one wave per (query row, head). Visible keys 0..p in tiles of 64:
// lane u scores key tile*64 + u under both maps against the query staged in LDS,
// the weights go through LDS, then lanes own output dims and sweep the tile's
// value rows once for both maps.
#define DIFF_MAX_ACC 8   // V <= 512
template <typename T>
__global__ void __launch_bounds__(WAVE) attn_diff_paged_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ kc, const T* __restrict__ vc,
    const int* __restrict__ block_tables, const int* __restrict__ token_seg, const int64_t* __restrict__ positions,
    float scale, float lam, float oscale, float eps, int H, int G, int D, int V, int BS, int bt_stride, int q_stride,
    int k4) {
  extern __shared__ float lds[];       // query [2 D] | weights [2][64] | cache row index [64] (as int)
  float* qs = lds;
  float* ps = lds + 2 * D;
  int* rows = (int*)(ps + 2 * WAVE);
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, g = h / (H / G);
  const int total = (int)positions[t] + 1;
  const int* bt = block_tables + (int64_t)token_seg[t] * bt_stride;
  const T* qr = q + (int64_t)t * q_stride + (int64_t)h * 2 * D;
  for (int i = lane; i < 2 * D; i += WAVE) qs[i] = ldf(qr + i);
  __syncthreads();
  float acc[2][DIFF_MAX_ACC], m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int i = 0; i < DIFF_MAX_ACC; ++i) acc[0][i] = acc[1][i] = 0.f;
  for (int base = 0; base < total; base += WAVE) {
    const int j = base + lane;
    float s[2] = {-INFINITY, -INFINITY};
    int row = 0;
    if (j < total) {
      row = (bt[j / BS] * G + g) * BS + (j % BS);
      const T* kr = kc + (int64_t)row * 2 * D;
#pragma unroll
      for (int mp = 0; mp < 2; ++mp) {
        const T* kp = kr + mp * D;
        const float* qp = qs + mp * D;
        float d = 0.f;
        if (k4) {
          for (int i = 0; i < D; i += 8) {
            float kv[8];
            ld8(kp + i, kv);
#pragma unroll
            for (int e = 0; e < 8; ++e) d += qp[i + e] * kv[e];
          }
        } else {
          for (int i = 0; i < D; ++i) d += qp[i] * ldf(kp + i);
        }
        s[mp] = d * scale;
      }
    }
    float corr[2];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
      const float m_new = fmaxf(m[mp], wave_max(s[mp]));
      const float wgt = j < total ? expf(s[mp] - m_new) : 0.f;
      corr[mp] = expf(m[mp] - m_new);                  // m = -inf on the first tile -> 0
      l[mp] = l[mp] * corr[mp] + wave_sum(wgt);
      m[mp] = m_new;
      ps[mp * WAVE + lane] = wgt;
    }
    rows[lane] = row;
    __syncthreads();
    const int n = min(WAVE, total - base);
#pragma unroll
    for (int i = 0; i < DIFF_MAX_ACC; ++i) { acc[0][i] *= corr[0]; acc[1][i] *= corr[1]; }
    for (int jj = 0; jj < n; ++jj) {
      const float p0 = ps[jj], p1 = ps[WAVE + jj];
      const T* vr = vc + (int64_t)rows[jj] * V;
#pragma unroll
      for (int i = 0; i < DIFF_MAX_ACC; ++i) {
        const int d = lane + i * WAVE;
        if (d < V) {
          const float v = ldf(vr + d);
          acc[0][i] += p0 * v;
          acc[1][i] += p1 * v;
        }
      }
    }
    __syncthreads();
  }
  const float i0 = 1.0f / l[0], i1 = lam / l[1];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < DIFF_MAX_ACC; ++i) {
    const float o = acc[0][i] * i0 - acc[1][i] * i1;   // dims beyond V hold zeros
    acc[0][i] = o;
    ss += o * o;
  }
  const float r = oscale / sqrtf(wave_sum(ss) / (float)V + eps);
  T* orow = out + ((int64_t)t * H + h) * V;
#pragma unroll
  for (int i = 0; i < DIFF_MAX_ACC; ++i) {
    const int d = lane + i * WAVE;
    if (d < V) stf(orow + d, acc[0][i] * r);
  }
}

// ---- MFMA attention kernels (bf16) ------------------------------------------------------
// v_mfma_f32_32x32x16_bf16 fragment maps:
//   A[i][k]: lane l holds i = l&31, k = (l>>5)*8 + j   (j = 0..7)
//   B[k][j]: lane l holds j = l&31, k = (l>>5)*8 + jj
//   C[i][j]: lane l holds j = l&31, i = (r&3) + 8*(r>>2) + 4*(l>>5)  (r = 0..15)
//
// All waves of a workgroup share staged tiles of 64 keys of one key/value head:
// the keys of both maps row by row (rows padded: 16-byte reads spread over the
// banks), the values transposed (pairs of keys packed, so a wave's stores spread
// too). The next tile's rows are on their way from memory meanwhile. A wave
// serves 32 query columns under ONE map:
//   S^T[key][col] = keys x query^T; a column's scores sit in a lane pair
//   (l, l ^ 32), so the online softmax is lane-local; O^T[d][col] += V^T x P
//   with P as a sum of two bf16 parts (the rounding of p and the rounding of
//   what that left): the weights keep 16 bits of mantissa.
// Form 0, query tiles (8 waves): four column tiles of 32 rows of one segment
// and one head each (heads of the key/value head side by side, or consecutive
// rows); the two waves of a column tile meet through LDS: combination, norm, store.
// Form 1, single rows (8 waves): the columns are the key/value head's query
// heads; per map two pairs of waves take half of each tile's keys each and deal
// the output tiles to the pair; gridDim.z workgroups take contiguous shares of the row's tiles and leave unnormalised partial
// results that attn_diff_merge_kernel combines in a fixed order.
typedef __bf16 df_bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 df_bf16x2 __attribute__((ext_vector_type(2)));
typedef float df_f32x16 __attribute__((ext_vector_type(16)));
typedef float df_f32x2 __attribute__((ext_vector_type(2)));

#define DIFF_KT 64           // keys per staged tile
#define DIFF_KPAD 8          // elements of padding per staged key row
#define DIFF_VS 72           // row stride of the transposed values: 64 keys + 8
#define DIFF_MAX_SPLIT 64
#define LOG2E 1.4426950408889634f

__device__ __forceinline__ int df_acc_row(int r, int half) { return (r & 3) + 8 * (r >> 2) + 4 * half; }

__device__ __forceinline__ uint32_t df_pack(float a, float b) {
  const df_f32x2 v = {a, b};
  df_bf16x2 r = __builtin_convertvector(v, df_bf16x2);
  return *reinterpret_cast<uint32_t*>(&r);
}
// max / sum over a lane and its partner in the other half
__device__ __forceinline__ float df_pair_max(float v) {
  auto sw = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(sw[0]), __uint_as_float(sw[1]));
}
__device__ __forceinline__ float df_pair_sum(float v) {
  auto sw = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(sw[0]) + __uint_as_float(sw[1]);
}
// workgroup barrier that orders LDS traffic only; global loads stay in flight
__device__ __forceinline__ void df_lds_barrier() {
  asm volatile("" ::: "memory");
  __builtin_amdgcn_s_waitcnt(0xc07f);      // vmcnt 63, expcnt 7, lgkmcnt 0
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
// 8 elements p[d .. d + 7] of a row of n (n a multiple of 8; zeros beyond it)
__device__ __forceinline__ uint4 df_load8(const bfraw* p, int d, int n) {
  return d < n ? *reinterpret_cast<const uint4*>(p + d) : make_uint4(0, 0, 0, 0);
}

template <int NSL, int NDT, bool SINGLE>
__global__ void __launch_bounds__(512, 2) attn_diff_mfma_kernel(
    bfraw* __restrict__ out, const bfraw* __restrict__ q, const bfraw* __restrict__ kc, const bfraw* __restrict__ vc,
    const int* __restrict__ block_tables, const int* __restrict__ token_seg, const int64_t* __restrict__ positions,
    const int* __restrict__ tiles, float scale, float lam, float oscale, float eps, int H, int G, int D, int V, int BS,
    int bt_stride, int q_stride, int hb, float* __restrict__ part_o, float* __restrict__ part_ml) {
  constexpr int NT = 512;
  constexpr int ODT = SINGLE ? NDT / 2 : NDT;         // 32-dim output tiles per wave: single rows deal them to two waves
  constexpr int TPK = NT / DIFF_KT;                   // threads per staged key
  constexpr int KI = 4 * NSL / TPK;                   // 16-byte key chunks per thread
  constexpr int VC = NT / 32;                         // 8-dim value chunks per pass
  constexpr int VI = (NDT * 4 + VC - 1) / VC;
  extern __shared__ __align__(16) unsigned char df_smem[];
  const int nsl = (D + 15) / 16, Dp = nsl * 16, ndt = (V + 31) / 32;
  const int KS = 2 * Dp + DIFF_KPAD;
  bfraw* k_lds = reinterpret_cast<bfraw*>(df_smem);                                         // [64][KS]
  bfraw* v_lds = reinterpret_cast<bfraw*>(df_smem + (size_t)DIFF_KT * KS * 2);              // [ndt*32][72]
  float* x_lds = reinterpret_cast<float*>(df_smem);                                         // epilogue: [tiles][16][64]

  const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
  const int half = lane >> 5, col = lane & 31;
  const int map = wave & 1, sub = SINGLE ? (wave >> 1) & 1 : wave >> 1, dg = SINGLE ? wave >> 2 : 0;
  constexpr int DG = SINGLE ? 2 : 1;                  // this wave's output tiles: i * DG + dg
  const int R = H / G, nhb = (R + hb - 1) / hb;
  const int g = blockIdx.x / nhb, hblk = blockIdx.x - g * nhb;
  const int h0 = g * R + hblk * hb, nh = min(hb, R - hblk * hb);

  // rows of this workgroup, this lane's column
  int row0, nrows, crow, chead;
  bool cvalid, active;
  if (SINGLE) {
    row0 = tiles != nullptr ? tiles[blockIdx.y] : (int)blockIdx.y;
    nrows = 1;
    cvalid = col < nh;
    chead = h0 + (cvalid ? col : 0);
    crow = row0;
    active = true;
  } else {
    row0 = tiles[2 * blockIdx.y];
    nrows = tiles[2 * blockIdx.y + 1];
    const int rt = sub / hb, hi = sub - rt * hb;       // hb is 1, 2 or 4 here
    active = hi < nh && rt * 32 < nrows;
    cvalid = active && rt * 32 + col < nrows;
    chead = h0 + (hi < nh ? hi : 0);
    crow = row0 + min(rt * 32 + col, nrows - 1);
  }
  const int cpos = (int)positions[crow];
  const int p_last = (int)positions[row0 + nrows - 1];
  const int w_last = SINGLE ? p_last : (int)positions[row0 + min((sub / hb) * 32 + 31, nrows - 1)];
  const int* bt = block_tables + (int64_t)token_seg[row0] * bt_stride;
  int k_begin = 0, k_end = p_last + 1;
  if (SINGLE) {
    const int ntl = p_last / DIFF_KT + 1, tps = (ntl + gridDim.z - 1) / gridDim.z;
    k_begin = (int)blockIdx.z * tps * DIFF_KT;
    k_end = min(k_end, k_begin + tps * DIFF_KT);
  }

  df_bf16x8 q_frag[NSL];
  {
    const bfraw* qp = q + (int64_t)crow * q_stride + ((int64_t)chead * 2 + map) * D;
#pragma unroll
    for (int s = 0; s < NSL; ++s) {
      uint4 val = df_load8(qp, s * 16 + half * 8, D);
      q_frag[s] = *reinterpret_cast<df_bf16x8*>(&val);
    }
  }
  df_f32x16 o_acc[ODT];
#pragma unroll
  for (int i = 0; i < ODT; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o_acc[i][r] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;
  const float scale2 = scale * LOG2E;

  // staging roles: keys — TPK threads per key; values — pairs of keys x 8 dims, 4 lanes on neighbouring chunks
  const int skey = tid / TPK, spart = tid % TPK;
  const int vkp = (tid >> 2) & 31, vch = (tid & 3) + 4 * (tid >> 7);
  uint4 kst[KI], vst[VI][2];
  auto fetch = [&](int kt0) {
    const int nk = min(DIFF_KT, k_end - kt0);
    {
      const int j = kt0 + min(skey, nk - 1);
      const bfraw* src = kc + ((int64_t)(bt[j / BS] * G + g) * BS + (j % BS)) * (2 * D);
#pragma unroll
      for (int i = 0; i < KI; ++i) {
        const int c = spart + i * TPK, mp = c >= 2 * nsl ? 1 : 0, d8 = (c - mp * 2 * nsl) * 8;
        kst[i] = skey < nk && c < 4 * nsl ? df_load8(src + mp * D, d8, D) : make_uint4(0, 0, 0, 0);
      }
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int key = 2 * vkp + u, j = kt0 + min(key, nk - 1);
      const bfraw* src = vc + ((int64_t)(bt[j / BS] * G + g) * BS + (j % BS)) * V;
#pragma unroll
      for (int i = 0; i < VI; ++i)
        vst[i][u] = key < nk ? df_load8(src, (vch + i * VC) * 8, V) : make_uint4(0, 0, 0, 0);
    }
  };
  if (k_begin < k_end) fetch(k_begin);
  for (int kt0 = k_begin; kt0 < k_end; kt0 += DIFF_KT) {
#pragma unroll
    for (int i = 0; i < KI; ++i) {
      const int c = spart + i * TPK;
      if (c < 4 * nsl) *reinterpret_cast<uint4*>(k_lds + skey * KS + c * 8) = kst[i];
    }
#pragma unroll
    for (int i = 0; i < VI; ++i) {
      const int c = vch + i * VC;
      if (c < ndt * 4) {
        const uint32_t* a = reinterpret_cast<const uint32_t*>(&vst[i][0]);
        const uint32_t* b = reinterpret_cast<const uint32_t*>(&vst[i][1]);
        uint32_t* dst = reinterpret_cast<uint32_t*>(v_lds + c * 8 * DIFF_VS) + vkp;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          dst[(2 * j) * (DIFF_VS / 2)] = (a[j] & 0xffffu) | (b[j] << 16);
          dst[(2 * j + 1) * (DIFF_VS / 2)] = (a[j] >> 16) | (b[j] & 0xffff0000u);
        }
      }
    }
    df_lds_barrier();
    if (kt0 + DIFF_KT < k_end) fetch(kt0 + DIFF_KT);
#pragma unroll 1
    for (int ks = SINGLE ? sub : 0; ks < (SINGLE ? sub + 1 : 2); ++ks) {
      const int kt = kt0 + ks * 32;
      if (!active || kt > w_last) continue;            // wave-uniform
      df_f32x16 s_acc;
#pragma unroll
      for (int r = 0; r < 16; ++r) s_acc[r] = 0.f;
      const bfraw* kr = k_lds + (ks * 32 + col) * KS + map * Dp + half * 8;
#pragma unroll
      for (int s = 0; s < NSL; ++s) {
        if (s < nsl) {
          const df_bf16x8 a = *reinterpret_cast<const df_bf16x8*>(kr + s * 16);
          s_acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, q_frag[s], s_acc, 0, 0, 0);
        }
      }
      float p[16], tmax = -INFINITY;
      const int room = cpos - kt;                      // keys kt + 0 .. kt + room are visible
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        p[r] = df_acc_row(r, half) <= room ? s_acc[r] * scale2 : -INFINITY;   // in units of ln 2
        tmax = fmaxf(tmax, p[r]);
      }
      const float m_new = fmaxf(m_run, df_pair_max(tmax));
      const float m_ref = m_new == -INFINITY ? 0.f : m_new;      // nothing seen yet: weights 2^-inf = 0
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_ref);
      m_run = m_new;
      float psum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        p[r] = __builtin_amdgcn_exp2f(p[r] - m_ref);
        psum += p[r];
      }
      l_run = l_run * alpha + psum;
      if (__builtin_amdgcn_ballot_w64(alpha != 1.0f)) {          // the running maximum moved in some column
#pragma unroll
        for (int i = 0; i < ODT; ++i)
#pragma unroll
          for (int r = 0; r < 16; ++r) o_acc[i][r] *= alpha;
      }
      // P as two bf16 parts; half swaps turn the accumulator layout into B fragments
      uint32_t hi[8], lo[8];
#pragma unroll
      for (int pr = 0; pr < 8; ++pr) {
        hi[pr] = df_pack(p[2 * pr], p[2 * pr + 1]);
        lo[pr] = df_pack(p[2 * pr] - __uint_as_float(hi[pr] << 16),
                         p[2 * pr + 1] - __uint_as_float(hi[pr] & 0xffff0000u));
      }
      df_bf16x8 pf[2][2];
#pragma unroll
      for (int k2 = 0; k2 < 2; ++k2) {
        auto h0_ = __builtin_amdgcn_permlane32_swap(hi[4 * k2], hi[4 * k2 + 2], false, false);
        auto h1_ = __builtin_amdgcn_permlane32_swap(hi[4 * k2 + 1], hi[4 * k2 + 3], false, false);
        auto l0_ = __builtin_amdgcn_permlane32_swap(lo[4 * k2], lo[4 * k2 + 2], false, false);
        auto l1_ = __builtin_amdgcn_permlane32_swap(lo[4 * k2 + 1], lo[4 * k2 + 3], false, false);
        uint4 wh = make_uint4(h0_[0], h1_[0], h0_[1], h1_[1]), wl = make_uint4(l0_[0], l1_[0], l0_[1], l1_[1]);
        pf[k2][0] = *reinterpret_cast<df_bf16x8*>(&wh);
        pf[k2][1] = *reinterpret_cast<df_bf16x8*>(&wl);
      }
      const bfraw* vr = v_lds + col * DIFF_VS + ks * 32 + half * 8;
#pragma unroll
      for (int i = 0; i < ODT; ++i) {
        if (i * DG + dg < ndt) {
#pragma unroll
          for (int k2 = 0; k2 < 2; ++k2) {
            const df_bf16x8 a = *reinterpret_cast<const df_bf16x8*>(vr + (i * DG + dg) * 32 * DIFF_VS + k2 * 16);
            o_acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pf[k2][0], o_acc[i], 0, 0, 0);
            o_acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pf[k2][1], o_acc[i], 0, 0, 0);
          }
        }
      }
    }
    df_lds_barrier();
  }
  l_run = df_pair_sum(l_run);

  if (SINGLE) {
    // the two halves of the keys meet: x_lds [2 tile sets][2 maps][16][64] per output tile, (max, sum) of the second behind it
    float* ml = x_lds + 4 * 16 * WAVE;
    if (sub == 1 && dg == 0 && half == 0) { ml[(map * 32 + col) * 2] = m_run; ml[(map * 32 + col) * 2 + 1] = l_run; }
    df_lds_barrier();
    const float m1 = ml[(map * 32 + col) * 2], l1 = ml[(map * 32 + col) * 2 + 1];
    const float M = fmaxf(m_run, m1), M_ref = M == -INFINITY ? 0.f : M;
    const float f0 = __builtin_amdgcn_exp2f(m_run - M_ref), f1 = __builtin_amdgcn_exp2f(m1 - M_ref);
    const int64_t slot = (((int64_t)blockIdx.y * H + chead) * 2 + map) * gridDim.z + blockIdx.z;
    if (sub == 0 && dg == 0 && cvalid && half == 0) {
      part_ml[2 * slot] = M;
      part_ml[2 * slot + 1] = l_run * f0 + l1 * f1;
    }
    float* po = part_o + slot * V;
    float* xw = x_lds + (dg * 2 + map) * 16 * WAVE + lane;
#pragma unroll
    for (int i = 0; i < ODT; ++i) {
      if (i * DG < ndt) {                              // the same for both tile sets: barriers inside
        if (sub == 1) {
#pragma unroll
          for (int r = 0; r < 16; ++r) xw[r * WAVE] = o_acc[i][r];
        }
        df_lds_barrier();
        if (sub == 0 && cvalid) {
#pragma unroll
          for (int g4 = 0; g4 < 4; ++g4) {             // regs 4 g4 .. 4 g4 + 3 hold 4 consecutive dims
            const int d = (i * DG + dg) * 32 + 8 * g4 + 4 * half;
            if (d < V)                                 // V is a multiple of 8
              *reinterpret_cast<float4*>(po + d) =
                  make_float4(o_acc[i][4 * g4] * f0 + xw[(4 * g4) * WAVE] * f1,
                              o_acc[i][4 * g4 + 1] * f0 + xw[(4 * g4 + 1) * WAVE] * f1,
                              o_acc[i][4 * g4 + 2] * f0 + xw[(4 * g4 + 2) * WAVE] * f1,
                              o_acc[i][4 * g4 + 3] * f0 + xw[(4 * g4 + 3) * WAVE] * f1);
          }
        }
        df_lds_barrier();
      }
    }
    return;
  }

  // query tiles: map 2's waves hand their outputs over, map 1's combine, norm and store
  const float inv = l_run > 0.f ? 1.0f / l_run : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < ODT; ++i) {
    if (i < ndt) {
      if (map == 1) {
#pragma unroll
        for (int r = 0; r < 16; ++r) x_lds[(sub * 16 + r) * WAVE + lane] = o_acc[i][r] * inv;
      }
      df_lds_barrier();
      if (map == 0) {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float o = o_acc[i][r] * inv - lam * x_lds[(sub * 16 + r) * WAVE + lane];
          o_acc[i][r] = o;                             // dims beyond V hold zeros
          ss += o * o;
        }
      }
      df_lds_barrier();
    }
  }
  if (map == 1) return;
  const float rs = oscale / sqrtf(df_pair_sum(ss) / (float)V + eps);
  if (!cvalid) return;
  bfraw* orow = out + ((int64_t)crow * H + chead) * V;
#pragma unroll
  for (int i = 0; i < ODT; ++i) {
    if (i < ndt) {
#pragma unroll
      for (int g4 = 0; g4 < 4; ++g4) {
        const int d = i * 32 + 8 * g4 + 4 * half;
        if (d < V) {                                   // V is a multiple of 8
          uint2 wd;
          wd.x = df_pack(o_acc[i][4 * g4] * rs, o_acc[i][4 * g4 + 1] * rs);
          wd.y = df_pack(o_acc[i][4 * g4 + 2] * rs, o_acc[i][4 * g4 + 3] * rs);
          *reinterpret_cast<uint2*>(orow + d) = wd;
        }
      }
    }
  }
}

// Merge of the key shares of single rows: grid (rows, H), 256 threads. Shares'
// factors 2^(m_z - M) per map go through LDS; threads own output dims and sum
// the shares in a fixed order; then the combination and its norm.
__global__ void __launch_bounds__(256) attn_diff_merge_kernel(
    bfraw* __restrict__ out, const float* __restrict__ part_o, const float* __restrict__ part_ml,
    const int* __restrict__ row_map, float lam, float oscale, float eps, int H, int V, int ns) {
  __shared__ float fz[2][DIFF_MAX_SPLIT];
  __shared__ float scratch[16];
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lane = tid & (WAVE - 1), wave = tid / WAVE;
  const int64_t base = ((int64_t)n * H + h) * 2 * ns;
  if (wave < 2) {                                      // wave m: map m's shares, one per lane
    const float* ml = part_ml + 2 * (base + (int64_t)wave * ns);
    const float m = lane < ns ? ml[2 * lane] : -INFINITY;
    const float l = lane < ns ? ml[2 * lane + 1] : 0.f;
    const float M = wave_max(m);
    const float f = l > 0.f ? __builtin_amdgcn_exp2f(m - M) : 0.f;
    const float L = wave_sum(l * f);
    if (lane < ns) fz[wave][lane] = f * ((wave == 0 ? 1.0f : lam) / L);
  }
  __syncthreads();
  const float* p0 = part_o + base * V;
  const float* p1 = p0 + (int64_t)ns * V;
  float ss = 0.f, o = 0.f;
  for (int d = tid; d < V; d += 256) {                 // V <= 256: one pass
    float a0 = 0.f, a1 = 0.f;
#pragma unroll 4
    for (int z = 0; z < ns; ++z) {
      a0 += p0[(int64_t)z * V + d] * fz[0][z];
      a1 += p1[(int64_t)z * V + d] * fz[1][z];
    }
    o = a0 - a1;
    ss = o * o;
  }
  ss = block_sum(ss, scratch);
  const int64_t row = row_map != nullptr ? row_map[n] : n;
  if (tid < V) stf(out + (row * H + h) * V + tid, o * (oscale / sqrtf(ss / (float)V + eps)));
}

// ---- launchers ---------------------------------------------------------------------------
extern "C" void seq_launch_conv_state_update(const void*, void*, const int*, const int*, const int*, int, int, int,
                                             int, int, hipStream_t);

extern "C" void seq_launch_conv_qkv_store(void* q_out, const void* y, const float* w, void* hist, const int* slots,
                                          const int* cu, const int* seg_start, const int* token_seg,
                                          const int64_t* positions, void* kc, void* vc, const int64_t* slot_map,
                                          int T_, int B, int C, int K, int y_stride, int qo, int qn, int ko, int kn,
                                          int vo, int vn, int D2, int V, int G, int BS, float coef, int every,
                                          int single, int is_f32, hipStream_t st) {
  bool v8 = C % 8 == 0 && y_stride % 8 == 0 && qo % 8 == 0 && qn % 8 == 0 && aligned16(q_out) && aligned16(y) &&
            aligned16(w) && aligned16(hist);
  if (kn > 0) v8 = v8 && ko % 8 == 0 && vo % 8 == 0 && D2 % 8 == 0 && V % 8 == 0 && aligned16(kc) && aligned16(vc);
  const int gx = (C / (v8 ? 8 : 1) + 255) / 256;
  // rows per thread: long enough to reuse the window, short enough to fill the chip
  int run = single ? 1 : 16;
  while (run > 1 && (int64_t)gx * ((T_ + run - 1) / run) < 1024) run >>= 1;
  while ((T_ + run - 1) / run > 65535) run <<= 1;
  const dim3 grid(gx, (T_ + run - 1) / run);
#define CONV_LAUNCH(VEC, KT)                                                                                       \
  DISPATCH_T(is_f32, hipLaunchKernelGGL((conv_qkv_store_kernel<T, VEC, KT>), grid, dim3(256), 0, st, (T*)q_out,    \
                                        (const T*)y, w, (T*)hist, slots, cu, seg_start, token_seg, positions,      \
                                        (T*)kc, (T*)vc, slot_map, T_, C, K, y_stride, qo, qn, ko, kn, vo, vn, D2,  \
                                        V, G, BS, coef, every, run, single);)
  if (v8 && K <= 4) { CONV_LAUNCH(8, 4) }
  else if (v8) { CONV_LAUNCH(8, 0) }
  else if (K <= 4) { CONV_LAUNCH(1, 4) }
  else { CONV_LAUNCH(1, 0) }
#undef CONV_LAUNCH
  if (K > 1 && !single) seq_launch_conv_state_update(y, hist, slots, cu, seg_start, B, C, K, y_stride, is_f32, st);
}

// what the MFMA kernels take (16-byte aligned rows besides)
extern "C" int seq_diff_mfma_fits(int D, int V) { return D % 8 == 0 && V % 8 == 0 && D <= 128 && V <= 256; }

template <int NSL, int NDT, bool SINGLE>
static hipError_t launch_diff_mfma(dim3 grid, size_t lds, hipStream_t st, bfraw* out, const bfraw* q, const bfraw* kc,
                                   const bfraw* vc, const int* bt, const int* seg, const int64_t* pos,
                                   const int* tiles, float scale, float lam, float oscale, float eps, int H, int G,
                                   int D, int V, int BS, int bt_stride, int q_stride, int hb, float* part_o,
                                   float* part_ml) {
  static bool wide = false;
  if (lds > 64 * 1024 && !wide) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_diff_mfma_kernel<NSL, NDT, SINGLE>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    if (e != hipSuccess) return e;
    wide = true;
  }
  hipLaunchKernelGGL((attn_diff_mfma_kernel<NSL, NDT, SINGLE>), grid, dim3(512), lds, st, out, q, kc, vc,
                     bt, seg, pos, tiles, scale, lam, oscale, eps, H, G, D, V, BS, bt_stride, q_stride, hb,
                     part_o, part_ml);
  return hipGetLastError();
}

// form 0: the plain kernel on every row; 1: query tiles [n, 2] (first row, rows); 2: n single rows
// (row list or nullptr = rows 0..n-1), part_o [n, H, 2, ns, V], part_ml [n, H, 2, ns, 2]. hb: heads
// of a key/value head side by side in one workgroup (form 1: 1, 2 or 4; form 2: up to 32)
extern "C" int seq_launch_attn_diff_paged(void* out, const void* q, const void* kc, const void* vc, const int* bt,
                                          const int* seg, const int64_t* pos, int form, const int* tiles, int n,
                                          float scale, float lam, float oscale, float eps, int T_, int H, int G, int D,
                                          int V, int BS, int bt_stride, int q_stride, int hb, int ns, float* part_o,
                                          float* part_ml, int is_f32, hipStream_t st) {
  if (form == 0) {
    const size_t lds = (size_t)(2 * D + 3 * WAVE) * sizeof(float);
    const int k4 = D % 8 == 0 && aligned16(kc) ? 1 : 0;
    DISPATCH_T(is_f32, hipLaunchKernelGGL(attn_diff_paged_kernel<T>, dim3(T_, H), dim3(WAVE), lds, st, (T*)out,
                                          (const T*)q, (const T*)kc, (const T*)vc, bt, seg, pos, scale, lam, oscale,
                                          eps, H, G, D, V, BS, bt_stride, q_stride, k4);)
    return (int)hipGetLastError();
  }
  const int R = H / G, nhb = (R + hb - 1) / hb;
  const int Dp = (D + 15) / 16 * 16, Vp = (V + 31) / 32 * 32;
  size_t lds = (size_t)DIFF_KT * (2 * Dp + DIFF_KPAD) * 2 + (size_t)Vp * DIFF_VS * 2;
  const size_t epi = form == 1 ? (size_t)4 * 16 * WAVE * 4 : (size_t)4 * 16 * WAVE * 4 + 2 * 32 * 2 * 4;
  if (lds < epi) lds = epi;
  const dim3 grid(G * nhb, n, form == 1 ? 1 : ns);
  hipError_t err = hipSuccess;
#define DIFF_GO(NSL, NDT)                                                                                           \
  err = form == 1                                                                                                   \
            ? launch_diff_mfma<NSL, NDT, false>(grid, lds, st, (bfraw*)out, (const bfraw*)q, (const bfraw*)kc,      \
                                                (const bfraw*)vc, bt, seg, pos, tiles, scale, lam, oscale, eps, H,  \
                                                G, D, V, BS, bt_stride, q_stride, hb, nullptr, nullptr)        \
            : launch_diff_mfma<NSL, NDT, true>(grid, lds, st, (bfraw*)out, (const bfraw*)q, (const bfraw*)kc,       \
                                               (const bfraw*)vc, bt, seg, pos, tiles, scale, lam, oscale, eps, H,   \
                                               G, D, V, BS, bt_stride, q_stride, hb, part_o, part_ml);
#define DIFF_NDT(NSL)                                    \
  if (V <= 64) { DIFF_GO(NSL, 2) }                       \
  else if (V <= 128) { DIFF_GO(NSL, 4) }                 \
  else { DIFF_GO(NSL, 8) }
  if (D <= 32) { DIFF_NDT(2) }
  else if (D <= 64) { DIFF_NDT(4) }
  else { DIFF_NDT(8) }
#undef DIFF_NDT
#undef DIFF_GO
  if (err != hipSuccess) return (int)err;
  if (form == 2)
    hipLaunchKernelGGL(attn_diff_merge_kernel, dim3(n, H), dim3(256), 0, st, (bfraw*)out, part_o, part_ml, tiles, lam,
                       oscale, eps, H, V, ns);
  return (int)hipGetLastError();
}
