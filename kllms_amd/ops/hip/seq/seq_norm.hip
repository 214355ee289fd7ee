// fp32-residual normalisation kernels and the clamped GLU activation.
// One workgroup per token row; rows are re-read from L1/L2 between passes
// instead of being held in registers, so any width works.

#include "seq_common.h"

// out[t] = rmsnorm(table[ids[t]] (+ pos_table[positions[t]])) * w   (fp32 residual stream)
template <typename T>
__global__ void embed_rmsnorm_kernel(float* __restrict__ out, const int64_t* __restrict__ ids,
                                     const T* __restrict__ table, const float* __restrict__ w,
                                     const T* __restrict__ pos_table, const int64_t* __restrict__ positions,
                                     int W, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const T* row = table + (int64_t)ids[t] * W;
  const T* prow = pos_table != nullptr ? pos_table + positions[t] * W : nullptr;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float v = ldf(row + i) + (prow != nullptr ? ldf(prow + i) : 0.f);
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x)
    out[(int64_t)t * W + i] = (ldf(row + i) + (prow != nullptr ? ldf(prow + i) : 0.f)) * r * w[i];
}

// out[t] = rmsnorm(x[t]) * w, x fp32, out in the activation type
template <typename T>
__global__ void rmsnorm_cast_kernel(T* __restrict__ out, const float* __restrict__ x,
                                    const float* __restrict__ w, int W, float eps) {
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * W;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) { float v = x[base + i]; ss += v * v; }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) stf(out + base + i, x[base + i] * r * w[i]);
}

// Fused sublayer epilogue:
//   y = a                                    (single branch)
//   y = (rms(a) wa + rms(b) wb) / 2          (two branches, DUAL)
//   x += rms(y) * w_post                     (fp32 residual, in place)
//   out = rms(x) * w_next                    (next sublayer's input; optional)
//   out = x                                  (w_next == nullptr, out != nullptr: the
//                                             stream itself in the activation type)
// y is staged in dynamic LDS (W floats).
template <typename T, bool DUAL>
__global__ void sandwich_residual_kernel(float* __restrict__ x, const T* __restrict__ a,
                                         const T* __restrict__ b, const float* __restrict__ wa,
                                         const float* __restrict__ wb, const float* __restrict__ w_post,
                                         const float* __restrict__ w_next, T* __restrict__ out,
                                         int W, float eps) {
  extern __shared__ __align__(16) float ybuf[];
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * W;
  const float invW = 1.0f / (float)W;
  float ssy = 0.f;
  if (DUAL) {
    float sa = 0.f, sb = 0.f;
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float va = ldf(a + base + i), vb = ldf(b + base + i);
      sa += va * va; sb += vb * vb;
    }
    sa = block_sum(sa, scratch);
    sb = block_sum(sb, scratch);
    const float ra = 1.0f / sqrtf(sa * invW + eps), rb = 1.0f / sqrtf(sb * invW + eps);
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float y = 0.5f * (ldf(a + base + i) * ra * wa[i] + ldf(b + base + i) * rb * wb[i]);
      ybuf[i] = y; ssy += y * y;
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float y = ldf(a + base + i);
      ybuf[i] = y; ssy += y * y;
    }
  }
  ssy = block_sum(ssy, scratch);
  const float ry = 1.0f / sqrtf(ssy * invW + eps);
  float ssx = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {   // each thread re-reads its own ybuf entries
    float v = x[base + i] + ybuf[i] * ry * w_post[i];
    x[base + i] = v; ybuf[i] = v; ssx += v * v;
  }
  if (out == nullptr) return;
  if (w_next == nullptr) {
    for (int i = threadIdx.x; i < W; i += blockDim.x) stf(out + base + i, ybuf[i]);
    return;
  }
  ssx = block_sum(ssx, scratch);
  const float rx = 1.0f / sqrtf(ssx * invW + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) stf(out + base + i, ybuf[i] * rx * w_next[i]);
}

// The same epilogue with 8-wide accesses (W % 8 == 0, 16-byte aligned rows).
template <typename T, bool DUAL>
__global__ void sandwich_residual_v8_kernel(float* __restrict__ x, const T* __restrict__ a,
                                            const T* __restrict__ b, const float* __restrict__ wa,
                                            const float* __restrict__ wb, const float* __restrict__ w_post,
                                            const float* __restrict__ w_next, T* __restrict__ out,
                                            int W, float eps) {
  extern __shared__ __align__(16) float ybuf[];
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * W;
  const float invW = 1.0f / (float)W;
  float ssy = 0.f;
  float va[8], vb[8], w1[8], w2[8], y[8];
  if (DUAL) {
    float sa = 0.f, sb = 0.f;
    for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {
      ld8(a + base + i, va); ld8(b + base + i, vb);
#pragma unroll
      for (int e = 0; e < 8; ++e) { sa += va[e] * va[e]; sb += vb[e] * vb[e]; }
    }
    sa = block_sum(sa, scratch);
    sb = block_sum(sb, scratch);
    const float ra = 1.0f / sqrtf(sa * invW + eps), rb = 1.0f / sqrtf(sb * invW + eps);
    for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {
      ld8(a + base + i, va); ld8(b + base + i, vb); ld8(wa + i, w1); ld8(wb + i, w2);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        y[e] = 0.5f * (va[e] * ra * w1[e] + vb[e] * rb * w2[e]);
        ssy += y[e] * y[e];
      }
      st8(ybuf + i, y);
    }
  } else {
    for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {
      ld8(a + base + i, y);
#pragma unroll
      for (int e = 0; e < 8; ++e) ssy += y[e] * y[e];
      st8(ybuf + i, y);
    }
  }
  ssy = block_sum(ssy, scratch);
  const float ry = 1.0f / sqrtf(ssy * invW + eps);
  float ssx = 0.f;
  for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {   // each thread re-reads its own ybuf entries
    ld8(ybuf + i, y); ld8(x + base + i, va); ld8(w_post + i, w1);
#pragma unroll
    for (int e = 0; e < 8; ++e) { va[e] += y[e] * ry * w1[e]; ssx += va[e] * va[e]; }
    st8(x + base + i, va);
    st8(ybuf + i, va);
  }
  if (out == nullptr) return;
  if (w_next == nullptr) {
    for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) { ld8(ybuf + i, va); st8(out + base + i, va); }
    return;
  }
  ssx = block_sum(ssx, scratch);
  const float rx = 1.0f / sqrtf(ssx * invW + eps);
  for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {
    ld8(ybuf + i, va); ld8(w_next + i, w1);
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = va[e] * rx * w1[e];
    st8(out + base + i, y);
  }
}

// Gate modes of the grouped norms:
//   GATE_SIGMOID     out[t, g*S + i] = o[t,g,i] / rms(o[t,g,:]) * w[i] * sigmoid(gate[t, g*S + i])
//   GATE_SILU_FIRST  the gate comes before the norm, the weight spans the whole
//                    row: y = o * silu(gate); out = y / rms(y[t,g,:]) * w[g*S + i]
//   GATE_SILU        as GATE_SIGMOID with silu
// w == nullptr: no weight.
#define GATE_SIGMOID 0
#define GATE_SILU_FIRST 1
#define GATE_SILU 2
__device__ __forceinline__ float gate_after(float g, int mode) {
  return mode == GATE_SIGMOID ? sigmoid_exact(g) : silu_exact(g);
}
__device__ __forceinline__ void ld_weight8(const float* w, int64_t i, float v[8]) {
  if (w != nullptr) { ld8(w + i, v); return; }
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = 1.0f;
}
template <typename T>
__global__ void gated_rmsnorm_kernel(T* __restrict__ out, const float* __restrict__ o,
                                     const float* __restrict__ w, const T* __restrict__ gate,
                                     int S, int gate_stride, float eps, int mode) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, g = blockIdx.y, G = gridDim.y;
  const float* row = o + ((int64_t)t * G + g) * S;
  const T* grow = gate + (int64_t)t * gate_stride + (int64_t)g * S;
  float ss = 0.f;
  for (int i = threadIdx.x; i < S; i += blockDim.x) {
    float v = row[i];
    if (mode == GATE_SILU_FIRST) v *= silu_exact(ldf(grow + i));
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)S + eps);
  T* orow = out + ((int64_t)t * G + g) * S;
  for (int i = threadIdx.x; i < S; i += blockDim.x) {
    const float gv = ldf(grow + i);
    const float wv = w == nullptr ? 1.0f : w[(mode == GATE_SILU_FIRST ? (int64_t)g * S : 0) + i];
    stf(orow + i, mode == GATE_SILU_FIRST ? row[i] * silu_exact(gv) * r * wv : row[i] * r * wv * gate_after(gv, mode));
  }
}

// 8-wide, single pass: each thread keeps its (up to two) chunks of the row in
// registers between the sum of squares and the scaling. One workgroup per row.
template <typename T>
__global__ void gated_rmsnorm_v8_kernel(T* __restrict__ out, const float* __restrict__ o,
                                        const float* __restrict__ w, const T* __restrict__ gate,
                                        int S, int gate_stride, float eps, int mode) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, g = blockIdx.y, G = gridDim.y;
  const float* row = o + ((int64_t)t * G + g) * S;
  const T* grow = gate + (int64_t)t * gate_stride + (int64_t)g * S;
  float v[2][8], ww[8], gg[8];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int i = (threadIdx.x + c * blockDim.x) * 8;
    if (i < S) {
      ld8(row + i, v[c]);
      if (mode == GATE_SILU_FIRST) {
        ld8(grow + i, gg);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[c][e] *= silu_exact(gg[e]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[c][e] * v[c][e];
    }
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)S + eps);
  T* orow = out + ((int64_t)t * G + g) * S;
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int i = (threadIdx.x + c * blockDim.x) * 8;
    if (i < S) {
      ld_weight8(w, (mode == GATE_SILU_FIRST ? (int64_t)g * S : 0) + i, ww);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[c][e] = v[c][e] * r * ww[e];
      if (mode != GATE_SILU_FIRST) {
        ld8(grow + i, gg);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[c][e] *= gate_after(gg[e], mode);
      }
      st8(orow + i, v[c]);
    }
  }
}

// Short rows (S = 8 * LPG, LPG a power of two <= 64): LPG lanes per row, 64/LPG
// rows per wave, reduction inside the lane group.
template <typename T>
__global__ void gated_rmsnorm_rows_kernel(T* __restrict__ out, const float* __restrict__ o,
                                          const float* __restrict__ w, const T* __restrict__ gate,
                                          int64_t rows, int G, int S, int LPG, int gate_stride, float eps,
                                          int mode) {
  const int64_t tid = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  const int64_t row = tid / LPG;
  const int i = (int)(tid - row * LPG) * 8;
  const bool on = row < rows;
  const int64_t t = row / G;
  const int g = (int)(row - t * G);
  float v[8], ww[8], gg[8];
  float ss = 0.f;
  if (on) {
    ld8(o + row * S + i, v);
    ld8(gate + t * gate_stride + (int64_t)g * S + i, gg);
    if (mode == GATE_SILU_FIRST) {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= silu_exact(gg[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
  }
  for (int off = 1; off < LPG; off <<= 1) ss += __shfl_xor(ss, off);
  if (!on) return;
  const float r = 1.0f / sqrtf(ss / (float)S + eps);
  ld_weight8(w, (mode == GATE_SILU_FIRST ? (int64_t)g * S : 0) + i, ww);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = v[e] * r * ww[e] * (mode == GATE_SILU_FIRST ? 1.0f : gate_after(gg[e], mode));
  st8(out + row * S + i, v);
}

// y = min(g, lim) * sigmoid(alpha * min(g, lim)) * (clamp(u, -lim, lim) + up_bias);
// lim = inf, alpha = 1, up_bias = 0 is silu(g) * u
template <typename T>
__global__ void clamped_glu_kernel(T* __restrict__ out, const T* __restrict__ gate,
                                   const T* __restrict__ up, int64_t n, int cols, int stride,
                                   float limit, float alpha, float up_bias) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = i / cols, c = i - r * cols;
    float g = fminf(ldf(gate + r * stride + c), limit);
    float u = fminf(fmaxf(ldf(up + r * stride + c), -limit), limit);
    stf(out + i, g * sigmoid_exact(alpha * g) * (u + up_bias));
  }
}

template <typename T>
__global__ void clamped_glu_v8_kernel(T* __restrict__ out, const T* __restrict__ gate,
                                      const T* __restrict__ up, int64_t n8, int cols8, int stride,
                                      float limit, float alpha, float up_bias) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n8;
       i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = i / cols8, c = (i - r * cols8) * 8;
    float g[8], u[8];
    ld8(gate + r * stride + c, g);
    ld8(up + r * stride + c, u);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float gc = fminf(g[e], limit), uc = fminf(fmaxf(u[e], -limit), limit);
      g[e] = gc * sigmoid_exact(alpha * gc) * (uc + up_bias);
    }
    st8(out + i * 8, g);
  }
}

// tanh-form gelu: 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))
__device__ __forceinline__ float gelu_tanh_exact(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <typename T>
__global__ void gelu_tanh_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t n, int cols, int stride) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = i / cols, c = i - r * cols;
    stf(out + i, gelu_tanh_exact(ldf(x + r * stride + c)));
  }
}

template <typename T>
__global__ void gelu_tanh_v8_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t n8, int cols8,
                                    int stride) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n8;
       i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = i / cols8, c = (i - r * cols8) * 8;
    float v[8];
    ld8(x + r * stride + c, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = gelu_tanh_exact(v[e]);
    st8(out + i * 8, v);
  }
}

// Elementwise activations of row views, in fp32 between load and store:
//   ACT_GELU_MUL    out = gelu(a) * b                (gated gelu feed-forward; a token's side row)
//   ACT_RELU2       out = max(a, 0)^2
//   ACT_SIGMOID_MUL out = a * sigmoid(b)
// Row r of b is b + r * b_stride, or with ids b + ids[r] * b_stride (b then
// already points at its first column). gelu in the form z * sigmoid(2 u), equal
// to z (1 + tanh(u)) / 2.
#define ACT_GELU_MUL 0
#define ACT_RELU2 1
#define ACT_SIGMOID_MUL 2
template <int OP>
__device__ __forceinline__ float act_pair(float a, float b) {
  if (OP == ACT_GELU_MUL) return a * sigmoid_exact(1.5957691216057308f * (a + 0.044715f * a * a * a)) * b;
  if (OP == ACT_RELU2) { const float p = fmaxf(a, 0.f); return p * p; }
  return a * sigmoid_exact(b);
}

template <typename T, int OP, int VEC>
__global__ void act_pair_kernel(T* __restrict__ out, const T* a, const T* __restrict__ b,
                                const int64_t* __restrict__ ids, int64_t n, int cols, int out_stride, int a_stride,
                                int64_t b_stride) {
  const int cv = cols / VEC;
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = i / cv, c = (i - r * cv) * VEC;
    const T* br = OP == ACT_RELU2 ? nullptr : b + (ids != nullptr ? ids[r] : r) * b_stride + c;
    if (VEC == 8) {
      float av[8], bv[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      ld8(a + r * a_stride + c, av);
      if (OP != ACT_RELU2) ld8(br, bv);
#pragma unroll
      for (int e = 0; e < 8; ++e) av[e] = act_pair<OP>(av[e], bv[e]);
      st8(out + r * out_stride + c, av);
    } else {
      stf(out + r * out_stride + c, act_pair<OP>(ldf(a + r * a_stride + c), OP == ACT_RELU2 ? 0.f : ldf(br)));
    }
  }
}

// z <- z * scale, then cap * tanh(z / cap) when cap > 0 (fp32 logits, in place)
__global__ void scale_softcap_kernel(float* __restrict__ z, int64_t n, float scale, float cap) {
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * blockDim.x) {
    const float v = z[i] * scale;
    z[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

// ---- dynamic-tanh norm: tanh(alpha v) w + b, no statistics -------------------------
// x (fp32 stream) += tanh(alpha_p a) w_p + b_p, then
// out = tanh(alpha_n x) w_n + b_n. With ids (and no a) the stream starts here:
// x = table row of the token times emb_scale. A thread keeps VEC columns of both norms in
// registers and walks the rows blockIdx.y, + gridDim.y, ...
template <typename T, int VEC>
__global__ void __launch_bounds__(256) dyt_residual_kernel(
    T* __restrict__ out, float* __restrict__ x, const T* __restrict__ a, const float* __restrict__ alpha_p,
    const float* __restrict__ w_p, const float* __restrict__ b_p, const float* __restrict__ alpha_n,
    const float* __restrict__ w_n, const float* __restrict__ b_n, const int64_t* __restrict__ ids,
    const T* __restrict__ table, float emb_scale, int T_, int W) {
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (c >= W) return;
  float wp[VEC], bp[VEC], wn[VEC], bn[VEC];
  const float an = alpha_n[0], ap = a != nullptr ? alpha_p[0] : 0.f;
  if constexpr (VEC == 8) {
    ld8(w_n + c, wn); ld8(b_n + c, bn);
    if (a != nullptr) { ld8(w_p + c, wp); ld8(b_p + c, bp); }
  } else {
    wn[0] = w_n[c]; bn[0] = b_n[c];
    if (a != nullptr) { wp[0] = w_p[c]; bp[0] = b_p[c]; }
  }
  for (int64_t t = blockIdx.y; t < T_; t += gridDim.y) {
    float xv[VEC], av[VEC];
    if (ids != nullptr) {
      const T* row = table + ids[t] * W + c;
      if constexpr (VEC == 8) ld8(row, xv); else xv[0] = ldf(row);
#pragma unroll
      for (int e = 0; e < VEC; ++e) xv[e] *= emb_scale;
      if constexpr (VEC == 8) st8(x + t * W + c, xv); else x[t * W + c] = xv[0];
    } else if constexpr (VEC == 8) {
      ld8(x + t * W + c, xv);
      if (a != nullptr) ld8(a + t * W + c, av);
    } else {
      xv[0] = x[t * W + c];
      if (a != nullptr) av[0] = ldf(a + t * W + c);
    }
    if (a != nullptr) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) xv[e] += tanhf(ap * av[e]) * wp[e] + bp[e];
      if constexpr (VEC == 8) st8(x + t * W + c, xv); else x[t * W + c] = xv[0];
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) xv[e] = tanhf(an * xv[e]) * wn[e] + bn[e];
    if constexpr (VEC == 8) st8(out + t * W + c, xv); else stf(out + t * W + c, xv[0]);
  }
}

// RMS norm of rows in the activation type (free row stride), one wave per row
template <typename T, int VEC>
__global__ void __launch_bounds__(256) rmsnorm_rows_kernel(T* __restrict__ out, const T* __restrict__ x,
                                                           const float* __restrict__ w, int T_, int C, int x_stride,
                                                           float eps) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int64_t t = (int64_t)blockIdx.x * (256 / WAVE) + threadIdx.x / WAVE;
  if (t >= T_) return;
  const T* row = x + t * x_stride;
  float ss = 0.f;
  for (int c = lane * VEC; c < C; c += WAVE * VEC) {
    float v[VEC];
    if constexpr (VEC == 8) ld8(row + c, v); else v[0] = ldf(row + c);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
  }
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)C + eps);
  for (int c = lane * VEC; c < C; c += WAVE * VEC) {
    float v[VEC], wv[VEC];
    if constexpr (VEC == 8) { ld8(row + c, v); ld8(w + c, wv); } else { v[0] = ldf(row + c); wv[0] = w[c]; }
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= r * wv[e];
    if constexpr (VEC == 8) st8(out + t * C + c, v); else stf(out + t * C + c, v[0]);
  }
}

#define DISPATCH_T(is_f32, ...)                                  \
  if (is_f32) { typedef float T; __VA_ARGS__ } else { typedef bfraw T; __VA_ARGS__ }

extern "C" void seq_launch_embed_rmsnorm(float* out, const int64_t* ids, const void* table,
                                         const float* w, const void* pos_table, const int64_t* positions,
                                         int T_, int W, float eps, int is_f32, hipStream_t st) {
  DISPATCH_T(is_f32, hipLaunchKernelGGL(embed_rmsnorm_kernel<T>, dim3(T_), dim3(256), 0, st, out, ids,
                                        (const T*)table, w, (const T*)pos_table, positions, W, eps);)
}

extern "C" void seq_launch_gelu_tanh(void* out, const void* x, int64_t rows, int cols, int stride, int is_f32,
                                     hipStream_t st) {
  if (cols % 8 == 0 && stride % 8 == 0 && aligned16(out) && aligned16(x)) {
    const int64_t n8 = rows * cols / 8;
    const int g8 = (int)((n8 + 255) / 256 < 16384 ? (n8 + 255) / 256 : 16384);
    DISPATCH_T(is_f32, hipLaunchKernelGGL(gelu_tanh_v8_kernel<T>, dim3(g8), dim3(256), 0, st, (T*)out,
                                          (const T*)x, n8, cols / 8, stride);)
    return;
  }
  const int64_t n = rows * cols;
  const int grid = (int)((n + 255) / 256 < 4096 ? (n + 255) / 256 : 4096);
  DISPATCH_T(is_f32, hipLaunchKernelGGL(gelu_tanh_kernel<T>, dim3(grid), dim3(256), 0, st, (T*)out, (const T*)x,
                                        n, cols, stride);)
}

template <typename T, int OP>
static void launch_act_pair(void* out, const void* a, const void* b, const int64_t* ids, int64_t rows, int cols,
                            int out_stride, int a_stride, int64_t b_stride, hipStream_t st) {
  const bool v8 = cols % 8 == 0 && out_stride % 8 == 0 && a_stride % 8 == 0 && b_stride % 8 == 0 && aligned16(out) &&
                  aligned16(a) && (b == nullptr || aligned16(b));
  const int64_t n = rows * cols / (v8 ? 8 : 1);
  const int grid = (int)((n + 255) / 256 < 16384 ? (n + 255) / 256 : 16384);
  if (v8) hipLaunchKernelGGL((act_pair_kernel<T, OP, 8>), dim3(grid), dim3(256), 0, st, (T*)out, (const T*)a,
                             (const T*)b, ids, n, cols, out_stride, a_stride, b_stride);
  else hipLaunchKernelGGL((act_pair_kernel<T, OP, 1>), dim3(grid), dim3(256), 0, st, (T*)out, (const T*)a,
                          (const T*)b, ids, n, cols, out_stride, a_stride, b_stride);
}

// op: ACT_*; ids: row indices into b, or nullptr
extern "C" void seq_launch_act_pair(void* out, const void* a, const void* b, const int64_t* ids, int64_t rows,
                                    int cols, int out_stride, int a_stride, int64_t b_stride, int op, int is_f32,
                                    hipStream_t st) {
  DISPATCH_T(is_f32,
             if (op == ACT_GELU_MUL)
               launch_act_pair<T, ACT_GELU_MUL>(out, a, b, ids, rows, cols, out_stride, a_stride, b_stride, st);
             else if (op == ACT_RELU2)
               launch_act_pair<T, ACT_RELU2>(out, a, b, ids, rows, cols, out_stride, a_stride, b_stride, st);
             else
               launch_act_pair<T, ACT_SIGMOID_MUL>(out, a, b, ids, rows, cols, out_stride, a_stride, b_stride, st);)
}

extern "C" void seq_launch_scale_softcap(float* z, int64_t n, float scale, float cap, hipStream_t st) {
  const int grid = (int)((n + 255) / 256 < 8192 ? (n + 255) / 256 : 8192);
  hipLaunchKernelGGL(scale_softcap_kernel, dim3(grid), dim3(256), 0, st, z, n, scale, cap);
}

extern "C" void seq_launch_rmsnorm_cast(void* out, const float* x, const float* w, int T_, int W,
                                        float eps, int is_f32, hipStream_t st) {
  DISPATCH_T(is_f32, hipLaunchKernelGGL(rmsnorm_cast_kernel<T>, dim3(T_), dim3(256), 0, st, (T*)out, x, w,
                                        W, eps);)
}

extern "C" void seq_launch_sandwich_residual(float* x, const void* a, const void* b, const float* wa,
                                             const float* wb, const float* w_post, const float* w_next,
                                             void* out, int T_, int W, float eps, int is_f32,
                                             hipStream_t st) {
  const size_t lds = (size_t)W * sizeof(float);
  const bool v8 = W % 8 == 0 && aligned16(x) && aligned16(a) && aligned16(b) && aligned16(out) &&
                  aligned16(wa) && aligned16(wb) && aligned16(w_post) && aligned16(w_next);
  if (v8 && b != nullptr) {
    DISPATCH_T(is_f32, hipLaunchKernelGGL((sandwich_residual_v8_kernel<T, true>), dim3(T_), dim3(256), lds, st,
                                          x, (const T*)a, (const T*)b, wa, wb, w_post, w_next, (T*)out, W, eps);)
  } else if (v8) {
    DISPATCH_T(is_f32, hipLaunchKernelGGL((sandwich_residual_v8_kernel<T, false>), dim3(T_), dim3(256), lds, st,
                                          x, (const T*)a, (const T*)b, wa, wb, w_post, w_next, (T*)out, W, eps);)
  } else if (b != nullptr) {
    DISPATCH_T(is_f32, hipLaunchKernelGGL((sandwich_residual_kernel<T, true>), dim3(T_), dim3(256), lds, st,
                                          x, (const T*)a, (const T*)b, wa, wb, w_post, w_next, (T*)out, W, eps);)
  } else {
    DISPATCH_T(is_f32, hipLaunchKernelGGL((sandwich_residual_kernel<T, false>), dim3(T_), dim3(256), lds, st,
                                          x, (const T*)a, (const T*)b, wa, wb, w_post, w_next, (T*)out, W, eps);)
  }
}

extern "C" void seq_launch_gated_rmsnorm(void* out, const float* o, const float* w, const void* gate,
                                         int T_, int G, int S, int gate_stride, float eps, int mode,
                                         int is_f32, hipStream_t st) {
  if (S % 8 == 0 && gate_stride % 8 == 0 && aligned16(out) && aligned16(o) && (w == nullptr || aligned16(w)) && aligned16(gate)) {
    const int lpg = S / 8;
    if (lpg <= 64 && (lpg & (lpg - 1)) == 0) {
      const int64_t rows = (int64_t)T_ * G;
      const int grid = (int)((rows * lpg + 255) / 256);
      DISPATCH_T(is_f32, hipLaunchKernelGGL(gated_rmsnorm_rows_kernel<T>, dim3(grid), dim3(256), 0, st, (T*)out,
                                            o, w, (const T*)gate, rows, G, S, lpg, gate_stride, eps, mode);)
      return;
    }
    int threads = ((lpg + 1) / 2 + WAVE - 1) / WAVE * WAVE;       // two chunks of 8 per thread
    if (threads <= 1024) {
      if (threads < WAVE) threads = WAVE;
      DISPATCH_T(is_f32, hipLaunchKernelGGL(gated_rmsnorm_v8_kernel<T>, dim3(T_, G), dim3(threads), 0, st,
                                            (T*)out, o, w, (const T*)gate, S, gate_stride, eps, mode);)
      return;
    }
  }
  const int threads = S >= 256 ? 256 : (S > 64 ? 128 : 64);
  DISPATCH_T(is_f32, hipLaunchKernelGGL(gated_rmsnorm_kernel<T>, dim3(T_, G), dim3(threads), 0, st, (T*)out,
                                        o, w, (const T*)gate, S, gate_stride, eps, mode);)
}

extern "C" void seq_launch_gated_act(void* out, const void* gate, const void* up, int64_t rows, int cols,
                                     int stride, float limit, float alpha, float up_bias, int is_f32,
                                     hipStream_t st) {
  if (cols % 8 == 0 && stride % 8 == 0 && aligned16(out) && aligned16(gate) && aligned16(up)) {
    const int64_t n8 = rows * cols / 8;
    const int g8 = (int)((n8 + 255) / 256 < 16384 ? (n8 + 255) / 256 : 16384);
    DISPATCH_T(is_f32, hipLaunchKernelGGL(clamped_glu_v8_kernel<T>, dim3(g8), dim3(256), 0, st, (T*)out,
                                          (const T*)gate, (const T*)up, n8, cols / 8, stride, limit, alpha, up_bias);)
    return;
  }
  const int64_t n = rows * cols;
  const int grid = (int)((n + 255) / 256 < 4096 ? (n + 255) / 256 : 4096);
  DISPATCH_T(is_f32, hipLaunchKernelGGL(clamped_glu_kernel<T>, dim3(grid), dim3(256), 0, st, (T*)out,
                                        (const T*)gate, (const T*)up, n, cols, stride, limit, alpha, up_bias);)
}

extern "C" void seq_launch_dyt_residual(void* out, float* x, const void* a, const float* alpha_p, const float* w_p,
                                        const float* b_p, const float* alpha_n, const float* w_n, const float* b_n,
                                        const int64_t* ids, const void* table, float emb_scale, int T_, int W,
                                        int is_f32, hipStream_t st) {
  const bool v8 = W % 8 == 0 && aligned16(out) && aligned16(x) && aligned16(w_n) && aligned16(b_n) &&
                  (ids == nullptr || aligned16(table)) &&
                  (a == nullptr || (aligned16(a) && aligned16(w_p) && aligned16(b_p)));
  const int cols = v8 ? W / 8 : W;
  const int threads = cols >= 256 ? 256 : (cols + WAVE - 1) / WAVE * WAVE;
  const int gx = (cols + threads - 1) / threads;
  int gy = (8192 * 256 / threads + gx - 1) / gx;
  if (gy > T_) gy = T_;
  if (gy > 65535) gy = 65535;
  DISPATCH_T(is_f32,
             if (v8) hipLaunchKernelGGL((dyt_residual_kernel<T, 8>), dim3(gx, gy), dim3(threads), 0, st, (T*)out, x,
                                        (const T*)a, alpha_p, w_p, b_p, alpha_n, w_n, b_n, ids, (const T*)table,
                                        emb_scale, T_, W);
             else hipLaunchKernelGGL((dyt_residual_kernel<T, 1>), dim3(gx, gy), dim3(threads), 0, st, (T*)out, x,
                                     (const T*)a, alpha_p, w_p, b_p, alpha_n, w_n, b_n, ids, (const T*)table,
                                     emb_scale, T_, W);)
}

extern "C" void seq_launch_rmsnorm_rows(void* out, const void* x, const float* w, int T_, int C, int x_stride,
                                        float eps, int is_f32, hipStream_t st) {
  const bool v8 = C % 8 == 0 && x_stride % 8 == 0 && aligned16(out) && aligned16(x) && aligned16(w);
  const int rows = 256 / WAVE;
  DISPATCH_T(is_f32,
             if (v8) hipLaunchKernelGGL((rmsnorm_rows_kernel<T, 8>), dim3((T_ + rows - 1) / rows), dim3(256), 0, st,
                                        (T*)out, (const T*)x, w, T_, C, x_stride, eps);
             else hipLaunchKernelGGL((rmsnorm_rows_kernel<T, 1>), dim3((T_ + rows - 1) / rows), dim3(256), 0, st,
                                     (T*)out, (const T*)x, w, T_, C, x_stride, eps);)
}
