// Retention: linear attention with one constant decay g per head and rotary
// positions on q and k,
//   S_t = g S_{t-1} + k_t v_t^T,   o_t = S_t^T q_t        (k scaled by D^-1/2 after the rotation)
// on segments whose state lives in fp32 slots [slot, H, D, V] (a segment with
// seg_start == 0 takes its state as zero). Everything between the projections
// and the read-out is fp32, matrix products included (v_mfma_f32_32x32x2_f32).
//
// Prompt portions run chunk-parallel: a segment's rows are cut into chunks of
// RET_L tokens. With i, j counted inside a chunk of n tokens and S0 the state
// before it,
//   o_i   = g^(i+1) S0^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j
//   S_end = g^n S0 + U,   U = sum_j g^(n-1-j) k_j v_j^T
//   retention_angles     cos / sin of every row's angles, once for all heads
//   retention_chunk_u    U of every (chunk, head), in parallel
//   retention_scan       per state entry: walks a segment's chunks, leaves S0 in
//                        U's place and the final state in the slot
//   retention_chunk_out  o of every (chunk, head), in parallel
// A step whose segments are all single rows (decode) is one kernel:
//   retention_step       rotation, update, read-out, RMS norm per head, silu gate

#include "seq_common.h"

#define RET_L 64               // tokens per chunk
#define RET_THREADS 256
#define RET_KU 8               // matrix steps per loop pass: 2 RET_KU divides RET_L and the staged widths

typedef float ret_f32x16 __attribute__((ext_vector_type(16)));

// accumulator map of the 32x32 product: register r of a lane holds row
// (r & 3) + 8 (r >> 2) + 4 (lane >> 5) of column lane & 31; an A (B) operand
// lane holds row (column) lane & 31 at k = lane >> 5
__device__ __forceinline__ int ret_acc_row(int r, int half) { return (r & 3) + 8 * (r >> 2) + 4 * half; }

// g^0 .. g^RET_L by binary powers (any g, zero included); one entry per thread
__device__ __forceinline__ void ret_powers(float* pw, float g) {
  for (int n = threadIdx.x; n <= RET_L; n += blockDim.x) {
    float p = 1.f, b = g;
    for (int e = n; e > 0; e >>= 1) { if (e & 1) p *= b; b *= b; }
    pw[n] = p;
  }
}

__global__ void retention_angles_kernel(float* __restrict__ cs, const int64_t* __restrict__ positions,
                                        const float* __restrict__ inv_freq, int64_t n, int R2) {
  const int64_t u = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (u >= n) return;
  const int64_t t = u / R2;
  const int i = (int)(u - t * R2);
  float s, c;
  sincosf((float)positions[t] * inv_freq[i], &s, &c);
  cs[t * 2 * R2 + i] = c;
  cs[t * 2 * R2 + R2 + i] = s;
}

// VEC entries from column c of a head row of D entries, rotated (entry i of the
// first 2 R2 with entry i + R2) with the row's cos [R2] | sin [R2]. VEC = 8:
// D and R2 are multiples of 8.
template <typename T, int VEC>
__device__ __forceinline__ void ret_load_rotated(const T* __restrict__ row, const float* __restrict__ cs, int c,
                                                 int R2, float x[VEC]) {
  float y[VEC], cc[VEC], sn[VEC];
  if constexpr (VEC == 8) ld8(row + c, x); else x[0] = ldf(row + c);
  if (c < 2 * R2) {
    const bool lo = c < R2;
    const int i = lo ? c : c - R2;
    if constexpr (VEC == 8) {
      ld8(row + (lo ? c + R2 : c - R2), y);
      ld8(cs + i, cc);
      ld8(cs + R2 + i, sn);
    } else {
      y[0] = ldf(row + (lo ? c + R2 : c - R2));
      cc[0] = cs[i];
      sn[0] = cs[R2 + i];
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] = x[e] * cc[e] + (lo ? -y[e] : y[e]) * sn[e];
  }
}

// Rotated rows of one head -> LDS [RET_L][DM + 1], zeros past n rows and D
// columns. The odd row stride puts both a row's and a column's 32 neighbours on
// 32 banks. pw != nullptr: row r is scaled by pw[n-1-r].
template <typename T, int DM, int VEC>
__device__ __forceinline__ void ret_stage(float* __restrict__ dst, const T* __restrict__ src, int64_t stride,
                                          const float* __restrict__ cs, int n, int D, int R2, float scale,
                                          const float* pw) {
  constexpr int CV = DM / VEC;
  for (int u = threadIdx.x; u < RET_L * CV; u += RET_THREADS) {
    const int r = u / CV, c = (u - r * CV) * VEC;
    float x[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] = 0.f;
    if (r < n && c < D) {
      ret_load_rotated<T, VEC>(src + r * stride, cs + (int64_t)r * 2 * R2, c, R2, x);
      const float f = pw != nullptr ? scale * pw[n - 1 - r] : scale;
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[e] *= f;
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) dst[r * (DM + 1) + c + e] = x[e];
  }
}

// chunks [NC, 4] int32: first row, rows, segment, -
// grid (NC, H): U [NC, H, D, V]
template <typename T, int DM, int VEC>
__global__ void __launch_bounds__(RET_THREADS, DM > 64 ? 2 : 4) retention_chunk_u_kernel(
    float* __restrict__ U, const T* __restrict__ k, const T* __restrict__ v, const float* __restrict__ cs,
    const float* __restrict__ decay, const int* __restrict__ chunks, float kscale, int H, int D, int V, int R2,
    int k_stride, int v_stride) {
  __shared__ float ks[RET_L * (DM + 1)];
  __shared__ float pw[RET_L + 1];
  const int c = blockIdx.x, h = blockIdx.y;
  const int row0 = chunks[4 * c], n = chunks[4 * c + 1];
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, half = lane >> 5, lr = lane & 31;
  ret_powers(pw, decay[h]);
  __syncthreads();
  ret_stage<T, DM, VEC>(ks, k + (int64_t)row0 * k_stride + (int64_t)h * D, k_stride, cs + (int64_t)row0 * 2 * R2, n,
                        D, R2, kscale, pw);
  __syncthreads();
  constexpr int DT = DM / 32;
  float* up = U + ((int64_t)c * H + h) * D * V;
  const T* vp = v + (int64_t)row0 * v_stride + (int64_t)h * V;
  for (int ct = wave; ct * 32 < V; ct += RET_THREADS / WAVE) {
    const int j = ct * 32 + lr, jc = min(j, V - 1);
    ret_f32x16 acc[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[d][r] = 0.f;
    const float* kp = ks + half * (DM + 1) + lr;
    for (int t = 0; t < n; t += 2 * RET_KU, kp += 2 * RET_KU * (DM + 1)) {
      float b[RET_KU];             // rows past n: the keys there are zero
#pragma unroll
      for (int u = 0; u < RET_KU; ++u) b[u] = ldf(vp + (uint32_t)(min(t + 2 * u + half, n - 1) * v_stride + jc));
#pragma unroll
      for (int u = 0; u < RET_KU; ++u)
#pragma unroll
        for (int d = 0; d < DT; ++d)
          acc[d] = __builtin_amdgcn_mfma_f32_32x32x2f32(kp[2 * u * (DM + 1) + d * 32], b[u], acc[d], 0, 0, 0);
    }
    if (j < V) {
#pragma unroll
      for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int dd = d * 32 + ret_acc_row(r, half);
          if (dd < D) up[(uint32_t)(dd * V + j)] = acc[d][r];
        }
    }
  }
}

// grid (B, H, ...): thread = VEC entries of the state matrix. seg_c0 [B + 1]:
// a segment's range of chunks. On return U holds the state before each chunk.
template <int VEC>
__global__ void __launch_bounds__(RET_THREADS) retention_scan_kernel(
    float* __restrict__ U, float* __restrict__ state, const float* __restrict__ decay,
    const int* __restrict__ chunks, const int* __restrict__ seg_c0, const int* __restrict__ slots,
    const int* __restrict__ seg_start, int H, int64_t DV) {
  __shared__ float pw[RET_L + 1];
  const int b = blockIdx.x, h = blockIdx.y;
  ret_powers(pw, decay[h]);
  __syncthreads();
  const int64_t e = ((int64_t)blockIdx.z * RET_THREADS + threadIdx.x) * VEC;
  const int c0 = seg_c0[b], c1 = seg_c0[b + 1];
  if (e >= DV || c0 == c1) return;
  float* sp = state + ((int64_t)slots[b] * H + h) * DV + e;
  float S[VEC];
  const bool fresh = seg_start[b] == 0;
#pragma unroll
  for (int i = 0; i < VEC; ++i) S[i] = fresh ? 0.f : sp[i];
  const int64_t step = (int64_t)H * DV;
  float* up = U + ((int64_t)c0 * H + h) * DV + e;
  constexpr int PF = 4;                       // chunks in flight
  for (int c = c0; c < c1; c += PF, up += PF * step) {
    float u[PF][VEC];
#pragma unroll
    for (int f = 0; f < PF; ++f)
      if (c + f < c1) {
        if constexpr (VEC == 4) *reinterpret_cast<float4*>(u[f]) = *reinterpret_cast<const float4*>(up + f * step);
        else u[f][0] = up[f * step];
      }
#pragma unroll
    for (int f = 0; f < PF; ++f)
      if (c + f < c1) {
        if constexpr (VEC == 4) *reinterpret_cast<float4*>(up + f * step) = *reinterpret_cast<float4*>(S);
        else up[f * step] = S[0];
        const float g = pw[chunks[4 * (c + f) + 1]];
#pragma unroll
        for (int i = 0; i < VEC; ++i) S[i] = g * S[i] + u[f][i];
      }
  }
#pragma unroll
  for (int i = 0; i < VEC; ++i) sp[i] = S[i];
}

// grid (NC, H): o [T, H, V]. S0: the state before each chunk [NC, H, D, V]
template <typename T, int DM, int VEC>
__global__ void __launch_bounds__(RET_THREADS, DM > 64 ? 2 : 3) retention_chunk_out_kernel(
    float* __restrict__ o, const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v,
    const float* __restrict__ S0, const float* __restrict__ cs, const float* __restrict__ decay,
    const int* __restrict__ chunks, float kscale, int H, int D, int V, int R2, int q_stride, int k_stride,
    int v_stride) {
  constexpr int QS = DM + 1, PS = RET_L + 1;                 // row strides of the staged rows and of the scores
  constexpr int KS = RET_L * (QS > PS ? QS : PS);            // the keys' buffer later holds the scores
  __shared__ float qs[RET_L * QS];
  __shared__ float ks[KS];
  __shared__ float pw[RET_L + 1];
  const int c = blockIdx.x, h = blockIdx.y;
  const int row0 = chunks[4 * c], n = chunks[4 * c + 1];
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, half = lane >> 5, lr = lane & 31;
  const float* csr = cs + (int64_t)row0 * 2 * R2;
  ret_powers(pw, decay[h]);
  ret_stage<T, DM, VEC>(qs, q + (int64_t)row0 * q_stride + (int64_t)h * D, q_stride, csr, n, D, R2, 1.0f, nullptr);
  ret_stage<T, DM, VEC>(ks, k + (int64_t)row0 * k_stride + (int64_t)h * D, k_stride, csr, n, D, R2, kscale, nullptr);
  __syncthreads();
  // scores q_i . k_j, one 32 x 32 tile per wave (the tile above the diagonal is never read)
  const int it = wave >> 1, jt = wave & 1;
  const bool tile = it >= jt;
  ret_f32x16 s;
#pragma unroll
  for (int r = 0; r < 16; ++r) s[r] = 0.f;
  if (tile) {
    const float* qr = qs + (it * 32 + lr) * QS + half;
    const float* kr = ks + (jt * 32 + lr) * QS + half;
#pragma unroll 16
    for (int d = 0; d < DM; d += 2) s = __builtin_amdgcn_mfma_f32_32x32x2f32(qr[d], kr[d], s, 0, 0, 0);
  }
  __syncthreads();
  float* ps = ks;                              // [RET_L][PS]
  if (tile) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = it * 32 + ret_acc_row(r, half), j = jt * 32 + lr;
      ps[i * PS + j] = i >= j ? s[r] * pw[i - j] : 0.f;
    }
  }
  __syncthreads();
  const float* sp = S0 + ((int64_t)c * H + h) * D * V;
  const T* vp = v + (int64_t)row0 * v_stride + (int64_t)h * V;
  float* op = o + ((int64_t)row0 * H + h) * V;
  const int HV = H * V;
  // rows past n, columns past V and entries past D are computed with the others (their staged queries or
  // scores are zero, so what the clamped loads bring does not matter) and not stored
  for (int ct = wave; ct * 32 < V; ct += RET_THREADS / WAVE) {
    const int j = ct * 32 + lr, jc = min(j, V - 1);
    ret_f32x16 a0, a1;
#pragma unroll
    for (int r = 0; r < 16; ++r) { a0[r] = 0.f; a1[r] = 0.f; }
    const float* qp = qs + lr * QS + half;
    for (int d = 0; d < D; d += 2 * RET_KU, qp += 2 * RET_KU) {
      float b[RET_KU];
#pragma unroll
      for (int u = 0; u < RET_KU; ++u) b[u] = sp[(uint32_t)(min(d + 2 * u + half, D - 1) * V + jc)];
#pragma unroll
      for (int u = 0; u < RET_KU; ++u) {
        a0 = __builtin_amdgcn_mfma_f32_32x32x2f32(qp[2 * u], b[u], a0, 0, 0, 0);
        a1 = __builtin_amdgcn_mfma_f32_32x32x2f32(qp[2 * u + 32 * QS], b[u], a1, 0, 0, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = ret_acc_row(r, half);
      a0[r] *= pw[i + 1];
      a1[r] *= pw[i + 33];
    }
    const float* pp = ps + lr * PS + half;
    for (int t = 0; t < n; t += 2 * RET_KU, pp += 2 * RET_KU) {
      float b[RET_KU];
#pragma unroll
      for (int u = 0; u < RET_KU; ++u) b[u] = ldf(vp + (uint32_t)(min(t + 2 * u + half, n - 1) * v_stride + jc));
      if (t < 32) {                            // tokens 32.. lie after rows 0..31
#pragma unroll
        for (int u = 0; u < RET_KU; ++u) a0 = __builtin_amdgcn_mfma_f32_32x32x2f32(pp[2 * u], b[u], a0, 0, 0, 0);
      }
#pragma unroll
      for (int u = 0; u < RET_KU; ++u)
        a1 = __builtin_amdgcn_mfma_f32_32x32x2f32(pp[2 * u + 32 * PS], b[u], a1, 0, 0, 0);
    }
    if (j < V) {
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int i = ret_acc_row(r, half);
        if (i < n) op[(uint32_t)(i * HV + j)] = a0[r];
        if (i + 32 < n) op[(uint32_t)((i + 32) * HV + j)] = a1[r];
      }
    }
  }
}

// ---- one row per segment (decode) -------------------------------------------------
// grid (B, H), row b of segment b: rotation, state update and read-out, the
// head's RMS norm (no weight) and silu gate in one pass over the state matrix.
// Threads = row lanes x groups of VEC state columns; the row lanes' partial
// read-outs meet in LDS.
template <typename T, int VEC>
__global__ void __launch_bounds__(RET_THREADS) retention_step_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v,
    const T* __restrict__ gate, const float* __restrict__ decay, const int64_t* __restrict__ positions,
    const float* __restrict__ inv_freq, float* __restrict__ state, const int* __restrict__ slots,
    const int* __restrict__ seg_start, float kscale, float eps, int H, int D, int V, int R2, int q_stride,
    int k_stride, int v_stride, int gate_stride) {
  extern __shared__ __align__(16) float sm[];        // q [D] | k [D] | partial read-outs [row lanes][V]
  __shared__ float scratch[16];
  float* qs = sm;
  float* ks = sm + D;
  float* part = sm + ((2 * D + 3) & ~3);
  const int64_t b = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const float pos = (float)positions[b];
  const T* qr = q + b * q_stride + (int64_t)h * D;
  const T* kr = k + b * k_stride + (int64_t)h * D;
  for (int u = tid; u < 2 * D; u += RET_THREADS) {
    const bool isk = u >= D;
    const int d = isk ? u - D : u;
    const T* row = isk ? kr : qr;
    float x = ldf(row + d);
    if (d < 2 * R2) {
      const bool lo = d < R2;
      const int i = lo ? d : d - R2;
      float s, c;
      sincosf(pos * inv_freq[i], &s, &c);
      const float y = ldf(row + (lo ? d + R2 : d - R2));
      x = x * c + (lo ? -y : y) * s;
    }
    (isk ? ks : qs)[d] = isk ? x * kscale : x;
  }
  __syncthreads();
  const int cg = V / VEC, lanes = RET_THREADS / cg;          // host: 1 <= cg <= RET_THREADS
  const int rl = tid / cg, j = (tid - rl * cg) * VEC;
  const float g = decay[h];
  const bool fresh = seg_start[b] == 0;
  if (rl < lanes) {
    const T* vr = v + b * v_stride + (int64_t)h * V + j;
    float vv[VEC], acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) { vv[e] = ldf(vr + e); acc[e] = 0.f; }
    float* sp = state + ((int64_t)slots[b] * H + h) * D * V + j;
#pragma unroll 4
    for (int d = rl; d < D; d += lanes) {
      float S[VEC];
      if (fresh) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) S[e] = 0.f;
      } else if constexpr (VEC == 4) {
        *reinterpret_cast<float4*>(S) = *reinterpret_cast<const float4*>(sp + (int64_t)d * V);
      } else {
        S[0] = sp[(int64_t)d * V];
      }
      const float kd = ks[d], qd = qs[d];
#pragma unroll
      for (int e = 0; e < VEC; ++e) { S[e] = g * S[e] + kd * vv[e]; acc[e] += S[e] * qd; }
      if constexpr (VEC == 4) *reinterpret_cast<float4*>(sp + (int64_t)d * V) = *reinterpret_cast<float4*>(S);
      else sp[(int64_t)d * V] = S[0];
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) part[rl * V + j + e] = acc[e];
  }
  __syncthreads();
  float ss = 0.f;
  for (int i = tid; i < V; i += RET_THREADS) {
    float x = 0.f;
    for (int r = 0; r < lanes; ++r) x += part[r * V + i];
    part[i] = x;                                             // row lane 0's entry i, read by this thread only
    ss += x * x;
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)V + eps);
  for (int i = tid; i < V; i += RET_THREADS)
    stf(out + (b * H + h) * V + i, part[i] * r * silu_exact(ldf(gate + b * gate_stride + (int64_t)h * V + i)));
}

#define DISPATCH_T(is_f32, ...)                                  \
  if (is_f32) { typedef float T; __VA_ARGS__ } else { typedef bfraw T; __VA_ARGS__ }

#define DISPATCH_D(D, ...)                                          \
  if (D <= 32) { constexpr int DM = 32; __VA_ARGS__ }               \
  else if (D <= 64) { constexpr int DM = 64; __VA_ARGS__ }          \
  else { constexpr int DM = 128; __VA_ARGS__ }

// cs [T, 2 R2], U [NC, H, D, V]: fp32 scratch; chunks [NC, 4], seg_c0 [B + 1]: the step's chunks. D <= 128
extern "C" void seq_launch_retention_chunks(float* o, const void* q, const void* k, const void* v, const float* decay,
                                            const int64_t* positions, const float* inv_freq, float* cs, float* U,
                                            float* state, const int* slots, const int* seg_start, const int* chunks,
                                            const int* seg_c0, int T_, int B, int NC, int H, int D, int V, int R2,
                                            int q_stride, int k_stride, int v_stride, int is_f32, hipStream_t st) {
  const float kscale = 1.0f / sqrtf((float)D);
  const int64_t na = (int64_t)T_ * R2;
  if (na > 0)
    hipLaunchKernelGGL(retention_angles_kernel, dim3((unsigned)((na + 255) / 256)), dim3(256), 0, st, cs, positions,
                       inv_freq, na, R2);
  const bool v8 = D % 8 == 0 && R2 % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 && aligned16(q) &&
                  aligned16(k) && aligned16(cs);
  DISPATCH_T(is_f32, DISPATCH_D(D,
             if (v8) hipLaunchKernelGGL((retention_chunk_u_kernel<T, DM, 8>), dim3(NC, H), dim3(RET_THREADS), 0, st, U,
                                        (const T*)k, (const T*)v, cs, decay, chunks, kscale, H, D, V, R2, k_stride,
                                        v_stride);
             else hipLaunchKernelGGL((retention_chunk_u_kernel<T, DM, 1>), dim3(NC, H), dim3(RET_THREADS), 0, st, U,
                                     (const T*)k, (const T*)v, cs, decay, chunks, kscale, H, D, V, R2, k_stride,
                                     v_stride);))
  const int64_t DV = (int64_t)D * V;
  if (DV % 4 == 0 && aligned16(U) && aligned16(state))
    hipLaunchKernelGGL(retention_scan_kernel<4>, dim3(B, H, (unsigned)((DV / 4 + RET_THREADS - 1) / RET_THREADS)),
                       dim3(RET_THREADS), 0, st, U, state, decay, chunks, seg_c0, slots, seg_start, H, DV);
  else
    hipLaunchKernelGGL(retention_scan_kernel<1>, dim3(B, H, (unsigned)((DV + RET_THREADS - 1) / RET_THREADS)),
                       dim3(RET_THREADS), 0, st, U, state, decay, chunks, seg_c0, slots, seg_start, H, DV);
  DISPATCH_T(is_f32, DISPATCH_D(D,
             if (v8) hipLaunchKernelGGL((retention_chunk_out_kernel<T, DM, 8>), dim3(NC, H), dim3(RET_THREADS), 0, st,
                                        o, (const T*)q, (const T*)k, (const T*)v, U, cs, decay, chunks, kscale, H, D,
                                        V, R2, q_stride, k_stride, v_stride);
             else hipLaunchKernelGGL((retention_chunk_out_kernel<T, DM, 1>), dim3(NC, H), dim3(RET_THREADS), 0, st, o,
                                     (const T*)q, (const T*)k, (const T*)v, U, cs, decay, chunks, kscale, H, D, V, R2,
                                     q_stride, k_stride, v_stride);))
}

// V <= RET_THREADS, or V % 4 == 0 and V <= 4 RET_THREADS; D <= 1024
extern "C" void seq_launch_retention_step(void* out, const void* q, const void* k, const void* v, const void* gate,
                                          const float* decay, const int64_t* positions, const float* inv_freq,
                                          float* state, const int* slots, const int* seg_start, float eps, int B,
                                          int H, int D, int V, int R2, int q_stride, int k_stride, int v_stride,
                                          int gate_stride, int is_f32, hipStream_t st) {
  const float kscale = 1.0f / sqrtf((float)D);
  const bool v4 = V % 4 == 0 && aligned16(state);
  const int cg = v4 ? V / 4 : V;
  const size_t lds = (size_t)(((2 * D + 3) & ~3) + (RET_THREADS / cg) * V) * sizeof(float);
  DISPATCH_T(is_f32,
             if (v4) hipLaunchKernelGGL((retention_step_kernel<T, 4>), dim3(B, H), dim3(RET_THREADS), lds, st, (T*)out,
                                        (const T*)q, (const T*)k, (const T*)v, (const T*)gate, decay, positions,
                                        inv_freq, state, slots, seg_start, kscale, eps, H, D, V, R2, q_stride,
                                        k_stride, v_stride, gate_stride);
             else hipLaunchKernelGGL((retention_step_kernel<T, 1>), dim3(B, H), dim3(RET_THREADS), lds, st, (T*)out,
                                     (const T*)q, (const T*)k, (const T*)v, (const T*)gate, decay, positions,
                                     inv_freq, state, slots, seg_start, kscale, eps, H, D, V, R2, q_stride, k_stride,
                                     v_stride, gate_stride);)
}
