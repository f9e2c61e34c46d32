// Linear attention with a constant decay per head over a flat token batch, chunk
// by chunk on the f32 matrix cores: the long feeds of the recurrence
//
//   S_t = lambda_h S_{t-1} + k_t v_t^T,    o_t = S_t^T q_t
//
// that state_scan_kernel (lightning.hip) runs token by token. A feed is cut into
// chunks of 64 tokens counted from its first one. With S the state before a chunk
// of n tokens (numbered from 0),
//
//   o_t   = lambda^(t + 1) S^T q_t + sum_{s <= t} lambda^(t - s) (q_t . k_s) v_s
//   S_end = lambda^n S + sum_s lambda^(n - 1 - s) k_s v_s^T
//
// and no power has a negative exponent, so nothing overflows for any decay in
// [0, 1]. Three launches: lc_local_kernel forms the last sum of every chunk,
// lc_pass_kernel walks each sequence's chunks in order, elementwise (what it leaves
// in the workspace is the state BEFORE each chunk) and stores the new state,
// lc_out_kernel forms the outputs. The first and the last are parallel over chunks,
// heads and value columns.
//
// Products run on v_mfma_f32_32x32x2_f32 (exact f32 multiply-adds): lane l holds
// row or column l % 32 and one of the two k indices of a step, and which k a half
// of the wave takes in which step is free as long as both operands agree: where an
// operand's k runs along LDS rows each half takes a contiguous part of the range, so
// that a lane reads its row in 16-byte runs; operands from global memory are read in
// 128-byte row pieces.
#include "seqmix.h"

#define LC_C 64

// lambda^n by squaring (0^0 = 1)
__device__ __forceinline__ float lc_pow(float x, int n) {
  float r = 1.f;
  for (; n; n >>= 1, x *= x)
    if (n & 1) r *= x;
  return r;
}

struct LcParams {
  const float* act; long ld; int H, D, Dv, q_off, k_off, v_off, hpg;
  float* state; const int* slots; const int* cu_q; const int* pos; const float* decay;
  float* ws; float* o; int B;
};

__device__ __forceinline__ float16v lc_zero() {
  float16v a;
#pragma unroll
  for (int i = 0; i < 16; ++i) a[i] = 0.f;
  return a;
}
// the row of accumulator register r in lane half h
__device__ __forceinline__ int lc_row(int r, int h) { return (r & 3) + 8 * (r >> 2) + 4 * h; }

__global__ __launch_bounds__(256, 2) void lc_local_kernel(LcParams p) {
  __shared__ float pw[LC_C];
  int b, t0, n;
  if (!seq_chunk<LC_C>(p.cu_q, p.B, blockIdx.x, b, t0, n)) return;
  const int h = blockIdx.y, wave = threadIdx.x >> 6, l = threadIdx.x & 31, hf = (threadIdx.x >> 5) & 1;
  if (threadIdx.x < LC_C) pw[threadIdx.x] = lc_pow(p.decay[h], threadIdx.x);
  __syncthreads();
  const int D = p.D, Dv = p.Dv, e = blockIdx.z * 32 + l;
  const float* vr = p.act + (size_t)t0 * p.ld + p.v_off + (size_t)h * Dv + min(e, Dv - 1);
  float* ws = p.ws + ((size_t)blockIdx.x * p.H + h) * D * Dv;
  const int steps = (n + 1) / 2;
  for (int dt = wave; dt * 32 < D; dt += 4) {
    const float* kr = p.act + (size_t)t0 * p.ld + p.k_off + (size_t)(h / p.hpg) * D +
                      min(dt * 32 + l, D - 1);
    float16v acc = lc_zero();
    for (int s0 = 0; s0 < steps; s0 += 16) {
      float a[16], v[16];
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        const size_t row = (size_t)min(2 * (s0 + j) + hf, n - 1) * p.ld;
        a[j] = kr[row];
        v[j] = vr[row];
      }
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        const int t = 2 * (s0 + j) + hf;
        const float f = t < n ? pw[n - 1 - t] : 0.f;
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a[j] * f, v[j], acc, 0, 0, 0);
      }
    }
    if (e < Dv)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int d = dt * 32 + lc_row(r, hf);
        if (d < D) ws[(size_t)d * Dv + e] = acc[r];
      }
  }
}

template <int N>
__global__ __launch_bounds__(256) void lc_pass_kernel(LcParams p) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int q0 = p.cu_q[b], len = p.cu_q[b + 1] - q0;
  if (len <= 0) return;
  const int before = seq_chunks_before<LC_C>(p.cu_q, b);
  const size_t n = (size_t)p.D * p.Dv, i = N * ((size_t)blockIdx.z * 256 + threadIdx.x);
  if (i >= n) return;
  const int nc = (len + LC_C - 1) / LC_C;
  const float lam = p.decay[h], full = lc_pow(lam, LC_C), last = lc_pow(lam, len - (nc - 1) * LC_C);
  float* st = p.state + ((size_t)p.slots[b] * p.H + h) * n + i;
  float* ws = p.ws + ((size_t)before * p.H + h) * n + i;
  const size_t step = (size_t)p.H * n;
  float S[N];
  if (p.pos[q0] == 0) {
#pragma unroll
    for (int k = 0; k < N; ++k) S[k] = 0.f;
  } else {
    ld_run<float, N>(st, S);
  }
  constexpr int U = 8;                               // chunks in flight
  for (int c0 = 0; c0 < nc; c0 += U) {
    float w[U][N];
#pragma unroll
    for (int c = 0; c < U; ++c) ld_run<float, N>(ws + (size_t)min(c0 + c, nc - 1) * step, w[c]);
#pragma unroll
    for (int c = 0; c < U; ++c) {
      if (c0 + c >= nc) break;
      st_run<float, N>(ws + (size_t)(c0 + c) * step, S);
      const float f = c0 + c == nc - 1 ? last : full;
#pragma unroll
      for (int k = 0; k < N; ++k) S[k] = f * S[k] + w[c][k];
    }
  }
  st_run<float, N>(st, S);
}

// A workgroup covers 64 value columns of a chunk: wave w the rows 32 (w / 2) .. and
// the columns 32 (w % 2) .. of them. The k range (the key size) goes in pieces of 32
// through LDS, where a lane reads its q and k rows in 16-byte runs; one walk over it
// forms both the scores (the same split over the 64 x 64 tokens, the tile above the
// diagonal left out) and the state's part. The next piece is in flight meanwhile.
// VEC: the rows allow 16-byte runs.
#define LC_K 32

template <bool VEC>
__global__ __launch_bounds__(256, 2) void lc_out_kernel(LcParams p) {
  constexpr int LD = LC_K + 4;
  __shared__ __attribute__((aligned(16))) float qs[LC_C][LD], ks[LC_C][LD];
  __shared__ __attribute__((aligned(16))) float P[LC_C][LC_C + 4];
  __shared__ float pw[LC_C + 1];
  int b, t0, n;
  if (!seq_chunk<LC_C>(p.cu_q, p.B, blockIdx.x, b, t0, n)) return;
  const int h = blockIdx.y, wave = threadIdx.x >> 6, l = threadIdx.x & 31, hf = (threadIdx.x >> 5) & 1;
  const int ti = wave >> 1, tj = wave & 1;
  if (threadIdx.x <= LC_C) pw[threadIdx.x] = lc_pow(p.decay[h], threadIdx.x);
  const int D = p.D, Dv = p.Dv;
  const float* base = p.act + (size_t)t0 * p.ld;
  const float* qb = base + p.q_off + (size_t)(h / p.hpg) * D;
  const float* kb = base + p.k_off + (size_t)(h / p.hpg) * D;
  const int e = blockIdx.z * 64 + tj * 32 + l, ec = min(e, Dv - 1);
  const float* S = p.ws + ((size_t)blockIdx.x * p.H + h) * D * Dv + ec;
  // staging: runs of four columns, thread -> row (tid / 8) and (tid / 8) + 32
  const int sr = threadIdx.x >> 3, sc4 = (threadIdx.x & 7) * 4;
  float rq[2][4], rk[2][4], w[16];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const size_t row = (size_t)min(sr + 32 * j, n - 1) * p.ld;
      if constexpr (VEC) {
        if (k0 + sc4 < D) {
          ld_run<float, 4>(qb + row + k0 + sc4, rq[j]);
          ld_run<float, 4>(kb + row + k0 + sc4, rk[j]);
          continue;
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool ok = !VEC && k0 + sc4 + i < D;
        rq[j][i] = ok ? qb[row + k0 + sc4 + i] : 0.f;
        rk[j][i] = ok ? kb[row + k0 + sc4 + i] : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) w[i] = S[(size_t)min(k0 + 16 * hf + i, D - 1) * Dv];
  };
  float16v acc = lc_zero(), sc = lc_zero();
  const bool scores = tj <= ti;                      // uniform over the wave
  fetch(0);
  for (int k0 = 0; k0 < D; k0 += LC_K) {
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      st_run<float, 4>(&qs[sr + 32 * j][sc4], rq[j]);
      st_run<float, 4>(&ks[sr + 32 * j][sc4], rk[j]);
    }
    float wc[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) wc[i] = w[i];
    __syncthreads();
    if (k0 + LC_K < D) fetch(k0 + LC_K);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float4 a = *reinterpret_cast<const float4*>(&qs[ti * 32 + l][16 * hf + 4 * j]);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, wc[4 * j], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, wc[4 * j + 1], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, wc[4 * j + 2], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, wc[4 * j + 3], acc, 0, 0, 0);
      if (scores) {
        const float4 k = *reinterpret_cast<const float4*>(&ks[tj * 32 + l][16 * hf + 4 * j]);
        sc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, k.x, sc, 0, 0, 0);
        sc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, k.y, sc, 0, 0, 0);
        sc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, k.z, sc, 0, 0, 0);
        sc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, k.w, sc, 0, 0, 0);
      }
    }
  }
  // the chunk's own values, up to the row tile's end
  const int half = 16 * (ti + 1), s_lo = hf * half;
  const float* vr = base + p.v_off + (size_t)h * Dv + ec;
  float v[32];
#pragma unroll
  for (int i = 0; i < 32; ++i) v[i] = i < half ? vr[(size_t)min(s_lo + i, n - 1) * p.ld] : 0.f;
  if (scores) {
    const int c = tj * 32 + l;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int t = ti * 32 + lc_row(r, hf);
      P[t][c] = c <= t && t < n ? sc[r] * pw[t - c] : 0.f;
    }
  }
#pragma unroll
  for (int r = 0; r < 16; ++r) acc[r] *= pw[ti * 32 + lc_row(r, hf) + 1];
  __syncthreads();
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    if (4 * j >= half) break;
    const float4 a = *reinterpret_cast<const float4*>(&P[ti * 32 + l][s_lo + 4 * j]);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, v[4 * j], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, v[4 * j + 1], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, v[4 * j + 2], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, v[4 * j + 3], acc, 0, 0, 0);
  }
  if (e < Dv)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int t = ti * 32 + lc_row(r, hf);
      if (t < n) p.o[(size_t)(t0 + t) * p.H * Dv + (size_t)h * Dv + e] = acc[r];
    }
}

// The arguments of loqa_state_scan with a constant decay; ws: f32 [T / 64 + B, H, D,
// Dv].
extern "C" int loqa_linear_chunks(const void* act, long ld, int H, int D, int Dv, int q_off,
                                  int k_off, int v_off, int hpg, void* state, const void* state_slots,
                                  const void* cu_q, const void* positions, const void* decay, void* ws,
                                  void* o, int B, int T, hipStream_t st) {
  if (T <= 0 || B <= 0) return 0;
  if (H <= 0 || D <= 0 || Dv <= 0 || hpg <= 0 || H % hpg || !decay || !ws)
    return (int)hipErrorInvalidValue;
  const LcParams p{(const float*)act, ld, H, D, Dv, q_off, k_off, v_off, hpg, (float*)state,
                   (const int*)state_slots, (const int*)cu_q, (const int*)positions,
                   (const float*)decay, (float*)ws, (float*)o, B};
  const int chunks = T / LC_C + B;                   // at least the number of chunks
  hipLaunchKernelGGL(lc_local_kernel, dim3(chunks, H, (Dv + 31) / 32), dim3(256), 0, st, p);
  const size_t n = (size_t)D * Dv;
  if (n % 4 == 0)
    hipLaunchKernelGGL(lc_pass_kernel<4>, dim3(B, H, (int)((n / 4 + 255) / 256)), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL(lc_pass_kernel<1>, dim3(B, H, (int)((n + 255) / 256)), dim3(256), 0, st, p);
  const bool vec = D % 4 == 0 && ld % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 &&
                   ((size_t)act & 15) == 0;
  const dim3 grid(chunks, H, (Dv + 63) / 64);
  if (vec) hipLaunchKernelGGL(lc_out_kernel<true>, grid, dim3(256), 0, st, p);
  else hipLaunchKernelGGL(lc_out_kernel<false>, grid, dim3(256), 0, st, p);
  return (int)hipGetLastError();
}
