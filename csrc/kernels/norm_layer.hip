// Layer norm with weight and bias, fused with the residual step of a pre-norm
// layer whose sublayer outputs may carry RMS norms of their own:
//
//   residual_ln_kernel:   resid += scale * (n_0(y_0) + n_1(y_1)) + vec
//                         n_i(y) = y / sqrt(mean(y^2) + eps) * w_i with a weight, else y
//                         then ONE of
//                           h = (resid - mean) / sqrt(var + eps) * nw + nb
//                           h = resid in the dtype of h (no norm weight given)
//
// Any part may be absent: no addends and no vec is the norm alone (row_idx
// gathers rows then), no h is the sum alone. With two normed addends it is the
// step after two mixers side by side, with one the step after a per-token side
// input, with vec the entry of a pass over a repeated stretch. h may be a
// column slice of a wider row.
//
// One workgroup per row. A row of up to 4096 entries (a multiple of 4) stays in
// registers from the sums to the output; the variance is the mean of the squared
// deviations from the mean, in a second pass over the registers. Other widths
// read the row again. Everything is f32 inside.
//
// bigram_embed_kernel: x = embed[token] + pairs[row], row a hash of the previous
// and the current token (the table's last row for a sequence's first token). The
// previous token of a feed's first token comes from the sequence's slot, which
// the same workgroup then sets to the feed's last token, so no other reads it.
#include "seqmix.h"

#define RL_THREADS 256
#define RL_NV 4                      // float4 chunks per thread held in registers

struct ResLnParams {
  float* resid; const long* row_idx;
  const void* y0; const float* w0; const void* y1; const float* w1; float scale;
  const float* vec; const float* nw; const float* nb; float eps;
  void* h; long h_ld; int d;
};

// the sums of a and b over the workgroup
__device__ __forceinline__ float2 rl_sum2(float a, float b, float2* scratch) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if (lane == 0) scratch[wid] = make_float2(a, b);
  __syncthreads();
  float2 t = make_float2(0.f, 0.f);
#pragma unroll
  for (int i = 0; i < RL_THREADS / 64; ++i) { t.x += scratch[i].x; t.y += scratch[i].y; }
  return t;
}

template <typename TY, typename TO>
__global__ __launch_bounds__(RL_THREADS) void residual_ln_kernel(ResLnParams p) {
  __shared__ float2 scratch[RL_THREADS / 64];
  const size_t r = blockIdx.x;
  const int d = p.d;
  const float fd = (float)d;
  float* xr = p.resid + (p.row_idx ? (size_t)p.row_idx[r] : r) * d;
  const TY* a0 = p.y0 ? (const TY*)p.y0 + r * d : nullptr;
  const TY* a1 = p.y1 ? (const TY*)p.y1 + r * d : nullptr;
  TO* hr = p.h ? (TO*)p.h + r * p.h_ld : nullptr;
  const bool adds = a0 || a1 || p.vec;
  const bool norms = p.w0 || p.w1;
  if (d % 4 == 0 && d <= 4 * RL_THREADS * RL_NV && p.h_ld % 4 == 0) {
    float v[RL_NV][4], s0[RL_NV][4], s1[RL_NV][4];
    float q0 = 0.f, q1 = 0.f;
#pragma unroll
    for (int i = 0; i < RL_NV; ++i) {
      const int c = 4 * (threadIdx.x + RL_THREADS * i);
#pragma unroll
      for (int k = 0; k < 4; ++k) v[i][k] = s0[i][k] = s1[i][k] = 0.f;
      if (c < d) {
        ld_run<float, 4>(xr + c, v[i]);
        if (a0) ld_run<TY, 4>(a0 + c, s0[i]);
        if (a1) ld_run<TY, 4>(a1 + c, s1[i]);
#pragma unroll
        for (int k = 0; k < 4; ++k) { q0 += s0[i][k] * s0[i][k]; q1 += s1[i][k] * s1[i][k]; }
      }
    }
    float i0 = 1.f, i1 = 1.f;
    if (norms) {
      const float2 q = rl_sum2(q0, q1, scratch);
      if (p.w0) i0 = 1.f / sqrtf(q.x / fd + p.eps);
      if (p.w1) i1 = 1.f / sqrtf(q.y / fd + p.eps);
    }
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < RL_NV; ++i) {
      const int c = 4 * (threadIdx.x + RL_THREADS * i);
      if (c >= d) continue;
      if (adds) {
        float w0[4] = {1.f, 1.f, 1.f, 1.f}, w1[4] = {1.f, 1.f, 1.f, 1.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
        if (p.w0) ld_run<float, 4>(p.w0 + c, w0);
        if (p.w1) ld_run<float, 4>(p.w1 + c, w1);
        if (p.vec) ld_run<float, 4>(p.vec + c, b);
#pragma unroll
        for (int k = 0; k < 4; ++k)
          v[i][k] += p.scale * (s0[i][k] * i0 * w0[k] + s1[i][k] * i1 * w1[k]) + b[k];
        st_run<float, 4>(xr + c, v[i]);
      }
      sum += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
    }
    if (!hr) return;
    if (!p.nw) {
#pragma unroll
      for (int i = 0; i < RL_NV; ++i) {
        const int c = 4 * (threadIdx.x + RL_THREADS * i);
        if (c < d) st_run<TO, 4>(hr + c, v[i]);
      }
      return;
    }
    const float mean = rl_sum2(sum, 0.f, scratch).x / fd;
    float var = 0.f;
#pragma unroll
    for (int i = 0; i < RL_NV; ++i)
      if (4 * (threadIdx.x + RL_THREADS * i) < d)
#pragma unroll
        for (int k = 0; k < 4; ++k) { v[i][k] -= mean; var += v[i][k] * v[i][k]; }
    const float inv = 1.f / sqrtf(rl_sum2(var, 0.f, scratch).x / fd + p.eps);
#pragma unroll
    for (int i = 0; i < RL_NV; ++i) {
      const int c = 4 * (threadIdx.x + RL_THREADS * i);
      if (c < d) {
        float w[4], b[4];
        ld_run<float, 4>(p.nw + c, w);
        ld_run<float, 4>(p.nb + c, b);
#pragma unroll
        for (int k = 0; k < 4; ++k) w[k] = v[i][k] * inv * w[k] + b[k];
        st_run<TO, 4>(hr + c, w);
      }
    }
    return;
  }
  // any width: a thread's own columns are read again in every pass
  float i0 = 1.f, i1 = 1.f;
  if (norms) {
    float q0 = 0.f, q1 = 0.f;
    for (int c = threadIdx.x; c < d; c += RL_THREADS) {
      const float u = a0 ? Act<TY>::ld(a0 + c) : 0.f, w = a1 ? Act<TY>::ld(a1 + c) : 0.f;
      q0 += u * u;
      q1 += w * w;
    }
    const float2 q = rl_sum2(q0, q1, scratch);
    if (p.w0) i0 = 1.f / sqrtf(q.x / fd + p.eps);
    if (p.w1) i1 = 1.f / sqrtf(q.y / fd + p.eps);
  }
  float sum = 0.f;
  for (int c = threadIdx.x; c < d; c += RL_THREADS) {
    float v = xr[c];
    if (adds) {
      float s = 0.f;
      if (a0) s += Act<TY>::ld(a0 + c) * i0 * (p.w0 ? p.w0[c] : 1.f);
      if (a1) s += Act<TY>::ld(a1 + c) * i1 * (p.w1 ? p.w1[c] : 1.f);
      v += p.scale * s + (p.vec ? p.vec[c] : 0.f);
      xr[c] = v;
    }
    if (hr && !p.nw) Act<TO>::st(hr + c, v);
    sum += v;
  }
  if (!hr || !p.nw) return;
  const float mean = rl_sum2(sum, 0.f, scratch).x / fd;
  float var = 0.f;
  for (int c = threadIdx.x; c < d; c += RL_THREADS) {
    const float v = xr[c] - mean;
    var += v * v;
  }
  const float inv = 1.f / sqrtf(rl_sum2(var, 0.f, scratch).x / fd + p.eps);
  for (int c = threadIdx.x; c < d; c += RL_THREADS)
    Act<TO>::st(hr + c, (xr[c] - mean) * inv * p.nw[c] + p.nb[c]);
}

// TE: dtype of the tables; TO: dtype of the copies at x2 (row stride x2_ld, or null).
template <typename TE, typename TO, int N>
__global__ __launch_bounds__(256) void bigram_embed_kernel(
    const int* __restrict__ tokens, const TE* __restrict__ embed, const TE* __restrict__ pairs,
    int vocab, long buckets, long mul_prev, long mul_cur, int* __restrict__ prev, int nslots,
    const int* __restrict__ slots, const int* __restrict__ cu_q, const int* __restrict__ pos, int B,
    float* __restrict__ x, TO* __restrict__ x2, long x2_ld, int copies, int d) {
  __shared__ long row_s;
  const int t = blockIdx.x;
  const int tok = min(max(tokens[t], 0), vocab - 1);
  if (threadIdx.x == 0) {
    long row = buckets;                           // a sequence's first token
    if (t < cu_q[B]) {
      int lo = 0, hi = B - 1;                     // the last feed that starts at or before t
      while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (cu_q[mid] <= t) lo = mid; else hi = mid - 1;
      }
      const int q0 = cu_q[lo], slot = min(max(slots[lo], 0), nslots - 1);
      const bool first = t == q0;
      if (pos[t] > 0) {
        const long before = first ? prev[slot] : tokens[t - 1];
        row = (before * mul_prev + (long)tok * mul_cur) % buckets;
        if (row < 0) row += buckets;
      }
      if (first) prev[slot] = tokens[cu_q[lo + 1] - 1];
    }
    row_s = row;
  }
  __syncthreads();
  const TE* er = embed + (size_t)tok * d;
  const TE* pr = pairs + (size_t)row_s * d;
  for (int c = N * threadIdx.x; c < d; c += N * blockDim.x) {
    float a[N], b[N];
    ld_run<TE, N>(er + c, a);
    ld_run<TE, N>(pr + c, b);
#pragma unroll
    for (int k = 0; k < N; ++k) a[k] += b[k];
    st_run<float, N>(x + (size_t)t * d + c, a);
    if (x2)
      for (int k = 0; k < copies; ++k) st_run<TO, N>(x2 + (size_t)t * x2_ld + (size_t)k * d + c, a);
  }
}

extern "C" int loqa_residual_ln(void* resid, const void* row_idx, const void* y0, const void* w0,
                                const void* y1, const void* w1, int y_dt, float scale,
                                const void* vec, const void* nw, const void* nb, float eps, void* h,
                                int h_dt, long h_ld, int rows, int d, hipStream_t st) {
  if (rows <= 0) return 0;
  if (d <= 0 || (nw && (!nb || !h)) || (h && h_ld < d) || (row_idx && (y0 || y1 || vec)))
    return (int)hipErrorInvalidValue;
  const ResLnParams p{(float*)resid, (const long*)row_idx, y0, y0 ? (const float*)w0 : nullptr, y1,
                      y1 ? (const float*)w1 : nullptr, scale, (const float*)vec, (const float*)nw,
                      (const float*)nb, eps, h, h_ld, d};
#define GO(TY, TO) \
  hipLaunchKernelGGL((residual_ln_kernel<TY, TO>), dim3(rows), dim3(RL_THREADS), 0, st, p)
  if (y_dt == 0 && h_dt == 0) GO(bf16_t, bf16_t);
  else if (y_dt == 0) GO(bf16_t, float);
  else if (h_dt == 0) GO(float, bf16_t);
  else GO(float, float);
#undef GO
  return (int)hipGetLastError();
}

extern "C" int loqa_bigram_embed(const void* tokens, const void* embed, const void* pairs, int e_dt,
                                 int vocab, long buckets, long mul_prev, long mul_cur, void* prev,
                                 int nslots, const void* slots, const void* cu_q, const void* pos,
                                 int B, int T, void* x, void* x2, int x2_dt, long x2_ld, int copies,
                                 int d, hipStream_t st) {
  if (T <= 0) return 0;
  if (B <= 0 || vocab <= 0 || buckets <= 0 || nslots <= 0 || d <= 0 || copies < 0 ||
      (x2 && x2_ld < (long)copies * d))
    return (int)hipErrorInvalidValue;
  const bool v4 = d % 4 == 0 && (!x2 || x2_ld % 4 == 0);
#define GO(TE, TO, N)                                                                            \
  hipLaunchKernelGGL((bigram_embed_kernel<TE, TO, N>), dim3(T), dim3(256), 0, st,                \
                     (const int*)tokens, (const TE*)embed, (const TE*)pairs, vocab, buckets,     \
                     mul_prev, mul_cur, (int*)prev, nslots, (const int*)slots, (const int*)cu_q, \
                     (const int*)pos, B, (float*)x, (TO*)x2, x2_ld, copies, d)
#define BY_N(TE, TO) do { if (v4) GO(TE, TO, 4); else GO(TE, TO, 1); } while (0)
  if (e_dt == 0 && x2_dt == 0) BY_N(bf16_t, bf16_t);
  else if (e_dt == 0) BY_N(bf16_t, float);
  else if (x2_dt == 0) BY_N(float, bf16_t);
  else BY_N(float, float);
#undef BY_N
#undef GO
  return (int)hipGetLastError();
}
