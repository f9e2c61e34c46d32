// Helpers shared by the sequence-mixer kernels of the hybrid decoders
// (norm_dyt.hip, attn_latent.hip, lightning.hip, moe.hip, seq_rows.hip,
// attn_sigmoid.hip, norm_scalar.hip, norm_rms1p.hip, attn_window.hip, mamba2.hip,
// matrix_memory.hip, delta_rule.hip, norm_layer.hip, linear_chunks.hip,
// delta_chunks.hip).
//
// Activations are bfloat16 or float32, chosen at run time by a dtype code
// (0: bf16, 1: f32); every kernel is a template over the storage type and does
// its arithmetic in f32. Small vectors (norm weights, sinks, decays, router
// corrections) are always f32.
#pragma once
#include "common.h"
#include <math.h>

template <typename T> struct Act;
template <> struct Act<bf16_t> {
  static __device__ __forceinline__ float ld(const bf16_t* p) { return bf2f(*p); }
  static __device__ __forceinline__ void st(bf16_t* p, float v) { *p = f2bf(v); }
};
template <> struct Act<float> {
  static __device__ __forceinline__ float ld(const float* p) { return *p; }
  static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
};

// tanh through one exponential: 1 - 2 / (1 + e^{2z}); absolute error of a few
// 1e-8 over the whole range (saturates to +-1 for large |z| without overflow
// trouble: e^{2z} = inf gives 1, 0 gives -1).
__device__ __forceinline__ float tanh_f(float z) { return 1.f - 2.f / (1.f + expf(2.f * z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
// The same through the hardware's exp2 and reciprocal (about 1 ulp each, a few
// 1e-6 relative for |z| up to 50): for results that are rounded to bfloat16.
__device__ __forceinline__ float sigmoid_fast(float z) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.44269504088896f * z));
}
template <typename T> __device__ __forceinline__ float sigmoid_for(float z) {
  return sizeof(T) == 2 ? sigmoid_fast(z) : sigmoid_f(z);
}

// Runs of N neighbouring entries (N = 4: one 16- or 8-byte access, N = 1: one
// entry) as f32.
template <typename T, int N> __device__ __forceinline__ void ld_run(const T* p, float* f) {
  if constexpr (N == 1) {
    f[0] = Act<T>::ld(p);
  } else if constexpr (sizeof(T) == 4) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  } else {
    const uint2 r = *reinterpret_cast<const uint2*>(p);
    f[0] = __uint_as_float(r.x << 16); f[1] = __uint_as_float(r.x & 0xffff0000u);
    f[2] = __uint_as_float(r.y << 16); f[3] = __uint_as_float(r.y & 0xffff0000u);
  }
}
template <typename T, int N> __device__ __forceinline__ void st_run(T* p, const float* f) {
  if constexpr (N == 1) {
    Act<T>::st(p, f[0]);
  } else if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
  } else {
    uint2 r;
    r.x = pack_bf16x2(f[0], f[1]);
    r.y = pack_bf16x2(f[2], f[3]);
    *reinterpret_cast<uint2*>(p) = r;
  }
}

// Side columns of a parallel layer's fused projection: the ungated feed-forward
// reads the same input as the mixer, so its up projection is a column slice of
// the same matrix product. src [T, src_ld] (the slice's first column) ->
// dst[t, 0 .. n) = relu(src)^2, and zeros in the columns zero_lo .. 0 (negative
// offsets: padding before the slice) and n .. zero_hi. The workgroups of a token
// (gridDim.y of them) share its row; vec: rows and bases are aligned for runs of
// four.
struct SideCols {
  const void* src; long src_ld;
  void* dst; long dst_ld;
  int n, zero_lo, zero_hi, vec;
};
template <typename T>
__device__ __forceinline__ void side_relu2(const SideCols& s, size_t t) {
  if (!s.dst) return;
  const T* a = (const T*)s.src + t * s.src_ld;
  T* o = (T*)s.dst + t * s.dst_ld;
  const int me = blockIdx.y * blockDim.x + threadIdx.x, all = gridDim.y * blockDim.x;
  if (s.vec) {
#pragma unroll 2
    for (int c = 4 * me; c < s.n; c += 4 * all) {
      float f[4];
      ld_run<T, 4>(a + c, f);
#pragma unroll
      for (int i = 0; i < 4; ++i) { f[i] = fmaxf(f[i], 0.f); f[i] *= f[i]; }
      st_run<T, 4>(o + c, f);
    }
  } else {
    for (int c = me; c < s.n; c += all) {
      const float f = fmaxf(Act<T>::ld(a + c), 0.f);
      Act<T>::st(o + c, f * f);
    }
  }
  for (int c = s.zero_lo + me; c < 0; c += all) Act<T>::st(o + c, 0.f);
  for (int c = s.n + me; c < s.zero_hi; c += all) Act<T>::st(o + c, 0.f);
}

// Feeds cut into chunks of C tokens counted from their first one. The chunk
// numbered i over all feeds: its sequence, first token and length; false past the
// last chunk. All lanes of the wave must be active.
template <int C>
__device__ __forceinline__ bool seq_chunk(const int* __restrict__ cu_q, int B, int i, int& b, int& t0,
                                          int& n) {
  const int lane = threadIdx.x & 63;
  for (int base = 0; base < B; base += 64) {
    const int s = base + lane;
    const int lo = s < B ? cu_q[s] : 0, hi = s < B ? cu_q[s + 1] : 0;
    const int nc = (hi - lo + C - 1) / C;
    int end = nc;                                    // inclusive prefix sum over the lanes
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(end, o, 64);
      if (lane >= o) end += v;
    }
    const unsigned long long past = __ballot(end > i);
    if (past) {
      const int w = __ffsll(past) - 1;
      b = base + w;
      t0 = __shfl(lo, w, 64) + (i - __shfl(end - nc, w, 64)) * C;
      n = min(C, __shfl(hi, w, 64) - t0);
      return true;
    }
    i -= __shfl(end, 63, 64);
  }
  return false;
}
// the number of chunks of the sequences before b (all lanes active)
template <int C>
__device__ __forceinline__ int seq_chunks_before(const int* __restrict__ cu_q, int b) {
  int c = 0;
  for (int s = threadIdx.x & 63; s < b; s += 64) c += (cu_q[s + 1] - cu_q[s] + C - 1) / C;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) c += __shfl_xor(c, o, 64);
  return c;
}

static inline int ceil_div(long a, long b) { return (int)((a + b - 1) / b); }
