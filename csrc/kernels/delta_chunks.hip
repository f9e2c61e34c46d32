// The gated delta rule over a flat token batch, chunk by chunk on the f32 matrix
// cores: the long feeds of the recurrence
//
//   S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//
// (g_t a number per head or, CHAN, one per head and key channel) that
// delta_scan_kernel (delta_rule.hip) runs token by token. Feeds are cut into chunks
// of 16 tokens counted from their first one. Write P(i, j) for the product of the
// decays g_{j+1} .. g_i (per channel), P(i) for g_1 .. g_i, S for the state before the
// chunk. Unrolling the definition within the chunk,
//
//   u_i = beta_i (v_i - (P(i) k_i)^T S - sum_{j < i} A_ij u_j)   A_ij = sum_d k_i P(i, j) k_j
//   o_i = (P(i) q_i)^T S + sum_{j <= i} B_ij u_j                 B_ij = sum_d q_i P(i, j) k_j
//   S_end = P(16) S + sum_j (P(16, j) k_j) u_j^T
//
// The first line is a unit lower triangular system in the u_i. Forward substitution
// on its two right-hand sides separately gives u = U - W S with U from the values and
// W from the keys, and neither depends on S. So
//
// delta_local_kernel (a workgroup per chunk and head, all chunks in parallel) forms
// A and B (16 lanes per row i; the rows k_i P(i, j) and q_i P(i, j) are carried down
// from j = i by one multiplication per step, so no decay is ever divided by or taken
// to a negative power), and W, U by forward substitution, a thread per column;
//
// delta_pass_kernel (a workgroup per sequence, head and 16 value columns) walks the
// chunks in order with the state in MFMA accumulators: W S and (P q) S, u = U - W S,
// S <- P(16) S + K^T u, o = (P q) S + B u. The four waves split the key channels and
// add up W S through LDS. With v_mfma_f32_16x16x4_f32 lane 16 g + m holds of an
// accumulator the rows 4 g + r (register r) of column m, and of a B operand row g of
// a step; taking the rows 4 g + r as step r's k indices makes an accumulator's
// registers the B operands of the next product as they are, and the A operand's four
// steps one 16-byte run.
//
// All products are exact f32 multiply-adds; the sums differ from the token-by-token
// kernel's in order only. Short chunks at a feed's end are filled with tokens that
// change nothing (k = q = v = 0, beta = 0, g = 1).
#include "seqmix.h"

#define DC_C 16

struct DcParams {
  const float* act; long ld; int H, D, Dv, q_off, k_off, v_off, g_off, hpg;
  float* state; const int* slots; const int* cu_q; const int* pos; const float* tok;
  float* ws; float* o; int B;
};

// Workspace of one (chunk, head), DP the padded key size: W [16][DP], P q [16][DP],
// (P(16, j) k_j) as [DP][16], P(16) [DP], U as [Dv][16], B [16][16].
__host__ __device__ __forceinline__ size_t dc_stride(int DP, int Dv) {
  return (size_t)49 * DP + 16 * Dv + 256;
}

template <int CTRL> __device__ __forceinline__ float dc_dpp(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, true));
}
// the sum over each run of 16 lanes, in every lane of the run
__device__ __forceinline__ float dc_sum16(float v) {
  v += dc_dpp<0xB1>(v);
  v += dc_dpp<0x4E>(v);
  v += dc_dpp<0x141>(v);
  v += dc_dpp<0x140>(v);
  return v;
}

// NT: key channels in units of 64 (DP = 64 NT)
template <int NT, bool CHAN>
__global__ __launch_bounds__(256) void delta_local_kernel(DcParams p) {
  constexpr int DP = 64 * NT, LD = DP + 4;
  __shared__ __attribute__((aligned(16))) float ks[DC_C][LD], qs[DC_C][LD], gs[DC_C][LD];
  __shared__ __attribute__((aligned(16))) float A[DC_C][DC_C];
  __shared__ float bs[DC_C];
  int b, t0, n;
  if (!seq_chunk<DC_C>(p.cu_q, p.B, blockIdx.x, b, t0, n)) return;
  const int h = blockIdx.y, tid = threadIdx.x, D = p.D, Dv = p.Dv;
  float* ws = p.ws + ((size_t)blockIdx.x * p.H + h) * dc_stride(DP, Dv);
  const float* base = p.act + (size_t)t0 * p.ld;
  {
    const float* qr = base + p.q_off + (size_t)(h / p.hpg) * D;
    const float* kr = base + p.k_off + (size_t)(h / p.hpg) * D;
    const float* gr = CHAN ? base + p.g_off + (size_t)h * D : nullptr;
    const float* tr = p.tok + ((size_t)t0 * p.H + h) * 2;
#pragma unroll
    for (int j = 0; j < DC_C * DP / 256; ++j) {
      const int i = (tid + 256 * j) / DP, d = (tid + 256 * j) % DP;
      const bool ok = i < n && d < D;
      const size_t row = (size_t)(i < n ? i : 0) * p.ld;
      qs[i][d] = ok ? qr[row + d] : 0.f;
      ks[i][d] = ok ? kr[row + d] : 0.f;
      gs[i][d] = ok ? (CHAN ? gr[row + d] : tr[(size_t)i * p.H * 2]) : 1.f;
    }
    if (tid < DC_C) bs[tid] = tid < n ? tr[(size_t)tid * p.H * 2 + 1] : 0.f;
  }
  __syncthreads();
  // A and B: row i on 16 lanes, lane q with the channels 64 m + 4 q ..
  const int i = tid >> 4, q = tid & 15;
  float a[NT][4], c[NT][4];
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    ld_run<float, 4>(&ks[i][64 * m + 4 * q], a[m]);
    ld_run<float, 4>(&qs[i][64 * m + 4 * q], c[m]);
  }
  float* Bw = ws + 49 * DP + 16 * Dv;
#pragma unroll 4
  for (int j = DC_C - 1; j >= 0; --j) {
    float sa = 0.f, sb = 0.f;
    if (j <= i) {
#pragma unroll
      for (int m = 0; m < NT; ++m) {
        float k[4], g[4];
        ld_run<float, 4>(&ks[j][64 * m + 4 * q], k);
        ld_run<float, 4>(&gs[j][64 * m + 4 * q], g);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          sa += a[m][e] * k[e];
          sb += c[m][e] * k[e];
          a[m][e] *= g[e];
          c[m][e] *= g[e];
        }
      }
    }
    sa = dc_sum16(sa);
    sb = dc_sum16(sb);
    if (q == 0) {
      A[i][j] = j < i ? sa : 0.f;
      Bw[i * DC_C + j] = j <= i ? sb : 0.f;
    }
  }
  // a = P(i) k_i, c = P(i) q_i now
#pragma unroll
  for (int m = 0; m < NT; ++m) st_run<float, 4>(ws + 16 * DP + i * DP + 64 * m + 4 * q, c[m]);
  // P(16, j) k_j and P(16), a thread per channel
  for (int d = tid; d < DP; d += 256) {
    float r = 1.f, kk[DC_C];
#pragma unroll
    for (int j = DC_C - 1; j >= 0; --j) {
      kk[j] = ks[j][d] * r;
      r *= gs[j][d];
    }
#pragma unroll
    for (int j = 0; j < DC_C; j += 4) st_run<float, 4>(ws + 32 * DP + (size_t)d * DC_C + j, kk + j);
    ws[48 * DP + d] = r;
  }
  __syncthreads();
#pragma unroll
  for (int m = 0; m < NT; ++m) st_run<float, 4>(&ks[i][64 * m + 4 * q], a[m]);
  __syncthreads();
  // forward substitution, a thread per column of [P k | v]
  for (int col = tid; col < DP + Dv; col += 256) {
    float x[DC_C];
    const bool key = col < DP;
    const float* vr = base + p.v_off + (size_t)h * Dv + (key ? 0 : col - DP);
#pragma unroll
    for (int t = 0; t < DC_C; ++t)
      x[t] = key ? ks[t][col] : (t < n ? vr[(size_t)t * p.ld] : 0.f);
#pragma unroll
    for (int t = 0; t < DC_C; ++t) {
      float s = x[t];
#pragma unroll
      for (int j = 0; j < t; ++j) s -= A[t][j] * x[j];
      x[t] = bs[t] * s;
    }
    if (key) {
#pragma unroll
      for (int t = 0; t < DC_C; ++t) ws[t * DP + col] = x[t];
    } else {
#pragma unroll
      for (int t = 0; t < DC_C; t += 4)
        st_run<float, 4>(ws + 49 * DP + (size_t)(col - DP) * DC_C + t, x + t);
    }
  }
}

// (2 workgroups per CU at least: the accumulators stay in ordinary registers, which
// the next products read as operands)
template <int NT>
__global__ __launch_bounds__(256, 2) void delta_pass_kernel(DcParams p) {
  constexpr int DP = 64 * NT, NS = NT <= 2 ? 4 : 2;
  __shared__ float4v xs[2][4][64], ys[2][4][64];
  const int b = blockIdx.x, h = blockIdx.y, e0 = blockIdx.z * 16;
  const int q0 = p.cu_q[b], len = p.cu_q[b + 1] - q0;
  if (len <= 0) return;
  const int before = seq_chunks_before<DC_C>(p.cu_q, b);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, m = lane & 15, g = lane >> 4;
  const int D = p.D, Dv = p.Dv, nc = (len + DC_C - 1) / DC_C;
  const bool col = e0 + m < Dv;
  const int ec = min(e0 + m, Dv - 1);
  // state [slots, H, Dv, D]: the wave's tile t holds the channels 16 (NT wave + t) ..
  float* Sg = p.state + (((size_t)p.slots[b] * p.H + h) * Dv + ec) * D;
  const bool fresh = p.pos[q0] == 0;
  float4v S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * (NT * wave + t) + 4 * g + r;
      S[t][r] = !fresh && d < D ? Sg[d] : 0.f;
    }
  const size_t st = dc_stride(DP, Dv), step = st * p.H;
  const float* ws = p.ws + ((size_t)before * p.H + h) * st;
  struct Set { float4v W[NT], Q[NT], K[NT], G[NT], U; float B; };
  auto fetch = [&](Set& f, int c) {
    const float* w = ws + (size_t)c * step;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int d0 = 16 * (NT * wave + t);
      f.W[t] = *reinterpret_cast<const float4v*>(w + m * DP + d0 + 4 * g);
      f.Q[t] = *reinterpret_cast<const float4v*>(w + 16 * DP + m * DP + d0 + 4 * g);
      f.K[t] = *reinterpret_cast<const float4v*>(w + 32 * DP + (d0 + m) * DC_C + 4 * g);
      f.G[t] = *reinterpret_cast<const float4v*>(w + 48 * DP + d0 + 4 * g);
    }
    f.U = *reinterpret_cast<const float4v*>(w + 49 * DP + (size_t)ec * DC_C + 4 * g);
    f.B = w[49 * DP + 16 * Dv + m * DC_C + 4 * g + wave];
  };
  // the outputs of chunk c: wave w takes the tokens 4 g + w
  auto outputs = [&](int c, int par) {
    const float* y = reinterpret_cast<const float*>(&ys[par][0][lane]) + wave;
    const float s = (y[0] + y[256]) + (y[512] + y[768]);
    const int t = c * DC_C + 4 * g + wave;
    if (col && t < len) p.o[(size_t)(q0 + t) * p.H * Dv + (size_t)h * Dv + e0 + m] = s;
  };
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  auto chunk = [&](Set& f, int c, int par) {
    float4v X = zero, Y = zero;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        X = __builtin_amdgcn_mfma_f32_16x16x4f32(f.W[t][r], S[t][r], X, 0, 0, 0);
    xs[par][wave][lane] = X;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        Y = __builtin_amdgcn_mfma_f32_16x16x4f32(f.Q[t][r], S[t][r], Y, 0, 0, 0);
    __syncthreads();
    const float4v u = f.U - ((xs[par][0][lane] + xs[par][1][lane]) +
                             (xs[par][2][lane] + xs[par][3][lane]));
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] *= f.G[t];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int t = 0; t < NT; ++t)
        S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.K[t][r], u[r], S[t], 0, 0, 0);
    const float uw = wave < 2 ? (wave == 0 ? u[0] : u[1]) : (wave == 2 ? u[2] : u[3]);
    ys[par][wave][lane] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.B, uw, Y, 0, 0, 0);
    // every wave wrote chunk c - 1's part before this chunk's barrier
    if (c > 0) outputs(c - 1, par ^ 1);
    fetch(f, min(c + NS, nc - 1));       // unconditional: the waits count loads
  };
  // NS chunks' inputs in flight: a chunk takes less time than a trip to memory
  Set f0, f1, f2, f3;
  fetch(f0, 0);
  fetch(f1, min(1, nc - 1));
  int c = 0;
  if constexpr (NS == 4) {
    fetch(f2, min(2, nc - 1));
    fetch(f3, min(3, nc - 1));
    for (; c + 3 < nc; c += 4) {
      chunk(f0, c, 0);
      chunk(f1, c + 1, 1);
      chunk(f2, c + 2, 0);
      chunk(f3, c + 3, 1);
    }
    if (c < nc) chunk(f0, c, 0);
    if (c + 1 < nc) chunk(f1, c + 1, 1);
    if (c + 2 < nc) chunk(f2, c + 2, 0);
  } else {
    for (; c + 1 < nc; c += 2) {
      chunk(f0, c, 0);
      chunk(f1, c + 1, 1);
    }
    if (c < nc) chunk(f0, c, 0);
  }
  __syncthreads();
  outputs(nc - 1, (nc - 1) & 1);
  if (col)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * (NT * wave + t) + 4 * g + r;
        if (d < D) Sg[d] = S[t][r];
      }
}

extern "C" long loqa_delta_chunks_ws(int H, int D, int Dv, int B, int T) {
  const int NT = D <= 64 ? 1 : (D <= 128 ? 2 : 4);
  return (long)(T / DC_C + B) * H * (long)dc_stride(64 * NT, Dv);
}

// The arguments of loqa_delta_scan; ws: f32, loqa_delta_chunks_ws entries.
extern "C" int loqa_delta_chunks(const void* act, long ld, int H, int D, int Dv, int q_off, int k_off,
                                 int v_off, int g_off, int hpg, void* state, const void* state_slots,
                                 const void* cu_q, const void* positions, const void* tok, void* ws,
                                 void* o, int B, int T, hipStream_t st) {
  if (T <= 0 || B <= 0) return 0;
  if (H <= 0 || D <= 0 || D > 256 || Dv <= 0 || hpg <= 0 || H % hpg || !tok || !ws)
    return (int)hipErrorInvalidValue;
  const DcParams p{(const float*)act, ld, H, D, Dv, q_off, k_off, v_off, g_off, hpg, (float*)state,
                   (const int*)state_slots, (const int*)cu_q, (const int*)positions,
                   (const float*)tok, (float*)ws, (float*)o, B};
  const dim3 gl(T / DC_C + B, H), gp(B, H, (Dv + 15) / 16);
#define GO(NT)                                                                                   \
  do {                                                                                           \
    if (g_off >= 0)                                                                              \
      hipLaunchKernelGGL((delta_local_kernel<NT, true>), gl, dim3(256), 0, st, p);               \
    else                                                                                         \
      hipLaunchKernelGGL((delta_local_kernel<NT, false>), gl, dim3(256), 0, st, p);              \
    hipLaunchKernelGGL(delta_pass_kernel<NT>, gp, dim3(256), 0, st, p);                          \
  } while (0)
  if (D <= 64) GO(1); else if (D <= 128) GO(2); else GO(4);
#undef GO
  return (int)hipGetLastError();
}
