// Latent (compressed-KV) attention over a paged latent cache.
//
// Every token caches ONE row [R latent | Dr rotary key part] shared by all
// heads; queries arrive already folded into latent space (qa = W_uk^T q), so
//   score(h, t, j) = (qa[h,t] . c_j + rot(qr[t,h]) . kr_j) * scale
//   out[h, t]      = sum_j softmax_j(score)[j] * c_j      (W_uv is applied after)
// with an optional learned sink per head that only joins the denominator, and
// an optional sliding window (the query at position p sees p - j < window).
//
// latent_inputs_kernel: everything between the fused projection and attention
//   that is no matrix product: RMS-norm of the latent part, interleaved rotary
//   on the key part (pairs 2i, 2i+1 of the first `dims` entries), store at the
//   slot; optionally the RMS norm of a query latent in the same rows, and the
//   side columns of a parallel layer.
// latent_attn_mfma_kernel (bf16; R a multiple of 16 up to 512, R + Dr one of 8 up
//   to 640): one workgroup per (query token, group of 16 heads, key split). Tiles
//   of 32 keys are staged in LDS once for the 16 heads; scores and outputs run on
//   the matrix cores with the head on the MFMA column, so the online softmax is
//   per lane.
// latent_attn_kernel (f32 and other sizes; latent_attn2_kernel is its form for
//   even sizes): one workgroup per (query token, group of 4 heads, key split). Key tiles are staged once in LDS (f32, odd row stride) for the
//   group's heads; each wave owns one head: a lane scores one key of the tile,
//   the online softmax runs across the wave, and for P.C each lane owns output
//   entries r = lane + 64 i. Prompt portions, single decode tokens and mixed
//   batches take this same kernel: a row's result depends only on its own
//   sequence's pages, in key order. Long contexts with few query rows split
//   the keys over workgroups; latent_combine_kernel merges the partials.
#include "seqmix.h"

#define LAT_THREADS 256
#define LAT_WAVES 4
#define LAT_MAXR 8      // R <= 64 * LAT_MAXR

struct LatInParams {
  const void* z; long ldz;               // [T, R + Dr]
  const float* nw; float eps;
  const int* pos; const float* cs; int max_pos;
  void* cache; long cache_rows; const int* slots;
  int R, Dr, dims;
  const void* dq; long lddq; const float* qw; int Rq; void* cq;   // query latent [T, Rq], or Rq == 0
  int vz, vq;                            // the rows can be accessed in runs of four
};

// The workgroups of a token: the last one norms and stores the cache row, the
// first one norms the query latent (the same workgroup when there is one), all
// share the side columns. Rows go in
// runs of N = 4 entries where they are aligned, else one by one.
template <typename T, int N>
__device__ __forceinline__ float li_sumsq(const T* x, int n) {
  float s = 0.f;
#pragma unroll 2
  for (int i = N * threadIdx.x; i < n; i += N * 128) {
    float f[N];
    ld_run<T, N>(x + i, f);
#pragma unroll
    for (int k = 0; k < N; ++k) s += f[k] * f[k];
  }
  return s;
}
template <typename T, int N>
__device__ __forceinline__ void li_scale(const T* x, const float* w, float inv, T* y, int n) {
#pragma unroll 2
  for (int i = N * threadIdx.x; i < n; i += N * 128) {
    float f[N], ww[N];
    ld_run<T, N>(x + i, f);
    ld_run<float, N>(w + i, ww);
#pragma unroll
    for (int k = 0; k < N; ++k) f[k] *= inv * ww[k];
    st_run<T, N>(y + i, f);
  }
}

template <typename T>
__global__ __launch_bounds__(128) void latent_inputs_kernel(LatInParams p, SideCols side) {
  __shared__ float part[2][2];
  const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const bool do_q = p.Rq && blockIdx.y == 0, do_z = blockIdx.y + 1 == gridDim.y;   // uniform
  const T* zr = (const T*)p.z + (size_t)t * p.ldz;
  const T* qr = p.Rq ? (const T*)p.dq + (size_t)t * p.lddq : nullptr;
  if (do_q || do_z) {
    float ss = 0.f, sq = 0.f;
    if (do_z) ss = p.vz ? li_sumsq<T, 4>(zr, p.R) : li_sumsq<T, 1>(zr, p.R);
    if (do_q) sq = p.vq ? li_sumsq<T, 4>(qr, p.Rq) : li_sumsq<T, 1>(qr, p.Rq);
    ss = wave_sum(ss);
    sq = wave_sum(sq);
    if (lane == 0) { part[0][wave] = ss; part[1][wave] = sq; }
    __syncthreads();
  }
  if (do_q) {
    const float inv = 1.f / sqrtf((part[1][0] + part[1][1]) / (float)p.Rq + p.eps);
    T* cq = (T*)p.cq + (size_t)t * p.Rq;
    if (p.vq) li_scale<T, 4>(qr, p.qw, inv, cq, p.Rq);
    else li_scale<T, 1>(qr, p.qw, inv, cq, p.Rq);
  }
  side_relu2<T>(side, t);
  if (!do_z) return;
  const int slot = p.slots[t];
  if (slot < 0 || slot >= p.cache_rows) return;    // padding row
  const float inv = 1.f / sqrtf((part[0][0] + part[0][1]) / (float)p.R + p.eps);
  T* row = (T*)p.cache + (size_t)slot * (p.R + p.Dr);
  if (p.vz) li_scale<T, 4>(zr, p.nw, inv, row, p.R);
  else li_scale<T, 1>(zr, p.nw, inv, row, p.R);
  const int pp = min(max(p.pos[t], 0), p.max_pos - 1);
  const float* csr = p.cs + (size_t)pp * p.dims;     // [dims/2][2]
  for (int i = threadIdx.x; i < p.Dr; i += 128) {
    float o;
    if (i < p.dims) {
      const float c = csr[(i >> 1) * 2], s = csr[(i >> 1) * 2 + 1];
      const float u = Act<T>::ld(zr + p.R + (i & ~1)), v = Act<T>::ld(zr + p.R + (i | 1));
      o = (i & 1) ? v * c + u * s : u * c - v * s;
    } else {
      o = Act<T>::ld(zr + p.R + i);
    }
    Act<T>::st(row + p.R + i, o);
  }
}

struct LatAttnParams {
  const void* qa; long qa_st, qa_sh;     // [H, T, R] strides in elements (token, head)
  const void* qr; long qr_st, qr_sh;     // [T, H, Dr]
  const void* cache; int blk;
  const int* cu_q; const int* ctx; const int* bt; int max_blocks;
  const int* pos; const float* cs; int max_pos;
  const float* sink; float scale;
  int B, H, T, R, Dr, dims;
  void* out;                             // [H, T, R]
  int num_splits, KT;
  float* ws;                             // [splits, T, H, R + 2] when num_splits > 1
  int window;                            // > 0: keys p - window + 1 .. p only
};

template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void latent_attn_kernel(LatAttnParams p) {
  extern __shared__ float lds[];
  const int W = p.R + p.Dr, Ws = W | 1, KT = p.KT;
  float* ktile = lds;                         // [KT][Ws]
  float* qs = ktile + (size_t)KT * Ws;        // [4][W]
  float* ps = qs + LAT_WAVES * W;             // [4][KT]
  const int t = blockIdx.x, split = blockIdx.z;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int h_raw = blockIdx.y * LAT_WAVES + wave;
  const bool live = h_raw < p.H;
  const int h = live ? h_raw : p.H - 1;       // idle waves shadow a head, write nothing
  T* out = (T*)p.out + ((size_t)h * p.T + t) * p.R;
  float* wsr = p.num_splits > 1
      ? p.ws + (((size_t)split * p.T + t) * p.H + h) * (p.R + 2) : nullptr;

  int nk = 0, lo = 0, b = 0;
  if (t < p.cu_q[p.B]) {
    while (b + 1 < p.B && t >= p.cu_q[b + 1]) ++b;
    nk = min(p.pos[t] + 1, p.ctx[b]);
    if (p.window > 0) lo = min(max(0, p.pos[t] + 1 - p.window), nk);
  }
  int k0 = lo, k1 = nk;
  if (p.num_splits > 1) {
    const int per = ((nk - lo + p.num_splits - 1) / p.num_splits + KT - 1) / KT * KT;
    k0 = min(nk, lo + split * per);
    k1 = min(nk, k0 + per);
  }
  // the wave's query in LDS, pre-scaled; its rotary part rotated here
  {
    const T* qa = (const T*)p.qa + (size_t)t * p.qa_st + (size_t)h * p.qa_sh;
    const T* qr = (const T*)p.qr + (size_t)t * p.qr_st + (size_t)h * p.qr_sh;
    const int pp = min(max(p.pos[t], 0), p.max_pos - 1);
    const float* csr = p.cs + (size_t)pp * p.dims;
    for (int i = lane; i < W; i += 64) {
      float v;
      if (i < p.R) {
        v = Act<T>::ld(qa + i);
      } else {
        const int j = i - p.R;
        if (j < p.dims) {
          const float c = csr[(j >> 1) * 2], s = csr[(j >> 1) * 2 + 1];
          const float u = Act<T>::ld(qr + (j & ~1)), w = Act<T>::ld(qr + (j | 1));
          v = (j & 1) ? w * c + u * s : u * c - w * s;
        } else {
          v = Act<T>::ld(qr + j);
        }
      }
      qs[wave * W + i] = v * p.scale;
    }
  }
  float m = -INFINITY, l = 0.f;
  float acc[LAT_MAXR];
#pragma unroll
  for (int i = 0; i < LAT_MAXR; ++i) acc[i] = 0.f;
  const T* cache = (const T*)p.cache;
  const int* bt = p.bt + (size_t)b * p.max_blocks;
  for (int kt = k0; kt < k1; kt += KT) {
    __syncthreads();                          // the previous tile is consumed
    for (int j = wave; j < KT; j += LAT_WAVES) {
      const int key = kt + j;
      float* dst = ktile + (size_t)j * Ws;
      if (key < k1) {
        const T* src = cache + ((size_t)bt[key / p.blk] * p.blk + key % p.blk) * W;
        for (int c = lane; c < W; c += 64) dst[c] = Act<T>::ld(src + c);
      } else {
        for (int c = lane; c < W; c += 64) dst[c] = 0.f;
      }
    }
    __syncthreads();
    float s = -INFINITY;
    if (lane < KT && kt + lane < k1) {
      const float* kr = ktile + (size_t)lane * Ws;
      const float* q = qs + wave * W;
      float a = 0.f;
      for (int c = 0; c < W; ++c) a += q[c] * kr[c];
      s = a;
    }
    const float mn = fmaxf(m, wave_max(s));   // finite: the tile holds >= 1 key
    const float pj = s == -INFINITY ? 0.f : expf(s - mn);
    const float corr = m == -INFINITY ? 0.f : expf(m - mn);
    l = l * corr + wave_sum(pj);
    m = mn;
    if (lane < KT) ps[wave * KT + lane] = pj;
    __syncthreads();                          // ps visible to the wave's other lanes
#pragma unroll
    for (int i = 0; i < LAT_MAXR; ++i) acc[i] *= corr;
    const int nj = min(KT, k1 - kt);
    for (int j = 0; j < nj; ++j) {
      const float pv = ps[wave * KT + j];
      const float* cr = ktile + (size_t)j * Ws;
#pragma unroll
      for (int i = 0; i < LAT_MAXR; ++i) {
        const int r = lane + 64 * i;
        if (r < p.R) acc[i] += pv * cr[r];
      }
    }
  }
  if (!live) return;
  if (wsr) {                                  // partial of this key split
    if (lane == 0) { wsr[0] = m; wsr[1] = l; }
#pragma unroll
    for (int i = 0; i < LAT_MAXR; ++i) {
      const int r = lane + 64 * i;
      if (r < p.R) wsr[2 + r] = acc[i];
    }
    return;
  }
  float M = m, den = l, f = 1.f;
  if (p.sink) {
    const float sk = p.sink[h];
    M = fmaxf(m, sk);
    f = m == -INFINITY ? 0.f : expf(m - M);
    den = l * f + expf(sk - M);
  }
  const float inv = den > 0.f ? f / den : 0.f;
#pragma unroll
  for (int i = 0; i < LAT_MAXR; ++i) {
    const int r = lane + 64 * i;
    if (r < p.R) Act<T>::st(out + r, acc[i] * inv);
  }
}

// The same computation for even R and R + Dr (every real configuration), laid
// out for throughput: the key tile sits in LDS in the activation dtype (twice
// the keys per tile for bf16), the score of a key is split over two lanes (each
// half of the wave takes half of the row, read two entries at a time, two
// independent accumulators), and for P.C a lane owns pairs of output entries.
#define LAT_MAXP 8      // R <= 128 * LAT_MAXP
#define LAT_MAXCH 10    // 16-byte chunks of a key tile per thread

template <typename T> struct Pair;
template <> struct Pair<bf16_t> {
  static __device__ __forceinline__ float2 ld(const bf16_t* p) {
    const uint32_t w = *reinterpret_cast<const uint32_t*>(p);
    return make_float2(__uint_as_float(w << 16), __uint_as_float(w & 0xffff0000u));
  }
};
template <> struct Pair<float> {
  static __device__ __forceinline__ float2 ld(const float* p) {
    return *reinterpret_cast<const float2*>(p);
  }
};

template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void latent_attn2_kernel(LatAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int W = p.R + p.Dr, Ws = W + 2, KT = p.KT;      // KT <= 32; Ws / 2 odd or even: rows shift banks
  float* qs = lds;                                      // [4][W] f32, pre-scaled
  float* ps = qs + LAT_WAVES * W;                       // [4][KT]
  T* ktile = reinterpret_cast<T*>(ps + LAT_WAVES * KT); // [KT][Ws]
  const int t = blockIdx.x, split = blockIdx.z;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int h_raw = blockIdx.y * LAT_WAVES + wave;
  const bool live = h_raw < p.H;
  const int h = live ? h_raw : p.H - 1;
  T* out = (T*)p.out + ((size_t)h * p.T + t) * p.R;
  float* wsr = p.num_splits > 1
      ? p.ws + (((size_t)split * p.T + t) * p.H + h) * (p.R + 2) : nullptr;
  int nk = 0, lo = 0, b = 0;
  if (t < p.cu_q[p.B]) {
    while (b + 1 < p.B && t >= p.cu_q[b + 1]) ++b;
    nk = min(p.pos[t] + 1, p.ctx[b]);
    if (p.window > 0) lo = min(max(0, p.pos[t] + 1 - p.window), nk);
  }
  int k0 = lo, k1 = nk;
  if (p.num_splits > 1) {
    const int per = ((nk - lo + p.num_splits - 1) / p.num_splits + KT - 1) / KT * KT;
    k0 = min(nk, lo + split * per);
    k1 = min(nk, k0 + per);
  }
  {
    const T* qa = (const T*)p.qa + (size_t)t * p.qa_st + (size_t)h * p.qa_sh;
    const T* qr = (const T*)p.qr + (size_t)t * p.qr_st + (size_t)h * p.qr_sh;
    const int pp = min(max(p.pos[t], 0), p.max_pos - 1);
    const float* csr = p.cs + (size_t)pp * p.dims;
    for (int i = lane; i < W; i += 64) {
      float v;
      if (i < p.R) {
        v = Act<T>::ld(qa + i);
      } else {
        const int j = i - p.R;
        if (j < p.dims) {
          const float c = csr[(j >> 1) * 2], s = csr[(j >> 1) * 2 + 1];
          const float u = Act<T>::ld(qr + (j & ~1)), w = Act<T>::ld(qr + (j | 1));
          v = (j & 1) ? w * c + u * s : u * c - w * s;
        } else {
          v = Act<T>::ld(qr + j);
        }
      }
      qs[wave * W + i] = v * p.scale;
    }
  }
  float m = -INFINITY, l = 0.f;
  float2 acc[LAT_MAXP];
#pragma unroll
  for (int i = 0; i < LAT_MAXP; ++i) acc[i] = make_float2(0.f, 0.f);
  const T* cache = (const T*)p.cache;
  const int* bt = p.bt + (size_t)b * p.max_blocks;
  const int key_l = lane & 31, half = lane >> 5;
  // the two halves of a row, in pairs: [0, hp) and [hp, W / 2)
  const int npair = W >> 1, hp = (npair + 1) >> 1;
  const int c_lo = half ? hp : 0, c_hi = half ? npair : hp;
  // Staging. Rows that are multiples of 16 bytes move as 16-byte chunks: the
  // tile's page lookups are done once (row offsets in LDS), then every thread
  // issues its chunks back to back, and the NEXT tile's chunks are in flight in
  // registers while this tile is scored. Other row sizes go 4 bytes at a time.
  long long* rowoff = reinterpret_cast<long long*>(ktile + (size_t)KT * Ws);   // [KT]
  const int epc = 16 / (int)sizeof(T);                  // entries per chunk
  const bool vec = (W % epc) == 0;
  const int cpr = W / epc, nch = KT * cpr;
  uint4 pre[LAT_MAXCH];
  auto plan_rows = [&](int kt) {
    if (threadIdx.x < KT) {
      const int key = kt + threadIdx.x;
      rowoff[threadIdx.x] = key < k1
          ? (long long)(((size_t)bt[key / p.blk] * p.blk + key % p.blk) * W) : -1ll;
    }
  };
  auto fetch = [&]() {
#pragma unroll
    for (int j = 0; j < LAT_MAXCH; ++j) {
      const int c = threadIdx.x + LAT_THREADS * j;
      pre[j] = make_uint4(0, 0, 0, 0);
      if (c < nch) {
        const int row = c / cpr, cc = c - row * cpr;
        const long long off = rowoff[row];
        if (off >= 0) pre[j] = *reinterpret_cast<const uint4*>(cache + off + cc * epc);
      }
    }
  };
  auto commit = [&]() {
#pragma unroll
    for (int j = 0; j < LAT_MAXCH; ++j) {
      const int c = threadIdx.x + LAT_THREADS * j;
      if (c < nch) {
        const int row = c / cpr, cc = c - row * cpr;
        uint32_t* dst = reinterpret_cast<uint32_t*>(ktile + (size_t)row * Ws + cc * epc);
        dst[0] = pre[j].x; dst[1] = pre[j].y; dst[2] = pre[j].z; dst[3] = pre[j].w;
      }
    }
  };
  if (vec && k0 < k1) {
    plan_rows(k0);
    __syncthreads();
    fetch();
  }
  for (int kt = k0; kt < k1; kt += KT) {
    __syncthreads();
    if (vec) {
      commit();
      if (kt + KT < k1) plan_rows(kt + KT);
    } else {
      for (int j = wave; j < KT; j += LAT_WAVES) {
        const int key = kt + j;
        uint32_t* dst = reinterpret_cast<uint32_t*>(ktile + (size_t)j * Ws);
        if (key < k1) {
          const T* src = cache + ((size_t)bt[key / p.blk] * p.blk + key % p.blk) * W;
          if (sizeof(T) == 2) {
            const uint32_t* s32 = reinterpret_cast<const uint32_t*>(src);
            for (int c = lane; c < npair; c += 64) dst[c] = s32[c];
          } else {
            const float* sf = reinterpret_cast<const float*>(src);
            float* df = reinterpret_cast<float*>(dst);
            for (int c = lane; c < W; c += 64) df[c] = sf[c];
          }
        }
      }
    }
    __syncthreads();
    if (vec && kt + KT < k1) fetch();
    float s = -INFINITY;
    const bool has = key_l < KT && kt + key_l < k1;
    if (has) {
      const T* kr = ktile + (size_t)key_l * Ws;
      const float* q = qs + wave * W;
      float a0 = 0.f, a1 = 0.f;
#pragma unroll 8
      for (int c = c_lo; c < c_hi; ++c) {    // 8 pairs in flight: LDS latency overlaps the FMAs
        const float2 kk = Pair<T>::ld(kr + 2 * c);
        const float2 qq = *reinterpret_cast<const float2*>(q + 2 * c);
        a0 += qq.x * kk.x;
        a1 += qq.y * kk.y;
      }
      s = a0 + a1;
    }
    {
      const float o = __shfl_xor(s, 32, 64);        // the other half of the row
      if (has) s += o;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float pj = (has && half == 0) ? expf(s - mn) : 0.f;
    const float corr = m == -INFINITY ? 0.f : expf(m - mn);
    l = l * corr + wave_sum(pj);
    m = mn;
    if (lane < KT) ps[wave * KT + lane] = pj;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < LAT_MAXP; ++i) { acc[i].x *= corr; acc[i].y *= corr; }
    const int nj = min(KT, k1 - kt);
#pragma unroll 4
    for (int j = 0; j < nj; ++j) {
      const float pv = ps[wave * KT + j];
      const T* cr = ktile + (size_t)j * Ws;
#pragma unroll
      for (int i = 0; i < LAT_MAXP; ++i) {
        const int r = 2 * (lane + 64 * i);
        if (r < p.R) {
          const float2 cc = Pair<T>::ld(cr + r);
          acc[i].x += pv * cc.x;
          acc[i].y += pv * cc.y;
        }
      }
    }
  }
  if (!live) return;
  if (wsr) {
    if (lane == 0) { wsr[0] = m; wsr[1] = l; }
#pragma unroll
    for (int i = 0; i < LAT_MAXP; ++i) {
      const int r = 2 * (lane + 64 * i);
      if (r < p.R) { wsr[2 + r] = acc[i].x; wsr[3 + r] = acc[i].y; }
    }
    return;
  }
  float M = m, den = l, f = 1.f;
  if (p.sink) {
    const float sk = p.sink[h];
    M = fmaxf(m, sk);
    f = m == -INFINITY ? 0.f : expf(m - M);
    den = l * f + expf(sk - M);
  }
  const float inv = den > 0.f ? f / den : 0.f;
#pragma unroll
  for (int i = 0; i < LAT_MAXP; ++i) {
    const int r = 2 * (lane + 64 * i);
    if (r < p.R) {
      Act<T>::st(out + r, acc[i].x * inv);
      Act<T>::st(out + r + 1, acc[i].y * inv);
    }
  }
}

// ------------------------------------------------------- matrix-core form (bf16)
#define LM_KT 32            // keys per tile = the depth of one v_mfma_f32_16x16x32_bf16
#define LM_MAXW 640         // R + Dr
#define LM_MAXR 512
#define LM_SST 36           // row stride of the score exchange (floats)
typedef short lm_v4s __attribute__((ext_vector_type(4)));
typedef unsigned lm_u32x4 __attribute__((ext_vector_type(4)));

static inline size_t latent_mfma_lds(int W) {
  const int Wp = (W + 31) / 32 * 32;
  return (size_t)LM_KT * (Wp + 8) * 2 + 2 * 16 * LM_SST * 4 + LM_KT * 8;
}

__global__ __launch_bounds__(256) void latent_attn_mfma_kernel(LatAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NKH = LM_MAXW / 32 / 2;                 // 32-entry score steps of half a row
  constexpr int NOB = LM_MAXR / 16 / 4;                 // 16-entry output blocks of a wave
  constexpr int NCH = LM_KT * (LM_MAXW / 8) / 256;      // 16-byte chunks of a tile per thread
  const int W = p.R + p.Dr, NK = (W + 31) / 32, Ws = NK * 32 + 8;
  float* sp = lds;                                      // [2 halves][16 heads][LM_SST]
  long long* rowoff = reinterpret_cast<long long*>(sp + 2 * 16 * LM_SST);   // [LM_KT]
  bf16_t* tile = reinterpret_cast<bf16_t*>(rowoff + LM_KT);                 // [LM_KT][Ws]
  const int t = blockIdx.x, split = blockIdx.z;
  // in a scalar register: matrix instructions ignore the lane mask, so branches
  // around them must be taken by whole waves
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int n = lane & 15, g = lane >> 4;
  const int h = blockIdx.y * 16 + n;
  const bool live = h < p.H;
  const bf16_t* cache = (const bf16_t*)p.cache;

  int nk = 0, lo = 0, b = 0;
  if (t < p.cu_q[p.B]) {
    while (b + 1 < p.B && t >= p.cu_q[b + 1]) ++b;
    nk = min(p.pos[t] + 1, p.ctx[b]);
    if (p.window > 0) lo = min(max(0, p.pos[t] + 1 - p.window), nk);
  }
  int k0 = lo, k1 = nk;
  if (p.num_splits > 1) {
    const int per = ((nk - lo + p.num_splits - 1) / p.num_splits + LM_KT - 1) / LM_KT * LM_KT;
    k0 = min(nk, lo + split * per);
    k1 = min(nk, k0 + per);
  }
  const int* bt = p.bt + (size_t)b * p.max_blocks;
  const int cpr = W / 8, nch = LM_KT * cpr;
  lm_u32x4 pre[NCH];
  auto plan_rows = [&](int kt) {
    if (threadIdx.x < LM_KT) {
      const int key = kt + threadIdx.x;
      rowoff[threadIdx.x] = key < k1
          ? (long long)(((size_t)bt[key / p.blk] * p.blk + key % p.blk) * W) : -1ll;
    }
  };
  auto fetch = [&]() {
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int c = threadIdx.x + 256 * j;
      pre[j] = lm_u32x4{0, 0, 0, 0};
      if (c < nch) {
        const int row = c / cpr, cc = c - row * cpr;
        const long long off = rowoff[row];
        if (off >= 0) pre[j] = *reinterpret_cast<const lm_u32x4*>(cache + off + cc * 8);
      }
    }
  };
  if (k0 < k1) plan_rows(k0);
  // columns W .. 32 NK of the tile stay zero (their query entries are zero too,
  // but what LDS holds at start may be no number)
  for (int i = threadIdx.x; i < LM_KT * (NK * 32 - W); i += 256) {
    const int row = i / (NK * 32 - W), c = W + i - row * (NK * 32 - W);
    tile[row * Ws + c] = 0;
  }
  __syncthreads();
  if (k0 < k1) fetch();

  // this wave scores keys 16 sub .. + 15 of a tile over half the row
  const int sub = wave & 1, half = wave >> 1;
  const int s_lo = half ? (NK + 1) / 2 : 0, s_n = half ? NK / 2 : (NK + 1) / 2;
  bf16x8 qf[NKH];
  {
    const bf16_t* qa = (const bf16_t*)p.qa + (size_t)t * p.qa_st + (size_t)(live ? h : 0) * p.qa_sh;
    const bf16_t* qr = (const bf16_t*)p.qr + (size_t)t * p.qr_st + (size_t)(live ? h : 0) * p.qr_sh;
    const int pp = min(max(p.pos[t], 0), p.max_pos - 1);
    const float* csr = p.cs + (size_t)pp * p.dims;
#pragma unroll
    for (int s = 0; s < NKH; ++s) {
      const int e0 = 32 * (s_lo + s) + 8 * g;           // 8 entries, all latent or all rotary (R % 8 == 0)
      short8 f;
#pragma unroll
      for (int i = 0; i < 8; ++i) f[i] = 0;
      if (live && s < s_n && e0 < W) {
        if (e0 < p.R) {
#pragma unroll
          for (int i = 0; i < 8; ++i) f[i] = (short)qa[e0 + i];
        } else {
          const int j0 = e0 - p.R;
#pragma unroll
          for (int i = 0; i < 8; i += 2) {
            const int j = j0 + i;
            const float u = bf2f(qr[j]), v = bf2f(qr[j + 1]);
            if (j < p.dims) {
              const float c = csr[j], sn = csr[j + 1];
              f[i] = (short)f2bf(u * c - v * sn);
              f[i + 1] = (short)f2bf(v * c + u * sn);
            } else {
              f[i] = (short)qr[j];
              f[i + 1] = (short)qr[j + 1];
            }
          }
        }
      }
      qf[s] = *reinterpret_cast<bf16x8*>(&f);
    }
  }
  float m = -INFINITY, l = 0.f;
  float4v acc[NOB];
#pragma unroll
  for (int i = 0; i < NOB; ++i) acc[i] = float4v{0.f, 0.f, 0.f, 0.f};

  for (int kt = k0; kt < k1; kt += LM_KT) {
    __syncthreads();                                    // the previous tile is consumed
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int c = threadIdx.x + 256 * j;
      if (c < nch) {
        const int row = c / cpr, cc = c - row * cpr;
        *reinterpret_cast<lm_u32x4*>(tile + row * Ws + cc * 8) = pre[j];
      }
    }
    if (kt + LM_KT < k1) plan_rows(kt + LM_KT);
    __syncthreads();
    if (kt + LM_KT < k1) fetch();
    {
      float4v s0{0.f, 0.f, 0.f, 0.f}, s1 = s0;          // two chains
      const bf16_t* kr = tile + (16 * sub + n) * Ws + 32 * s_lo + 8 * g;
#pragma unroll
      for (int s = 0; s < NKH; ++s)
        if (s < s_n) {
          const bf16x8 a = *reinterpret_cast<const bf16x8*>(kr + 32 * s);
          if (s & 1) s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qf[s], s1, 0, 0, 0);
          else s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qf[s], s0, 0, 0, 0);
        }
      // lane: head n, keys 16 sub + 4 g .. + 3
      *reinterpret_cast<float4v*>(sp + (half * 16 + n) * LM_SST + 16 * sub + 4 * g) = s0 + s1;
    }
    __syncthreads();
    // every wave: head n, keys 8 g .. 8 g + 7 of the tile
    bf16x8 pf;
    float corr;
    {
      float sv[8];
      float mx = -INFINITY;
#pragma unroll
      for (int q4 = 0; q4 < 2; ++q4) {
        const float4v x = *reinterpret_cast<const float4v*>(sp + n * LM_SST + 8 * g + 4 * q4);
        const float4v y = *reinterpret_cast<const float4v*>(sp + (16 + n) * LM_SST + 8 * g + 4 * q4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int k = 4 * q4 + i;
          sv[k] = kt + 8 * g + k < k1 ? (x[i] + y[i]) * p.scale : -INFINITY;
          mx = fmaxf(mx, sv[k]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m, mx);                    // finite: the tile holds at least one key
      corr = m == -INFINITY ? 0.f : expf(m - mn);
      float ls = 0.f;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const float e = sv[k] == -INFINITY ? 0.f : expf(sv[k] - mn);
        ls += e;
        pf[k] = (__bf16)e;
      }
      ls += __shfl_xor(ls, 16, 64);
      ls += __shfl_xor(ls, 32, 64);
      l = l * corr + ls;
      m = mn;
    }
    // O^T[entry, head] += C^T[entry, key] P^T[key, head]; C^T by transposed reads:
    // a group of 16 lanes names 4 rows x 16 entries and gets its entry of the 4 rows
#pragma unroll
    for (int i = 0; i < NOB; ++i) {
      const int c0 = 16 * (4 * i + wave);
      if (c0 < p.R) {
        const bf16_t* src = tile + (8 * g + (n >> 2)) * Ws + c0 + 4 * (n & 3);
        const lm_v4s a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) lm_v4s*)(src));
        const lm_v4s a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) lm_v4s*)(src + 4 * Ws));
        short8 a8;
        a8[0] = a0[0]; a8[1] = a0[1]; a8[2] = a0[2]; a8[3] = a0[3];
        a8[4] = a1[0]; a8[5] = a1[1]; a8[6] = a1[2]; a8[7] = a1[3];
        acc[i] *= corr;
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<bf16x8*>(&a8), pf, acc[i],
                                                         0, 0, 0);
      }
    }
  }
  if (!live) return;
  if (p.num_splits > 1) {                               // partial of this key split
    float* wsr = p.ws + (((size_t)split * p.T + t) * p.H + h) * (p.R + 2);
    if (wave == 0 && g == 0) { wsr[0] = m; wsr[1] = l; }
#pragma unroll
    for (int i = 0; i < NOB; ++i) {
      const int r = 16 * (4 * i + wave) + 4 * g;
      if (r < p.R) {
#pragma unroll
        for (int k = 0; k < 4; ++k) wsr[2 + r + k] = acc[i][k];
      }
    }
    return;
  }
  float M = m, den = l, f = 1.f;
  if (p.sink) {
    const float sk = p.sink[h];
    M = fmaxf(m, sk);
    f = m == -INFINITY ? 0.f : expf(m - M);
    den = l * f + expf(sk - M);
  }
  const float inv = den > 0.f ? f / den : 0.f;
  bf16_t* out = (bf16_t*)p.out + ((size_t)h * p.T + t) * p.R;
#pragma unroll
  for (int i = 0; i < NOB; ++i) {
    const int r = 16 * (4 * i + wave) + 4 * g;
    if (r < p.R) {
      uint2 w;
      w.x = pack_bf16x2(acc[i][0] * inv, acc[i][1] * inv);
      w.y = pack_bf16x2(acc[i][2] * inv, acc[i][3] * inv);
      *reinterpret_cast<uint2*>(out + r) = w;
    }
  }
}

// out[h, t] from the key splits' (m, l, acc) partials, merged in split order.
// One wave per (token, head): lane s first turns split s's (m, l) into its
// weight e^{m_s - M} (M = the largest m, or the sink), then the partial
// accumulators stream through in split order, four splits in flight.
template <typename T>
__global__ __launch_bounds__(64) void latent_combine_kernel(
    const float* __restrict__ ws, const float* __restrict__ sink, T* __restrict__ out, int Tn, int H,
    int R, int S) {
  __shared__ float fs[64];
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const size_t stride = (size_t)Tn * H * (R + 2);
  const float* base = ws + ((size_t)t * H + h) * (R + 2);
  const float ms = lane < S ? base[lane * stride] : -INFINITY;
  const float ls = lane < S ? base[lane * stride + 1] : 0.f;
  float M = wave_max(ms);
  if (sink) M = fmaxf(M, sink[h]);
  const float f = ms == -INFINITY ? 0.f : expf(ms - M);
  fs[lane] = f;
  float den = wave_sum(ls * f);
  if (sink) den += expf(sink[h] - M);
  __syncthreads();
  float acc[LAT_MAXR];
#pragma unroll
  for (int i = 0; i < LAT_MAXR; ++i) acc[i] = 0.f;
  // unconditional (clamped) loads, so several splits' rows are in flight at once
#pragma unroll 4
  for (int s = 0; s < S; ++s) {
    const float* w = base + s * stride + 2;
    const float fw = fs[s];
    float v[LAT_MAXR];
#pragma unroll
    for (int i = 0; i < LAT_MAXR; ++i) v[i] = w[min(lane + 64 * i, R - 1)];
#pragma unroll
    for (int i = 0; i < LAT_MAXR; ++i) acc[i] += v[i] * fw;
  }
  const float inv = den > 0.f ? 1.f / den : 0.f;
#pragma unroll
  for (int i = 0; i < LAT_MAXR; ++i) {
    const int r = lane + 64 * i;
    if (r < R) Act<T>::st(out + ((size_t)h * Tn + t) * R + r, acc[i] * inv);
  }
}

extern "C" int loqa_latent_inputs(const void* z, int dt, long ldz, const void* nw, float eps,
                                  const void* pos, const void* cs, int max_pos, void* cache, int blk,
                                  int nblocks, const void* slots, int T, int R, int Dr, int dims,
                                  const void* dq, long lddq, const void* qw, int Rq, void* cq,
                                  const void* s_src, long s_src_ld, void* s_dst, long s_dst_ld,
                                  int s_n, int s_lo, int s_hi, int s_vec, hipStream_t st) {
  if (T <= 0) return 0;
  if (R <= 0 || Dr < 0 || dims < 0 || dims > Dr || Rq < 0 || (Rq && (!dq || !qw || !cq)))
    return (int)hipErrorInvalidValue;
  const size_t run = dt == 0 ? 8 : 16;
  auto runs = [&](const void* a, long lda, const void* w, const void* b, long ldb, int n) {
    return n % 4 == 0 && lda % 4 == 0 && ldb % 4 == 0 && (size_t)a % run == 0 &&
           (size_t)b % run == 0 && (size_t)w % 16 == 0;
  };
  const LatInParams p{z, ldz, (const float*)nw, eps, (const int*)pos, (const float*)cs, max_pos,
                      cache, (long)blk * nblocks, (const int*)slots, R, Dr, dims, dq, lddq,
                      (const float*)qw, Rq, cq, runs(z, ldz, nw, cache, R + Dr, R),
                      Rq ? runs(dq, lddq, qw, cq, Rq, Rq) : 0};
  // a decode step has few tokens: a token's row spreads over workgroups
  const dim3 grid(T, T >= 256 ? 1 : (s_n > 0 ? 2 + ceil_div(s_n, 1024) : (Rq ? 2 : 1)));
  const SideCols side{s_src, s_src_ld, s_dst, s_dst_ld, s_n, s_lo, s_hi, s_vec};
  if (dt == 0) hipLaunchKernelGGL(latent_inputs_kernel<bf16_t>, grid, dim3(128), 0, st, p, side);
  else hipLaunchKernelGGL(latent_inputs_kernel<float>, grid, dim3(128), 0, st, p, side);
  return (int)hipGetLastError();
}

extern "C" int loqa_latent_attention(
    const void* qa, long qa_st, long qa_sh, const void* qr, long qr_st, long qr_sh, int dt,
    const void* cache, int blk, int nblocks, const void* cu_q, const void* ctx, const void* bt,
    int max_blocks, const void* pos, const void* cs, int max_pos, const void* sink, float scale,
    int B, int H, int T, int R, int Dr, int dims, void* out, int num_splits, void* ws, int window,
    int mfma, hipStream_t st) {
  if (T <= 0 || H <= 0) return 0;
  if (R > 64 * LAT_MAXR || R <= 0 || B <= 0) return (int)hipErrorInvalidValue;
  if (num_splits > 1 && !ws) return (int)hipErrorInvalidValue;
  if (num_splits > 64) return (int)hipErrorInvalidValue;      // one combine lane per split
  LatAttnParams p;
  p.qa = qa; p.qa_st = qa_st; p.qa_sh = qa_sh; p.qr = qr; p.qr_st = qr_st; p.qr_sh = qr_sh;
  p.cache = cache; p.blk = blk; p.cu_q = (const int*)cu_q; p.ctx = (const int*)ctx;
  p.bt = (const int*)bt; p.max_blocks = max_blocks; p.pos = (const int*)pos;
  p.cs = (const float*)cs; p.max_pos = max_pos; p.sink = (const float*)sink; p.scale = scale;
  p.B = B; p.H = H; p.T = T; p.R = R; p.Dr = Dr; p.dims = dims; p.out = out;
  p.num_splits = num_splits < 1 ? 1 : num_splits; p.ws = (float*)ws;
  p.window = window;
  const int W = R + Dr, Ws = W | 1;
  if (mfma) {
    // 16-byte rows and queries, whole output blocks
    if (dt != 0 || R % 16 || W % 8 || R > LM_MAXR || W > LM_MAXW || dims % 2 || dims > Dr ||
        ((size_t)cache & 15))
      return (int)hipErrorInvalidValue;
    hipLaunchKernelGGL(latent_attn_mfma_kernel, dim3(T, (H + 15) / 16, p.num_splits), dim3(256),
                       latent_mfma_lds(W), st, p);
    int rc = (int)hipGetLastError();
    if (rc || p.num_splits == 1) return rc;
    hipLaunchKernelGGL(latent_combine_kernel<bf16_t>, dim3(T, H), dim3(64), 0, st, (const float*)ws,
                       (const float*)sink, (bf16_t*)out, T, H, R, p.num_splits);
    return (int)hipGetLastError();
  }
  if (W % 2 == 0 && R % 2 == 0 && R <= 128 * LAT_MAXP) {
    const size_t esz = dt == 0 ? 2 : 4;
    int KT2 = 32;
    const size_t chunks_per_row = ((size_t)W * esz + 15) / 16;
    while (KT2 > 4 && ((size_t)(LAT_WAVES * W + LAT_WAVES * KT2) * 4 + (size_t)KT2 * (W + 2) * esz +
                       KT2 * 8 > 60 * 1024 || KT2 * chunks_per_row > (size_t)LAT_THREADS * LAT_MAXCH))
      KT2 >>= 1;
    const size_t smem2 = (size_t)(LAT_WAVES * W + LAT_WAVES * KT2) * 4 + (size_t)KT2 * (W + 2) * esz +
                         KT2 * 8 + 8;
    if (smem2 <= 64 * 1024 && KT2 * chunks_per_row <= (size_t)LAT_THREADS * LAT_MAXCH) {
      p.KT = KT2;
      const dim3 grid2(T, (H + LAT_WAVES - 1) / LAT_WAVES, p.num_splits);
      if (dt == 0) hipLaunchKernelGGL(latent_attn2_kernel<bf16_t>, grid2, dim3(LAT_THREADS), smem2, st, p);
      else hipLaunchKernelGGL(latent_attn2_kernel<float>, grid2, dim3(LAT_THREADS), smem2, st, p);
      int rc2 = (int)hipGetLastError();
      if (rc2 || p.num_splits == 1) return rc2;
      if (dt == 0)
        hipLaunchKernelGGL(latent_combine_kernel<bf16_t>, dim3(T, H), dim3(64), 0, st,
                           (const float*)ws, (const float*)sink, (bf16_t*)out, T, H, R, p.num_splits);
      else
        hipLaunchKernelGGL(latent_combine_kernel<float>, dim3(T, H), dim3(64), 0, st,
                           (const float*)ws, (const float*)sink, (float*)out, T, H, R, p.num_splits);
      return (int)hipGetLastError();
    }
  }
  int KT = 64;
  while (KT > 4 && ((size_t)KT * Ws + LAT_WAVES * W + LAT_WAVES * KT) * 4 > 60 * 1024) KT >>= 1;
  p.KT = KT;
  const size_t smem = ((size_t)KT * Ws + LAT_WAVES * W + LAT_WAVES * KT) * 4;
  if (smem > 64 * 1024) return (int)hipErrorInvalidValue;
  const dim3 grid(T, (H + LAT_WAVES - 1) / LAT_WAVES, p.num_splits);
  if (dt == 0) hipLaunchKernelGGL(latent_attn_kernel<bf16_t>, grid, dim3(LAT_THREADS), smem, st, p);
  else hipLaunchKernelGGL(latent_attn_kernel<float>, grid, dim3(LAT_THREADS), smem, st, p);
  int rc = (int)hipGetLastError();
  if (rc || p.num_splits == 1) return rc;
  if (dt == 0)
    hipLaunchKernelGGL(latent_combine_kernel<bf16_t>, dim3(T, H), dim3(64), 0, st, (const float*)ws,
                       (const float*)sink, (bf16_t*)out, T, H, R, p.num_splits);
  else
    hipLaunchKernelGGL(latent_combine_kernel<float>, dim3(T, H), dim3(64), 0, st, (const float*)ws,
                       (const float*)sink, (float*)out, T, H, R, p.num_splits);
  return (int)hipGetLastError();
}
