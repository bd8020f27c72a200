// Hyper-connections: the residual is a bundle of S fp32 streams a token, and a
// sublayer reads a weighted sum of them and writes back to all of them:
//
//   hyper_rmsnorm   y = sublayer result (a row, and / or the weighted gather of
//                   a token's expert rows, and / or a shared expert's row);
//                   X_o <- sum_s mix[s, o] X_s + out[o] y; then the NEXT
//                   sublayer's input: u = sum_s in[s] X_s, h = u / rms(u) *
//                   weight. Every stream is read and written once.
//
//   relu_sq         max(z, 0)^2 in place, elementwise (ungated feed-forward)
//
// X is [T, S, W] (a token's streams are neighbours). The first update of a step
// may take all streams from one row (x_in [T, W], the embedding output); the
// last one need not write the streams at all.
#include "mix_common.h"

struct HyperArgs {
  float* x;                // [T, S, W]
  const float* x_in;       // [T, W]: every stream starts as this row
  const void* y;           // [T, W]
  const void* rows;        // expert rows
  const int* padpos;       // [T, k]
  const float* wts;        // [T, k] (null: every pair weighs wconst)
  float wconst;
  int k;
  const void* y2;          // [T, W]
  const float* mix;        // [S, S] [from, to] (null: no update)
  const float* out;        // [S]
  const float* in;         // [S]
  const float* nw;         // [W]
  float eps;
  void* h;                 // [T, W] (null: no read)
  int write, S, W;
};

// the sublayer result at columns c .. c + V - 1
template <typename A, int V>
__device__ __forceinline__ void hyper_result(const HyperArgs& P, long t, int c,
                                             float* yv) {
  typedef A vec_t __attribute__((ext_vector_type(V)));
#pragma unroll
  for (int e = 0; e < V; ++e) yv[e] = 0.f;
  auto add = [&](const void* base, long row, float f) {
    const vec_t v = *(const vec_t*)((const A*)base + row * P.W + c);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      A ve = v[e];
      yv[e] += f * ldf<A>(&ve);
    }
  };
  if (P.y) add(P.y, t, 1.f);
  if (P.rows)
    for (int j = 0; j < P.k; ++j)
      add(P.rows, P.padpos[t * P.k + j], P.wts ? P.wts[t * P.k + j] : P.wconst);
  if (P.y2) add(P.y2, t, 1.f);
}

template <typename A, int V>
__device__ __forceinline__ void hyper_norm_out(const HyperArgs& P, long t,
                                               const float* us, float ssq,
                                               float* red) {
  typedef A vec_t __attribute__((ext_vector_type(V)));
  const float inv =
      1.f / sqrtf(block_sum_256(ssq, red) / (float)P.W + P.eps);
  A* hr = (A*)P.h + t * P.W;
  // a thread reads back the columns it left in LDS itself
  for (int c = threadIdx.x * V; c < P.W; c += 256 * V) {
    vec_t o;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      A oe;
      stf<A>(&oe, us[c + e] * inv * P.nw[c + e]);
      o[e] = oe;
    }
    *(vec_t*)(hr + c) = o;
  }
}

// One 256-thread block a token, V columns of all S streams a thread and turn.
template <typename A, int V, int S>
__global__ void __launch_bounds__(256) hyper_rmsnorm_kernel(HyperArgs P) {
  typedef float fvec __attribute__((ext_vector_type(V)));
  extern __shared__ __attribute__((aligned(16))) float us[];  // [W]
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int W = P.W;
  float* xr = P.x + t * S * W;
  float ssq = 0.f;
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    fvec xv[S];
    if (P.x_in) {
      xv[0] = *(const fvec*)(P.x_in + t * W + c);
#pragma unroll
      for (int s = 1; s < S; ++s) xv[s] = xv[0];
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) xv[s] = *(const fvec*)(xr + (long)s * W + c);
    }
    if (P.mix) {
      float yv[V];
      hyper_result<A, V>(P, t, c, yv);
      fvec nx[S];
#pragma unroll
      for (int o = 0; o < S; ++o) {
        const float b = P.out[o];
#pragma unroll
        for (int e = 0; e < V; ++e) nx[o][e] = b * yv[e];
#pragma unroll
        for (int s = 0; s < S; ++s) {
          const float m = P.mix[s * S + o];
#pragma unroll
          for (int e = 0; e < V; ++e) nx[o][e] += m * xv[s][e];
        }
        if (P.write) *(fvec*)(xr + (long)o * W + c) = nx[o];
      }
#pragma unroll
      for (int s = 0; s < S; ++s) xv[s] = nx[s];
    }
    if (P.h) {
      fvec u;
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = 0.f;
#pragma unroll
      for (int s = 0; s < S; ++s) {
        const float a = P.in[s];
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] += a * xv[s][e];
      }
      *(fvec*)(us + c) = u;
#pragma unroll
      for (int e = 0; e < V; ++e) ssq += u[e] * u[e];
    }
  }
  if (P.h) hyper_norm_out<A, V>(P, t, us, ssq, red);
}

// Any number of streams and any width: one column a thread and turn, the old
// streams of the turn's columns in LDS.
template <typename A>
__global__ void __launch_bounds__(256) hyper_rmsnorm_any_kernel(HyperArgs P) {
  extern __shared__ __attribute__((aligned(16))) float us[];  // [W] | [S][256]
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int W = P.W, S = P.S;
  float* xr = P.x + t * S * W;
  float* old = us + W + threadIdx.x;  // private to the thread
  float ssq = 0.f;
  for (int c = threadIdx.x; c < W; c += 256) {
    for (int s = 0; s < S; ++s)
      old[s * 256] = P.x_in ? P.x_in[t * W + c] : xr[(long)s * W + c];
    float yv = 0.f;
    if (P.mix) hyper_result<A, 1>(P, t, c, &yv);
    float u = 0.f;
    for (int o = 0; o < S; ++o) {
      float v = old[o * 256];
      if (P.mix) {
        v = P.out[o] * yv;
        for (int s = 0; s < S; ++s) v += P.mix[s * S + o] * old[s * 256];
        if (P.write) xr[(long)o * W + c] = v;
      }
      if (P.h) u += P.in[o] * v;
    }
    if (P.h) {
      us[c] = u;
      ssq += u * u;
    }
  }
  if (P.h) hyper_norm_out<A, 1>(P, t, us, ssq, red);
}

// LDS of a launch: what fits is W + (S > 8 or odd width ? 256 S : 0) floats in
// HYPER_LDS bytes
#define HYPER_LDS (64 * 1024 - 64)

extern "C" long mix_hyper_lds(int S, int W) {
  return ((long)W + (S > 8 || W % 4 ? 256L * S : 0)) * (long)sizeof(float);
}

extern "C" int mix_hyper_rmsnorm(float* x, const float* x_in, const void* y,
                                 const void* rows, const int* padpos,
                                 const float* wts, float wconst, int k,
                                 const void* y2, const float* mix,
                                 const float* out, const float* in,
                                 const float* nw, float eps, void* h, int write,
                                 long T, int S, int W, int f32, hipStream_t s) {
  const size_t smem = (size_t)mix_hyper_lds(S, W);
  if (smem > HYPER_LDS) return 0;
  if (T == 0) return 1;
  HyperArgs P;
  P.x = x; P.x_in = x_in; P.y = y; P.rows = rows; P.padpos = padpos;
  P.wts = wts; P.wconst = wconst; P.k = k; P.y2 = y2; P.mix = mix; P.out = out;
  P.in = in; P.nw = nw; P.eps = eps; P.h = h; P.write = write; P.S = S; P.W = W;
  const dim3 grid((unsigned)T), block(256);
#define LAUNCH_HY(SS)                                                         \
  case SS:                                                                    \
    if (f32)                                                                  \
      hipLaunchKernelGGL((hyper_rmsnorm_kernel<float, 4, SS>), grid, block,   \
                         smem, s, P);                                         \
    else                                                                      \
      hipLaunchKernelGGL((hyper_rmsnorm_kernel<u16, 4, SS>), grid, block,     \
                         smem, s, P);                                         \
    return 1
  if (W % 4 == 0) switch (S) {
      LAUNCH_HY(1);
      LAUNCH_HY(2);
      LAUNCH_HY(3);
      LAUNCH_HY(4);
      LAUNCH_HY(5);
      LAUNCH_HY(6);
      LAUNCH_HY(7);
      LAUNCH_HY(8);
      default:
        break;
    }
#undef LAUNCH_HY
  if (f32)
    hipLaunchKernelGGL(hyper_rmsnorm_any_kernel<float>, grid, block, smem, s, P);
  else
    hipLaunchKernelGGL(hyper_rmsnorm_any_kernel<u16>, grid, block, smem, s, P);
  return 1;
}

// ---- relu_sq ---------------------------------------------------------------
template <typename A, int V>
__global__ void __launch_bounds__(256) relu_sq_kernel(A* __restrict__ z,
                                                      long n) {
  typedef A vec_t __attribute__((ext_vector_type(V)));
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  vec_t v = *(const vec_t*)(z + i);
#pragma unroll
  for (int e = 0; e < V; ++e) {
    A ve = v[e];
    const float f = fmaxf(ldf<A>(&ve), 0.f);
    stf<A>(&ve, f * f);
    v[e] = ve;
  }
  *(vec_t*)(z + i) = v;
}

extern "C" void mix_relu_sq(void* z, long n, int f32, hipStream_t s) {
  if (n == 0) return;
  const int V = n % (f32 ? 4 : 8) ? 1 : (f32 ? 4 : 8);
  const unsigned grid = (unsigned)((n / V + 255) / 256);
#define LAUNCH_RQ(AA, VV)                                                     \
  hipLaunchKernelGGL((relu_sq_kernel<AA, VV>), dim3(grid), dim3(256), 0, s,   \
                     (AA*)z, n)
  if (f32) {
    if (V == 4) LAUNCH_RQ(float, 4); else LAUNCH_RQ(float, 1);
  } else {
    if (V == 8) LAUNCH_RQ(u16, 8); else LAUNCH_RQ(u16, 1);
  }
#undef LAUNCH_RQ
}
