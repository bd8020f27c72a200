// Projection post-processing of attention variants that norm a whole
// projection at once:
//   tied_attn_prep    q and k sections RMS-normed over ALL heads together
//                     (weights of the section's size); q times a temperature
//                     1 + coef * ln(floor((p + 1) / every) + 1) of its
//                     position p; normed k into the paged K cache and the RAW
//                     k section into the paged V cache (values are the keys)
//   section_rmsnorm   out[row(t)] = n(section of proj[t]) * w; row(t) = t, or
//                     an index list (scatter into cache pages: a latent)
//   sigmoid_gate_mul  v *= sigmoid(gate section), elementwise
//   latent_prep       latent attention with a rotated key part: normed latent
//                     and rotated key part of every token into its cache row,
//                     rotated query parts behind the folded queries; pairs
//                     (i, i + rd/2) or neighbours (2i, 2i + 1)
//   rope_table        cos | sin rows of the positions of a step
// One 256-thread block a token (and section); fp32 math.
#include "mix_common.h"

template <typename A>
__global__ void tied_attn_prep_kernel(
    A* __restrict__ q_out, const A* __restrict__ proj, long ld, int q_off,
    int k_off, const float* __restrict__ q_w, const float* __restrict__ k_w,
    float eps, const long* __restrict__ pos, float temp_coef, int temp_every,
    const long* __restrict__ slots, A* __restrict__ k_cache,
    A* __restrict__ v_cache, int H, int G, int dk, int page) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const bool is_q = blockIdx.y == 0;
  const int n = (is_q ? H : G) * dk;
  const A* src = proj + t * ld + (is_q ? q_off : k_off);
  float ssq = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const float v = ldf<A>(src + c);
    ssq += v * v;
  }
  float inv = 1.f / sqrtf(block_sum_256(ssq, red) / (float)n + eps);
  if (is_q) {
    if (temp_every > 0) {
      const long steps = (pos[t] + 1) / temp_every;
      inv *= 1.f + temp_coef * logf((float)steps + 1.f);
    }
    A* dst = q_out + t * (long)n;
    for (int c = threadIdx.x; c < n; c += blockDim.x)
      stf<A>(dst + c, ldf<A>(src + c) * q_w[c] * inv);
    return;
  }
  const long slot = slots[t];
  const long blk = slot / page, off = slot - blk * page;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const int g = c / dk, i = c - g * dk;
    const long at = ((blk * G + g) * page + off) * (long)dk + i;
    const float v = ldf<A>(src + c);
    stf<A>(k_cache + at, v * inv * k_w[c]);
    stf<A>(v_cache + at, v);
  }
}

template <typename A>
__global__ void section_rmsnorm_kernel(A* __restrict__ out, long ldo,
                                       const A* __restrict__ proj, long ld,
                                       int off, const float* __restrict__ w,
                                       float eps, const long* __restrict__ rows,
                                       int n) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const A* src = proj + t * ld + off;
  float ssq = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const float v = ldf<A>(src + c);
    ssq += v * v;
  }
  const float inv = 1.f / sqrtf(block_sum_256(ssq, red) / (float)n + eps);
  A* dst = out + (rows ? rows[t] : t) * ldo;
  for (int c = threadIdx.x; c < n; c += blockDim.x)
    stf<A>(dst + c, ldf<A>(src + c) * inv * w[c]);
}

// 16-byte form: one vector a thread (sections up to 256 vectors long), the
// section is read once. Needs n, the offset and both row strides to be
// multiples of the vector (8 bf16 or 4 fp32).
template <typename A, int V>
__global__ void __launch_bounds__(256) section_rmsnorm_vec_kernel(
    A* __restrict__ out, long ldo, const A* __restrict__ proj, long ld,
    int off, const float* __restrict__ w, float eps,
    const long* __restrict__ rows, int n) {
  typedef A vec_t __attribute__((ext_vector_type(V)));
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int c = threadIdx.x * V;
  float x[V];
  float ssq = 0.f;
  if (c < n) {
    const vec_t v = *(const vec_t*)(proj + t * ld + off + c);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      A ve = v[e];
      x[e] = ldf<A>(&ve);
      ssq += x[e] * x[e];
    }
  }
  const float inv = 1.f / sqrtf(block_sum_256(ssq, red) / (float)n + eps);
  if (c < n) {
    vec_t o;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      A oe;
      stf<A>(&oe, x[e] * inv * w[c + e]);
      o[e] = oe;
    }
    *(vec_t*)(out + (rows ? rows[t] : t) * ldo + c) = o;
  }
}

// One 256-thread block a token. q [T, H, *] rows of the query (strides sqt,
// sqh; the rotated part starts at q0), qa [T, H, R + rd]; the cache row is
// latent [R] | rotated key [rd]. cs row t: cos[rd/2] | sin[rd/2].
template <typename A>
__global__ void __launch_bounds__(256) latent_prep_kernel(
    A* __restrict__ cache, const long* __restrict__ rows,
    const A* __restrict__ proj, long ld, int off, const float* __restrict__ w,
    float eps, const float* __restrict__ cos_sin, int R, int rd, int adjacent,
    const A* __restrict__ q, long sqt, long sqh, A* __restrict__ qa, int H) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const A* src = proj + t * ld + off;
  float ssq = 0.f;
  for (int c = threadIdx.x; c < R; c += 256) {
    const float v = ldf<A>(src + c);
    ssq += v * v;
  }
  const float inv = 1.f / sqrtf(block_sum_256(ssq, red) / (float)R + eps);
  A* dst = cache + rows[t] * (long)(R + rd);
  for (int c = threadIdx.x; c < R; c += 256)
    stf<A>(dst + c, ldf<A>(src + c) * inv * w[c]);
  // pair i of query head u < H, or of the shared key part (u == H)
  const int half = rd / 2;
  const float* cs = cos_sin + t * (long)rd;
  for (int e = threadIdx.x; e < (H + 1) * half; e += 256) {
    const int u = e / half, i = e - u * half;
    const A* in = u < H ? q + t * sqt + u * sqh : src + R;
    A* o = u < H ? qa + (t * H + u) * (long)(R + rd) + R : dst + R;
    const int ia = adjacent ? 2 * i : i, ib = adjacent ? 2 * i + 1 : half + i;
    const float a = ldf<A>(in + ia), b = ldf<A>(in + ib);
    const float c = cs[i], sn = cs[half + i];
    stf<A>(o + ia, a * c - b * sn);
    stf<A>(o + ib, b * c + a * sn);
  }
}

// bf16, 16 bytes a lane: the first wave of a workgroup norms the latent (kept
// in registers up to 512 wide), the other two turn 8 pairs a lane. Needs R,
// half the rotated part and every offset and stride to be multiples of 8.
template <bool ADJ>
__global__ void __launch_bounds__(192) latent_prep_vec_kernel(
    u16* __restrict__ cache, const long* __restrict__ rows,
    const u16* __restrict__ proj, long ld, int off, const float* __restrict__ w,
    float eps, const float* __restrict__ cos_sin, int R, int rd,
    const u16* __restrict__ q, long sqt, long sqh, u16* __restrict__ qa,
    int H) {
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const u16* src = proj + t * ld + off;
  u16* dst = cache + rows[t] * (long)(R + rd);
  if (tid < 64) {
    float x[8], ssq = 0.f;
    for (int c = tid * 8; c < R; c += 512) {
      bf8_to_f32(*(const u16x8*)(src + c), x);
#pragma unroll
      for (int e = 0; e < 8; ++e) ssq += x[e] * x[e];
    }
    const float inv = 1.f / sqrtf(wave_sum_f32(ssq) / (float)R + eps);
    for (int c = tid * 8; c < R; c += 512) {
      if (R > 512) bf8_to_f32(*(const u16x8*)(src + c), x);
      const f32x4 w0 = *(const f32x4*)(w + c), w1 = *(const f32x4*)(w + c + 4);
      u16x8 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[e] = f2bf(x[e] * inv * w0[e]);
        o[e + 4] = f2bf(x[e + 4] * inv * w1[e]);
      }
      *(u16x8*)(dst + c) = o;
    }
    return;
  }
  const int half = rd / 2, per = half / 8;
  const float* cs = cos_sin + t * (long)rd;
  for (int j = tid - 64; j < (H + 1) * per; j += 128) {
    const int u = j / per, i = (j - u * per) * 8;
    const u16* in = u < H ? q + t * sqt + u * sqh : src + R;
    u16* o = u < H ? qa + (t * H + u) * (long)(R + rd) + R : dst + R;
    // the 8 pairs lie in two vectors: first and second members (halves), or
    // pairs 0..3 and pairs 4..7 (neighbours)
    const int p0 = ADJ ? 2 * i : i, p1 = ADJ ? 2 * i + 8 : half + i;
    float a[8], b[8];
    bf8_to_f32(*(const u16x8*)(in + p0), a);
    bf8_to_f32(*(const u16x8*)(in + p1), b);
    if (ADJ) {
      float x[16];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        x[e] = a[e];
        x[8 + e] = b[e];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        a[e] = x[2 * e];
        b[e] = x[2 * e + 1];
      }
    }
    u16x8 oa, ob;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const f32x4 c = *(const f32x4*)(cs + i + 4 * h);
      const f32x4 s = *(const f32x4*)(cs + half + i + 4 * h);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int k = 4 * h + e;
        const u16 ya = f2bf(a[k] * c[e] - b[k] * s[e]);
        const u16 yb = f2bf(b[k] * c[e] + a[k] * s[e]);
        if (ADJ) {
          if (h == 0) {
            oa[2 * e] = ya;
            oa[2 * e + 1] = yb;
          } else {
            ob[2 * e] = ya;
            ob[2 * e + 1] = yb;
          }
        } else {
          oa[k] = ya;
          ob[k] = yb;
        }
      }
    }
    *(u16x8*)(o + p0) = oa;
    *(u16x8*)(o + p1) = ob;
  }
}

extern "C" void mix_latent_prep(void* cache, const long* rows, const void* proj,
                                long ld, int off, const float* w, float eps,
                                const float* cos_sin, int R, int rd,
                                int adjacent, const void* q, long sqt,
                                long sqh, void* qa, long T, int H, int f32,
                                hipStream_t s) {
  if (T == 0) return;
  if (!f32 && R % 8 == 0 && rd % 16 == 0 && off % 8 == 0 && ld % 8 == 0 &&
      sqt % 8 == 0 && sqh % 8 == 0 && (size_t)q % 16 == 0 &&
      (size_t)proj % 16 == 0 && (size_t)qa % 16 == 0 &&
      (size_t)cache % 16 == 0) {
    if (adjacent)
      hipLaunchKernelGGL(latent_prep_vec_kernel<true>, dim3((unsigned)T),
                         dim3(192), 0, s, (u16*)cache, rows, (const u16*)proj,
                         ld, off, w, eps, cos_sin, R, rd, (const u16*)q, sqt,
                         sqh, (u16*)qa, H);
    else
      hipLaunchKernelGGL(latent_prep_vec_kernel<false>, dim3((unsigned)T),
                         dim3(192), 0, s, (u16*)cache, rows, (const u16*)proj,
                         ld, off, w, eps, cos_sin, R, rd, (const u16*)q, sqt,
                         sqh, (u16*)qa, H);
    return;
  }
  if (f32)
    hipLaunchKernelGGL(latent_prep_kernel<float>, dim3((unsigned)T), dim3(256),
                       0, s, (float*)cache, rows, (const float*)proj, ld, off,
                       w, eps, cos_sin, R, rd, adjacent, (const float*)q, sqt,
                       sqh, (float*)qa, H);
  else
    hipLaunchKernelGGL(latent_prep_kernel<u16>, dim3((unsigned)T), dim3(256),
                       0, s, (u16*)cache, rows, (const u16*)proj, ld, off, w,
                       eps, cos_sin, R, rd, adjacent, (const u16*)q, sqt, sqh,
                       (u16*)qa, H);
}

// out[t]: amp * cos(pos f_i) [half] | amp * sin(pos f_i) [half], fp32 angles
__global__ void __launch_bounds__(256) rope_table_kernel(
    float* __restrict__ out, const long* __restrict__ pos,
    const float* __restrict__ inv_freq, int half, float amp, long T) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= T * half) return;
  const long t = i / half;
  const int c = (int)(i - t * half);
  const float ang = (float)pos[t] * inv_freq[c];
  out[t * 2 * half + c] = cosf(ang) * amp;
  out[t * 2 * half + half + c] = sinf(ang) * amp;
}

extern "C" void mix_rope_table(float* out, const long* pos,
                               const float* inv_freq, int half, float amp,
                               long T, hipStream_t s) {
  const long n = T * half;
  if (n == 0) return;
  hipLaunchKernelGGL(rope_table_kernel, dim3((unsigned)((n + 255) / 256)),
                     dim3(256), 0, s, out, pos, inv_freq, half, amp, T);
}

template <typename A>
__global__ void sigmoid_gate_mul_kernel(A* __restrict__ v, long ldv,
                                        const A* __restrict__ proj, long ld,
                                        int g_off, long T, int N) {
  const long total = T * (long)N;
  for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += (long)gridDim.x * blockDim.x) {
    const long row = idx / N;
    const int c = (int)(idx - row * N);
    A* p = v + row * ldv + c;
    stf<A>(p, ldf<A>(p) * sigmoid_f(ldf<A>(proj + row * ld + g_off + c)));
  }
}

// 16-byte form: needs N, both row strides and the gate offset to be multiples
// of the vector (8 bf16 or 4 fp32)
template <typename A, int V>
__global__ void sigmoid_gate_mul_vec_kernel(A* __restrict__ v, long ldv,
                                            const A* __restrict__ proj,
                                            long ld, int g_off, long T, int N) {
  typedef A vec_t __attribute__((ext_vector_type(V)));
  const int vpr = N / V;
  const long total = T * (long)vpr;
  for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
       idx += (long)gridDim.x * blockDim.x) {
    const long row = idx / vpr;
    const int c = (int)(idx - row * vpr) * V;
    vec_t* p = (vec_t*)(v + row * ldv + c);
    const vec_t x = *p;
    const vec_t g = *(const vec_t*)(proj + row * ld + g_off + c);
    vec_t o;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      A xj = x[j], gj = g[j], r;
      stf<A>(&r, ldf<A>(&xj) * sigmoid_f(ldf<A>(&gj)));
      o[j] = r;
    }
    *p = o;
  }
}

extern "C" void mix_tied_attn_prep(void* q_out, const void* proj, long ld,
                                   int q_off, int k_off, const float* q_w,
                                   const float* k_w, float eps,
                                   const long* pos, float temp_coef,
                                   int temp_every, const long* slots,
                                   void* k_cache, void* v_cache, long T, int H,
                                   int G, int dk, int page, int f32,
                                   hipStream_t s) {
  if (T == 0) return;
  const dim3 grid((unsigned)T, 2);
  if (f32)
    hipLaunchKernelGGL(tied_attn_prep_kernel<float>, grid, dim3(256), 0, s,
                       (float*)q_out, (const float*)proj, ld, q_off, k_off,
                       q_w, k_w, eps, pos, temp_coef, temp_every, slots,
                       (float*)k_cache, (float*)v_cache, H, G, dk, page);
  else
    hipLaunchKernelGGL(tied_attn_prep_kernel<u16>, grid, dim3(256), 0, s,
                       (u16*)q_out, (const u16*)proj, ld, q_off, k_off, q_w,
                       k_w, eps, pos, temp_coef, temp_every, slots,
                       (u16*)k_cache, (u16*)v_cache, H, G, dk, page);
}

extern "C" void mix_section_rmsnorm(void* out, long ldo, const void* proj,
                                    long ld, int off, const float* w,
                                    float eps, const long* rows, long T, int n,
                                    int f32, hipStream_t s) {
  if (T == 0) return;
  const int V = f32 ? 4 : 8;
  if (n % V == 0 && n <= 256 * V && off % V == 0 && ld % V == 0 &&
      ldo % V == 0 && (size_t)out % 16 == 0 && (size_t)proj % 16 == 0) {
    if (f32)
      hipLaunchKernelGGL((section_rmsnorm_vec_kernel<float, 4>),
                         dim3((unsigned)T), dim3(256), 0, s, (float*)out, ldo,
                         (const float*)proj, ld, off, w, eps, rows, n);
    else
      hipLaunchKernelGGL((section_rmsnorm_vec_kernel<u16, 8>),
                         dim3((unsigned)T), dim3(256), 0, s, (u16*)out, ldo,
                         (const u16*)proj, ld, off, w, eps, rows, n);
    return;
  }
  if (f32)
    hipLaunchKernelGGL(section_rmsnorm_kernel<float>, dim3((unsigned)T),
                       dim3(256), 0, s, (float*)out, ldo, (const float*)proj,
                       ld, off, w, eps, rows, n);
  else
    hipLaunchKernelGGL(section_rmsnorm_kernel<u16>, dim3((unsigned)T),
                       dim3(256), 0, s, (u16*)out, ldo, (const u16*)proj, ld,
                       off, w, eps, rows, n);
}

extern "C" void mix_sigmoid_gate_mul(void* v, long ldv, const void* proj,
                                     long ld, int g_off, long T, int N,
                                     int f32, hipStream_t s) {
  const long total = T * (long)N;
  if (total == 0) return;
  const int V = f32 ? 4 : 8;
  if (N % V == 0 && ldv % V == 0 && ld % V == 0 && g_off % V == 0 &&
      (size_t)v % 16 == 0 && (size_t)proj % 16 == 0) {
    long vb = (total / V + 255) / 256;
    if (vb > 65536) vb = 65536;
    if (f32)
      hipLaunchKernelGGL((sigmoid_gate_mul_vec_kernel<float, 4>),
                         dim3((unsigned)vb), dim3(256), 0, s, (float*)v, ldv,
                         (const float*)proj, ld, g_off, T, N);
    else
      hipLaunchKernelGGL((sigmoid_gate_mul_vec_kernel<u16, 8>),
                         dim3((unsigned)vb), dim3(256), 0, s, (u16*)v, ldv,
                         (const u16*)proj, ld, g_off, T, N);
    return;
  }
  long blocks = (total + 255) / 256;
  if (blocks > 65536) blocks = 65536;
  if (f32)
    hipLaunchKernelGGL(sigmoid_gate_mul_kernel<float>, dim3((unsigned)blocks),
                       dim3(256), 0, s, (float*)v, ldv, (const float*)proj, ld,
                       g_off, T, N);
  else
    hipLaunchKernelGGL(sigmoid_gate_mul_kernel<u16>, dim3((unsigned)blocks),
                       dim3(256), 0, s, (u16*)v, ldv, (const u16*)proj, ld,
                       g_off, T, N);
}
