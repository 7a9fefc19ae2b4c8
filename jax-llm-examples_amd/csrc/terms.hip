// The residual, up to three weighted branch outputs, and what is formed from their sum in the same launch:
//     y = x + vec * (fa a + fb b + fc c)         a, b, c: rows of one type (each optional), vec: float32 [D] (optional)
//   norm:    x <- y,  h = (y - mean) / sqrt(mean((y - mean)^2) + eps) * w + bias      (CENTER: a layer norm)
//            or       h = y / sqrt(mean(y^2) + eps) * w                               in the run dtype (and float32)
//   joined:  (x stays) the rows that a looped stretch's input product takes: [y | rows] in float32, or in bfloat16
//            [leading term of y | rows | remainder of y]
// One block per row, the row in registers (THREADS * PIECES pieces of V neighbours; wider rows are formed again); every
// sum in an order that depends on the width alone.
#include "common.h"
#include "rows.h"

using namespace jle;

namespace {

template <typename T>
struct TermArgs {
  float* x;  // [N, D]
  const T* t[3];
  float f[3];
  const float* vec;
  const float* w;
  const float* bias;
  void* h;     // [N, D] run dtype or null (the sum only)
  float* h32;  // [N, D] or null
  float eps;
  int h_bf16, D;
  const float* rows;  // joined: [N, D]
};

// V neighbouring elements
template <typename T, int V>
__device__ __forceinline__ f32x4_t get(const T* p) {
  if (V == 4) return load4<T>(p);
  return f32x4_t{Num<T>::load(p), 0.f, 0.f, 0.f};
}
template <typename T, int V>
__device__ __forceinline__ void put(T* p, f32x4_t v) {
  if (V == 4) store4<T>(p, v);
  else Num<T>::store(p, v[0]);
}

template <typename T, int V>
__device__ __forceinline__ f32x4_t summed(const TermArgs<T>& p, size_t base, int d, f32x4_t x) {
  f32x4_t t = {0.f, 0.f, 0.f, 0.f};
  if (p.t[0] == nullptr) return x;
  t = get<T, V>(p.t[0] + base + d) * p.f[0];
#pragma unroll
  for (int j = 1; j < 3; ++j)
    if (p.t[j] != nullptr) {
      const f32x4_t u = get<T, V>(p.t[j] + base + d);
#pragma unroll
      for (int i = 0; i < V; ++i) t[i] = __builtin_fmaf(p.f[j], u[i], t[i]);
    }
  if (p.vec != nullptr) t *= get<float, V>(p.vec + d);
  return x + t;
}

template <typename T, int V>
__device__ __forceinline__ void put_h(const TermArgs<T>& p, size_t at, f32x4_t h) {
  if (p.h_bf16) put<bf16_t, V>((bf16_t*)p.h + at, h);
  else put<float, V>((float*)p.h + at, h);
  if (p.h32 != nullptr) put<float, V>(p.h32 + at, h);
}

template <typename T, int V>
__device__ __forceinline__ void put_joined(const TermArgs<T>& p, size_t n, int d, f32x4_t y) {
  const size_t D = p.D;
  const f32x4_t r = get<float, V>(p.rows + n * D + d);
  if (!p.h_bf16) {
    float* o = (float*)p.h + n * 2 * D + d;
    put<float, V>(o, y);
    put<float, V>(o + D, r);
    return;
  }
  bf16_t* o = (bf16_t*)p.h + n * 3 * D + d;
  f32x4_t rest;
#pragma unroll
  for (int i = 0; i < 4; ++i) rest[i] = y[i] - Num<bf16_t>::round(y[i]);
  put<bf16_t, V>(o, y);
  put<bf16_t, V>(o + D, r);
  put<bf16_t, V>(o + 2 * D, rest);
}

template <typename T, int V, int THREADS, int PIECES, bool CENTER, bool JOIN>
__global__ __launch_bounds__(THREADS) void terms_kernel(TermArgs<T> p) {
  __shared__ float red[THREADS / 64];
  const size_t n = blockIdx.x, base = n * p.D;
  const int D = p.D;
  f32x4_t v[PIECES];
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int d = (threadIdx.x + THREADS * i) * V;
    v[i] = d < D ? get<float, V>(p.x + base + d) : f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int d = (threadIdx.x + THREADS * i) * V;
    if (d < D) v[i] = summed<T, V>(p, base, d, v[i]);
  }
  if (JOIN) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int d = (threadIdx.x + THREADS * i) * V;
      if (d < D) put_joined<T, V>(p, n, d, v[i]);
    }
    return;
  }
  if (p.t[0] != nullptr) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int d = (threadIdx.x + THREADS * i) * V;
      if (d < D) put<float, V>(p.x + base + d, v[i]);
    }
  }
  if (p.h == nullptr) return;
  if (CENTER) {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
#pragma unroll
      for (int e = 0; e < V; ++e) sum += v[i][e];
    const float mean = block_sum<THREADS>(sum, red) / (float)D;
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const bool in = (int)(threadIdx.x + THREADS * i) * V < D;
#pragma unroll
      for (int e = 0; e < V; ++e) v[i][e] = in ? v[i][e] - mean : 0.f;
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PIECES; ++i)
#pragma unroll
    for (int e = 0; e < V; ++e) ss = __builtin_fmaf(v[i][e], v[i][e], ss);
  const float inv = 1.0f / sqrtf(block_sum<THREADS>(ss, red) / (float)D + p.eps);
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int d = (threadIdx.x + THREADS * i) * V;
    if (d < D) {
      f32x4_t h = v[i] * inv;
      if (p.w != nullptr) h *= get<float, V>(p.w + d);
      if (p.bias != nullptr) h += get<float, V>(p.bias + d);
      put_h<T, V>(p, base + d, h);
    }
  }
}

// Rows wider than the registers hold: the sums are stored and the row read again.
template <typename T, int THREADS, bool CENTER, bool JOIN>
__global__ __launch_bounds__(THREADS) void terms_wide_kernel(TermArgs<T> p) {
  __shared__ float red[THREADS / 64];
  const size_t n = blockIdx.x, base = n * p.D;
  const int D = p.D;
  float sum = 0.f, ss = 0.f;
  for (int d = threadIdx.x; d < D; d += THREADS) {
    const f32x4_t y = summed<T, 1>(p, base, d, f32x4_t{p.x[base + d], 0.f, 0.f, 0.f});
    if (JOIN) {
      put_joined<T, 1>(p, n, d, y);
    } else {
      p.x[base + d] = y[0];
      sum += y[0];
    }
  }
  if (JOIN || p.h == nullptr) return;
  const float mean = CENTER ? block_sum<THREADS>(sum, red) / (float)D : 0.f;
  for (int d = threadIdx.x; d < D; d += THREADS) {  // (this thread's own stores)
    const float v = p.x[base + d] - mean;
    ss = __builtin_fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum<THREADS>(ss, red) / (float)D + p.eps);
  for (int d = threadIdx.x; d < D; d += THREADS) {
    float h = (p.x[base + d] - mean) * inv;
    if (p.w != nullptr) h *= p.w[d];
    if (p.bias != nullptr) h += p.bias[d];
    put_h<T, 1>(p, base + d, f32x4_t{h, 0.f, 0.f, 0.f});
  }
}

template <typename T, bool CENTER, bool JOIN>
int launch(const TermArgs<T>& p, int N, hipStream_t s) {
  const int D = p.D;
  // (which kernel: by the width and the arrays' alignment alone, never by the step's size)
  const uintptr_t all = (uintptr_t)p.x | (uintptr_t)p.t[0] | (uintptr_t)p.t[1] | (uintptr_t)p.t[2] | (uintptr_t)p.vec |
                        (uintptr_t)p.w | (uintptr_t)p.bias | (uintptr_t)p.h | (uintptr_t)p.h32 | (uintptr_t)p.rows;
#define TERMS(V, TH, P) hipLaunchKernelGGL((terms_kernel<T, V, TH, P, CENTER, JOIN>), dim3(N), dim3(TH), 0, s, p)
  if (D % 4 == 0 && all % 16 == 0 && D <= 16384) {
    if (D <= 256) TERMS(4, 64, 1);
    else if (D <= 1024) TERMS(4, 256, 1);
    else if (D <= 2048) TERMS(4, 256, 2);
    else if (D <= 4096) TERMS(4, 256, 4);
    else if (D <= 8192) TERMS(4, 512, 4);
    else TERMS(4, 512, 8);
  } else if (D <= 256) {
    TERMS(1, 64, 4);
  } else if (D <= 2048) {
    TERMS(1, 256, 8);
  } else {
    hipLaunchKernelGGL((terms_wide_kernel<T, 512, CENTER, JOIN>), dim3(N), dim3(512), 0, s, p);
  }
#undef TERMS
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename T>
int run(float* x, const void* const* t, const float* f, const float* vec, const float* w, const float* bias, float eps,
        int mode, void* h, int h_bf16, float* h32, const float* rows, int N, int D, hipStream_t s) {
  TermArgs<T> p{x, {(const T*)t[0], (const T*)t[1], (const T*)t[2]}, {f[0], f[1], f[2]}, vec, w, bias, h, h32, eps, h_bf16,
                D, rows};
  if (mode == 2) return launch<T, false, true>(p, N, s);
  return mode == 1 ? launch<T, true, false>(p, N, s) : launch<T, false, false>(p, N, s);
}

}  // namespace

// The terms a, b, c (bfloat16 if t_bf16, else float32; b needs a, c needs b).  mode 0: root-mean-square norm, 1: layer
// norm (h null: the sum only); 2: joined rows into h (x is not written; rows: float32 [N, D]).
JLE_API int jle_terms(float* x, const void* a, float fa, const void* b, float fb, const void* c, float fc, int t_bf16,
                      const float* vec, const float* w, const float* bias, float eps, int mode, void* h, int h_bf16,
                      float* h32, const float* rows, int N, int D, hipStream_t s) {
  if (N <= 0) return 0;
  if (D <= 0 || x == nullptr || (b != nullptr && a == nullptr) || (c != nullptr && b == nullptr) || mode < 0 || mode > 2 ||
      (h == nullptr && h32 != nullptr) || (mode == 2 && (rows == nullptr || h == nullptr || h32 != nullptr)))
    return JLE_BAD_ARG;
  const void* t[3] = {a, b, c};
  const float f[3] = {fa, fb, fc};
  return t_bf16 ? run<bf16_t>(x, t, f, vec, w, bias, eps, mode, h, h_bf16, h32, rows, N, D, s)
                : run<float>(x, t, f, vec, w, bias, eps, mode, h, h_bf16, h32, rows, N, D, s);
}
