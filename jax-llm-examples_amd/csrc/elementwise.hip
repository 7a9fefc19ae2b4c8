// Embedding gather, residual add + RMS norm, SiLU*up, row gather, expert output combine.
#include "common.h"
#include "rows.h"

using namespace jle;


// ------------------------------------------------------------------ embedding
template <typename T>
__global__ void embed_kernel(const int* __restrict__ tok, const T* __restrict__ table, float* __restrict__ out, int D) {
  const size_t row = blockIdx.x;
  const T* src = table + (size_t)tok[row] * D;
  float* dst = out + row * D;
  for (int d = threadIdx.x; d < D; d += blockDim.x) dst[d] = Num<T>::load(src + d);
}

JLE_API int jle_embed(const int* tok, const void* table, int is_bf16, float* out, int N, int D, hipStream_t s) {
  if (N <= 0) return 0;
  if (is_bf16)
    hipLaunchKernelGGL(embed_kernel<bf16_t>, dim3(N), dim3(256), 0, s, tok, (const bf16_t*)table, out, D);
  else
    hipLaunchKernelGGL(embed_kernel<float>, dim3(N), dim3(256), 0, s, tok, (const float*)table, out, D);
  JLE_LAUNCH_CHECK();
  return 0;
}

// out = table[tok] + pair[(prev * mul_prev + tok * mul_cur) mod buckets], and row `buckets` of the pair table for a
// token without a token before it (prev < 0); the hash in 64 bits.
template <typename T>
__global__ void embed_pair_kernel(const int* __restrict__ tok, const int* __restrict__ prev,
                                  const T* __restrict__ table, const T* __restrict__ pair, float* __restrict__ out,
                                  int D, int buckets, long long mul_prev, long long mul_cur) {
  const size_t row = blockIdx.x;
  const int t = tok[row], p = prev[row];
  const long long r = p < 0 ? (long long)buckets : ((long long)p * mul_prev + (long long)t * mul_cur) % buckets;
  const T* a = table + (size_t)t * D;
  const T* b = pair + (size_t)r * D;
  float* dst = out + row * D;
  for (int d = threadIdx.x; d < D; d += blockDim.x) dst[d] = Num<T>::load(a + d) + Num<T>::load(b + d);
}

JLE_API int jle_embed_pair(const int* tok, const int* prev, const void* table, const void* pair, int is_bf16,
                           float* out, int N, int D, int buckets, long long mul_prev, long long mul_cur,
                           hipStream_t s) {
  if (N <= 0) return 0;
  if (buckets <= 0 || mul_prev < 0 || mul_cur < 0) return JLE_BAD_ARG;
  if (is_bf16)
    hipLaunchKernelGGL(embed_pair_kernel<bf16_t>, dim3(N), dim3(256), 0, s, tok, prev, (const bf16_t*)table,
                       (const bf16_t*)pair, out, D, buckets, mul_prev, mul_cur);
  else
    hipLaunchKernelGGL(embed_pair_kernel<float>, dim3(N), dim3(256), 0, s, tok, prev, (const float*)table,
                       (const float*)pair, out, D, buckets, mul_prev, mul_cur);
  JLE_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ add + rmsnorm
// x (float32, the residual) += delta; out = x * rsqrt(mean(x^2) + eps) * weight.
// delta is either a plain tensor or the sum of a token's expert outputs and the shared expert's:
//   delta[n] = sum_j routed[inv[n * k + j]] + shared[n]
// One block per row.  Rows up to 8192 wide stay in registers (THREADS * EPT elements); wider rows
// are read twice.  The sum of squares is formed in a fixed order that depends on the width only.
template <typename DT, typename OT, int THREADS, int EPT>
__global__ __launch_bounds__(THREADS) void add_rmsnorm_reg_kernel(float* __restrict__ x, Delta<DT> delta,
                                                                  const float* __restrict__ w, float eps,
                                                                  OT* __restrict__ out, float* __restrict__ out32,
                                                                  int D) {
  __shared__ float red[THREADS / 64];
  const size_t n = blockIdx.x;
  const size_t base = n * D;
  float v[EPT];
  float ss = 0.f;
  const bool add = delta.any();
#pragma unroll
  for (int i = 0; i < EPT; ++i) {
    const int d = threadIdx.x + THREADS * i;
    v[i] = 0.f;
    if (d < D) {
      v[i] = x[base + d];
      if (add) {
        v[i] += delta.at(n, d, D);
        x[base + d] = v[i];
      }
      ss += v[i] * v[i];
    }
  }
  const float tot = block_sum<THREADS>(ss, red);
  const float inv = 1.0f / sqrtf(tot / (float)D + eps);
#pragma unroll
  for (int i = 0; i < EPT; ++i) {
    const int d = threadIdx.x + THREADS * i;
    if (d < D) {
      float h = v[i] * inv;
      if (w != nullptr) h *= w[d];
      if (out != nullptr) Num<OT>::store(out + base + d, h);
      if (out32 != nullptr) out32[base + d] = h;
    }
  }
}

// Rows whose width is a multiple of 8 (and 16-byte aligned arrays): a thread takes CPT pieces of 4
// neighbouring elements, piece = thread, thread + THREADS, ...; up to THREADS * CPT * 4 wide.
template <typename DT, typename OT, int THREADS, int CPT, bool STREAM>
__global__ __launch_bounds__(THREADS, 4) void add_rmsnorm_vec_kernel(float* __restrict__ x, Delta<DT> delta,
                                                                  const float* __restrict__ w, float eps,
                                                                  OT* __restrict__ out, float* __restrict__ out32,
                                                                  int D) {
  __shared__ float red[THREADS / 64];
  const size_t n = blockIdx.x;
  const size_t base = n * D;
  // (the weights are asked for first: they wait for nothing)
  f32x4_t wv[CPT];
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int d = (threadIdx.x + THREADS * i) * 4;
    wv[i] = (w != nullptr && d < D) ? load4<float>(w + d) : f32x4_t{1.f, 1.f, 1.f, 1.f};
  }
  f32x4_t v[CPT];
  float ss = 0.f;
  const bool add = delta.any();
  const DeltaRow<DT> drow = delta_row(delta, n, D);
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int d = (threadIdx.x + THREADS * i) * 4;
    v[i] = d < D ? load4_as<STREAM, float>(x + base + d) : f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  // (every load before the first store: a store in between would make the loads after it wait, since the
  // compiler cannot know that x is none of the arrays they read.  The pieces past the row's end are selects,
  // not branches around an update of v[i]: with those the compiler carries the whole array as one wide value
  // and needs 211 registers instead of 118, which halves the rows a compute unit works on at once.)
  if (add) {
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int d = (threadIdx.x + THREADS * i) * 4;
      v[i] += d < D ? delta_row_at4<STREAM, DT>(delta, drow, n, d, D) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int d = (threadIdx.x + THREADS * i) * 4;
      if (d < D) {
        if (STREAM) __builtin_nontemporal_store(v[i], reinterpret_cast<f32x4_t*>(x + base + d));
        else store4<float>(x + base + d, v[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < CPT; ++i) ss = add_squares4(ss, v[i]);
  const float tot = block_sum<THREADS>(ss, red);
  const float inv = 1.0f / sqrtf(tot / (float)D + eps);
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int d = (threadIdx.x + THREADS * i) * 4;
    if (d < D) {
      f32x4_t h = v[i] * inv;
      if (w != nullptr) h *= wv[i];
      if (out != nullptr) store4<OT>(out + base + d, h);
      if (out32 != nullptr) store4<float>(out32 + base + d, h);
    }
  }
}

template <typename DT, typename OT>
__global__ __launch_bounds__(256) void add_rmsnorm_wide_kernel(float* __restrict__ x, Delta<DT> delta,
                                                               const float* __restrict__ w, float eps,
                                                               OT* __restrict__ out, float* __restrict__ out32,
                                                               int D) {
  __shared__ float red[4];
  const size_t n = blockIdx.x;
  const size_t base = n * D;
  float ss = 0.f;
  const bool add = delta.any();
  for (int d = threadIdx.x; d < D; d += 256) {
    float v = x[base + d];
    if (add) {
      v += delta.at(n, d, D);
      x[base + d] = v;
    }
    ss += v * v;
  }
  const float tot = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(tot / (float)D + eps);
  for (int d = threadIdx.x; d < D; d += 256) {
    float h = x[base + d] * inv;
    if (w != nullptr) h *= w[d];
    if (out != nullptr) Num<OT>::store(out + base + d, h);
    if (out32 != nullptr) out32[base + d] = h;
  }
}

template <typename DT, typename OT>
static void launch_add_rmsnorm(float* x, Delta<DT> delta, const float* w, float eps, void* out, float* out32, int N,
                               int D, hipStream_t s) {
  dim3 g(N);
  // (which kernel: by the width and the arrays' alignment only, so a row's result is the same in any batch)
  const uintptr_t all = (uintptr_t)x | (uintptr_t)delta.plain | (uintptr_t)delta.routed | (uintptr_t)delta.shared |
                        (uintptr_t)delta.self | (uintptr_t)w | (uintptr_t)out | (uintptr_t)out32;
  if (D % 8 == 0 && (all & 15) == 0 && D > 1024 && D <= 8192) {  // (rows of any of the arrays then start 16-byte aligned)
    // (the same arithmetic either way: only where the data are kept differs)
    if ((size_t)N * D >= ((size_t)4 << 20))
      hipLaunchKernelGGL((add_rmsnorm_vec_kernel<DT, OT, 256, 8, true>), g, dim3(256), 0, s, x, delta, w, eps,
                         (OT*)out, out32, D);
    else
      hipLaunchKernelGGL((add_rmsnorm_vec_kernel<DT, OT, 256, 8, false>), g, dim3(256), 0, s, x, delta, w, eps,
                         (OT*)out, out32, D);
  }
  else if (D <= 1024)
    hipLaunchKernelGGL((add_rmsnorm_reg_kernel<DT, OT, 256, 4>), g, dim3(256), 0, s, x, delta, w, eps, (OT*)out, out32,
                       D);
  else if (D <= 8192)
    hipLaunchKernelGGL((add_rmsnorm_reg_kernel<DT, OT, 1024, 8>), g, dim3(1024), 0, s, x, delta, w, eps, (OT*)out,
                       out32, D);
  else
    hipLaunchKernelGGL((add_rmsnorm_wide_kernel<DT, OT>), g, dim3(256), 0, s, x, delta, w, eps, (OT*)out, out32, D);
}

// delta_kind: 0 none, 1 plain (delta), 2 expert sum (routed, inv, k, shared; self, self_w, self_k: see Delta)
JLE_API int jle_add_rmsnorm(float* x, int delta_kind, const void* delta, const void* routed, const int* inv, int k,
                            const void* shared, int delta_is_bf16, const float* w, float eps, void* out,
                            int out_is_bf16, float* out32, int N, int D, const void* self, const float* self_w,
                            int self_k, hipStream_t s) {
  if (N <= 0) return 0;
#define GO(DT, OT)                                                                              \
  do {                                                                                          \
    Delta<DT> dl = {delta_kind == 1 ? (const DT*)delta : nullptr,                               \
                    delta_kind == 2 ? (const DT*)routed : nullptr, inv, (const DT*)shared, k,  \
                    (const DT*)self, self_w, self_k};                                           \
    launch_add_rmsnorm<DT, OT>(x, dl, w, eps, out, out32, N, D, s);                             \
  } while (0)
  if (delta_is_bf16) {
    if (out_is_bf16) GO(bf16_t, bf16_t); else GO(bf16_t, float);
  } else {
    if (out_is_bf16) GO(float, bf16_t); else GO(float, float);
  }
#undef GO
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename DT>
__global__ void add_residual_kernel(float* __restrict__ x, const DT* __restrict__ delta, size_t n) {
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) x[i] += Num<DT>::load(delta + i);
}

JLE_API int jle_add_residual(float* x, const void* delta, int delta_is_bf16, long long n, hipStream_t s) {
  if (n <= 0) return 0;
  dim3 g((unsigned)((n + 255) / 256)), b(256);
  if (delta_is_bf16)
    hipLaunchKernelGGL(add_residual_kernel<bf16_t>, g, b, 0, s, x, (const bf16_t*)delta, (size_t)n);
  else
    hipLaunchKernelGGL(add_residual_kernel<float>, g, b, 0, s, x, (const float*)delta, (size_t)n);
  JLE_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ row gather (any dtype)
template <typename W>
__global__ void gather_rows_kernel(const W* __restrict__ src, const int* __restrict__ idx, W* __restrict__ out,
                                   int words) {
  const W* s = src + (size_t)idx[blockIdx.x] * words;
  W* d = out + (size_t)blockIdx.x * words;
  for (int i = threadIdx.x; i < words; i += blockDim.x) d[i] = s[i];
}

JLE_API int jle_gather_rows(const void* src, const int* idx, void* out, int M, int row_bytes, hipStream_t s) {
  if (M <= 0) return 0;
  if (row_bytes % 4 == 0)
    hipLaunchKernelGGL(gather_rows_kernel<uint32_t>, dim3(M), dim3(256), 0, s, (const uint32_t*)src, idx,
                       (uint32_t*)out, row_bytes / 4);
  else if (row_bytes % 2 == 0)
    hipLaunchKernelGGL(gather_rows_kernel<uint16_t>, dim3(M), dim3(256), 0, s, (const uint16_t*)src, idx,
                       (uint16_t*)out, row_bytes / 2);
  else
    return JLE_BAD_ARG;
  JLE_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ act(gate) * up
// in: [N, 2F] (gate columns, then up columns); out: [N, F].  ACT 0: silu, z / (1 + exp(-z)); 1: the tanh form of
// gelu, 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))).
template <int ACT>
__device__ __forceinline__ float gate_act(float g) {
  if (ACT == 1) return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
  return g / (1.0f + expf(-g));
}

template <typename T, int ACT>
__global__ void silu_mul_kernel(const T* __restrict__ in, T* __restrict__ out, int F) {
  const size_t row = blockIdx.y;
  const int f = blockIdx.x * blockDim.x + threadIdx.x;
  if (f >= F) return;
  const float g = Num<T>::load(in + row * 2 * F + f);
  const float u = Num<T>::load(in + row * 2 * F + F + f);
  Num<T>::store(out + row * F + f, gate_act<ACT>(g) * u);
}

// bfloat16 rows whose halves are 16-byte aligned: 8 elements per thread
template <int ACT>
__global__ void silu_mul_bf16x8_kernel(const bf16_t* __restrict__ in, bf16_t* __restrict__ out, int F) {
  const size_t row = blockIdx.y;
  const int f = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
  if (f >= F) return;
  const uint4 gv = *reinterpret_cast<const uint4*>(in + row * 2 * F + f);
  const uint4 uv = *reinterpret_cast<const uint4*>(in + row * 2 * F + F + f);
  const uint32_t gw[4] = {gv.x, gv.y, gv.z, gv.w}, uw[4] = {uv.x, uv.y, uv.z, uv.w};
  uint32_t o[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float g0 = __uint_as_float(gw[i] << 16), g1 = __uint_as_float(gw[i] & 0xffff0000u);
    const float u0 = __uint_as_float(uw[i] << 16), u1 = __uint_as_float(uw[i] & 0xffff0000u);
    o[i] = pack_bf16(gate_act<ACT>(g0) * u0, gate_act<ACT>(g1) * u1);
  }
  *reinterpret_cast<uint4*>(out + row * F + f) = uint4{o[0], o[1], o[2], o[3]};
}

template <int ACT>
static int launch_act_mul(const void* in, void* out, int is_bf16, int N, int F, hipStream_t s) {
  if (N <= 0 || F <= 0) return 0;
  if (N > 65535 * 16) return JLE_BAD_ARG;
  dim3 g((F + 255) / 256, N), b(256);
  if (is_bf16 && F % 8 == 0 && (((uintptr_t)in | (uintptr_t)out) & 15) == 0) {
    dim3 g8((F / 8 + 255) / 256, N);
    hipLaunchKernelGGL(silu_mul_bf16x8_kernel<ACT>, g8, b, 0, s, (const bf16_t*)in, (bf16_t*)out, F);
  } else if (is_bf16) {
    hipLaunchKernelGGL((silu_mul_kernel<bf16_t, ACT>), g, b, 0, s, (const bf16_t*)in, (bf16_t*)out, F);
  } else {
    hipLaunchKernelGGL((silu_mul_kernel<float, ACT>), g, b, 0, s, (const float*)in, (float*)out, F);
  }
  JLE_LAUNCH_CHECK();
  return 0;
}

JLE_API int jle_silu_mul(const void* in, void* out, int is_bf16, int N, int F, hipStream_t s) {
  return launch_act_mul<0>(in, out, is_bf16, N, F, s);
}

// act: 0 silu, 1 gelu (tanh form)
JLE_API int jle_act_mul(const void* in, void* out, int is_bf16, int N, int F, int act, hipStream_t s) {
  if (act == 0) return launch_act_mul<0>(in, out, is_bf16, N, F, s);
  if (act == 1) return launch_act_mul<1>(in, out, is_bf16, N, F, s);
  return JLE_BAD_ARG;
}

// x = cap * tanh(x / cap), in place
__global__ void softcap_kernel(float* __restrict__ x, long long n, float cap) {
  const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] / cap);
}

JLE_API int jle_softcap(float* x, long long n, float cap, hipStream_t s) {
  if (n <= 0) return 0;
  if (!(cap > 0.f) || (n + 255) / 256 > 0x7fffffffll) return JLE_BAD_ARG;
  hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, x, n, cap);
  JLE_LAUNCH_CHECK();
  return 0;
}

// out[n, c] = o[n, c] * sigmoid(gate[n * gate_ld + c]): the gate's rows are a slice of wider rows.
template <typename T>
__global__ void sigmoid_mul_kernel(const T* __restrict__ o, const T* __restrict__ gate, int gate_ld,
                                   T* __restrict__ out, int C, int share) {
  const size_t row = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= C) return;
  const float g = Num<T>::load(gate + row * gate_ld + (share == 1 ? c : c / share));
  Num<T>::store(out + row * C + c, Num<T>::load(o + row * C + c) / (1.0f + expf(-g)));
}

// share: so many neighbouring elements of o have one gate (1: a gate each)
JLE_API int jle_sigmoid_mul(const void* o, const void* gate, int gate_ld, void* out, int is_bf16, int N, int C,
                            int share, hipStream_t s) {
  if (N <= 0 || C <= 0) return 0;
  if (share < 1 || C % share || gate_ld < C / share || (C + 255) / 256 > 65535) return JLE_BAD_ARG;
  dim3 g(N, (C + 255) / 256), b(256);
  if (is_bf16)
    hipLaunchKernelGGL(sigmoid_mul_kernel<bf16_t>, g, b, 0, s, (const bf16_t*)o, (const bf16_t*)gate, gate_ld,
                       (bf16_t*)out, C, share);
  else
    hipLaunchKernelGGL(sigmoid_mul_kernel<float>, g, b, 0, s, (const float*)o, (const float*)gate, gate_ld,
                       (float*)out, C, share);
  JLE_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ combine expert outputs
// out[n] = sum_j routed[inv[n * k + j]] + shared[n]   (float32 result; see Delta for negative rows)
template <typename T>
__global__ void moe_combine_kernel(const T* __restrict__ routed, const int* __restrict__ inv,
                                   const T* __restrict__ shared, float* __restrict__ out, int k, int D,
                                   const T* __restrict__ self, const float* __restrict__ self_w, int self_k) {
  const size_t n = blockIdx.x;
  const Delta<T> delta = {nullptr, routed, inv, shared, k, self, self_w, self_k};
  for (int d = threadIdx.x; d < D; d += blockDim.x) out[n * D + d] = delta.at(n, d, D);
}

JLE_API int jle_moe_combine(const void* routed, const int* inv, const void* shared, float* out, int is_bf16, int N,
                            int k, int D, const void* self, const float* self_w, int self_k, hipStream_t s) {
  if (N <= 0) return 0;
  if (is_bf16)
    hipLaunchKernelGGL(moe_combine_kernel<bf16_t>, dim3(N), dim3(256), 0, s, (const bf16_t*)routed, inv,
                       (const bf16_t*)shared, out, k, D, (const bf16_t*)self, self_w, self_k);
  else
    hipLaunchKernelGGL(moe_combine_kernel<float>, dim3(N), dim3(256), 0, s, (const float*)routed, inv,
                       (const float*)shared, out, k, D, (const float*)self, self_w, self_k);
  JLE_LAUNCH_CHECK();
  return 0;
}
