// Queries and keys normed over the whole projection, then queries to their rows and keys and values to their pages.
//
// rows: [N][Hq dk] (queries only) or [N][Hq dk + Hk dk + Hk dv].  One RMS norm over all Hq dk queries of a token
// (weights wq of that size) and one over all its Hk dk keys (wk); then (rd > 0) the leading rd elements of every q and
// k head turned by pos * inv_freq[j], element j paired with j + rd / 2 (angles float32); the queries times 1 + attn_scale * ln(1 +
// floor((pos + 1) / floor_scale)) (floor_scale <= 0: no factor).  Heads are stored PD elements wide (PD >= dk, dv),
// zeros behind the real ones: q_out [N][Hq][PD]; pages [page][2][Hk][..]: keys [ps][PD], values [PD][ps].
// One block per token; statistics, weights and the factor in float32; sums of squares in an order that depends on the
// sizes only.
#include "common.h"

using namespace jle;

template <typename T>
__global__ __launch_bounds__(256) void span_prepare_kernel(const T* __restrict__ rows, T* __restrict__ q_out,
                                                           T* __restrict__ kv, const int* __restrict__ positions,
                                                           const int* __restrict__ slot_mapping,
                                                           const float* __restrict__ wq, const float* __restrict__ wk,
                                                           float eps, float floor_scale, float attn_scale, int Hq,
                                                           int Hk, int dk, int dv, int PD, int ps, int own_kv,
                                                           const float* __restrict__ inv_freq, int rd) {
  __shared__ float red[4];
  extern __shared__ float turn[];  // [rd / 2][2]: the token's cosines and sines
  const int hr = rd / 2;
  const size_t n = blockIdx.x;
  const int nq = Hq * dk, nk = Hk * dk, nv = Hk * dv;
  const int width = own_kv ? nq + nk + nv : nq;
  const T* r = rows + n * width;
  for (int j = threadIdx.x; j < hr; j += 256) {  // (visible to all behind block_sum's barriers)
    float sn, cs;
    sincosf((float)positions[n] * inv_freq[j], &sn, &cs);
    turn[2 * j] = cs;
    turn[2 * j + 1] = sn;
  }
  // element d of a head whose weighted (not yet divided) elements lie at x * w
  auto turned = [&](const T* x, const float* w, int d) {
    const float v = Num<T>::load(x + d) * w[d];
    if (d >= rd) return v;
    const bool first = d < hr;
    const int j = first ? d : d - hr, p = first ? d + hr : d - hr;
    const float o = Num<T>::load(x + p) * w[p], cs = turn[2 * j], sn = turn[2 * j + 1];
    return first ? v * cs - o * sn : v * cs + o * sn;
  };
  float ssq = 0.f, ssk = 0.f;
  for (int c = threadIdx.x; c < nq; c += 256) {
    const float v = Num<T>::load(r + c);
    ssq = fmaf(v, v, ssq);
  }
  const bool write = own_kv && kv != nullptr;
  if (write)
    for (int c = threadIdx.x; c < nk; c += 256) {
      const float v = Num<T>::load(r + nq + c);
      ssk = fmaf(v, v, ssk);
    }
  const float tq = block_sum<256>(ssq, red);
  float inv_q = 1.0f / sqrtf(tq / (float)nq + eps);
  if (floor_scale > 0.f)
    inv_q *= 1.0f + attn_scale * log1pf(floorf(((float)positions[n] + 1.0f) / floor_scale));
  T* qo = q_out + n * (size_t)Hq * PD;
  for (int c = threadIdx.x; c < Hq * PD; c += 256) {
    const int h = c / PD, d = c - h * PD;
    float v = 0.f;
    if (d < dk) v = turned(r + h * dk, wq + h * dk, d) * inv_q;
    Num<T>::store(qo + c, v);
  }
  if (!write) return;
  const float tk = block_sum<256>(ssk, red);
  const float inv_k = 1.0f / sqrtf(tk / (float)nk + eps);
  const int slot = slot_mapping[n];
  const int page = slot / ps, off = slot - page * ps;
  const size_t plane = (size_t)ps * PD;
  T* kpage = kv + (size_t)page * 2 * Hk * plane;
  T* vpage = kpage + (size_t)Hk * plane;
  for (int c = threadIdx.x; c < Hk * PD; c += 256) {
    const int h = c / PD, d = c - h * PD;
    float kx = 0.f, vx = 0.f;
    if (d < dk) kx = turned(r + nq + h * dk, wk + h * dk, d) * inv_k;
    if (d < dv) vx = Num<T>::load(r + nq + nk + h * dv + d);
    Num<T>::store(kpage + h * plane + (size_t)off * PD + d, kx);
    Num<T>::store(vpage + h * plane + (size_t)d * ps + off, vx);
  }
}

// The same, eight neighbouring elements at a time (dk, PD and the half of the turned elements multiples of 8, every array
// 16-byte aligned): the row's q and k part is read once, into shared memory, where a turned element finds its partner.
template <typename T>
struct Eight;
template <>
struct Eight<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t* p, float* v) {
    const uint4 r = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {r.x, r.y, r.z, r.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float* v) {
    *reinterpret_cast<uint4*>(p) = uint4{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7])};
  }
};
template <>
struct Eight<float> {
  static __device__ __forceinline__ void load(const float* p, float* v) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
  }
  static __device__ __forceinline__ void store(float* p, const float* v) {
    *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<float4*>(p + 4) = float4{v[4], v[5], v[6], v[7]};
  }
};

constexpr int kVecThreads = 512;

template <typename T>
__global__ __launch_bounds__(kVecThreads) void span_prepare_vec_kernel(
    const T* __restrict__ rows, T* __restrict__ q_out, T* __restrict__ kv, const int* __restrict__ positions,
    const int* __restrict__ slot_mapping, const float* __restrict__ wq, const float* __restrict__ wk, float eps,
    float floor_scale, float attn_scale, int Hq, int Hk, int dk, int dv, int PD, int ps, int own_kv,
    const float* __restrict__ inv_freq, int rd) {
  constexpr int TH = kVecThreads;
  extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
  __shared__ float red_q[TH / 64], red_k[TH / 64];
  const size_t n = blockIdx.x;
  const int nq = Hq * dk, nk = Hk * dk, nv = Hk * dv, hr = rd / 2;
  const bool write = own_kv && kv != nullptr;
  const int held = write ? nq + nk : nq;  // the elements that are normed
  T* x = reinterpret_cast<T*>(lds);                                     // [held], as the projection left them
  float* turn = reinterpret_cast<float*>(lds + ((size_t)held * sizeof(T) + 15) / 16 * 16);  // cosines [hr], sines [hr]
  const T* r = rows + n * (own_kv ? nq + nk + nv : nq);
  float ssq = 0.f, ssk = 0.f;
  for (int c = threadIdx.x * 8; c < held; c += TH * 8) {
    float v[8];
    Eight<T>::load(r + c, v);
    Eight<T>::store(x + c, v);
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) s = fmaf(v[i], v[i], s);
    if (c < nq) ssq += s;
    else ssk += s;
  }
  for (int j = threadIdx.x; j < hr; j += TH) {
    float sn, cs;
    sincosf((float)positions[n] * inv_freq[j], &sn, &cs);
    turn[j] = cs;
    turn[hr + j] = sn;
  }
  ssq = wave_sum(ssq);
  ssk = wave_sum(ssk);
  if ((threadIdx.x & 63) == 0) {
    red_q[threadIdx.x >> 6] = ssq;
    red_k[threadIdx.x >> 6] = ssk;
  }
  __syncthreads();
  float tq = 0.f, tk = 0.f;
#pragma unroll
  for (int i = 0; i < TH / 64; ++i) {
    tq += red_q[i];
    tk += red_k[i];
  }
  float inv_q = 1.0f / sqrtf(tq / (float)nq + eps);
  if (floor_scale > 0.f) inv_q *= 1.0f + attn_scale * log1pf(floorf(((float)positions[n] + 1.0f) / floor_scale));
  const float inv_k = 1.0f / sqrtf(tk / (float)nk + eps);
  int page = 0, off = 0;
  if (write) {
    const int slot = slot_mapping[n];
    page = slot / ps;
    off = slot - page * ps;
  }
  const size_t plane = (size_t)ps * PD;
  T* kpage = write ? kv + (size_t)page * 2 * Hk * plane : nullptr;
  T* qo = q_out + n * (size_t)Hq * PD;
  const int heads = write ? Hq + Hk : Hq;
  for (int c = threadIdx.x * 8; c < heads * PD; c += TH * 8) {
    const int h = c / PD, d = c - h * PD;
    const bool is_q = h < Hq;
    const T* xh = x + h * dk;  // (the keys' heads follow the queries')
    const float* w = is_q ? wq + h * dk : wk + (h - Hq) * dk;
    const float inv = is_q ? inv_q : inv_k;
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = 0.f;
    if (d < dk) {
      float ww[8];
      Eight<T>::load(xh + d, v);
      Eight<float>::load(w + d, ww);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] *= ww[i];
      if (d < rd) {
        const bool first = d < hr;
        const int p = first ? d + hr : d - hr, j = first ? d : d - hr;
        float o[8], cs[8], sn[8];
        Eight<T>::load(xh + p, o);
        Eight<float>::load(w + p, ww);
        Eight<float>::load(turn + j, cs);
        Eight<float>::load(turn + hr + j, sn);
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float y = o[i] * ww[i];
          v[i] = first ? v[i] * cs[i] - y * sn[i] : v[i] * cs[i] + y * sn[i];
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] *= inv;
    }
    Eight<T>::store(is_q ? qo + c : kpage + (size_t)(h - Hq) * plane + (size_t)off * PD + d, v);
  }
  if (!write) return;
  T* vpage = kpage + (size_t)Hk * plane;
  const T* vr = r + nq + nk;
  for (int c = threadIdx.x; c < Hk * PD; c += TH) {
    const int h = c / PD, d = c - h * PD;
    Num<T>::store(vpage + h * plane + (size_t)d * ps + off, d < dv ? Num<T>::load(vr + h * dv + d) : 0.f);
  }
}

template <typename T>
static bool launch_span_vec(const void* rows, void* q_out, void* kv, const int* positions, const int* slot_mapping,
                            const float* wq, const float* wk, float eps, float floor_scale, float attn_scale, int N,
                            int Hq, int Hk, int dk, int dv, int PD, int ps, int own_kv, const float* inv_freq, int rd,
                            hipStream_t s) {
  // (by the sizes and the arrays' alignment alone, never by the step's size)
  const int width = own_kv ? (Hq + Hk) * dk + Hk * dv : Hq * dk;
  const uintptr_t all = (uintptr_t)rows | (uintptr_t)q_out | (uintptr_t)kv | (uintptr_t)wq | (uintptr_t)wk;
  const size_t held = (size_t)(own_kv ? Hq + Hk : Hq) * dk * sizeof(T);
  const size_t lds = (held + 15) / 16 * 16 + rd * sizeof(float);
  if (dk % 8 || PD % 8 || (rd / 2) % 8 || width % 8 || all % 16 || lds > 60 * 1024) return false;
  hipLaunchKernelGGL(span_prepare_vec_kernel<T>, dim3(N), dim3(kVecThreads), lds, s, (const T*)rows, (T*)q_out, (T*)kv,
                     positions, slot_mapping, wq, wk, eps, floor_scale, attn_scale, Hq, Hk, dk, dv, PD, ps, own_kv,
                     inv_freq, rd);
  return true;
}

JLE_API int jle_span_prepare(const void* rows, void* q_out, void* kv, const int* positions, const int* slot_mapping,
                             const float* wq, const float* wk, float eps, float floor_scale, float attn_scale,
                             int is_bf16, int N, int Hq, int Hk, int dk, int dv, int PD, int ps, int own_kv,
                             const float* inv_freq, int rd, hipStream_t s) {
  if (N <= 0) return 0;
  if (Hq < 1 || Hk < 1 || dk < 1 || dv < 1 || PD < dk || PD < dv || ps < 1 || wq == nullptr) return JLE_BAD_ARG;
  if (rd < 0 || rd % 2 || rd > dk || rd > 4096 || (rd > 0 && (inv_freq == nullptr || positions == nullptr))) return JLE_BAD_ARG;
  if (kv != nullptr && (!own_kv || wk == nullptr || slot_mapping == nullptr)) return JLE_BAD_ARG;
  if (is_bf16 ? launch_span_vec<bf16_t>(rows, q_out, kv, positions, slot_mapping, wq, wk, eps, floor_scale, attn_scale, N, Hq,
                                        Hk, dk, dv, PD, ps, own_kv, inv_freq, rd, s)
              : launch_span_vec<float>(rows, q_out, kv, positions, slot_mapping, wq, wk, eps, floor_scale, attn_scale, N, Hq,
                                       Hk, dk, dv, PD, ps, own_kv, inv_freq, rd, s)) {
    JLE_LAUNCH_CHECK();
    return 0;
  }
  if (is_bf16)
    hipLaunchKernelGGL(span_prepare_kernel<bf16_t>, dim3(N), dim3(256), rd * sizeof(float), s, (const bf16_t*)rows, (bf16_t*)q_out,
                       (bf16_t*)kv, positions, slot_mapping, wq, wk, eps, floor_scale, attn_scale, Hq, Hk, dk, dv, PD,
                       ps, own_kv, inv_freq, rd);
  else
    hipLaunchKernelGGL(span_prepare_kernel<float>, dim3(N), dim3(256), rd * sizeof(float), s, (const float*)rows, (float*)q_out,
                       (float*)kv, positions, slot_mapping, wq, wk, eps, floor_scale, attn_scale, Hq, Hk, dk, dv, PD, ps,
                       own_kv, inv_freq, rd);
  JLE_LAUNCH_CHECK();
  return 0;
}

// rows[n][:] *= sigmoid(h32[n] . w): one number a token, the product and the sigmoid in float32.  One block per row.
template <typename T>
__global__ __launch_bounds__(256) void row_gate_kernel(T* __restrict__ rows, const float* __restrict__ h32,
                                                       const float* __restrict__ w, int K, int D) {
  __shared__ float red[4];
  const size_t n = blockIdx.x;
  float dot = 0.f;
  for (int c = threadIdx.x; c < K; c += 256) dot = fmaf(h32[n * K + c], w[c], dot);
  const float z = block_sum<256>(dot, red);
  const float gate = 1.0f / (1.0f + expf(-z));
  for (int d = threadIdx.x; d < D; d += 256) Num<T>::store(rows + n * D + d, Num<T>::load(rows + n * D + d) * gate);
}

JLE_API int jle_row_gate(void* rows, int is_bf16, const float* h32, const float* w, int N, int K, int D,
                         hipStream_t s) {
  if (N <= 0) return 0;
  if (K < 1 || D < 1) return JLE_BAD_ARG;
  if (is_bf16)
    hipLaunchKernelGGL(row_gate_kernel<bf16_t>, dim3(N), dim3(256), 0, s, (bf16_t*)rows, h32, w, K, D);
  else
    hipLaunchKernelGGL(row_gate_kernel<float>, dim3(N), dim3(256), 0, s, (float*)rows, h32, w, K, D);
  JLE_LAUNCH_CHECK();
  return 0;
}
