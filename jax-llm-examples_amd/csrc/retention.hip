// Retention: a matrix memory per head with a fixed decay, float32 memory:
//
//   q, k turned by the position (pairs of the leading rd elements, angles float32), k times 1 / sqrt(dk)
//   S <- decay S + k v^T;   o = S^T q;   out = o / rms(o) * silu(gate)                  (per head; S: dk x dv)
//
// rows: [N][2 H dk + 2 H dv] (T) = q | k | v | gate.  A head's memory lies [dv][dk] (a value column's dk numbers side by
// side); a step reads the half `phase` of the request's memory and writes the other.  Turned queries and keys are float32
// numbers and are used as such.
//
// Three ways through a step:
//  tokens (every row a segment of its own): a block takes a (segment, head), streams the memory through its registers
//    once, and forms norm and gate.
//  scan: token after token, the memory in registers, a wavefront 16 value columns of one (segment, head); both dtypes.
//  chunks (bfloat16 rows): 128 tokens of one segment at a time, all chunks side by side, on the bfloat16 matrix
//    instructions.  With place t of a token in its chunk, n the chunk's tokens and S0 the memory in front of it:
//      o_t = decay^(t+1) S0^T q_t + sum_{s <= t} decay^(t-s) (q_t . k_s) v_s
//      S   = decay^n S0 + sum_s decay^(n-1-s) k_s v_s^T
//    Values enter exactly (they are bfloat16 numbers); what is float32 - queries, keys, the memory that is read, the
//    weighted scores - is split into a leading bfloat16 term and its remainder (16 bits together), whose products are
//    added up (remainder times remainder left out).  Four kernels: prepare (turn, split, and the operands whose inner
//    index is the token laid out along it), the chunks' own contributions to the memory, the walk over a segment's
//    chunks (elementwise, float32), the outputs.
#include "common.h"

using namespace jle;

namespace {

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4;  // (register arrays of HIP's uint4 may end up in scratch)

struct Heads {
  int H, dk, dv, rd, half_pairs;
  const float* inv_freq;  // [rd / 2]
  float k_scale, magnitude;
  __device__ __forceinline__ int width() const { return 2 * H * (dk + dv); }
};

struct Memory {
  float* state;  // [slots][2][H][dv][dk]
  const int* cu;
  const int* slots;
  const int* phase;
  const float* decays;  // [2][H]: the decays, their base-2 logarithms
};

__device__ __forceinline__ float silu_(float x) { return x / (1.0f + expf(-x)); }

// Element e of a head's row x, turned; cs / sn of pair j by `angle(j)`
template <typename T, typename A>
__device__ __forceinline__ float turned(const T* x, int e, const Heads& z, A angle) {
  const float v = Num<T>::load(x + e);
  if (e >= z.rd) return v;
  const int hr = z.rd / 2;
  const bool first = z.half_pairs ? e < hr : (e & 1) == 0;
  const int j = z.half_pairs ? (first ? e : e - hr) : e >> 1;
  const int p = z.half_pairs ? (first ? e + hr : e - hr) : e ^ 1;
  const float o = Num<T>::load(x + p);
  const float2 a = angle(j);
  return first ? v * a.x - o * a.y : v * a.x + o * a.y;
}

__device__ __forceinline__ float2 cos_sin(int pos, const Heads& z, int j) {
  float sn, cs;
  sincosf((float)pos * z.inv_freq[j], &sn, &cs);
  return float2{cs * z.magnitude, sn * z.magnitude};
}

// [N][rd / 2]: cosine and sine of every token's angles
__global__ __launch_bounds__(256) void retention_angles_kernel(const int* __restrict__ positions, Heads z,
                                                               float2* __restrict__ out, int N) {
  const int hr = z.rd / 2;
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long long)N * hr) return;
  const int n = (int)(i / hr);
  out[i] = cos_sin(positions[n], z, (int)(i - (long long)n * hr));
}

// out[N][2 H dk]: q and k of all heads turned, k scaled, float32 (for the scan)
template <typename T>
__global__ __launch_bounds__(256) void retention_turn_kernel(const T* __restrict__ rows, const float2* __restrict__ angles,
                                                             Heads z, float* __restrict__ out) {
  const int n = blockIdx.x, hd = z.H * z.dk, hr = z.rd / 2;
  const T* r = rows + (size_t)n * z.width();
  for (int c = threadIdx.x; c < 2 * hd; c += 256) {
    const int e = c % z.dk;
    const float v = turned(r + (c - e), e, z, [&](int j) { return angles[(size_t)n * hr + j]; });
    out[(size_t)n * 2 * hd + c] = c < hd ? v : v * z.k_scale;
  }
}

template <bool VEC>
__device__ __forceinline__ f32x4 load_up_to4(const float* p, int count) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    if (count > 0) v = *reinterpret_cast<const f32x4*>(p);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < count) v[i] = p[i];
  }
  return v;
}
template <bool VEC>
__device__ __forceinline__ void store_up_to4(float* p, f32x4 v, int count) {
  if (VEC) {
    if (count > 0) *reinterpret_cast<f32x4*>(p) = v;
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < count) p[i] = v[i];
  }
}

// over the 16 lanes of a row
__device__ __forceinline__ float row16_sum(float v) {
#pragma unroll
  for (int m = 8; m > 0; m >>= 1) v += __shfl_xor(v, m, 64);
  return v;
}

// -------------------------------------------------------------------------------------------------- single tokens
constexpr int kTokenThreads = 512;

// KN: 64s of a value column's numbers.  VEC: dk a multiple of 4, the memory 16-byte aligned.  Shared memory: q and k
// [KN 64] each, the outputs [dv].
template <typename T, int KN, bool VEC>
__global__ __launch_bounds__(kTokenThreads) void retention_tokens_kernel(const T* __restrict__ rows,
                                                                         const int* __restrict__ positions, Heads z,
                                                                         Memory mem, T* __restrict__ out, float eps) {
  extern __shared__ float sh[];
  __shared__ float red[kTokenThreads / 64];
  float *sq = sh, *sk = sh + KN * 64, *so = sh + 2 * KN * 64;
  const int n = blockIdx.x / z.H, h = blockIdx.x - n * z.H;
  const int tid = threadIdx.x, lane = tid & 63, w = wave_index(), l = lane & 15, pg = lane >> 4;
  const T* r = rows + (size_t)n * z.width();
  const int pos = positions[n], hd = z.H * z.dk;
  for (int c = tid; c < 2 * KN * 64; c += kTokenThreads) {
    const int e = c & (KN * 64 - 1);
    const bool is_q = c < KN * 64;
    float v = 0.f;
    if (e < z.dk) {
      v = turned(r + (is_q ? 0 : hd) + h * z.dk, e, z, [&](int j) { return cos_sin(pos, z, j); });
      if (!is_q) v *= z.k_scale;
    }
    sh[c] = v;
  }
  __syncthreads();
  f32x4 q[KN], k[KN];
#pragma unroll
  for (int i = 0; i < KN; ++i) {
    q[i] = *reinterpret_cast<const f32x4*>(sq + 64 * i + 4 * l);
    k[i] = *reinterpret_cast<const f32x4*>(sk + 64 * i + 4 * l);
  }
  const size_t head = (size_t)z.dv * z.dk, half = z.H * head;
  const size_t slot = (size_t)mem.slots[n] * 2;
  const int ph = mem.phase[n];
  const float* st_in = mem.state + (slot + ph) * half + h * head;
  float* st_out = mem.state + (slot + 1 - ph) * half + h * head;
  const float keep = mem.decays[h];
  const T* vr = r + 2 * hd + h * z.dv;
  constexpr int STEP = 4 * (kTokenThreads / 64), U = KN <= 2 ? 4 : KN <= 4 ? 2 : 1;
  for (int p0 = 4 * w + pg; p0 < z.dv + pg; p0 += STEP * U) {  // (the same number of rounds in all lanes of a wavefront)
    f32x4 M[U][KN];
    float v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + STEP * u;
      v[u] = p < z.dv ? Num<T>::load(vr + p) : 0.f;
#pragma unroll
      for (int i = 0; i < KN; ++i) {
        const int e = 64 * i + 4 * l;
        M[u][i] = load_up_to4<VEC>(st_in + (size_t)p * z.dk + e, p < z.dv ? z.dk - e : 0);
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + STEP * u;
      f32x4 part = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < KN; ++i) {
        const int e = 64 * i + 4 * l;
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          M[u][i][x] = __builtin_fmaf(keep, M[u][i][x], v[u] * k[i][x]);
          part[x] = __builtin_fmaf(M[u][i][x], q[i][x], part[x]);
        }
        store_up_to4<VEC>(st_out + (size_t)p * z.dk + e, M[u][i], p < z.dv ? z.dk - e : 0);
      }
      const float o = row16_sum((part[0] + part[1]) + (part[2] + part[3]));
      if (l == 0 && p < z.dv) so[p] = o;
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int p = tid; p < z.dv; p += kTokenThreads) ss = __builtin_fmaf(so[p], so[p], ss);
  const float inv = 1.0f / sqrtf(block_sum<kTokenThreads>(ss, red) / (float)z.dv + eps);
  const T* gr = vr + z.H * z.dv;
  T* o = out + ((size_t)n * z.H + h) * z.dv;
  for (int p = tid; p < z.dv; p += kTokenThreads) Num<T>::store(o + p, so[p] * inv * silu_(Num<T>::load(gr + p)));
}

// -------------------------------------------------------------------------------------------------- scan
constexpr int kCols = 4;  // value columns a lane holds (16 a wavefront)

template <typename T, int KN, bool VEC>
__global__ __launch_bounds__(64) void retention_scan_kernel(const float* __restrict__ qk, const T* __restrict__ rows,
                                                            Heads z, Memory mem, float* __restrict__ y) {
  const int seg = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * 16;
  const int lane = threadIdx.x, l = lane & 15, pg = lane >> 4;
  const int t0 = mem.cu[seg], t1 = mem.cu[seg + 1], hd = z.H * z.dk;
  const size_t head = (size_t)z.dv * z.dk, half = z.H * head;
  const float* st_in = mem.state + ((size_t)mem.slots[seg] * 2 + mem.phase[seg]) * half + h * head;
  float* st_out = mem.state + ((size_t)mem.slots[seg] * 2 + (1 - mem.phase[seg])) * half + h * head;
  f32x4 M[kCols][KN];
#pragma unroll
  for (int c = 0; c < kCols; ++c) {
    const int p = p0 + pg + 4 * c;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int e = 64 * i + 4 * l;
      M[c][i] = load_up_to4<VEC>(st_in + (size_t)p * z.dk + e, p < z.dv ? z.dk - e : 0);
    }
  }
  const float keep = mem.decays[h];
  f32x4 qn[KN], kn[KN];
  float vn[kCols];
  auto fetch = [&](int t) {
    const float* r = qk + (size_t)t * 2 * hd + h * z.dk;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int e = 64 * i + 4 * l;
      qn[i] = load_up_to4<VEC>(r + e, z.dk - e);
      kn[i] = load_up_to4<VEC>(r + hd + e, z.dk - e);
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      const int p = p0 + pg + 4 * c;
      vn[c] = p < z.dv ? Num<T>::load(rows + (size_t)t * z.width() + 2 * hd + h * z.dv + p) : 0.f;
    }
  };
  if (t0 < t1) fetch(t0);
  for (int t = t0; t < t1; ++t) {
    f32x4 q[KN], k[KN];
    float v[kCols], o[kCols];
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      q[i] = qn[i];
      k[i] = kn[i];
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) v[c] = vn[c];
    if (t + 1 < t1) fetch(t + 1);
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      f32x4 part = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < KN; ++i)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          M[c][i][x] = __builtin_fmaf(keep, M[c][i][x], v[c] * k[i][x]);
          part[x] = __builtin_fmaf(M[c][i][x], q[i][x], part[x]);
        }
      o[c] = row16_sum((part[0] + part[1]) + (part[2] + part[3]));
    }
    float mine = o[0];  // lane l < kCols of every group stores column pg + 4 l
#pragma unroll
    for (int c = 1; c < kCols; ++c)
      if (l == c) mine = o[c];
    const int p = p0 + pg + 4 * l;
    if (l < kCols && p < z.dv) y[((size_t)t * z.H + h) * z.dv + p] = mine;
  }
#pragma unroll
  for (int c = 0; c < kCols; ++c) {
    const int p = p0 + pg + 4 * c;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int e = 64 * i + 4 * l;
      store_up_to4<VEC>(st_out + (size_t)p * z.dk + e, M[c][i], p < z.dv ? z.dk - e : 0);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(64) void retention_gate_kernel(const float* __restrict__ y, const T* __restrict__ rows, Heads z,
                                                            T* __restrict__ out, float eps) {
  const int n = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const size_t at = ((size_t)n * z.H + h) * z.dv;
  const T* gr = rows + (size_t)n * z.width() + 2 * z.H * z.dk + z.H * z.dv + h * z.dv;
  float ss = 0.f;
  for (int p = lane; p < z.dv; p += 64) ss = __builtin_fmaf(y[at + p], y[at + p], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)z.dv + eps);
  for (int p = lane; p < z.dv; p += 64) Num<T>::store(out + at + p, y[at + p] * inv * silu_(Num<T>::load(gr + p)));
}

// -------------------------------------------------------------------------------------------------- chunks
constexpr int kChunk = 128;
constexpr int kPrep = 64;  // tokens of a block of the preparing kernel

__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ bf16x8 piece(const bf16_t* p) {
  return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p));
}
// a float32 number as its leading bfloat16 term (low half) and the remainder's
__device__ __forceinline__ uint32_t split(float v) {
  const bf16_t hi = float_to_bf16(v);
  return (uint32_t)hi | ((uint32_t)float_to_bf16(v - bf16_to_float(hi)) << 16);
}

// The chunks' operands.  dkp, dvp: dk and dv filled up (zeros) to what the kernels below are laid out for.
struct Operands {
  // [nc][H][kChunk][dkp]: queries and keys, leading terms and remainders (a chunk's rows of a head side by side: rows that
  // lie all heads apart fall on few of the caches' sets and channels)
  bf16_t *qh, *ql, *kh, *kl;
  bf16_t *dh, *dl;            // [nc][H][dkp][kChunk]: keys times decay^(n-1-s), a row the chunk's tokens (zeros behind its last)
  bf16_t* vt;                 // [nc][H][dvp][kChunk]: values, the same way
  bf16_t *sh, *sl;            // [nc][H][dvp][dkp]: the memory in front of the chunk
  float* kv;                  // [nc][H][dv][dk]: the chunk's contribution
  int dkp, dvp;
};

__device__ __forceinline__ void unpack8(uint4 r, float* v) {
  const uint32_t w[4] = {r.x, r.y, r.z, r.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    v[2 * i] = __uint_as_float(w[i] << 16);
    v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}
// eight numbers' leading terms and remainders, eight of each side by side
__device__ __forceinline__ void deal8(const uint32_t* w, uint4& hi, uint4& lo) {
  uint32_t h[4], l[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    h[j] = (w[2 * j] & 0xffffu) | (w[2 * j + 1] << 16);
    l[j] = (w[2 * j] >> 16) | (w[2 * j + 1] & 0xffff0000u);
  }
  hi = uint4{h[0], h[1], h[2], h[3]};
  lo = uint4{l[0], l[1], l[2], l[3]};
}
// Elements e .. e + 7 of a head's row x, turned.  VEC: dk and the half of the turned elements are multiples of 8, half-split
// pairs, rows aligned; a: the token's angles.
template <bool VEC>
__device__ __forceinline__ void turned8(const bf16_t* x, int e, const Heads& z, const float2* a, float* v) {
  if (VEC) {
    unpack8(*reinterpret_cast<const uint4*>(x + e), v);
    if (e < z.rd) {
      const int hr = z.rd / 2;
      const bool first = e < hr;
      float o[8];
      unpack8(*reinterpret_cast<const uint4*>(x + (first ? e + hr : e - hr)), o);
      const float4* t = reinterpret_cast<const float4*>(a + (first ? e : e - hr));
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float4 c = t[i];  // (two pairs' cosines and sines)
        v[2 * i] = first ? v[2 * i] * c.x - o[2 * i] * c.y : v[2 * i] * c.x + o[2 * i] * c.y;
        v[2 * i + 1] = first ? v[2 * i + 1] * c.z - o[2 * i + 1] * c.w : v[2 * i + 1] * c.z + o[2 * i + 1] * c.w;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = e + i < z.dk ? turned(x, e + i, z, [&](int j) { return a[j]; }) : 0.f;
  }
}

// blockIdx: (chunk, half of it, head).  Shared memory: [kPrep][max(dkp + 4, dvp / 2 + 4)] words.
template <bool VEC>
__global__ __launch_bounds__(256) void retention_prepare_kernel(const bf16_t* __restrict__ rows,
                                                                const float2* __restrict__ angles, Heads z,
                                                                const float* __restrict__ decays,
                                                                const int* __restrict__ chunks, Operands o) {
  extern __shared__ uint32_t words[];
  const int c = blockIdx.x, h = blockIdx.z, s0 = blockIdx.y * kPrep;
  const int t0 = chunks[3 * c + 1], n = chunks[3 * c + 2], m = min(kPrep, n - s0);  // (m <= 0: zeros only)
  const int hd = z.H * z.dk, hr = z.rd / 2, W = z.width(), dkp = o.dkp, dvp = o.dvp;
  const float log2_decay = decays[z.H + h];
  const size_t own = ((size_t)c * z.H + h) * kChunk + s0;  // this block's first row of q and k
  const int e8 = dkp / 8;  // (a power of two)
  for (int i = threadIdx.x; i < m * e8; i += 256) {
    const int t = i / e8, e = (i - t * e8) * 8;
    const size_t row = (size_t)(t0 + s0 + t);
    uint32_t w[8] = {0u, 0u, 0u, 0u, 0u, 0u, 0u, 0u};
    if (e < z.dk) {
      float v[8];
      turned8<VEC>(rows + row * W + h * z.dk, e, z, angles + row * hr, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] = split(v[j]);
    }
    uint4 hi, lo;
    deal8(w, hi, lo);
    const size_t at = (own + t) * dkp + e;
    *reinterpret_cast<uint4*>(o.qh + at) = hi;
    *reinterpret_cast<uint4*>(o.ql + at) = lo;
  }
  const int ldk = dkp + 4;
  for (int i = threadIdx.x; i < kPrep * e8; i += 256) {
    const int t = i / e8, e = (i - t * e8) * 8;
    uint32_t d[8] = {0u, 0u, 0u, 0u, 0u, 0u, 0u, 0u};
    if (t < m) {
      const size_t row = (size_t)(t0 + s0 + t);
      uint32_t w[8] = {0u, 0u, 0u, 0u, 0u, 0u, 0u, 0u};
      if (e < z.dk) {
        float v[8];
        turned8<VEC>(rows + row * W + hd + h * z.dk, e, z, angles + row * hr, v);
        const float fade = __builtin_amdgcn_exp2f((float)(n - 1 - s0 - t) * log2_decay);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float k = v[j] * z.k_scale;
          w[j] = split(k);
          d[j] = split(k * fade);
        }
      }
      uint4 hi, lo;
      deal8(w, hi, lo);
      const size_t at = (own + t) * dkp + e;
      *reinterpret_cast<uint4*>(o.kh + at) = hi;
      *reinterpret_cast<uint4*>(o.kl + at) = lo;
    }
    *reinterpret_cast<uint4*>(words + t * ldk + e) = uint4{d[0], d[1], d[2], d[3]};
    *reinterpret_cast<uint4*>(words + t * ldk + e + 4) = uint4{d[4], d[5], d[6], d[7]};
  }
  __syncthreads();
  const size_t kt = ((size_t)c * z.H + h) * dkp * kChunk + s0;
  for (int i = threadIdx.x; i < dkp * (kPrep / 8); i += 256) {
    const int e = i / (kPrep / 8), tg = (i - e * (kPrep / 8)) * 8;
    uint32_t w[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) w[j] = words[(tg + j) * ldk + e];
    uint4 hi, lo;
    deal8(w, hi, lo);
    *reinterpret_cast<uint4*>(o.dh + kt + (size_t)e * kChunk + tg) = hi;
    *reinterpret_cast<uint4*>(o.dl + kt + (size_t)e * kChunk + tg) = lo;
  }
  __syncthreads();
  bf16_t* sv = reinterpret_cast<bf16_t*>(words);
  const int ldv = dvp + 8, v8 = dvp / 8;
  for (int i = threadIdx.x; i < kPrep * v8; i += 256) {
    const int t = i / v8, e = (i - t * v8) * 8;
    uint4 v = {0u, 0u, 0u, 0u};
    if (t < m && e < z.dv) {
      const bf16_t* src = rows + (size_t)(t0 + s0 + t) * W + 2 * hd + h * z.dv + e;
      if (VEC) {
        v = *reinterpret_cast<const uint4*>(src);
      } else {
        uint32_t w[4] = {0u, 0u, 0u, 0u};
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (e + j < z.dv) w[j >> 1] |= (uint32_t)src[j] << (16 * (j & 1));
        v = uint4{w[0], w[1], w[2], w[3]};
      }
    }
    *reinterpret_cast<uint4*>(sv + t * ldv + e) = v;
  }
  __syncthreads();
  const size_t vt = ((size_t)c * z.H + h) * dvp * kChunk + s0;
  for (int i = threadIdx.x; i < dvp * (kPrep / 8); i += 256) {
    const int e = i / (kPrep / 8), tg = (i - e * (kPrep / 8)) * 8;
    uint32_t w[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) w[j] = (uint32_t)sv[(tg + 2 * j) * ldv + e] | ((uint32_t)sv[(tg + 2 * j + 1) * ldv + e] << 16);
    *reinterpret_cast<uint4*>(o.vt + vt + (size_t)e * kChunk + tg) = uint4{w[0], w[1], w[2], w[3]};
  }
}

// kv[c][h] = sum_s decay^(n-1-s) v_s k_s^T, a wavefront 64 x 64 of it.  blockIdx: (chunk * H + head, 64 x 64 tiles).
__global__ __launch_bounds__(64) void retention_chunk_memory_kernel(Operands o, Heads z) {
  const int lane = threadIdx.x, c16 = lane & 15, g = lane >> 4;
  const int kt = o.dkp / 64, v0 = (blockIdx.y / kt) * 64, k0 = (blockIdx.y % kt) * 64;
  const bf16_t* va = o.vt + (size_t)blockIdx.x * o.dvp * kChunk;
  const size_t kb = (size_t)blockIdx.x * o.dkp * kChunk;
  f32x4 acc[4][4];
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int b = 0; b < 4; ++b) acc[a][b] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < kChunk; s += 32) {
    bf16x8 v[4], kh[4], kl[4];
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      v[a] = piece(va + (size_t)(v0 + 16 * a + c16) * kChunk + s + 8 * g);
      const size_t at = kb + (size_t)(k0 + 16 * a + c16) * kChunk + s + 8 * g;
      kh[a] = piece(o.dh + at);
      kl[a] = piece(o.dl + at);
    }
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        acc[a][b] = mma(v[a], kl[b], acc[a][b]);
        acc[a][b] = mma(v[a], kh[b], acc[a][b]);
      }
  }
  float* out = o.kv + (size_t)blockIdx.x * z.dv * z.dk;
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int vr = v0 + 16 * a + 4 * g + i;
      if (vr >= z.dv) continue;
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const int kc = k0 + 16 * b + c16;
        if (kc < z.dk) out[(size_t)vr * z.dk + kc] = acc[a][b][i];
      }
    }
}

// The memory in front of every chunk, as two bfloat16 terms, and the segment's last one.  A thread one number of a
// (segment, head)'s memory.  blockIdx: (256 of dvp * dkp, head, segment); first: [R + 1], the segments' first chunks.
__global__ __launch_bounds__(256) void retention_walk_kernel(Operands o, Heads z, Memory mem, const int* __restrict__ chunks,
                                                             const int* __restrict__ first) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= o.dvp * o.dkp) return;
  const int h = blockIdx.y, seg = blockIdx.z;
  const int v = i / o.dkp, k = i - v * o.dkp;
  const bool there = v < z.dv && k < z.dk;
  const int lo = first[seg], hi = first[seg + 1];
  const size_t head = (size_t)z.dv * z.dk, half = z.H * head, e = (size_t)v * z.dk + k;
  const size_t slot = (size_t)mem.slots[seg] * 2;
  const int ph = mem.phase[seg];
  float S = there ? mem.state[(slot + ph) * half + h * head + e] : 0.f;
  const float log2_decay = mem.decays[z.H + h];
  constexpr int U = 4;  // (chunks whose contributions are asked for at once)
  for (int c = lo; c < hi; c += U) {
    float kv[U];
    int n[U];
#pragma unroll
    for (int j = 0; j < U; ++j) {
      const int cc = min(c + j, hi - 1);
      kv[j] = there ? o.kv[((size_t)cc * z.H + h) * head + e] : 0.f;
      n[j] = chunks[3 * cc + 2];
    }
#pragma unroll
    for (int j = 0; j < U; ++j)
      if (c + j < hi) {
        const size_t at = ((size_t)(c + j) * z.H + h) * o.dvp * o.dkp + i;
        const uint32_t s = split(S);
        o.sh[at] = (bf16_t)(s & 0xffffu);
        o.sl[at] = (bf16_t)(s >> 16);
        S = __builtin_fmaf(__builtin_amdgcn_exp2f((float)n[j] * log2_decay), S, kv[j]);
      }
  }
  if (there) mem.state[(slot + 1 - ph) * half + h * head + e] = S;
}

// The outputs of a chunk for one head: a block of eight wavefronts, 16 tokens each.  Everything is kept transposed (rows:
// keys or value elements, columns: tokens), so that the weighted scores are the second product's operand where the first
// left them: row r of the scores' key tile tt is key 8 (r / 4) + 4 tt + r % 4 of a step's 32, so a lane's eight scores are
// those of eight consecutive keys.
// All wavefronts read the same memory, keys and values: they come through shared memory, once per block, in stages - 32
// value columns of the memory, then 32 keys with their values -, the next stage's on its way in registers while one is
// worked on; two buffers, one barrier a stage.
// DKS: dkp / 32, DVT: dvp / 16.  VEC: gate and output rows are aligned for four neighbours.  blockIdx: chunk * H + head
constexpr int kOutThreads = kChunk * 4;

template <int DKS, int DVT>
constexpr size_t output_lds() {  // bytes of the two buffers
  return 2 * sizeof(bf16_t) * (2 * 32 * (32 * DKS + 8) + 16 * DVT * 40);
}

template <int DKS, int DVT, bool VEC>
__global__ __launch_bounds__(kOutThreads) void retention_outputs_kernel(const bf16_t* __restrict__ rows, Operands o, Heads z,
                                                                        const float* __restrict__ decays,
                                                                        const int* __restrict__ chunks,
                                                                        bf16_t* __restrict__ out, float eps) {
  constexpr int dkp = 32 * DKS, dvp = 16 * DVT, TH = kOutThreads;
  constexpr int LK = dkp + 8, LV = 40;                      // from one row to the next in shared memory
  constexpr int HALF = 32 * LK, BUF = 2 * HALF + dvp * LV;  // leading terms, remainders, values
  constexpr int RP = 32 * dkp / 8, KP = 2 * RP / TH;        // eights of a stage's rows (one kind), and a thread's of both
  constexpr int VE = dvp * 4, VP = (VE + TH - 1) / TH;      // the same of its values
  constexpr int SS = DVT / 2;                               // stages of the memory
  static_assert(2 * RP % TH == 0, "whole rounds of rows");
  extern __shared__ __attribute__((aligned(16))) bf16_t buffers[];
  const int tid = threadIdx.x, lane = tid & 63, w = wave_index(), c16 = lane & 15, g = lane >> 4;
  const int c = blockIdx.x / z.H, h = blockIdx.x - c * z.H;
  const int t0 = chunks[3 * c + 1], n = chunks[3 * c + 2];
  const int q0 = w * 16;        // the wavefront's first place in the chunk
  const bool live = q0 < n;
  const float log2_decay = decays[z.H + h];
  const int t = q0 + c16;
  const size_t own = (size_t)blockIdx.x * kChunk * dkp;
  const bf16_t* vt = o.vt + (size_t)blockIdx.x * dvp * kChunk;
  const size_t mem_at = (size_t)blockIdx.x * dvp * dkp;
  const int stages = SS + (n + 31) / 32;

  u32x4 reg[KP + VP];
  auto fetch = [&](int stage) {
    const bool keys = stage >= SS;
    const size_t at = keys ? own + (size_t)(stage - SS) * 32 * dkp : mem_at + (size_t)stage * 32 * dkp;
    const bf16_t *hi = (keys ? o.kh : o.sh) + at, *lo = (keys ? o.kl : o.sl) + at;
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int idx = tid + TH * i;
      reg[i] = *reinterpret_cast<const u32x4*>((idx < RP ? hi : lo) + (size_t)(idx < RP ? idx : idx - RP) * 8);
    }
    if (keys) {
#pragma unroll
      for (int i = 0; i < VP; ++i) {
        const int idx = min(tid + TH * i, VE - 1);
        reg[KP + i] = *reinterpret_cast<const u32x4*>(vt + (size_t)(idx >> 2) * kChunk + (stage - SS) * 32 + (idx & 3) * 8);
      }
    }
  };
  auto put = [&](int stage) {
    bf16_t* b = buffers + (stage & 1) * BUF;
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int idx = tid + TH * i, in = idx < RP ? idx : idx - RP;
      *reinterpret_cast<u32x4*>(b + (idx < RP ? 0 : HALF) + (in / (dkp / 8)) * LK + (in % (dkp / 8)) * 8) = reg[i];
    }
    if (stage >= SS) {
#pragma unroll
      for (int i = 0; i < VP; ++i) {
        const int idx = tid + TH * i;
        if (idx < VE) *reinterpret_cast<u32x4*>(b + 2 * HALF + (idx >> 2) * LV + (idx & 3) * 8) = reg[KP + i];
      }
    }
    __syncthreads();
    if (stage + 1 < stages) fetch(stage + 1);
  };

  fetch(0);
  bf16x8 qh[DKS], ql[DKS];
  {
    const size_t at = own + (size_t)min(t, n - 1) * dkp + 8 * g;
#pragma unroll
    for (int k = 0; k < DKS; ++k) {
      qh[k] = piece(o.qh + at + 32 * k);
      ql[k] = piece(o.ql + at + 32 * k);
    }
  }
  f32x4 acc[DVT];
#pragma unroll
  for (int d = 0; d < DVT; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  // the memory's part
#pragma unroll
  for (int st = 0; st < SS; ++st) {
    put(st);
    if (!live) continue;
    const bf16_t* b = buffers + (st & 1) * BUF + c16 * LK + 8 * g;
#pragma unroll
    for (int k = 0; k < DKS; ++k) {
      bf16x8 sh[2], sl[2];
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        sh[x] = piece(b + 16 * x * LK + 32 * k);
        sl[x] = piece(b + HALF + 16 * x * LK + 32 * k);
      }
#pragma unroll
      for (int x = 0; x < 2; ++x) acc[2 * st + x] = mma(sl[x], qh[k], acc[2 * st + x]);
#pragma unroll
      for (int x = 0; x < 2; ++x) acc[2 * st + x] = mma(sh[x], ql[k], acc[2 * st + x]);
#pragma unroll
      for (int x = 0; x < 2; ++x) acc[2 * st + x] = mma(sh[x], qh[k], acc[2 * st + x]);
    }
  }
  {
    const float f = __builtin_amdgcn_exp2f((float)(t + 1) * log2_decay);
#pragma unroll
    for (int d = 0; d < DVT; ++d) acc[d] *= f;
  }
  // the chunk's own tokens
  for (int stage = SS; stage < stages; ++stage) {
    put(stage);
    const int s0 = (stage - SS) * 32;
    if (!live || s0 > q0 + 15) continue;
    const bf16_t* b = buffers + (stage & 1) * BUF;
    f32x4 st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    const bf16_t* kr = b + (8 * (c16 >> 2) + (c16 & 3)) * LK + 8 * g;
#pragma unroll
    for (int k = 0; k < DKS; ++k) {
      bf16x8 kh[2], kl[2];
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        kh[tt] = piece(kr + 4 * tt * LK + 32 * k);
        kl[tt] = piece(kr + HALF + 4 * tt * LK + 32 * k);
      }
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) st[tt] = mma(kl[tt], qh[k], st[tt]);
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) st[tt] = mma(kh[tt], ql[k], st[tt]);
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) st[tt] = mma(kh[tt], qh[k], st[tt]);
    }
    uint32_t s[8];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int back = t - (s0 + 8 * g + 4 * tt + i);
        s[4 * tt + i] = split(back >= 0 ? st[tt][i] * __builtin_amdgcn_exp2f((float)back * log2_decay) : 0.f);
      }
    uint4 hi, lo;
    deal8(s, hi, lo);
    const bf16x8 ph = __builtin_bit_cast(bf16x8, hi), pl = __builtin_bit_cast(bf16x8, lo);
    const bf16_t* vr = b + 2 * HALF + c16 * LV + 8 * g;
#pragma unroll
    for (int d = 0; d < DVT; ++d) {
      const bf16x8 v = piece(vr + 16 * d * LV);
      acc[d] = mma(v, pl, acc[d]);
      acc[d] = mma(v, ph, acc[d]);
    }
  }
  if (!live) return;
  // norm and gate: a token's elements lie in the four lanes of its column
  float ss = 0.f;
#pragma unroll
  for (int d = 0; d < DVT; ++d)
#pragma unroll
    for (int i = 0; i < 4; ++i) ss = __builtin_fmaf(acc[d][i], acc[d][i], ss);  // (zeros behind the real elements)
  ss += __shfl_xor(ss, 16, 64);
  ss += __shfl_xor(ss, 32, 64);
  if (t >= n) return;
  const float inv = 1.0f / sqrtf(ss / (float)z.dv + eps);
  const size_t row = (size_t)(t0 + t);
  const bf16_t* gr = rows + row * z.width() + 2 * z.H * z.dk + z.H * z.dv + h * z.dv + 4 * g;
  bf16_t* dst = out + (row * z.H + h) * z.dv + 4 * g;
#pragma unroll
  for (int d = 0; d < DVT; ++d) {
    const int e = 16 * d + 4 * g;
    if (VEC) {
      if (e < z.dv) {
        const uint2 r = *reinterpret_cast<const uint2*>(gr + 16 * d);
        const float g0 = __uint_as_float(r.x << 16), g1 = __uint_as_float(r.x & 0xffff0000u);
        const float g2 = __uint_as_float(r.y << 16), g3 = __uint_as_float(r.y & 0xffff0000u);
        *reinterpret_cast<uint2*>(dst + 16 * d) = uint2{pack_bf16(acc[d][0] * inv * silu_(g0), acc[d][1] * inv * silu_(g1)),
                                                        pack_bf16(acc[d][2] * inv * silu_(g2), acc[d][3] * inv * silu_(g3))};
      }
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (e + i < z.dv) dst[16 * d + i] = float_to_bf16(acc[d][i] * inv * silu_(bf16_to_float(gr[16 * d + i])));
    }
  }
}

// dk and dv filled up to what the chunk kernels are laid out for (0: too large)
int padded_keys(int dk) { return dk <= 64 ? 64 : dk <= 128 ? 128 : dk <= 256 ? 256 : 0; }
int padded_values(int dv) { return dv <= 64 ? 64 : dv <= 128 ? 128 : dv <= 256 ? 256 : dv <= 512 ? 512 : 0; }

size_t align16(size_t n) { return (n + 15) / 16 * 16; }

// the operands' places in the workspace; with base null: its size
size_t place(Operands& o, char* base, int nc, int H, int dk, int dv) {
  o.dkp = padded_keys(dk);
  o.dvp = padded_values(dv);
  size_t at = 0;
  auto take = [&](size_t bytes) {
    char* p = base == nullptr ? nullptr : base + at;
    at += align16(bytes);
    return p;
  };
  const size_t kt = (size_t)nc * H * o.dkp * kChunk * 2, ch = (size_t)nc * H;
  o.qh = (bf16_t*)take(kt);
  o.ql = (bf16_t*)take(kt);
  o.kh = (bf16_t*)take(kt);
  o.kl = (bf16_t*)take(kt);
  o.dh = (bf16_t*)take(kt);
  o.dl = (bf16_t*)take(kt);
  o.vt = (bf16_t*)take(ch * o.dvp * kChunk * 2);
  o.sh = (bf16_t*)take(ch * o.dvp * o.dkp * 2);
  o.sl = (bf16_t*)take(ch * o.dvp * o.dkp * 2);
  o.kv = (float*)take(ch * dv * dk * 4);
  return at;
}

template <int DKS, int DVT, bool VEC>
int launch_outputs(const bf16_t* rows, const Operands& o, const Heads& z, const float* decays, const int* chunks, int nc,
                   bf16_t* out, float eps, hipStream_t s) {
  constexpr size_t lds = output_lds<DKS, DVT>();
  static_assert(lds <= 160 * 1024, "the two buffers fit a compute unit");
  static bool allowed = false;
  if (!allowed) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_outputs_kernel<DKS, DVT, VEC>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
    allowed = true;
  }
  hipLaunchKernelGGL((retention_outputs_kernel<DKS, DVT, VEC>), dim3(nc * z.H), dim3(kOutThreads), lds, s, rows, o, z, decays,
                     chunks, out, eps);
  JLE_LAUNCH_CHECK();
  return 0;
}

template <int DKS>
int pick_outputs(const bf16_t* rows, const Operands& o, const Heads& z, const float* decays, const int* chunks, int nc,
                 bf16_t* out, float eps, bool vec, hipStream_t s) {
#define OUTPUTS(DVT)                                                                                          \
  return vec ? launch_outputs<DKS, DVT, true>(rows, o, z, decays, chunks, nc, out, eps, s)                    \
             : launch_outputs<DKS, DVT, false>(rows, o, z, decays, chunks, nc, out, eps, s)
  switch (o.dvp) {
    case 64: OUTPUTS(4);
    case 128: OUTPUTS(8);
    case 256: OUTPUTS(16);
    default: OUTPUTS(32);
  }
#undef OUTPUTS
}

int run_chunks(const bf16_t* rows, const float2* angles, const Heads& z, const Memory& mem, const int* chunks, int nc,
               const int* first, char* ws, bf16_t* out, int R, float eps, hipStream_t s) {
  Operands o;
  place(o, ws, nc, z.H, z.dk, z.dv);
  const size_t lds = sizeof(uint32_t) * kPrep * (size_t)(o.dkp > o.dvp / 2 ? o.dkp + 4 : o.dvp / 2 + 4);
  const bool vec8 = z.dk % 8 == 0 && z.dv % 8 == 0 && (z.rd == 0 || z.half_pairs) && (z.rd / 2) % 8 == 0 &&
                    ((uintptr_t)rows | (uintptr_t)angles) % 16 == 0;  // (then a row's width is a multiple of 8 too)
  auto prepare = vec8 ? retention_prepare_kernel<true> : retention_prepare_kernel<false>;
  static bool allowed[2] = {false, false};
  if (!allowed[vec8]) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(prepare), hipFuncAttributeMaxDynamicSharedMemorySize,
                                       80 * 1024);
    if (e != hipSuccess) return (int)e;
    allowed[vec8] = true;
  }
  hipLaunchKernelGGL(prepare, dim3(nc, kChunk / kPrep, z.H), dim3(256), lds, s, rows, angles, z, mem.decays,
                     chunks, o);
  JLE_LAUNCH_CHECK();
  hipLaunchKernelGGL(retention_chunk_memory_kernel, dim3(nc * z.H, (o.dkp / 64) * (o.dvp / 64)), dim3(64), 0, s, o, z);
  JLE_LAUNCH_CHECK();
  hipLaunchKernelGGL(retention_walk_kernel, dim3(o.dkp * o.dvp / 256, z.H, R), dim3(256), 0, s, o, z, mem, chunks, first);
  JLE_LAUNCH_CHECK();
  const bool vec = z.dv % 4 == 0 && (2 * z.H * z.dk) % 4 == 0 && ((uintptr_t)rows | (uintptr_t)out) % 8 == 0;
  switch (o.dkp) {
    case 64: return pick_outputs<2>(rows, o, z, mem.decays, chunks, nc, out, eps, vec, s);
    case 128: return pick_outputs<4>(rows, o, z, mem.decays, chunks, nc, out, eps, vec, s);
    default: return pick_outputs<8>(rows, o, z, mem.decays, chunks, nc, out, eps, vec, s);
  }
}

template <typename T>
int run_tokens(const T* rows, const int* positions, const Heads& z, const Memory& mem, T* out, int N, float eps, bool vec,
               hipStream_t s) {
  const int need = (z.dk + 63) / 64;
#define TOKENS(KN)                                                                                                       \
  do {                                                                                                                   \
    const size_t lds = sizeof(float) * (2 * KN * 64 + (size_t)z.dv);                                                     \
    if (vec)                                                                                                             \
      hipLaunchKernelGGL((retention_tokens_kernel<T, KN, true>), dim3(N * z.H), dim3(kTokenThreads), lds, s, rows,       \
                         positions, z, mem, out, eps);                                                                   \
    else                                                                                                                 \
      hipLaunchKernelGGL((retention_tokens_kernel<T, KN, false>), dim3(N * z.H), dim3(kTokenThreads), lds, s, rows,      \
                         positions, z, mem, out, eps);                                                                   \
  } while (0)
  if (need <= 1) TOKENS(1);
  else if (need <= 2) TOKENS(2);
  else if (need <= 4) TOKENS(4);
  else TOKENS(8);
#undef TOKENS
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename T>
int run_scan(const T* rows, const float2* angles, const Heads& z, const Memory& mem, float* ws, T* out, int N, int R,
             float eps, bool vec, hipStream_t s) {
  float *qk = ws, *y = ws + (size_t)N * 2 * z.H * z.dk;
  hipLaunchKernelGGL(retention_turn_kernel<T>, dim3(N), dim3(256), 0, s, rows, angles, z, qk);
  JLE_LAUNCH_CHECK();
  const dim3 grid(R, z.H, (z.dv + 15) / 16);
#define SCAN(KN)                                                                                                       \
  do {                                                                                                                 \
    if (vec)                                                                                                           \
      hipLaunchKernelGGL((retention_scan_kernel<T, KN, true>), grid, dim3(64), 0, s, qk, rows, z, mem, y);             \
    else                                                                                                               \
      hipLaunchKernelGGL((retention_scan_kernel<T, KN, false>), grid, dim3(64), 0, s, qk, rows, z, mem, y);            \
  } while (0)
  const int need = (z.dk + 63) / 64;
  if (need <= 1) SCAN(1);
  else if (need <= 2) SCAN(2);
  else if (need <= 4) SCAN(4);
  else SCAN(8);
#undef SCAN
  JLE_LAUNCH_CHECK();
  hipLaunchKernelGGL(retention_gate_kernel<T>, dim3(N, z.H), dim3(64), 0, s, y, rows, z, out, eps);
  JLE_LAUNCH_CHECK();
  return 0;
}

bool sizes_ok(int H, int dk, int dv, int rd, const float* inv_freq) {
  return H >= 1 && H <= 65535 && dk >= 1 && dk <= 512 && dv >= 1 && dv <= 8192 && rd >= 0 && rd % 2 == 0 && rd <= dk &&
         (rd == 0 || inv_freq != nullptr);
}

Heads heads_of(int H, int dk, int dv, const float* inv_freq, int rd, int half_pairs, float magnitude) {
  return Heads{H, dk, dv, rd, half_pairs, inv_freq, 1.0f / sqrtf((float)dk), magnitude};
}

}  // namespace

JLE_API int jle_retention_chunk_tokens() { return kChunk; }
JLE_API int jle_retention_chunked_supported(int dk, int dv) { return dk >= 1 && dv >= 1 && padded_keys(dk) && padded_values(dv); }
// bytes of the chunk kernels' workspace, in units of 1,024
JLE_API int jle_retention_workspace_kib(int nc, int H, int dk, int dv) {
  Operands o;
  return (int)((place(o, nullptr, nc, H, dk, dv) + 1023) / 1024);
}

// cosines and sines of every token's angles: out [N][rd / 2][2] float32
JLE_API int jle_retention_angles(const int* positions, const float* inv_freq, int rd, float magnitude, float* out, int N,
                                 hipStream_t s) {
  if (N <= 0 || rd == 0) return 0;
  if (rd < 0 || rd % 2 || inv_freq == nullptr || positions == nullptr || out == nullptr) return JLE_BAD_ARG;
  const Heads z = heads_of(1, rd, 1, inv_freq, rd, 1, magnitude);
  const long long items = (long long)N * (rd / 2);
  hipLaunchKernelGGL(retention_angles_kernel, dim3((unsigned)((items + 255) / 256)), dim3(256), 0, s, positions, z,
                     (float2*)out, N);
  JLE_LAUNCH_CHECK();
  return 0;
}

// state: [slots][2][H][dv][dk] float32; decays: [2][H].  how 0: every row a segment of its own (N == R; positions; no
// workspace); 1: scan (angles; ws: N (2 H dk + H dv) floats); 2: chunks (bfloat16; angles; chunks [nc][3] = (segment,
// first token, tokens), first [R + 1]; ws: see jle_retention_workspace_kib).  ws 16-byte aligned.
JLE_API int jle_retention(const void* rows, int is_bf16, const int* positions, const float* inv_freq, int rd,
                          int half_pairs, float magnitude, const float* decays, float* state, const int* cu,
                          const int* slots, const int* phase, void* out, int N, int R, int H, int dk, int dv, float eps,
                          int how, const float* angles, const int* chunks, int nc, const int* first, void* ws,
                          hipStream_t s) {
  if (N <= 0 || R <= 0) return 0;
  if (!sizes_ok(H, dk, dv, rd, inv_freq) || R > 65535 || rows == nullptr || out == nullptr || state == nullptr ||
      decays == nullptr || slots == nullptr || phase == nullptr)
    return JLE_BAD_ARG;
  const Heads z = heads_of(H, dk, dv, inv_freq, rd, half_pairs, magnitude);
  const Memory mem = {state, cu, slots, phase, decays};
  const bool vec = dk % 4 == 0 && ((uintptr_t)state | (uintptr_t)ws) % 16 == 0;
  if (how == 0) {
    if (N != R || positions == nullptr) return JLE_BAD_ARG;
    return is_bf16 ? run_tokens<bf16_t>((const bf16_t*)rows, positions, z, mem, (bf16_t*)out, N, eps, vec, s)
                   : run_tokens<float>((const float*)rows, positions, z, mem, (float*)out, N, eps, vec, s);
  }
  if (cu == nullptr || ws == nullptr || (rd > 0 && angles == nullptr)) return JLE_BAD_ARG;
  if (how == 1)
    return is_bf16 ? run_scan<bf16_t>((const bf16_t*)rows, (const float2*)angles, z, mem, (float*)ws, (bf16_t*)out, N, R, eps, vec, s)
                   : run_scan<float>((const float*)rows, (const float2*)angles, z, mem, (float*)ws, (float*)out, N, R, eps, vec, s);
  if (how != 2 || !is_bf16 || nc < 1 || chunks == nullptr || first == nullptr || !jle_retention_chunked_supported(dk, dv) ||
      (uintptr_t)ws % 16)
    return JLE_BAD_ARG;
  return run_chunks((const bf16_t*)rows, (const float2*)angles, z, mem, chunks, nc, first, (char*)ws, (bf16_t*)out, R, eps, s);
}
