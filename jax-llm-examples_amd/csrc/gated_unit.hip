// A recurrence with one number of memory per channel whose decay and input gate are products of the token's own row (a
// real-gated linear recurrent unit), float32 memory:
//
//   per block of `size` channels:  r = sigmoid(A u + ab),  i = sigmoid(B u + bb);   log a = -rate r softplus(lam)
//   S <- a S + sqrt(1 - a^2) i u;    out = S gelu(y + yb)
//
// u: [N][W] (T), y: rows of stride y_ld (T), A and B: [blocks][out][in] (T).  The gates' products are formed on the matrix
// instructions of T's type with float32 sums, which are never rounded (bfloat16 operands enter exactly; float32 ones on
// the float32 instructions).  A wavefront takes 16 channels: the products' results lie with the lane (c, g), c = lane %
// 16, g = lane / 16, holding the tokens 4 g .. 4 g + 3 of every 16 for channel c.
//
// Two ways through a step:
//  steps of single tokens (every row a segment of its own): one kernel forms gates, memory and output.
//  segments of several tokens: chunks of up to 64 tokens of one segment, worked on side by side.  A token of a chunk maps
//    the memory in front of it as S -> a S + b; the maps of the tokens up to and including each one are put together
//    within the wavefront (4 tokens in a lane, across the lanes of a channel, 16 tokens after 16) and kept; a second
//    kernel walks over a segment's chunks (one multiply-add each), a third forms S and the output from the two.
#include "common.h"
#include "rows.h"

using namespace jle;

namespace {

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

// A product step: every lane brings `kLane` neighbouring elements of a row of either operand (lane (c, g): row c,
// elements kLane g .. of the step's 4 kLane).
template <typename T>
struct Step;
template <>
struct Step<bf16_t> {
  static constexpr int kLane = 8;
  typedef bf16x8 Frag;
  template <bool VEC>
  static __device__ __forceinline__ Frag load(const bf16_t* p, int count) {
    uint4 v = {0u, 0u, 0u, 0u};
    if (VEC) {
      if (count > 0) v = *reinterpret_cast<const uint4*>(p);
    } else {
      uint32_t w[4] = {0u, 0u, 0u, 0u};
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (i < count) w[i >> 1] |= (uint32_t)p[i] << (16 * (i & 1));
      v = uint4{w[0], w[1], w[2], w[3]};
    }
    return __builtin_bit_cast(bf16x8, v);
  }
  static __device__ __forceinline__ void store(bf16_t* p, Frag f) { *reinterpret_cast<uint4*>(p) = __builtin_bit_cast(uint4, f); }
  static __device__ __forceinline__ f32x4 mma(Frag a, Frag b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
  }
};
template <>
struct Step<float> {
  static constexpr int kLane = 4;
  typedef f32x4 Frag;
  template <bool VEC>
  static __device__ __forceinline__ Frag load(const float* p, int count) {
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
  static __device__ __forceinline__ void store(float* p, Frag f) { *reinterpret_cast<f32x4*>(p) = f; }
  static __device__ __forceinline__ f32x4 mma(Frag a, Frag b, f32x4 c) {
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
  }
};

// exp, 1 / (1 + exp(-x)) and the square root: float32 runs by the library, bfloat16 ones by the hardware's instructions
// (a unit in the last place each, and half a one of the exponent's argument)
template <typename T>
struct Math {
  static __device__ __forceinline__ float exp(float x) { return expf(x); }
  static __device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
  static __device__ __forceinline__ float root(float x) { return sqrtf(x); }
};
template <>
struct Math<bf16_t> {
  static __device__ __forceinline__ float exp(float x) { return __builtin_amdgcn_exp2f(1.4426950408889634f * x); }
  static __device__ __forceinline__ float sigmoid(float x) { return __builtin_amdgcn_rcpf(1.0f + exp(-x)); }
  static __device__ __forceinline__ float root(float x) { return __builtin_amdgcn_sqrtf(x); }
};
__device__ __forceinline__ float softplus_(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// gelu in its tanh form: 0.5 (1 + tanh t) = sigmoid(2 t)
template <typename T>
__device__ __forceinline__ float gelu_(float z) {
  return z * Math<T>::sigmoid(1.5957691216057308f * __builtin_fmaf(0.044715f * z, z * z, z));
}
// sqrt(1 - a^2) for a = exp(l), l <= 0: 1 - exp(x), x = 2 l, by its series near zero, where the difference would cancel
template <typename T>
__device__ __forceinline__ float taken(float l, float a) {
  const float x = 2.0f * l;
  float e = 1.0f / 40320.0f;
  e = __builtin_fmaf(e, x, 1.0f / 5040.0f);
  e = __builtin_fmaf(e, x, 1.0f / 720.0f);
  e = __builtin_fmaf(e, x, 1.0f / 120.0f);
  e = __builtin_fmaf(e, x, 1.0f / 24.0f);
  e = __builtin_fmaf(e, x, 1.0f / 6.0f);
  e = __builtin_fmaf(e, x, 0.5f);
  e = __builtin_fmaf(e, x, 1.0f);
  const float near = -e * x, far = __builtin_fmaf(-a, a, 1.0f);
  return Math<T>::root(x > -0.5f ? near : far);
}

template <typename T>
struct UnitArgs {
  const T* u;  // [N][W]
  const T* y;
  const float* y_bias;  // [W]
  const T* wr;          // [blocks][size][size]
  const T* wi;
  const float* br;  // [W]
  const float* bi;
  const float* lam;
  float rate;
  int y_ld, W, size;
  float* state;  // [slots][2][W]
  const int* slots;
  const int* phase;
};

// what a token does to the memory of its channel
struct Map {
  float a, b;
};
__device__ __forceinline__ Map then(Map f, Map s) { return Map{f.a * s.a, __builtin_fmaf(s.a, f.b, s.b)}; }

template <typename T>
struct Channel {  // a channel's constants
  float fall, br, bi;  // fall = -rate softplus(lam)
  __device__ __forceinline__ Channel(const UnitArgs<T>& p, int ch)
      : fall(-p.rate * softplus_(p.lam[ch])), br(p.br[ch]), bi(p.bi[ch]) {}
  __device__ __forceinline__ Map map(float pre_r, float pre_i, float u) const {
    const float l = fall * Math<T>::sigmoid(pre_r + br), a = Math<T>::exp(l);
    return Map{a, taken<T>(l, a) * Math<T>::sigmoid(pre_i + bi) * u};
  }
};

// ------------------------------------------------------------------------------------------------- single tokens
// A wavefront: 16 channels, RT * 16 rows.  blockIdx: (channel tile of a block, rows), tiles of a block side by side.
template <typename T, int RT, bool VEC>
__global__ __launch_bounds__(64) void gated_unit_tokens_kernel(UnitArgs<T> p, T* __restrict__ out, int N, int tiles) {
  typedef Step<T> S;
  typedef typename S::Frag Frag;
  constexpr int KL = S::kLane, KS = 4 * KL;
  const int lane = threadIdx.x, c16 = lane & 15, g = lane >> 4;
  const int blk = blockIdx.x / tiles, c0 = (blockIdx.x - blk * tiles) * 16, n0 = blockIdx.y * 16 * RT;
  const int size = p.size, in_blk = c0 + c16;
  const bool there = in_blk < size;
  const size_t row_w = ((size_t)blk * size + min(in_blk, size - 1)) * size;
  f32x4 ar[RT], ai[RT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) ar[rt] = ai[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const T* urow[RT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) urow[rt] = p.u + (size_t)min(n0 + 16 * rt + c16, N - 1) * p.W + (size_t)blk * size;
#pragma unroll 2
  for (int k = KL * g; k < size + KL * g; k += KS) {  // (the same number of steps in all lanes)
    const int left = size - k;
    const Frag fr = S::template load<VEC>(p.wr + row_w + k, left), fi = S::template load<VEC>(p.wi + row_w + k, left);
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      const Frag fu = S::template load<VEC>(urow[rt] + k, left);
      ar[rt] = S::mma(fu, fr, ar[rt]);
      ai[rt] = S::mma(fu, fi, ai[rt]);
    }
  }
  if (!there) return;
  const int ch = blk * size + in_blk;
  const Channel<T> k(p, ch);
  const float yb = p.y_bias[ch];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n0 + 16 * rt + 4 * g + i;
      if (n >= N) continue;
      const Map m = k.map(ar[rt][i], ai[rt][i], Num<T>::load(p.u + (size_t)n * p.W + ch));
      float* st = p.state + (size_t)p.slots[n] * 2 * p.W + ch;
      const int ph = p.phase[n];
      const float s = __builtin_fmaf(m.a, st[(size_t)ph * p.W], m.b);
      st[(size_t)(1 - ph) * p.W] = s;
      Num<T>::store(out + (size_t)n * p.W + ch, s * gelu_<T>(Num<T>::load(p.y + (size_t)n * p.y_ld + ch) + yb));
    }
}

// ------------------------------------------------------------------------------------------------- chunks
constexpr int kChunk = 64;
constexpr int kChunkWaves = 4;

// chunks: [nc][3] = (segment, first token, tokens).  Writes every token's map of the memory in front of its chunk
// ([N][W] each of wa, wb) and the chunk's ([nc][W] each of ca, cb).  blockIdx: (chunk, channel tile).
template <typename T, int CT, bool VEC>
__global__ __launch_bounds__(kChunkWaves * 64) void gated_unit_chunk_kernel(UnitArgs<T> p, const int* __restrict__ chunks,
                                                                            float* __restrict__ wa, float* __restrict__ wb,
                                                                            float* __restrict__ ca, float* __restrict__ cb,
                                                                            int tiles) {
  typedef Step<T> S;
  typedef typename S::Frag Frag;
  constexpr int KL = S::kLane, KS = 4 * KL;
  constexpr int SLAB = 8 * KS;       // elements of a row that lie in shared memory at a time
  constexpr int ROW = SLAB + KL;     // (16 bytes more than a row)
  constexpr int RT = kChunk / 16;
  __shared__ __attribute__((aligned(16))) T su[kChunk * ROW];
  const int tid = threadIdx.x, lane = tid & 63, w = wave_index(), c16 = lane & 15, g = lane >> 4;
  const int t0 = chunks[3 * blockIdx.x + 1], n = chunks[3 * blockIdx.x + 2];
  const int blk = blockIdx.y / tiles, c0 = (blockIdx.y - blk * tiles) * (16 * CT * kChunkWaves) + 16 * CT * w;
  const int size = p.size;
  size_t row_w[CT];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) row_w[ct] = ((size_t)blk * size + min(c0 + 16 * ct + c16, size - 1)) * size;
  f32x4 ar[CT][RT], ai[CT][RT];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct)
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) ar[ct][rt] = ai[ct][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const T* ub = p.u + (size_t)t0 * p.W + (size_t)blk * size;
  for (int k0 = 0; k0 < size; k0 += SLAB) {
    // the chunk's rows, elements k0 .. of this block's part (zeros behind the part's end and behind the chunk's last row)
#pragma unroll
    for (int j = tid; j < kChunk * (SLAB / KL); j += kChunkWaves * 64) {
      const int row = j / (SLAB / KL), e = (j - row * (SLAB / KL)) * KL;
      const Frag f = S::template load<VEC>(ub + (size_t)min(row, n - 1) * p.W + k0 + e, row < n ? size - k0 - e : 0);
      S::store(su + row * ROW + e, f);
    }
    __syncthreads();
    const int steps = min(8, (size - k0 + KS - 1) / KS);
#pragma unroll 4
    for (int s = 0; s < steps; ++s) {
      const int k = s * KS + KL * g, left = size - k0 - k;
      Frag fr[CT], fi[CT];
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        fr[ct] = S::template load<VEC>(p.wr + row_w[ct] + k0 + k, left);
        fi[ct] = S::template load<VEC>(p.wi + row_w[ct] + k0 + k, left);
      }
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) {
        if (16 * rt >= n) break;
        const Frag fu = *reinterpret_cast<const Frag*>(su + (16 * rt + c16) * ROW + k);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          ar[ct][rt] = S::mma(fu, fr[ct], ar[ct][rt]);
          ai[ct][rt] = S::mma(fu, fi[ct], ai[ct][rt]);
        }
      }
    }
    if (k0 + SLAB < size) __syncthreads();
  }
  // (a block's part of a row that is no wider than the slab is still there)
  const bool held = size <= SLAB;
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    const int in_blk = c0 + 16 * ct + c16;
    const bool there = in_blk < size;
    const int ch = blk * size + min(in_blk, size - 1);
    const Channel<T> k(p, ch);
    Map before = {1.f, 0.f};  // the chunk's tokens in front of this 16
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      if (16 * rt >= n) break;  // (the same in all lanes)
      Map m[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * rt + 4 * g + i;
        m[i] = Map{1.f, 0.f};
        if (t < n)
          m[i] = k.map(ar[ct][rt][i], ai[ct][rt][i],
                       held ? Num<T>::load(su + t * ROW + min(in_blk, size - 1)) : Num<T>::load(p.u + (size_t)(t0 + t) * p.W + ch));
        if (i > 0) m[i] = then(m[i - 1], m[i]);
      }
      // across the channel's four lanes
      Map sum = m[3];
#pragma unroll
      for (int o = 16; o < 64; o <<= 1) {
        const Map f = {__shfl_up(sum.a, o, 64), __shfl_up(sum.b, o, 64)};
        if (lane >= o) sum = then(f, sum);
      }
      Map front = {__shfl_up(sum.a, 16, 64), __shfl_up(sum.b, 16, 64)};
      front = g > 0 ? then(before, front) : before;
      before = then(before, Map{__shfl(sum.a, 48 + c16, 64), __shfl(sum.b, 48 + c16, 64)});
      if (!there) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * rt + 4 * g + i;
        if (t < n) {
          const Map all = then(front, m[i]);
          wa[(size_t)(t0 + t) * p.W + ch] = all.a;
          wb[(size_t)(t0 + t) * p.W + ch] = all.b;
        }
      }
    }
    if (there && g == 0) {
      ca[(size_t)blockIdx.x * p.W + ch] = before.a;
      cb[(size_t)blockIdx.x * p.W + ch] = before.b;
    }
  }
}

// The memory in front of every chunk (into cb's place) and the segment's last one, a thread a channel.  blockIdx: (segment,
// 64 channels); first: [R + 1], the segments' first chunks.
__global__ __launch_bounds__(64) void gated_unit_carry_kernel(const float* __restrict__ ca, float* __restrict__ cb,
                                                              const int* __restrict__ first, float* __restrict__ state,
                                                              const int* __restrict__ slots,
                                                              const int* __restrict__ phase, int W) {
  const int seg = blockIdx.x, ch = blockIdx.y * 64 + threadIdx.x;
  if (ch >= W) return;
  const int lo = first[seg], hi = first[seg + 1], ph = phase[seg];
  float* st = state + (size_t)slots[seg] * 2 * W + ch;
  float S = st[(size_t)ph * W];
  constexpr int U = 8;  // (chunks whose maps are asked for at once)
  for (int c = lo; c < hi; c += U) {
    float a[U], b[U];
#pragma unroll
    for (int j = 0; j < U; ++j) {
      const size_t at = (size_t)min(c + j, hi - 1) * W + ch;
      a[j] = ca[at];
      b[j] = cb[at];
    }
#pragma unroll
    for (int j = 0; j < U; ++j)
      if (c + j < hi) {
        cb[(size_t)(c + j) * W + ch] = S;
        S = __builtin_fmaf(a[j], S, b[j]);
      }
  }
  st[(size_t)(1 - ph) * W] = S;
}

// out = (wa S0 + wb) gelu(y + yb), S0 the memory in front of the token's chunk.  blockIdx: (chunk, 64 V channels, 16 tokens)
template <typename T, int V>
__global__ __launch_bounds__(256) void gated_unit_out_kernel(const int* __restrict__ chunks, const float* __restrict__ wa,
                                                             const float* __restrict__ wb, const float* __restrict__ s0,
                                                             const T* __restrict__ y, int y_ld,
                                                             const float* __restrict__ y_bias, T* __restrict__ out, int W) {
  const int t0 = chunks[3 * blockIdx.x + 1], n = chunks[3 * blockIdx.x + 2];
  const int ch = (blockIdx.y * 64 + (threadIdx.x & 63)) * V;
  if (ch >= W) return;
  float S[V], yb[V];
#pragma unroll
  for (int e = 0; e < V; ++e) {
    S[e] = s0[(size_t)blockIdx.x * W + ch + e];
    yb[e] = y_bias[ch + e];
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 16 * blockIdx.z + 4 * r + wave_index();
    if (t >= n) continue;
    const size_t at = (size_t)(t0 + t) * W + ch;
    const T* yr = y + (size_t)(t0 + t) * y_ld + ch;
    if (V == 4) {
      const f32x4_t a = load4<float>(wa + at), b = load4<float>(wb + at), z = load4<T>(yr);
      f32x4_t o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = __builtin_fmaf(a[e], S[e < V ? e : 0], b[e]) * gelu_<T>(z[e] + yb[e < V ? e : 0]);
      store4<T>(out + at, o);
    } else {
      Num<T>::store(out + at, __builtin_fmaf(wa[at], S[0], wb[at]) * gelu_<T>(Num<T>::load(yr) + yb[0]));
    }
  }
}

template <typename T>
int run_tokens(const UnitArgs<T>& p, T* out, int N, int blocks, bool vec, hipStream_t s) {
  const int tiles = (p.size + 15) / 16;
#define TOKENS(RT, VEC)                                                                                            \
  hipLaunchKernelGGL((gated_unit_tokens_kernel<T, RT, VEC>), dim3(blocks * tiles, (N + 16 * RT - 1) / (16 * RT)), \
                     dim3(64), 0, s, p, out, N, tiles)
  if (vec) {
    // (more rows a wavefront read the matrices less often; up to two wavefronts a SIMD it is their number that counts)
    const long long waves = (long long)blocks * tiles * ((N + 15) / 16);
    if (waves <= 2048) TOKENS(1, true);
    else if (waves <= 4096) TOKENS(2, true);
    else TOKENS(4, true);
  } else {
    TOKENS(1, false);
  }
#undef TOKENS
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename T>
int run_chunks(const UnitArgs<T>& p, T* out, int N, int R, int blocks, const int* chunks, int nc, const int* first,
               float* ws, bool vec, bool vec_out, hipStream_t s) {
  float *wa = ws, *wb = ws + (size_t)N * p.W, *ca = wb + (size_t)N * p.W, *cb = ca + (size_t)nc * p.W;
  const bool wide = vec && p.size % (32 * kChunkWaves) == 0;  // (whole tiles of 128 channels)
  const int per = 16 * kChunkWaves * (wide ? 2 : 1), tiles = (p.size + per - 1) / per;
  const dim3 grid(nc, blocks * tiles), block(kChunkWaves * 64);
  if (grid.y > 65535) return JLE_BAD_ARG;
#define CHUNK(CT, VEC) \
  hipLaunchKernelGGL((gated_unit_chunk_kernel<T, CT, VEC>), grid, block, 0, s, p, chunks, wa, wb, ca, cb, tiles)
  if (wide) CHUNK(2, true);
  else if (vec) CHUNK(1, true);
  else CHUNK(1, false);
#undef CHUNK
  JLE_LAUNCH_CHECK();
  hipLaunchKernelGGL(gated_unit_carry_kernel, dim3(R, (p.W + 63) / 64), dim3(64), 0, s, ca, cb, first, p.state, p.slots,
                     p.phase, p.W);
  JLE_LAUNCH_CHECK();
  if (vec_out)
    hipLaunchKernelGGL((gated_unit_out_kernel<T, 4>), dim3(nc, (p.W + 255) / 256, kChunk / 16), dim3(256), 0, s, chunks, wa,
                       wb, cb, p.y, p.y_ld, p.y_bias, out, p.W);
  else
    hipLaunchKernelGGL((gated_unit_out_kernel<T, 1>), dim3(nc, (p.W + 63) / 64, kChunk / 16), dim3(256), 0, s, chunks, wa, wb,
                       cb, p.y, p.y_ld, p.y_bias, out, p.W);
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename T>
int run(const void* u, const void* y, int y_ld, const float* y_bias, const void* wr, const float* br, const void* wi,
        const float* bi, const float* lam, float rate, float* state, const int* slots, const int* phase, void* out, int N,
        int R, int W, int blocks, const int* chunks, int nc, const int* first, float* ws, hipStream_t s) {
  const UnitArgs<T> p{(const T*)u, (const T*)y, y_bias, (const T*)wr, (const T*)wi, br, bi, lam, rate, y_ld, W, W / blocks,
                      state, slots, phase};
  const bool vec = p.size % Step<T>::kLane == 0 && ((uintptr_t)u | (uintptr_t)wr | (uintptr_t)wi) % 16 == 0;
  if (chunks == nullptr) return run_tokens<T>(p, (T*)out, N, blocks, vec, s);
  const bool vec_out = W % 4 == 0 && y_ld % 4 == 0 && (uintptr_t)y % (4 * sizeof(T)) == 0 &&
                       ((uintptr_t)out | (uintptr_t)ws) % 16 == 0;
  return run_chunks<T>(p, (T*)out, N, R, blocks, chunks, nc, first, ws, vec, vec_out, s);
}

}  // namespace

JLE_API int jle_gated_unit_chunk_tokens() { return kChunk; }

// state: [slots][2][W] float32.  chunks null: every row is a segment of its own (N == R).  Else [nc][3] = (segment, first
// token, tokens <= 64) and first: [R + 1], the segments' first chunks; ws: (2 N + 2 nc) W floats, 16-byte aligned.
JLE_API int jle_gated_unit(const void* u, const void* y, int y_ld, const float* y_bias, const void* wr, const float* br,
                           const void* wi, const float* bi, const float* lam, float rate, float* state, const int* slots,
                           const int* phase, void* out, int is_bf16, int N, int R, int W, int blocks, const int* chunks,
                           int nc, const int* first, float* ws, hipStream_t s) {
  if (N <= 0 || R <= 0) return 0;
  if (W < 1 || blocks < 1 || W % blocks || y_ld < W || rate <= 0.f || u == nullptr || y == nullptr || out == nullptr ||
      state == nullptr || slots == nullptr || phase == nullptr || R > 65535 * 16)
    return JLE_BAD_ARG;
  if (chunks == nullptr ? N != R : (nc < 1 || first == nullptr || ws == nullptr)) return JLE_BAD_ARG;
  return is_bf16 ? run<bf16_t>(u, y, y_ld, y_bias, wr, br, wi, bi, lam, rate, state, slots, phase, out, N, R, W, blocks,
                               chunks, nc, first, ws, s)
                 : run<float>(u, y, y_ld, y_bias, wr, br, wi, bi, lam, rate, state, slots, phase, out, N, R, W, blocks,
                              chunks, nc, first, ws, s);
}
