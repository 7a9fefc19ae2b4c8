// A matrix memory per head with one decay and one write strength a token (the Mamba-2 recurrence), float32 memory:
//
//   d = softplus(dt + dt_bias);  a = -exp(A_log) d;   S <- exp(a) S + d B x^T;   y = S^T C + skip x
//
// and what follows it, y * silu(z) normed in equal parts.  proj: the projection's rows [N][2 H P + 2 G S + H] (T) = gate z |
// (values, write keys, read keys before their convolution) | dt; rows: [N][H P + 2 G S] (T) = x | B | C behind it.
// A head's memory lies [P][S] (a value column's S numbers side by side); a step reads the half `phase` of the
// request's memory and writes the other.
//
// Two kernels walk through a segment's tokens.
//  scan: token after token.  A wavefront takes 16 value columns of one (segment, head): lane (pg, l), pg = lane / 16, l =
//    lane % 16, holds the columns pg, pg + 4, .. and of each the numbers 4 l .. 4 l + 3 of every 64; the products with C
//    are summed over l by lane exchanges.  Both dtypes; steps of single tokens and of short segments.
//  chunks (bfloat16 rows): a block of eight wavefronts takes 64 value columns of one (segment, head) and goes through the
//    segment 64 tokens at a time, the memory in registers (two wavefronts share 16 columns, each holds half of a
//    column's numbers).  With L_t the running sum of a in the chunk and S0 the memory in front of it:
//      y_t = exp(L_t) S0^T C_t + sum_{s <= t} exp(L_t - L_s) d_s (C_t . B_s) x_s + skip x_t
//      S   = exp(L_end) S0 + sum_s exp(L_end - L_s) d_s B_s x_s^T
//    as products on the bfloat16 matrix instructions.  B, C and x enter exactly (they are bfloat16 numbers); what is not -
//    the weighted scores, the memory that is read, the weighted values that are written - is split into bfloat16
//    terms that are multiplied one after the other: the written values into three (all 24 bits of them, so the memory
//    is as a float32 recurrence leaves it), the scores and the memory's read-out into two (16 bits).  The sums L are
//    formed in float64: under strong decay they reach hundreds, and it is their differences that count.
#include "common.h"

using namespace jle;

namespace {

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

__device__ __forceinline__ float softplus_(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

struct Sizes {
  int H, P, S, G;
  int ld;      // of proj
  int dt_off;  // where dt begins in a row of proj
  __device__ __forceinline__ int inner() const { return H * P; }
  __device__ __forceinline__ int width() const { return H * P + 2 * G * S; }
};

struct Memory {
  float* state;  // [slots][2][H][P][S]
  const int* cu;
  const int* slots;
  const int* phase;
};

template <typename T>
__device__ __forceinline__ f32x4 load4(const T* p);
template <>
__device__ __forceinline__ f32x4 load4<float>(const float* p) {
  return *reinterpret_cast<const f32x4*>(p);
}
template <>
__device__ __forceinline__ f32x4 load4<bf16_t>(const bf16_t* p) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  return f32x4{__uint_as_float(r.x << 16), __uint_as_float(r.x & 0xffff0000u), __uint_as_float(r.y << 16),
               __uint_as_float(r.y & 0xffff0000u)};
}
// up to four neighbours, `count` of them there
template <typename T, bool VEC>
__device__ __forceinline__ f32x4 load_up_to4(const T* p, int count) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    if (count > 0) v = load4<T>(p);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < count) v[i] = Num<T>::load(p + i);
  }
  return v;
}

constexpr int kCols = 4;  // value columns a lane holds in the scan (16 a wavefront)

// VEC: S is a multiple of 4 and every array is aligned to what four neighbours take
template <typename T, int KN, bool VEC>
__global__ __launch_bounds__(64) void mamba2_scan_kernel(const T* __restrict__ proj, const T* __restrict__ rows,
                                                         const float* __restrict__ dt_bias,
                                                         const float* __restrict__ a_log,
                                                         const float* __restrict__ skip, Memory mem,
                                                         float* __restrict__ y, Sizes z) {
  const int seg = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * 16;
  const int lane = threadIdx.x, l = lane & 15, pg = lane >> 4;
  const int t0 = mem.cu[seg], t1 = mem.cu[seg + 1];
  const size_t half = (size_t)z.H * z.P * z.S;
  const float* st_in = mem.state + ((size_t)mem.slots[seg] * 2 + mem.phase[seg]) * half + (size_t)h * z.P * z.S;
  float* st_out = mem.state + ((size_t)mem.slots[seg] * 2 + (1 - mem.phase[seg])) * half + (size_t)h * z.P * z.S;
  f32x4 M[kCols][KN];
#pragma unroll
  for (int q = 0; q < kCols; ++q) {
    const int p = p0 + pg + 4 * q;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int s = 4 * l + 64 * i;
      M[q][i] = p < z.P ? load_up_to4<float, VEC>(st_in + (size_t)p * z.S + s, z.S - s) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }
  const float neg_rate = -expf(a_log[h]), bias = dt_bias[h], sk = skip[h];
  const int g = h / (z.H / z.G), W = z.width();
  f32x4 Bn[KN], Cn[KN];
  float xn[kCols], dn = 0.f;
  auto fetch = [&](int t) {
    const T* r = rows + (size_t)t * W;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int s = 4 * l + 64 * i;
      Bn[i] = load_up_to4<T, VEC>(r + z.inner() + g * z.S + s, z.S - s);
      Cn[i] = load_up_to4<T, VEC>(r + z.inner() + (z.G + g) * z.S + s, z.S - s);
    }
#pragma unroll
    for (int q = 0; q < kCols; ++q) {
      const int p = p0 + pg + 4 * q;
      xn[q] = p < z.P ? Num<T>::load(r + h * z.P + p) : 0.f;
    }
    dn = Num<T>::load(proj + (size_t)t * z.ld + z.dt_off + h);
  };
  if (t0 < t1) fetch(t0);
  for (int t = t0; t < t1; ++t) {
    f32x4 B[KN], C[KN];
    float x[kCols];
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      B[i] = Bn[i];
      C[i] = Cn[i];
    }
#pragma unroll
    for (int q = 0; q < kCols; ++q) x[q] = xn[q];
    const float d = softplus_(dn + bias);
    if (t + 1 < t1) fetch(t + 1);
    const float keep = expf(neg_rate * d);
    float o[kCols];
#pragma unroll
    for (int q = 0; q < kCols; ++q) {
      const float dx = d * x[q];
      f32x4 part = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < KN; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          M[q][i][e] = fmaf(keep, M[q][i][e], dx * B[i][e]);
          part[e] = fmaf(M[q][i][e], C[i][e], part[e]);
        }
      o[q] = (part[0] + part[1]) + (part[2] + part[3]);
    }
#pragma unroll
    for (int m = 8; m > 0; m >>= 1)
#pragma unroll
      for (int q = 0; q < kCols; ++q) o[q] += __shfl_xor(o[q], m, 64);
    // lane l < kCols of every group stores column pg + 4 l
    float mine = o[0], mx = x[0];
#pragma unroll
    for (int q = 1; q < kCols; ++q)
      if (l == q) {
        mine = o[q];
        mx = x[q];
      }
    const int p = p0 + pg + 4 * l;
    if (l < kCols && p < z.P) y[(size_t)t * z.inner() + h * z.P + p] = fmaf(sk, mx, mine);
  }
#pragma unroll
  for (int q = 0; q < kCols; ++q) {
    const int p = p0 + pg + 4 * q;
    if (p >= z.P) continue;
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int s = 4 * l + 64 * i;
      float* dst = st_out + (size_t)p * z.S + s;
      if (VEC) {
        if (s < z.S) *reinterpret_cast<f32x4*>(dst) = M[q][i];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (s + e < z.S) dst[e] = M[q][i][e];
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------------------ chunks
constexpr int kChunk = 64;          // tokens of a chunk, and value columns of a block
constexpr int kTS = kChunk + 8;     // from one row of a transposed array (or of the scores) to the next
constexpr int kPadS = 8;            // numbers behind a row of B or C
constexpr int kChunkThreads = 512;

__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ bf16x8 piece(const bf16_t* p) {
  return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p));
}
__device__ __forceinline__ bf16x8 pack8(const float* v) {
  const uint4 r = {pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7])};
  return __builtin_bit_cast(bf16x8, r);
}
// the leading bfloat16 term of eight numbers; v keeps what it leaves
__device__ __forceinline__ bf16x8 take_term(float* v) {
  const bf16x8 t = pack8(v);
  const uint4 r = __builtin_bit_cast(uint4, t);
  const uint32_t w[4] = {r.x, r.y, r.z, r.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    v[2 * i] -= __uint_as_float(w[i] << 16);
    v[2 * i + 1] -= __uint_as_float(w[i] & 0xffff0000u);
  }
  return t;
}

// Eight neighbouring numbers.  VEC: what lies past the end is read from the end instead (one load, no branch, so that
// nothing waits for it before it is used) and made zero by `there` when it has come; else only what is there is read.
template <bool VEC>
__device__ __forceinline__ uint4 load8(const bf16_t* row, int col, int cols) {
  if (VEC) return *reinterpret_cast<const uint4*>(row + min(col, cols - 8));
  uint32_t w[4] = {0u, 0u, 0u, 0u};
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (col + i < cols) w[i >> 1] |= (uint32_t)row[col + i] << (16 * (i & 1));
  return uint4{w[0], w[1], w[2], w[3]};
}
__device__ __forceinline__ uint4 there(uint4 v, bool ok) {
  return uint4{ok ? v.x : 0u, ok ? v.y : 0u, ok ? v.z : 0u, ok ? v.w : 0u};
}
// Four rows of them (a piece of B or x, to be stored both ways round)
struct Piece {
  uint4 r[4];
};
template <bool VEC>
__device__ __forceinline__ Piece load_piece(const bf16_t* rows, size_t width, int row, int n, int col, int cols) {
  Piece q;
#pragma unroll
  for (int i = 0; i < 4; ++i) q.r[i] = load8<VEC>(rows + (size_t)min(row + i, n - 1) * width, col, cols);
  return q;
}
__device__ __forceinline__ void piece_there(Piece& q, int row, int n, bool cols_there) {
#pragma unroll
  for (int i = 0; i < 4; ++i) q.r[i] = there(q.r[i], cols_there && row + i < n);
}
// dst[column][row .. row + 3]: the piece turned round, eight stores of four numbers
__device__ __forceinline__ void store_turned(const Piece& q, bf16_t* dst) {
  const uint32_t w[4][4] = {{q.r[0].x, q.r[0].y, q.r[0].z, q.r[0].w}, {q.r[1].x, q.r[1].y, q.r[1].z, q.r[1].w},
                            {q.r[2].x, q.r[2].y, q.r[2].z, q.r[2].w}, {q.r[3].x, q.r[3].y, q.r[3].z, q.r[3].w}};
#pragma unroll
  for (int c = 0; c < 8; ++c) {
    const int i = c >> 1;
    uint32_t a, b;
    if (c & 1) {
      a = (w[0][i] >> 16) | (w[1][i] & 0xffff0000u);
      b = (w[2][i] >> 16) | (w[3][i] & 0xffff0000u);
    } else {
      a = (w[0][i] & 0xffffu) | (w[1][i] << 16);
      b = (w[2][i] & 0xffffu) | (w[3][i] << 16);
    }
    *reinterpret_cast<uint2*>(dst + c * kTS) = uint2{a, b};
  }
}

// the sum over the lanes up to and including this one, by lane permutations that ride on an operand (rows of 16 lanes,
// then the rows' and the halves' last lanes handed on)
template <int CTRL, int ROWS>
__device__ __forceinline__ double moved_up(double v) {
  const unsigned long long u = __double_as_longlong(v);
  const uint32_t lo = (uint32_t)__builtin_amdgcn_update_dpp(0, (int)(uint32_t)u, CTRL, ROWS, 0xf, false);
  const uint32_t hi = (uint32_t)__builtin_amdgcn_update_dpp(0, (int)(uint32_t)(u >> 32), CTRL, ROWS, 0xf, false);
  return __longlong_as_double((long long)(((unsigned long long)hi << 32) | lo));
}
__device__ __forceinline__ double sum_up_to_lane(double v) {
  v += moved_up<0x111, 0xf>(v);
  v += moved_up<0x112, 0xf>(v);
  v += moved_up<0x114, 0xf>(v);
  v += moved_up<0x118, 0xf>(v);
  v += moved_up<0x142, 0xa>(v);
  v += moved_up<0x143, 0xc>(v);
  return v;
}
__device__ __forceinline__ double last_lane(double v) {
  const unsigned long long u = __double_as_longlong(v);
  const uint32_t lo = (uint32_t)__builtin_amdgcn_readlane((int)(uint32_t)u, 63);
  const uint32_t hi = (uint32_t)__builtin_amdgcn_readlane((int)(uint32_t)(u >> 32), 63);
  return __longlong_as_double((long long)(((unsigned long long)hi << 32) | lo));
}

template <int NT>
constexpr size_t chunk_lds() {  // bytes
  constexpr int NP = 32 * NT, SB = NP + kPadS;
  return sizeof(bf16_t) * (2 * kChunk * SB + NP * kTS + 3 * kChunk * kTS) + sizeof(double) * kChunk +
         3 * sizeof(float) * kChunk + 16 * 64 * sizeof(f32x4);
}

// NT: S, filled up to a multiple of 32, over 32.  VEC: S, P and the rows' width are multiples of 8, rows aligned.
template <int NT, bool VEC>
__global__ __launch_bounds__(kChunkThreads) void mamba2_chunk_kernel(const bf16_t* __restrict__ proj,
                                                           const bf16_t* __restrict__ rows,
                                                           const float* __restrict__ dt_bias,
                                                           const float* __restrict__ a_log,
                                                           const float* __restrict__ skip, Memory mem,
                                                           float* __restrict__ y, Sizes z) {
  constexpr int NP = 32 * NT, SB = NP + kPadS;
  constexpr int TH = kChunkThreads;
  constexpr int PP = (NT * 64 + 128 + TH - 1) / TH;  // pieces of B and x a thread takes
  constexpr int CP = (NT * 256 + TH - 1) / TH;       // eights of C
  constexpr int KH = (NT + 1) / 2;                   // 32s of a column's numbers that a wavefront holds
  extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
  double* s_L = reinterpret_cast<double*>(lds);               // [64] running sums of a, in units of ln 2
  float* s_d = reinterpret_cast<float*>(s_L + kChunk);        // [64] step sizes
  float* s_w = s_d + kChunk;                                  // [64] exp(L_end - L_s) d_s
  float* s_e = s_w + kChunk;                                  // [64] exp(L_t)
  bf16_t* sB = reinterpret_cast<bf16_t*>(s_e + kChunk);       // [64][SB] write keys, token by token
  bf16_t* sC = sB + kChunk * SB;                              // [64][SB] read keys
  bf16_t* bT = sC + kChunk * SB;                              // [NP][kTS] write keys, turned round
  bf16_t* xT = bT + NP * kTS;                                 // [64][kTS] this block's value columns, turned round
  bf16_t* Ph = xT + kChunk * kTS;                             // [64][kTS] weighted scores [query][key], leading term
  bf16_t* Pl = Ph + kChunk * kTS;                             // and the next
  f32x4* sF = reinterpret_cast<f32x4*>(Pl + kChunk * kTS);    // [16][64] what two wavefronts hand each other
  const int seg = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * kChunk;
  const int tid = threadIdx.x, lane = tid & 63, w = wave_index(), c16 = lane & 15, g = lane >> 4;
  const int t_begin = mem.cu[seg], t_end = mem.cu[seg + 1];
  const size_t half = (size_t)z.H * z.P * z.S;
  const float* st_in = mem.state + ((size_t)mem.slots[seg] * 2 + mem.phase[seg]) * half + (size_t)h * z.P * z.S;
  float* st_out = mem.state + ((size_t)mem.slots[seg] * 2 + (1 - mem.phase[seg])) * half + (size_t)h * z.P * z.S;
  const int grp = h / (z.H / z.G), W = z.width(), inner = z.inner();
  const float neg_rate = -expf(a_log[h]), bias = dt_bias[h], sk = skip[h];

  // this wavefront's value columns: p0 + 16 pt + c16; element r of M[k][u]: number 32 (k0 + k) + 8 g + 4 u + r of the
  // column; the queries whose outputs it forms: 32 hf .. 32 hf + 31 of a chunk
  const int pt = w & 3, hf = w >> 2, k0 = hf * KH;
  const int p = p0 + 16 * pt + c16;
  const bool wave_live = p0 + 16 * pt < z.P;
  f32x4 M[KH][2];
#pragma unroll
  for (int k = 0; k < KH; ++k)
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int s = 32 * (k0 + k) + 8 * g + 4 * u;
      M[k][u] = p < z.P ? load_up_to4<float, VEC>(st_in + (size_t)p * z.S + s, z.S - s) : f32x4{0.f, 0.f, 0.f, 0.f};
    }

  // the next chunk's rows, asked for while this chunk is worked on.  A thread takes PP pieces of the write keys and the
  // values (which of them: by the thread's number, without a branch, so that no load is waited for before its use)
  Piece nP[PP];
  uint4 nC[CP];
  bf16_t nd = 0;
  auto fetch = [&](int t0) {
    const int n = min(kChunk, t_end - t0);
    const bf16_t* base = rows + (size_t)t0 * W;
#pragma unroll
    for (int i = 0; i < PP; ++i) {
      const int idx = min(tid + TH * i, NT * 64 + 127);
      const bool keys = idx < NT * 64;
      const int at = keys ? idx : idx - NT * 64;
      nP[i] = load_piece<VEC>(base + (keys ? inner + grp * z.S : h * z.P + p0), W, (at & 15) * 4, n, (at >> 4) * 8,
                              keys ? z.S : z.P - p0);
    }
    nd = proj[(size_t)(t0 + min(lane, n - 1)) * z.ld + z.dt_off + h];
#pragma unroll
    for (int i = 0; i < CP; ++i) {
      const int idx = tid + TH * i;
      const int s = idx / (4 * NT), c8 = (idx - s * (4 * NT)) * 8;
      nC[i] = load8<VEC>(base + (size_t)min(s, n - 1) * W + inner + (z.G + grp) * z.S, c8, z.S);
    }
  };
  // vmcnt(0): the memory has come (left pending, it would be waited for inside the loop, and the next chunk's rows with it)
  __builtin_amdgcn_s_waitcnt(0x0F70);
  asm volatile("" ::: "memory");
  if (t_begin < t_end) fetch(t_begin);
  for (int t0 = t_begin; t0 < t_end; t0 += kChunk) {
    const int n = min(kChunk, t_end - t0);
    // the chunk into shared memory
#pragma unroll
    for (int i = 0; i < PP; ++i) {
      const int idx = tid + TH * i;
      const bool keys = idx < NT * 64;
      const int at = keys ? idx : idx - NT * 64;
      const int s4 = (at & 15) * 4, c8 = (at >> 4) * 8;
      if (idx < NT * 64 + 128) {
        piece_there(nP[i], s4, n, c8 < (keys ? z.S : z.P - p0));
        store_turned(nP[i], (keys ? bT : xT) + c8 * kTS + s4);
        if (keys) {
#pragma unroll
          for (int r = 0; r < 4; ++r) *reinterpret_cast<uint4*>(sB + (s4 + r) * SB + c8) = nP[i].r[r];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < CP; ++i) {
      const int idx = tid + TH * i;
      const int s = idx / (4 * NT), c8 = (idx - s * (4 * NT)) * 8;
      if (s < kChunk) *reinterpret_cast<uint4*>(sC + s * SB + c8) = there(nC[i], s < n && c8 < z.S);
    }
    if (w == 7) {
      const bool ok = lane < n;
      const float d = ok ? softplus_(bf16_to_float(nd) + bias) : 0.f;
      const double L = sum_up_to_lane((double)(neg_rate * d) * 1.4426950408889634);
      const double end = last_lane(L);  // (tokens behind the chunk's last add nothing)
      s_L[lane] = L;
      s_d[lane] = d;
      s_w[lane] = __builtin_amdgcn_exp2f((float)(end - L)) * d;
      s_e[lane] = __builtin_amdgcn_exp2f((float)L);
    }
    __syncthreads();
    if (t0 + kChunk < t_end) fetch(t0 + kChunk);
    // the weighted scores of 16 queries (two wavefronts share them, every other key block each), key block by key block
    // up to the diagonal, and zeros up to the end of the 32 keys that a product takes at a time
    if (16 * pt < n) {
      const int t = 16 * pt + c16;
      const double Lt = s_L[t];
      bf16x8 cq[NT];
#pragma unroll
      for (int kk = 0; kk < NT; ++kk) cq[kk] = piece(sC + t * SB + 32 * kk + 8 * g);
      f32x4 acc[2];  // (both key blocks' products side by side)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (hf + 2 * i > pt) continue;
#pragma unroll
        for (int kk = 0; kk < NT; ++kk)
          acc[i] = mma(piece(sB + (16 * (hf + 2 * i) + c16) * SB + 32 * kk + 8 * g), cq[kk], acc[i]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int sb = hf + 2 * i;
        if (sb > (pt | 1)) continue;
        float v[4], lo[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int s = 16 * sb + 4 * g + r;
          v[r] = s <= t ? acc[i][r] * (__builtin_amdgcn_exp2f((float)(Lt - s_L[s])) * s_d[s]) : 0.f;
        }
        const uint2 hi = {pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
        lo[0] = v[0] - __uint_as_float(hi.x << 16);
        lo[1] = v[1] - __uint_as_float(hi.x & 0xffff0000u);
        lo[2] = v[2] - __uint_as_float(hi.y << 16);
        lo[3] = v[3] - __uint_as_float(hi.y & 0xffff0000u);
        *reinterpret_cast<uint2*>(Ph + t * kTS + 16 * sb + 4 * g) = hi;
        *reinterpret_cast<uint2*>(Pl + t * kTS + 16 * sb + 4 * g) = uint2{pack_bf16(lo[0], lo[1]), pack_bf16(lo[2], lo[3])};
      }
    }
    __syncthreads();
    // values of this wavefront's columns, a column a lane row: tokens 32 ks + 8 g .. + 7
    bf16x8 xa[2];
    f32x4 inside[2];  // the chunk's own part of this wavefront's two query tiles
    f32x4 mine[2];    // this wavefront's half of the memory's part of them
    if (wave_live) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) xa[ks] = piece(xT + (16 * pt + c16) * kTS + 32 * ks + 8 * g);
      f32x4 front[4];  // S0^T C_t of the four query tiles (rows: value columns)
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) front[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KH; ++k) {
        const int kk = k0 + k;
        if (kk >= NT) break;
        float v[8] = {M[k][0][0], M[k][0][1], M[k][0][2], M[k][0][3], M[k][1][0], M[k][1][1], M[k][1][2], M[k][1][3]};
        const bf16x8 m_hi = take_term(v), m_lo = pack8(v);
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          const bf16x8 c = piece(sC + (16 * tt + c16) * SB + 32 * kk + 8 * g);
          front[tt] = mma(m_lo, c, front[tt]);
          front[tt] = mma(m_hi, c, front[tt]);
        }
      }
      // the other wavefront's queries' part goes to it, its comes back behind the barrier
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        mine[i] = hf == 0 ? front[i] : front[2 + i];
        sF[(w * 2 + i) * 64 + lane] = hf == 0 ? front[2 + i] : front[i];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        inside[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int t = 32 * hf + 16 * i + c16;
        if (32 * hf + 16 * i >= n) continue;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          if (ks > hf) break;
          inside[i] = mma(xa[ks], piece(Pl + t * kTS + 32 * ks + 8 * g), inside[i]);
          inside[i] = mma(xa[ks], piece(Ph + t * kTS + 32 * ks + 8 * g), inside[i]);
        }
      }
    }
    __syncthreads();
    if (wave_live) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int t = 32 * hf + 16 * i + c16;
        if (t < n) {
          const float e = s_e[t];
          const f32x4 other = sF[((w ^ 4) * 2 + i) * 64 + lane];
          f32x4 o;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float x = bf16_to_float(xT[(16 * pt + 4 * g + r) * kTS + t]);
            o[r] = fmaf(e, mine[i][r] + other[r], inside[i][r]) + sk * x;
          }
          const int pc = p0 + 16 * pt + 4 * g;
          float* dst = y + (size_t)(t0 + t) * inner + h * z.P + pc;
          if (VEC) {
            if (pc < z.P) *reinterpret_cast<f32x4*>(dst) = o;
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (pc + r < z.P) dst[r] = o[r];
          }
        }
      }
      // the memory behind the chunk
      const float fade = s_e[kChunk - 1];
#pragma unroll
      for (int k = 0; k < KH; ++k)
#pragma unroll
        for (int u = 0; u < 2; ++u) M[k][u] *= fade;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        if (32 * ks >= n) break;
        const uint4 raw = __builtin_bit_cast(uint4, xa[ks]);
        const uint32_t xw[4] = {raw.x, raw.y, raw.z, raw.w};
        float v[8];
#pragma unroll
        for (int j = 0; j < 8; ++j)
          v[j] = __uint_as_float((j & 1) ? (xw[j >> 1] & 0xffff0000u) : (xw[j >> 1] << 16)) * s_w[32 * ks + 8 * g + j];
        const bf16x8 v1 = take_term(v), v2 = take_term(v), v3 = pack8(v);
#pragma unroll
        for (int k = 0; k < KH; ++k)
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            if (k0 + k >= NT) break;
            const int s = 32 * (k0 + k) + 8 * (c16 >> 2) + 4 * u + (c16 & 3);
            const bf16x8 b = piece(bT + s * kTS + 32 * ks + 8 * g);
            M[k][u] = mma(b, v3, M[k][u]);
            M[k][u] = mma(b, v2, M[k][u]);
            M[k][u] = mma(b, v1, M[k][u]);
          }
      }
    }
    __syncthreads();
  }
  if (p < z.P) {
#pragma unroll
    for (int k = 0; k < KH; ++k)
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int s = 32 * (k0 + k) + 8 * g + 4 * u;
        float* dst = st_out + (size_t)p * z.S + s;
        if (VEC) {
          if (s < z.S) *reinterpret_cast<f32x4*>(dst) = M[k][u];
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (s + e < z.S) dst[e] = M[k][u][e];
        }
      }
  }
}

// ------------------------------------------------------------------------------------------------------ gate and norm
// out[t][part] = U(y silu(z)) * w, U: divided by the part's own root mean square; a block per (token, part).  VEC: parts of
// a multiple of 4 numbers, every array aligned for four.
template <typename T, bool VEC, int THREADS>
__global__ __launch_bounds__(THREADS) void mamba2_out_kernel(const float* __restrict__ y, const T* __restrict__ proj, int ld,
                                                             const float* __restrict__ w, T* __restrict__ out, int inner,
                                                             int part, float eps) {
  constexpr int V = VEC ? 4 : 1, KEEP = 8;  // pieces a thread keeps in registers
  __shared__ float red[THREADS / 64];
  const size_t t = blockIdx.x;
  const int c0 = blockIdx.y * part;
  const float* yr = y + t * inner + c0;
  const T* zr = proj + t * ld + c0;
  auto gated = [&](int c, float* o) {
    if (VEC) {
      const f32x4 a = load4<float>(yr + c), b = load4<T>(zr + c);
#pragma unroll
      for (int i = 0; i < V; ++i) o[i] = a[i] * (b[i] / (1.0f + expf(-b[i])));
    } else {
      const float b = Num<T>::load(zr + c);
      o[0] = yr[c] * (b / (1.0f + expf(-b)));
    }
  };
  float v[KEEP][V];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + THREADS * k) * V;
    if (c < part) {
      gated(c, v[k]);
#pragma unroll
      for (int i = 0; i < V; ++i) ss = __builtin_fmaf(v[k][i], v[k][i], ss);
    }
  }
  for (int c = (threadIdx.x + THREADS * KEEP) * V; c < part; c += THREADS * V) {  // (what does not fit is formed twice)
    float o[V];
    gated(c, o);
#pragma unroll
    for (int i = 0; i < V; ++i) ss = __builtin_fmaf(o[i], o[i], ss);
  }
  const float inv = 1.0f / sqrtf(block_sum<THREADS>(ss, red) / (float)part + eps);
  auto put = [&](int c, const float* o) {
    T* dst = out + t * inner + c0 + c;
    if (VEC) {
      const f32x4 ww = load4<float>(w + c0 + c);
      if (sizeof(T) == 4) {
        *reinterpret_cast<f32x4*>(dst) = f32x4{o[0] * inv * ww[0], o[V > 1 ? 1 : 0] * inv * ww[1],
                                               o[V > 2 ? 2 : 0] * inv * ww[2], o[V > 3 ? 3 : 0] * inv * ww[3]};
      } else {
        *reinterpret_cast<uint2*>(dst) = uint2{pack_bf16(o[0] * inv * ww[0], o[V > 1 ? 1 : 0] * inv * ww[1]),
                                               pack_bf16(o[V > 2 ? 2 : 0] * inv * ww[2], o[V > 3 ? 3 : 0] * inv * ww[3])};
      }
    } else {
      Num<T>::store(dst, o[0] * inv * w[c0 + c]);
    }
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + THREADS * k) * V;
    if (c < part) put(c, v[k]);
  }
  for (int c = (threadIdx.x + THREADS * KEEP) * V; c < part; c += THREADS * V) {
    float o[V];
    gated(c, o);
    put(c, o);
  }
}

template <typename T>
int launch_scan(const void* proj, const void* rows, const float* dt_bias, const float* a_log, const float* skip,
                const Memory& mem, float* y, const Sizes& z, int R, bool vec, hipStream_t s) {
  const dim3 grid(R, z.H, (z.P + 15) / 16);
#define SCAN(KN)                                                                                                       \
  do {                                                                                                                 \
    if (vec)                                                                                                           \
      hipLaunchKernelGGL((mamba2_scan_kernel<T, KN, true>), grid, dim3(64), 0, s, (const T*)proj, (const T*)rows,      \
                         dt_bias, a_log, skip, mem, y, z);                                                             \
    else                                                                                                               \
      hipLaunchKernelGGL((mamba2_scan_kernel<T, KN, false>), grid, dim3(64), 0, s, (const T*)proj, (const T*)rows,     \
                         dt_bias, a_log, skip, mem, y, z);                                                             \
  } while (0)
  const int need = (z.S + 63) / 64;
  if (need <= 1) SCAN(1);
  else if (need <= 2) SCAN(2);
  else if (need <= 4) SCAN(4);
  else SCAN(8);
#undef SCAN
  JLE_LAUNCH_CHECK();
  return 0;
}

template <int NT, bool VEC>
int launch_chunks(const bf16_t* proj, const bf16_t* rows, const float* dt_bias, const float* a_log, const float* skip,
                  const Memory& mem, float* y, const Sizes& z, int R, hipStream_t s) {
  static bool allowed = false;
  constexpr size_t smem = chunk_lds<NT>();
  if (!allowed) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&mamba2_chunk_kernel<NT, VEC>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    if (e != hipSuccess) return (int)e;
    allowed = true;
  }
  hipLaunchKernelGGL((mamba2_chunk_kernel<NT, VEC>), dim3(R, z.H, (z.P + kChunk - 1) / kChunk), dim3(kChunkThreads), smem, s, proj,
                     rows, dt_bias, a_log, skip, mem, y, z);
  JLE_LAUNCH_CHECK();
  return 0;
}

template <typename T>
int launch_out(const float* y, const void* proj, int ld, const float* w, void* out, int N, int inner, int parts, float eps,
               bool vec, hipStream_t s) {
  const int part = inner / parts;
  const dim3 grid(N, parts);
#define OUT(VEC, TH)                                                                                                  \
  hipLaunchKernelGGL((mamba2_out_kernel<T, VEC, TH>), grid, dim3(TH), 0, s, y, (const T*)proj, ld, w, (T*)out, inner,  \
                     part, eps)
  if (vec) {
    if (part <= 2048) OUT(true, 64);
    else OUT(true, 256);
  } else {
    if (part <= 512) OUT(false, 64);
    else OUT(false, 256);
  }
#undef OUT
  JLE_LAUNCH_CHECK();
  return 0;
}

}  // namespace

JLE_API int jle_mamba2_chunked_supported(int S, int is_bf16) { return is_bf16 && S >= 1 && S <= 256; }

// state: [slots][2][H][P][S] float32; y: float32 [N][H P] scratch; out [N][H P] in the run dtype.  chunked: the kernel
// that goes through segments 64 tokens at a time (see jle_mamba2_chunked_supported), else token after token.
JLE_API int jle_mamba2(const void* proj, int ld, const void* rows, int is_bf16, const float* dt_bias, const float* a_log,
                       const float* skip, const float* norm_w, float* state, const int* cu, const int* slots,
                       const int* phase, float* y, void* out, int N, int R, int H, int P, int S, int G, int norm_groups,
                       float eps, int chunked, hipStream_t s) {
  if (N <= 0 || R <= 0) return 0;
  if (H < 1 || P < 1 || S < 1 || S > 512 || G < 1 || H % G || norm_groups < 1 || (H * P) % norm_groups || H > 65535 ||
      norm_groups > 65535 || (P + 15) / 16 > 65535 || ld < 2 * H * P + 2 * G * S + H)
    return JLE_BAD_ARG;
  if (chunked && !jle_mamba2_chunked_supported(S, is_bf16)) return JLE_BAD_ARG;
  const Sizes z = {H, P, S, G, ld, ld - H};
  const Memory mem = {state, cu, slots, phase};
  const uintptr_t base = (uintptr_t)rows | (uintptr_t)state | (uintptr_t)y;
  int rc;
  if (chunked) {
    const bf16_t *pj = (const bf16_t*)proj, *rw = (const bf16_t*)rows;
    const bool vec = S % 8 == 0 && P % 8 == 0 && base % 16 == 0;  // (then a row's width is a multiple of 8 too)
#define CHUNKS(NT)                                                                            \
  rc = vec ? launch_chunks<NT, true>(pj, rw, dt_bias, a_log, skip, mem, y, z, R, s)           \
           : launch_chunks<NT, false>(pj, rw, dt_bias, a_log, skip, mem, y, z, R, s)
    if (S <= 32) CHUNKS(1);
    else if (S <= 64) CHUNKS(2);
    else if (S <= 128) CHUNKS(4);
    else CHUNKS(8);
#undef CHUNKS
  } else {
    const bool vec = S % 4 == 0 && P % 4 == 0 && base % 16 == 0;
    rc = is_bf16 ? launch_scan<bf16_t>(proj, rows, dt_bias, a_log, skip, mem, y, z, R, vec, s)
                 : launch_scan<float>(proj, rows, dt_bias, a_log, skip, mem, y, z, R, vec, s);
  }
  if (rc) return rc;
  const int inner = H * P;
  const uintptr_t all = (uintptr_t)y | (uintptr_t)proj | (uintptr_t)norm_w | (uintptr_t)out;
  const bool vec = (inner / norm_groups) % 4 == 0 && ld % 4 == 0 && all % 16 == 0;
  return is_bf16 ? launch_out<bf16_t>(y, proj, ld, norm_w, out, N, inner, norm_groups, eps, vec, s)
                 : launch_out<float>(y, proj, ld, norm_w, out, N, inner, norm_groups, eps, vec, s);
}
