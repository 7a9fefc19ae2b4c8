// Pieces shared by the kernels that choose experts and group the choices: data handed between blocks within a launch,
// the choice by scores, and the grouping of (token, choice) pairs by expert.
#pragma once
#include <limits.h>

#include "common.h"

namespace jle {

// A float written to / read from where all compute units of the GPU see it at once (the caches of one die are
// written through and read past): for data that blocks on different dies hand each other within a launch.
__device__ __forceinline__ void put_shared(float* p, float v) {
  __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
__device__ __forceinline__ float get_shared(const float* p) {
  return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}

// What a choice by scores takes.  Scores s: sigmoid of the logit, or (softmax) the softmax over the router's E rows;
// choice scores c = s + correction.  With groups (equal groups of neighbours): a group's score is the sum of its
// `terms` largest c, the `keep` best groups stay.  The top_k largest c among the experts that stay, lowest index first
// among equals.  Weights: the chosen s, divided by their sum plus floor_ if that is not negative, times scale.
struct Choice {
  const float* correction;  // [E] or null
  int E, top_k, groups, keep, terms, softmax;
  float floor_, scale;
};
constexpr int kChoiceMaxE = 4096, kChoiceMaxGroups = 64, kChoiceMaxTop = 64, kChoiceMaxTerms = 4;

static inline bool choice_ok(const Choice& c) {
  return c.E >= 1 && c.E <= kChoiceMaxE && c.top_k >= 1 && c.top_k <= kChoiceMaxTop && c.top_k <= c.E && c.groups >= 0 &&
         c.groups <= kChoiceMaxGroups &&
         (c.groups == 0 || (c.E % c.groups == 0 && c.keep >= 1 && c.keep <= c.groups && c.terms >= 1 &&
                            c.terms <= kChoiceMaxTerms && c.keep * (c.E / c.groups) >= c.top_k));
}

// what a wavefront's lanes wrote to shared memory is there for its other lanes
__device__ __forceinline__ void wave_sees_own_writes() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Over all lanes without a trip through shared memory: within rows of 16 lanes by lane permutations that ride on an
// operand (neighbour, neighbour's neighbour, mirrored half row, mirrored row), then rows and halves swapped.
template <int CTRL>
__device__ __forceinline__ uint32_t permuted(uint32_t v) {
  return (uint32_t)__builtin_amdgcn_mov_dpp((int)v, CTRL, 0xf, 0xf, true);
}
template <typename F>
__device__ __forceinline__ float lanes_reduce(float x, F f) {
  uint32_t u = __float_as_uint(x);
  u = __float_as_uint(f(__uint_as_float(u), __uint_as_float(permuted<0xB1>(u))));
  u = __float_as_uint(f(__uint_as_float(u), __uint_as_float(permuted<0x4E>(u))));
  u = __float_as_uint(f(__uint_as_float(u), __uint_as_float(permuted<0x141>(u))));
  u = __float_as_uint(f(__uint_as_float(u), __uint_as_float(permuted<0x140>(u))));
  auto r = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  u = __float_as_uint(f(__uint_as_float(r[0]), __uint_as_float(r[1])));
  r = __builtin_amdgcn_permlane32_swap(u, u, false, false);
  return f(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float lanes_sum(float x) {
  return lanes_reduce(x, [](float a, float b) { return a + b; });
}
__device__ __forceinline__ float lanes_max(float x) {
  return lanes_reduce(x, [](float a, float b) { return fmaxf(a, b); });
}

// the larger of two (value, index) pairs in all lanes, the lower index among equals; INT_MAX: none
__device__ __forceinline__ void wave_best(float& v, int& at) {
  auto better = [&](float ov, int oa) {
    if (oa != INT_MAX && (at == INT_MAX || ov > v || (ov == v && oa < at))) {
      v = ov;
      at = oa;
    }
  };
  better(__uint_as_float(permuted<0xB1>(__float_as_uint(v))), (int)permuted<0xB1>((uint32_t)at));
  better(__uint_as_float(permuted<0x4E>(__float_as_uint(v))), (int)permuted<0x4E>((uint32_t)at));
  better(__uint_as_float(permuted<0x141>(__float_as_uint(v))), (int)permuted<0x141>((uint32_t)at));
  better(__uint_as_float(permuted<0x140>(__float_as_uint(v))), (int)permuted<0x140>((uint32_t)at));
  {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    const auto b = __builtin_amdgcn_permlane16_swap((uint32_t)at, (uint32_t)at, false, false);
    v = __uint_as_float(a[0]);
    at = (int)b[0];
    better(__uint_as_float(a[1]), (int)b[1]);
  }
  const auto a = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  const auto b = __builtin_amdgcn_permlane32_swap((uint32_t)at, (uint32_t)at, false, false);
  v = __uint_as_float(a[0]);
  at = (int)b[0];
  better(__uint_as_float(a[1]), (int)b[1]);
}

// how many of the lanes 0 .. n - 1 whose bit is set in `open` come before this lane when they are ordered by their
// values, largest first, the lower lane first among equals
__device__ __forceinline__ int lanes_rank(float v, int n, unsigned long long open) {
  const int lane = threadIdx.x & 63;
  int rank = 0;
  for (int i = 0; i < n; ++i) {
    if (!((open >> i) & 1ull)) continue;
    const float o = __uint_as_float((uint32_t)__builtin_amdgcn_readlane((int)__float_as_uint(v), i));
    rank += (o > v || (o == v && i < lane)) ? 1 : 0;
  }
  return rank;
}

// A wavefront chooses for one token.  z: the token's logits; scores, choices: E floats of shared memory each, the
// wavefront's own.  Lane r < top_k returns the r-th choice and its weight.  Lane l looks after the experts l, l + 64,
// ...; the order of every sum depends on the sizes alone.  ACROSS: z was written by other blocks of this launch.
template <bool ACROSS>
__device__ __forceinline__ void choose_by_wave(const float* z, const Choice& a, float* scores, float* choices, int& id,
                                               float& weight) {
  const int lane = threadIdx.x & 63;
  const int E = a.E;
  wave_sees_own_writes();  // (what the wavefront's last token left in shared memory has been read)
  float top = -INFINITY;
  for (int e = lane; e < E; e += 64) {
    const float v = ACROSS ? get_shared(z + e) : z[e];
    scores[e] = v;  // (read back by this lane only)
    top = fmaxf(top, v);
  }
  float inv = 1.0f;
  if (a.softmax) {
    top = lanes_max(top);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) {
      const float p = expf(scores[e] - top);
      scores[e] = p;
      sum += p;
    }
    inv = lanes_sum(sum);
  }
  for (int e = lane; e < E; e += 64) {
    const float s = a.softmax ? scores[e] / inv : 1.0f / (1.0f + expf(-scores[e]));
    scores[e] = s;
    choices[e] = s + (a.correction != nullptr ? a.correction[e] : 0.f);
  }
  wave_sees_own_writes();
  unsigned long long kept = ~0ull;  // bit g: group g's experts can be chosen
  const int per = a.groups > 0 ? E / a.groups : E;
  if (a.groups > 0) {
    float mine = 0.f;
    if (lane < a.groups) {
      float best[kChoiceMaxTerms];
#pragma unroll
      for (int i = 0; i < kChoiceMaxTerms; ++i) best[i] = -INFINITY;
      for (int e = lane * per; e < (lane + 1) * per; ++e) {
        float c = choices[e];
#pragma unroll
        for (int i = 0; i < kChoiceMaxTerms; ++i) {  // (kept in descending order)
          if (i < a.terms && c > best[i]) {
            const float t = best[i];
            best[i] = c;
            c = t;
          }
        }
      }
#pragma unroll
      for (int i = 0; i < kChoiceMaxTerms; ++i)
        if (i < a.terms && i < per) mine += best[i];
    }
    kept = __ballot(lane < a.groups && lanes_rank(mine, a.groups, ~0ull) < a.keep);
  }
  unsigned long long open = 0ull;  // bit j: this lane's expert lane + 64 j can still be chosen
  for (int j = 0, e = lane; e < E; ++j, e += 64)
    if (a.groups == 0 || ((kept >> (e / per)) & 1ull)) open |= 1ull << j;
  id = lane < E ? lane : 0;
  weight = 0.f;
  if (E <= 64) {  // an expert a lane: every lane counts those ahead of it, and leaves its number at its place
    const bool mine = (open & 1ull) != 0ull;
    const float c = lane < E ? choices[lane] : 0.f;
    const float s = lane < E ? scores[lane] : 0.f;
    const int rank = lanes_rank(c, E, __ballot(mine));
    wave_sees_own_writes();  // (the lanes have read their scores)
    int* place = reinterpret_cast<int*>(choices);
    if (lane < a.top_k) place[lane] = lane;  // (what stays there if no order can be told: a number all the same)
    wave_sees_own_writes();
    if (mine && rank < a.top_k) place[rank] = lane;
    wave_sees_own_writes();
    if (lane < a.top_k) id = place[lane];
    weight = __shfl(s, id, 64);
    if (lane >= a.top_k) weight = 0.f;
  }
  for (int r = 0; E > 64 && r < a.top_k; ++r) {
    float v = 0.f;
    int at = INT_MAX;
    for (int j = 0, e = lane; e < E; ++j, e += 64) {
      if (!((open >> j) & 1ull)) continue;
      const float c = choices[e];
      if (at == INT_MAX || c > v) {
        v = c;
        at = e;
      }
    }
    wave_best(v, at);
    if ((at & 63) == lane) open &= ~(1ull << (at >> 6));
    if (lane == r) {
      id = at;
      weight = scores[at];
    }
  }
  if (a.floor_ >= 0.f) {
    const float total = lanes_sum(lane < a.top_k ? weight : 0.f) + a.floor_;
    weight = weight / total;
  }
  weight *= a.scale;
}

// Where the grouping notes a pair's row: inv[n * inv_ld + j] (inv_ld = k, or k + 1 where a token's row in the extra
// group is noted behind its choices' rows).
//
// Stable counting sort of the M = N * k pairs by expert, by one block.
//   offsets[e] .. offsets[e + 1]: rows of expert e in sorted order
//   sorted_token[s]: the token of sorted row s;  sorted_gate[s]: its gate;  inv: sorted row of every pair
// A pair whose expert is E or more (an identity expert) has no row: its inv is -1.
// ids and gates may lie in shared memory; counts[E] and starts[E + 1] do.
// extra > 0: one more group behind the experts' that holds every token once, in order, with gate 1 (offsets[E + 1] =
// offsets[E] + extra): the rows of a shared expert.
__device__ __forceinline__ void extra_group(int base, int* __restrict__ offsets, int* __restrict__ sorted_token,
                                            float* __restrict__ sorted_gate, int* __restrict__ inv, int E, int k,
                                            int extra, int inv_ld) {
  if (extra <= 0) return;
  if (threadIdx.x == 0) offsets[E + 1] = base + extra;
  for (int i = threadIdx.x; i < extra; i += blockDim.x) {
    sorted_token[base + i] = i;
    sorted_gate[base + i] = 1.0f;
    if (inv_ld > k) inv[i * inv_ld + k] = base + i;
  }
}

__device__ __forceinline__ void align_by_block(const int* ids, const float* gates, int* counts, int* starts,
                                               int* __restrict__ offsets, int* __restrict__ sorted_token,
                                               float* __restrict__ sorted_gate, int* __restrict__ inv, int M, int E,
                                               int k, int extra, int inv_ld) {
  for (int e = threadIdx.x; e < E; e += blockDim.x) counts[e] = 0;
  __syncthreads();
  for (int r = threadIdx.x; r < M; r += blockDim.x) {
    const int e = ids[r];
    if (e < E) atomicAdd(&counts[e], 1);
    else inv[(r / k) * inv_ld + r % k] = -1;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int run = 0;
    for (int e = 0; e < E; ++e) {
      starts[e] = run;
      run += counts[e];
    }
    starts[E] = run;
  }
  __syncthreads();
  extra_group(starts[E], offsets, sorted_token, sorted_gate, inv, E, k, extra, inv_ld);
  for (int e = threadIdx.x; e <= E; e += blockDim.x) offsets[e] = starts[e];
  const int lane = threadIdx.x & 63, wave = wave_index(), waves = blockDim.x >> 6;
  for (int e = wave; e < E; e += waves) {
    if (counts[e] == 0) continue;
    int run = starts[e];
    for (int base = 0; base < M; base += 64) {
      const int r = base + lane;
      const bool match = r < M && ids[r] == e;
      const unsigned long long bal = __ballot(match);
      if (match) {
        const int pos = run + __popcll(bal & ((1ull << lane) - 1ull));
        sorted_token[pos] = r / k;
        sorted_gate[pos] = gates[r];
        inv[(r / k) * inv_ld + r % k] = pos;
      }
      run += __popcll(bal);
    }
  }
}

}  // namespace jle
