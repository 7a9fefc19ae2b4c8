// The choice of experts by scores (see Choice, route.h): a wavefront per token; in steps of few tokens one block chooses
// for all of them and groups the choices by expert in the same launch.  And the experts' activation relu(x)^2,
// element by element.
#include "common.h"
#include "route.h"

using namespace jle;

namespace {

constexpr int kFewTokens = 16;  // up to here one block chooses and groups (with 64 it takes 15 us, two launches 9)

__global__ __launch_bounds__(256) void moe_choose_kernel(const float* __restrict__ logits, Choice a, int* __restrict__ ids,
                                                         float* __restrict__ weights, int N) {
  extern __shared__ float lds[];  // [waves][2 E]
  const int wave = wave_index(), lane = threadIdx.x & 63;
  const int n = blockIdx.x * (blockDim.x >> 6) + wave;
  if (n >= N) return;  // (no barrier below)
  float* scores = lds + (size_t)wave * 2 * a.E;
  int id;
  float weight;
  choose_by_wave<false>(logits + (size_t)n * a.E, a, scores, scores + a.E, id, weight);
  if (lane < a.top_k) {
    ids[(size_t)n * a.top_k + lane] = id;
    weights[(size_t)n * a.top_k + lane] = weight;
  }
}

__global__ __launch_bounds__(1024) void moe_choose_align_kernel(const float* __restrict__ logits, Choice a,
                                                                int* __restrict__ ids, float* __restrict__ weights,
                                                                int* __restrict__ offsets, int* __restrict__ sorted_token,
                                                                float* __restrict__ sorted_weight, int* __restrict__ inv,
                                                                int N, int experts, int extra, int inv_ld) {
  extern __shared__ int smem[];  // counts[experts], starts[experts + 1], ids[N k], weights[N k], [waves][2 E] floats
  const int k = a.top_k, M = N * k;
  int* ids_s = smem + 2 * experts + 1;
  float* weights_s = reinterpret_cast<float*>(ids_s + M);
  const int wave = wave_index(), lane = threadIdx.x & 63;
  float* scores = weights_s + M + (size_t)wave * 2 * a.E;
  for (int n = wave; n < N; n += (int)(blockDim.x >> 6)) {
    int id;
    float weight;
    choose_by_wave<false>(logits + (size_t)n * a.E, a, scores, scores + a.E, id, weight);
    if (lane < k) {
      ids[n * k + lane] = id;
      weights[n * k + lane] = weight;
      ids_s[n * k + lane] = id;
      weights_s[n * k + lane] = weight;
    }
  }
  __syncthreads();
  align_by_block(ids_s, weights_s, smem, smem + experts, offsets, sorted_token, sorted_weight, inv, M, experts, k, extra,
                 inv_ld);
}

template <typename T>
__global__ __launch_bounds__(256) void relu2_kernel(const T* __restrict__ x, T* __restrict__ y, long long count) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= count) return;
  const float v = fmaxf(Num<T>::load(x + i), 0.f);
  Num<T>::store(y + i, v * v);
}

}  // namespace

// groups == 0: no groups; correction null: none; floor_ < 0: the weights are not divided by their sum.  logits float32
// [N, E].  experts > 0 (and few tokens: see jle_moe_choose_groups): also the grouping of the choices among the first
// `experts` of the router's rows, as by jle_moe_align.
JLE_API int jle_moe_choose_groups(int N, int E, int top_k, int experts) {
  const size_t words = (size_t)2 * experts + 1 + (size_t)2 * N * top_k + (size_t)32 * E;
  return N <= kFewTokens && words * sizeof(int) <= 64 * 1024;
}

JLE_API int jle_moe_choose(const float* logits, const float* correction, int* ids, float* weights, int N, int E,
                           int top_k, int groups, int keep, int terms, int softmax, float floor_, float scale, int experts,
                           int* offsets, int* sorted_token, float* sorted_weight, int* inv, int extra_group, int inv_ld,
                           hipStream_t s) {
  if (N <= 0) return 0;
  const Choice a = {correction, E, top_k, groups, keep, terms, softmax, floor_, scale};
  if (logits == nullptr || ids == nullptr || weights == nullptr || !choice_ok(a)) return JLE_BAD_ARG;
  if (experts > 0) {
    if (experts > E || !jle_moe_choose_groups(N, E, top_k, experts) || offsets == nullptr || sorted_token == nullptr ||
        sorted_weight == nullptr || inv == nullptr || inv_ld < top_k || inv_ld > top_k + 1)
      return JLE_BAD_ARG;
    const size_t words = (size_t)2 * experts + 1 + (size_t)2 * N * top_k + (size_t)32 * E;
    hipLaunchKernelGGL(moe_choose_align_kernel, dim3(1), dim3(1024), words * sizeof(int), s, logits, a, ids, weights,
                       offsets, sorted_token, sorted_weight, inv, N, experts, extra_group ? N : 0, inv_ld);
    JLE_LAUNCH_CHECK();
    return 0;
  }
  const int waves = E <= 1024 ? 4 : 1;
  hipLaunchKernelGGL(moe_choose_kernel, dim3((N + waves - 1) / waves), dim3(64 * waves),
                     (size_t)waves * 2 * E * sizeof(float), s, logits, a, ids, weights, N);
  JLE_LAUNCH_CHECK();
  return 0;
}

JLE_API int jle_relu2(const void* x, void* y, int is_bf16, long long count, hipStream_t s) {
  if (count <= 0) return 0;
  if (x == nullptr || y == nullptr || (count + 255) / 256 > 2147483647LL) return JLE_BAD_ARG;
  if (is_bf16)
    hipLaunchKernelGGL(relu2_kernel<bf16_t>, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, s, (const bf16_t*)x,
                       (bf16_t*)y, count);
  else
    hipLaunchKernelGGL(relu2_kernel<float>, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, s, (const float*)x,
                       (float*)y, count);
  JLE_LAUNCH_CHECK();
  return 0;
}
