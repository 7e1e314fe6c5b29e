// Mixture-of-experts bookkeeping around the grouped products of nv_linear:
//   nv_moe_route   : per token the `top` largest router logits (fp32) and the softmax over just those (mode 0), or
//                    the softmax over all experts, the chosen scores divided by (their sum + 1e-20) (mode 1), or
//                    the sigmoid of each chosen logit as it is (mode 2)
//   nv_moe_sort    : (token, choice) pairs ordered by expert -> group offsets, the token behind every sorted row and
//                    the sorted row of every pair
//   nv_moe_plan    : both, in one launch for short steps, with the weight of every sorted row and a shared expert that
//                    every token has as its last choice
//   nv_moe_combine : weighted sum of a token's expert rows (+ a sigmoid-gated shared expert)
// The sum over a token's experts runs in the order of its choices, so it does not depend on what else is in the batch.
#include "anyt.h"

namespace {

// One wavefront routes one token.  Choices come out in descending order, ties go to the lower index: the next choice is
// the best among what comes after the previous one in that order, so nothing has to be marked as taken.
__device__ __forceinline__ void route_token(const float* __restrict__ row, int E, int top, int mode, int32_t* ti, float* tw,
                                            int lane) {
  constexpr int NONE = 0x7fffffff;
  float pv = INFINITY;
  int pe = -1;
  for (int j = 0; j < top; ++j) {
    float bv = -INFINITY;
    int be = NONE;
    for (int e = lane; e < E; e += 64) {
      const float v = row[e];
      if ((v < pv || (v == pv && e > pe)) && (be == NONE || v > bv)) {
        bv = v;
        be = e;
      }
    }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float v2 = __shfl_xor(bv, o, 64);
      const int e2 = __shfl_xor(be, o, 64);
      if (e2 != NONE && (be == NONE || v2 > bv || (v2 == bv && e2 < be))) {
        bv = v2;
        be = e2;
      }
    }
    if (be == NONE) be = j;          // only logits that are no numbers: any expert within range
    if (lane == 0) {
      ti[j] = be;
      tw[j] = bv;
    }
    pv = bv;
    pe = be;
  }
  float all = 0.0f, m = 0.0f;
  if (mode == 1) {
    m = -INFINITY;
    for (int e = lane; e < E; e += 64) m = fmaxf(m, row[e]);
    m = wave_max(m);
    for (int e = lane; e < E; e += 64) all += expf(row[e] - m);
    all = wave_sum(all);
  }
  if (lane != 0) return;
  if (mode == 2) {                   // the sigmoid of each chosen logit, as it is
    for (int j = 0; j < top; ++j) tw[j] = sigmoid_f32(tw[j]);
    return;
  }
  float sum = 0.0f;
  if (mode == 1) {                   // scores of the softmax over every expert, renormalised over the chosen ones
    for (int j = 0; j < top; ++j) {
      tw[j] = expf(tw[j] - m) / all;
      sum += tw[j];
    }
    for (int j = 0; j < top; ++j) tw[j] /= sum + 1e-20f;
    return;
  }
  m = tw[0];
  for (int j = 0; j < top; ++j) {
    tw[j] = expf(tw[j] - m);
    sum += tw[j];
  }
  for (int j = 0; j < top; ++j) tw[j] /= sum;
}

__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, int64_t rs, int E, int top,
                                                        int32_t* __restrict__ idx, float* __restrict__ wt, int64_t T_,
                                                        int mode) {
  const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= T_) return;
  route_token(logits + t * rs, E, top, mode, idx + t * top, wt + t * top, threadIdx.x & 63);
}

struct SortArgs {
  const int32_t* idx;        // [tokens, top]
  const float* wt;           // [tokens, top]
  int64_t tokens;
  int E, top, shared;        // shared 1: every token also has choice `top`, expert E with weight 1
  int32_t* offsets;          // [E + shared + 1]
  int32_t* sorted_token;     // [tokens * (top + shared)]
  float* sorted_weight;      // the same, or null
  int32_t* slot_of;          // [tokens, top + shared]
};

// cnt [E] LDS counts -> starts, and the offsets of the groups; one wavefront scans 64 experts per round
__device__ __forceinline__ void counts_to_starts(int32_t* cnt, const SortArgs& p) {
  if (threadIdx.x >= 64) return;
  const int lane = threadIdx.x;
  int run = 0;
  for (int e0 = 0; e0 < p.E; e0 += 64) {
    const int n = e0 + lane < p.E ? cnt[e0 + lane] : 0;
    int inc = n;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(inc, o, 64);
      if (lane >= o) inc += v;
    }
    if (e0 + lane < p.E) {
      cnt[e0 + lane] = run + inc - n;
      p.offsets[e0 + lane] = run + inc - n;
    }
    run += __shfl(inc, 63, 64);
  }
  if (lane == 0) {
    p.offsets[p.E] = run;
    if (p.shared) p.offsets[p.E + 1] = run + (int32_t)p.tokens;
  }
}

// the (token, choice) pairs go to their expert's next free place; idx may be a copy in LDS
__device__ __forceinline__ void scatter_pairs(int32_t* cnt, const int32_t* idx, const SortArgs& p) {
  const int64_t pairs = p.tokens * p.top;
  const int C = p.top + p.shared;
  for (int64_t i = threadIdx.x; i < pairs; i += blockDim.x) {
    const int slot = atomicAdd(&cnt[idx[i]], 1);
    p.sorted_token[slot] = (int32_t)(i / p.top);
    if (p.sorted_weight) p.sorted_weight[slot] = p.wt[i];
    p.slot_of[i / p.top * C + i % p.top] = slot;
  }
  if (!p.shared) return;
  for (int64_t t = threadIdx.x; t < p.tokens; t += blockDim.x) {
    const int64_t slot = pairs + t;
    p.sorted_token[slot] = (int32_t)t;
    if (p.sorted_weight) p.sorted_weight[slot] = 1.0f;
    p.slot_of[t * C + p.top] = (int32_t)slot;
  }
}

__global__ __launch_bounds__(1024) void moe_sort_kernel(SortArgs p) {
  extern __shared__ int32_t cnt[];   // [E] counts, then cursors
  const int64_t pairs = p.tokens * p.top;
  for (int e = threadIdx.x; e < p.E; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  for (int64_t i = threadIdx.x; i < pairs; i += blockDim.x) atomicAdd(&cnt[p.idx[i]], 1);
  __syncthreads();
  counts_to_starts(cnt, p);
  __syncthreads();
  scatter_pairs(cnt, p.idx, p);
}

// routing and ordering of a short step in one launch: sixteen wavefronts route a token each, then sort together
__global__ __launch_bounds__(1024) void moe_plan_kernel(const float* __restrict__ logits, int64_t rs, int mode, int32_t* idx_out,
                                                        float* wt_out, SortArgs p) {
  extern __shared__ int32_t cnt[];                                   // [E] | choices [tokens * top] | their weights
  int32_t* choice = cnt + p.E;
  const int64_t pairs = p.tokens * p.top;
  float* weight = reinterpret_cast<float*>(choice + pairs);
  for (int e = threadIdx.x; e < p.E; e += blockDim.x) cnt[e] = 0;
  for (int64_t t = threadIdx.x >> 6; t < p.tokens; t += blockDim.x >> 6)
    route_token(logits + t * rs, p.E, p.top, mode, choice + t * p.top, weight + t * p.top, threadIdx.x & 63);
  __syncthreads();
  for (int64_t i = threadIdx.x; i < pairs; i += blockDim.x) {
    atomicAdd(&cnt[choice[i]], 1);
    idx_out[i] = choice[i];
    wt_out[i] = weight[i];
  }
  __syncthreads();
  counts_to_starts(cnt, p);
  __syncthreads();
  p.wt = weight;
  scatter_pairs(cnt, choice, p);
}

__global__ __launch_bounds__(256) void moe_combine_kernel(const float* __restrict__ y, const int32_t* __restrict__ slot_of,
                                                          const float* __restrict__ wt, int top,
                                                          const float* __restrict__ shared, const float* __restrict__ sg,
                                                          int64_t sg_rs, float* __restrict__ out, int width) {
  const int64_t t = blockIdx.x;
  const float gate = !shared ? 0.0f : sg ? sigmoid_f32(sg[t * sg_rs]) : 1.0f;   // no gate logits: a plain addend
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float a = 0.0f;
    for (int j = 0; j < top; ++j) a += wt[t * top + j] * y[(int64_t)slot_of[t * top + j] * width + c];
    if (shared) a += gate * shared[t * width + c];
    out[t * width + c] = a;
  }
}

}  // namespace

extern "C" int nv_moe_route(const float* logits, int64_t row_stride, int32_t* idx, float* weights, int64_t tokens,
                            int experts, int top, int mode, nv_stream_t stream) {
  NV_CHECK_ARG(logits && idx && weights, "nv_moe_route: null pointer");
  NV_CHECK_ARG(mode >= 0 && mode <= 2, "nv_moe_route: bad mode %d", mode);
  NV_CHECK_ARG(tokens >= 0 && experts > 0 && top > 0 && top <= experts, "nv_moe_route: bad shape experts=%d top=%d",
               experts, top);
  if (tokens == 0) return NV_OK;
  moe_route_kernel<<<dim3((unsigned)((tokens + 3) / 4)), dim3(256), 0, (hipStream_t)stream>>>(
      logits, row_stride, experts, top, idx, weights, tokens, mode);
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_moe_sort(const int32_t* idx, int64_t tokens, int experts, int top, int32_t* offsets,
                           int32_t* sorted_token, int32_t* slot_of, nv_stream_t stream) {
  NV_CHECK_ARG(idx && offsets && sorted_token && slot_of, "nv_moe_sort: null pointer");
  NV_CHECK_ARG(tokens >= 0 && experts > 0 && experts <= 8192 && top > 0, "nv_moe_sort: bad shape");
  SortArgs p{idx, nullptr, tokens, experts, top, 0, offsets, sorted_token, nullptr, slot_of};
  moe_sort_kernel<<<dim3(1), dim3(1024), (size_t)experts * sizeof(int32_t), (hipStream_t)stream>>>(p);
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_moe_plan(const float* logits, int64_t row_stride, int64_t tokens, int experts, int top, int mode, int shared,
                           int32_t* idx, float* weights, int32_t* offsets, int32_t* sorted_token, float* sorted_weight,
                           int32_t* slot_of, nv_stream_t stream) {
  NV_CHECK_ARG(logits && idx && weights && offsets && sorted_token && slot_of, "nv_moe_plan: null pointer");
  NV_CHECK_ARG(mode >= 0 && mode <= 2 && (shared == 0 || shared == 1), "nv_moe_plan: bad mode %d / %d", mode, shared);
  NV_CHECK_ARG(tokens >= 0 && tokens * (top + 1) < (1ll << 31) && experts > 0 && experts <= 8192 && top > 0 && top <= experts,
               "nv_moe_plan: bad shape experts=%d top=%d", experts, top);
  if (tokens == 0) return NV_OK;
  hipStream_t s = (hipStream_t)stream;
  SortArgs p{idx, weights, tokens, experts, top, shared, offsets, sorted_token, sorted_weight, slot_of};
  if (tokens <= 64 && tokens * top <= 2048) {
    const size_t lds = (experts + 2 * tokens * top) * sizeof(int32_t);
    moe_plan_kernel<<<dim3(1), dim3(1024), lds, s>>>(logits, row_stride, mode, idx, weights, p);
    NV_CHECK_LAUNCH();
    return NV_OK;
  }
  moe_route_kernel<<<dim3((unsigned)((tokens + 3) / 4)), dim3(256), 0, s>>>(logits, row_stride, experts, top, idx, weights,
                                                                            tokens, mode);
  NV_CHECK_LAUNCH();
  moe_sort_kernel<<<dim3(1), dim3(1024), (size_t)experts * sizeof(int32_t), s>>>(p);
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_moe_combine(const float* y, const int32_t* slot_of, const float* weights, int top, const float* shared,
                              const float* shared_gate, int64_t shared_gate_stride, float* out, int64_t tokens,
                              int width, nv_stream_t stream) {
  NV_CHECK_ARG(y && slot_of && weights && out, "nv_moe_combine: null pointer");
  NV_CHECK_ARG(tokens >= 0 && top > 0 && width > 0, "nv_moe_combine: bad shape");
  if (tokens == 0) return NV_OK;
  moe_combine_kernel<<<dim3((unsigned)tokens), dim3(256), 0, (hipStream_t)stream>>>(y, slot_of, weights, top, shared,
                                                                                   shared_gate, shared_gate_stride, out,
                                                                                   width);
  NV_CHECK_LAUNCH();
  return NV_OK;
}
