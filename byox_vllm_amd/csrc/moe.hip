// Mixture-of-experts bookkeeping around the grouped products of nv_linear:
//   nv_moe_route   : per token the `top` largest router logits (fp32) and the softmax over just those (mode 0), or
//                    the softmax over all experts, the chosen scores divided by (their sum + 1e-20) (mode 1), or
//                    the sigmoid of each chosen logit as it is (mode 2), or the softmax over all experts as it is (mode 3)
//   nv_moe_sort    : (token, choice) pairs ordered by expert -> group offsets, the token behind every sorted row and
//                    the sorted row of every pair
//   nv_moe_plan    : both, in one launch for short steps, with the weight of every sorted row and a shared expert that
//                    every token has as its last choice.  Options of the choice (modes 1 - 3): a correction added to the
//                    scores where they are compared, only the best groups of neighbouring experts to choose from, a
//                    factor on the weights, and router outputs behind the experts whose "expert" is the identity: they
//                    take part in everything but own no rows, a token's weights of them are summed instead
//   nv_moe_combine : weighted sum of a token's expert rows (+ a sigmoid-gated shared expert)
// The sum over a token's experts runs in the order of its choices, so it does not depend on what else is in the batch.
#include <type_traits>

#include "anyt.h"

namespace {

constexpr int ROUTE_NONE = 0x7fffffff;

// How a token's experts are chosen and weighed.  ``n`` counts the router's outputs, identity experts included.
struct RouteArgs {
  int n, top, mode;
  const float* correction;   // [n] added to the scores where they are compared (not to the weights), or null
  int groups, keep;          // > 0: n / groups neighbours form a group; only the `keep` groups with the best member count
  float scale;               // factor on the weights
  // the choice compares scores and not plain logits
  __host__ __device__ bool scored() const { return correction != nullptr || groups > 0; }
  // numbers of LDS per token at work: what is compared, then best members of the groups, each padded to whole 16 bytes
  __host__ __device__ int n4() const { return (n + 3) & ~3; }
  __host__ __device__ int lds_words() const { return n <= 128 || scored() ? n4() + ((groups + 3) & ~3) : 0; }
};

// The best of v[0 .. n) that comes after (pv, pe) in descending order, ties to the lower index: taking one after the
// other this way, nothing has to be marked as taken.  Every lane of the wavefront gets the result.
__device__ __forceinline__ void next_best(const float* v, int n, int lane, float pv, int pe, float& bv, int& be) {
  bv = -INFINITY;
  be = ROUTE_NONE;
  for (int e = lane; e < n; e += 64) {
    const float x = v[e];
    if ((x < pv || (x == pv && e > pe)) && (be == ROUTE_NONE || x > bv)) {
      bv = x;
      be = e;
    }
  }
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float v2 = __shfl_xor(bv, o, 64);
    const int e2 = __shfl_xor(be, o, 64);
    if (e2 != ROUTE_NONE && (be == ROUTE_NONE || v2 > bv || (v2 == bv && e2 < be))) {
      bv = v2;
      be = e2;
    }
  }
}

// LDS written by one lane and read by another of the same wavefront
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// At most ROUTE_RANKED outputs: a lane owns one of them (of more than 64: two) and counts how many come before its own in
// descending order (ties: the lower index first), which is the place of its choice; nothing is searched for step by step.
// LP lanes serve a token, 64 / LP tokens share a wavefront (LP 128: 64 lanes with two outputs each).  ``lds``: p.lds_words()
// numbers of this token.  What is no number is compared as -inf, so the places are always a permutation.  Every lane of the
// wavefront takes part; with live == false nothing is read or written.
constexpr int ROUTE_RANKED = 128;

// how many of v[0 .. n) come before (x, at) in descending order; v is padded with -inf to whole 16 bytes
__device__ __forceinline__ int count_before(const float* v, int n, float x, int at) {
  int before = 0;
#pragma unroll 2
  for (int o = 0; o < n; o += 4) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(v + o);
#pragma unroll
    for (int i = 0; i < 4; ++i) before += (a[i] > x || (a[i] == x && o + i < at)) ? 1 : 0;
  }
  return before;
}

template <int LP> __device__ __forceinline__ float token_sum(float v) {
  float a, b;
  v = lanes_sum<16>(v);
  if constexpr (LP >= 32) {
    rows_pair16(v, a, b);
    v = a + b;
  }
  if constexpr (LP >= 64) {
    rows_pair32(v, a, b);
    v = a + b;
  }
  return v;
}
template <int LP> __device__ __forceinline__ float token_max(float v) {
  float a, b;
  v = lanes_max<16>(v);
  if constexpr (LP >= 32) {
    rows_pair16(v, a, b);
    v = fmaxf(a, b);
  }
  if constexpr (LP >= 64) {
    rows_pair32(v, a, b);
    v = fmaxf(a, b);
  }
  return v;
}

template <int LP>
__device__ __forceinline__ void route_token_ranked(const float* __restrict__ row, bool live, const RouteArgs& p, int32_t* ti,
                                                   float* tw, float* lds, int lane) {
  constexpr int W = LP < 64 ? LP : 64, NV = LP / W;
  const int n = p.n, top = p.top, mode = p.mode;
  float z[NV], s[NV], c[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    z[i] = live && lane + W * i < n ? row[lane + W * i] : -INFINITY;
    if (z[i] != z[i]) z[i] = -INFINITY;
  }
  float all = 1.0f;
  if (mode == 2) {
#pragma unroll
    for (int i = 0; i < NV; ++i) s[i] = sigmoid_f32(z[i]);
  } else {
    float m = z[0];
    if constexpr (NV == 2) m = fmaxf(z[0], z[1]);
    m = token_max<LP>(m);
    float sum = 0.0f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      s[i] = lane + W * i < n ? expf(z[i] - m) : 0.0f;
      sum += s[i];
    }
    if (mode != 0) {
      all = 1.0f / token_sum<LP>(sum);
#pragma unroll
      for (int i = 0; i < NV; ++i) s[i] *= all;
    }
  }
  const bool scored = p.scored();
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = lane + W * i;
    c[i] = z[i];
    if (scored) {
      c[i] = s[i] + (p.correction && e < n ? p.correction[e] : 0.0f);
      if (e >= n || c[i] != c[i]) c[i] = -INFINITY;
    }
    if (live && e < p.n4()) lds[e] = c[i];
  }
  wave_lds_fence();
  if (p.groups > 0 && p.keep < p.groups) {
    float* best = lds + p.n4();        // [groups] best member of each group
    const int size = n / p.groups;
    for (int g = lane; live && g < ((p.groups + 3) & ~3); g += W) {
      float b = -INFINITY;
      if (g < p.groups) {
#pragma unroll 4
        for (int e = g * size; e < (g + 1) * size; ++e) b = fmaxf(b, lds[e]);
      }
      best[g] = b;
    }
    wave_lds_fence();
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = lane + W * i;
      if (!live || e >= n) continue;
      const int g = e / size;
      if (count_before(best, p.groups, best[g], g) >= p.keep) {
        c[i] = -INFINITY;
        lds[e] = c[i];
      }
    }
    wave_lds_fence();
  }
  float chosen = 0.0f;
  int rank[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    rank[i] = live && lane + W * i < n ? count_before(lds, n, c[i], lane + W * i) : top;
    if (rank[i] < top) chosen += s[i];
  }
  float factor = p.scale;
  if (mode <= 1) factor /= token_sum<LP>(chosen) + (mode == 1 ? 1e-20f : 0.0f);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    if (rank[i] >= top) continue;
    ti[rank[i]] = lane + W * i;
    tw[rank[i]] = s[i] * factor;
  }
  wave_lds_fence();                    // the next token's scores take this one's place
}

// Any number of outputs: one wavefront routes one token, one choice after the other in descending order.  ``lds``:
// p.lds_words() numbers of this wavefront.
__device__ __forceinline__ void route_token(const float* __restrict__ row, const RouteArgs& p, int32_t* ti, float* tw,
                                            float* lds, int lane) {
  const int n = p.n, top = p.top, mode = p.mode;
  float all = 0.0f, m = 0.0f;
  if (mode == 1 || mode == 3) {
    m = -INFINITY;
    for (int e = lane; e < n; e += 64) m = fmaxf(m, row[e]);
    m = wave_max(m);
    for (int e = lane; e < n; e += 64) all += expf(row[e] - m);
    all = wave_sum(all);
  }
  const float* compare = row;
  const bool scored = p.scored();
  if (scored) {
    float* best = lds + p.n4();      // [groups] best member of each group
    for (int e = lane; e < n; e += 64) {
      const float s = mode == 2 ? sigmoid_f32(row[e]) : expf(row[e] - m) / all;
      lds[e] = s + (p.correction ? p.correction[e] : 0.0f);
    }
    wave_lds_fence();
    if (p.groups > 0 && p.keep < p.groups) {
      const int size = n / p.groups;
      for (int g = lane; g < p.groups; g += 64) {
        float b = -INFINITY;
        for (int e = g * size; e < (g + 1) * size; ++e) b = fmaxf(b, lds[e]);
        best[g] = b;
      }
      wave_lds_fence();
      float pv = INFINITY;
      int pe = -1;
      for (int j = 0; j < p.keep; ++j) {
        float bv;
        int be;
        next_best(best, p.groups, lane, pv, pe, bv, be);
        if (be == ROUTE_NONE) break;
        pv = bv;
        pe = be;
      }
      // (pv, pe) is the last group kept
      for (int e = lane; e < n; e += 64) {
        const int g = e / size;
        if (best[g] < pv || (best[g] == pv && g > pe)) lds[e] = -INFINITY;
      }
      wave_lds_fence();
    }
    compare = lds;
  }
  float pv = INFINITY;
  int pe = -1;
  for (int j = 0; j < top; ++j) {
    float bv;
    int be;
    next_best(compare, n, lane, pv, pe, bv, be);
    if (be == ROUTE_NONE) be = j;    // only logits that are no numbers: any expert within range
    if (lane == 0) {
      ti[j] = be;
      tw[j] = scored ? row[be] : bv;
    }
    pv = bv;
    pe = be;
  }
  if (scored) wave_lds_fence();      // the next token's scores take this one's place
  if (lane != 0) return;
  if (mode == 2) {                   // the sigmoid of each chosen logit, as it is
    for (int j = 0; j < top; ++j) tw[j] = sigmoid_f32(tw[j]) * p.scale;
    return;
  }
  if (mode == 3) {                   // scores of the softmax over every expert, as they are
    for (int j = 0; j < top; ++j) tw[j] = expf(tw[j] - m) / all * p.scale;
    return;
  }
  float sum = 0.0f;
  if (mode == 1) {                   // scores of the softmax over every expert, renormalised over the chosen ones
    for (int j = 0; j < top; ++j) {
      tw[j] = expf(tw[j] - m) / all;
      sum += tw[j];
    }
    for (int j = 0; j < top; ++j) tw[j] = tw[j] / (sum + 1e-20f) * p.scale;
    return;
  }
  m = tw[0];
  for (int j = 0; j < top; ++j) {
    tw[j] = expf(tw[j] - m);
    sum += tw[j];
  }
  for (int j = 0; j < top; ++j) tw[j] = tw[j] / sum * p.scale;
}

// the wavefront's tokens t0 .. t0 + tokens_per_wave<LP>() - 1; LP 0: by search
template <int LP> __host__ __device__ constexpr int tokens_per_wave() { return LP > 0 && LP < 64 ? 64 / LP : 1; }

template <int LP>
__device__ __forceinline__ void route_wave(const float* logits, int64_t rs, int64_t t0, int64_t tokens, const RouteArgs& p,
                                           int32_t* ti, float* tw, float* lds, int lane) {
  if constexpr (LP == 0) {
    route_token(logits + t0 * rs, p, ti + t0 * p.top, tw + t0 * p.top, lds, lane);
  } else {
    constexpr int W = LP < 64 ? LP : 64;
    const int64_t t = t0 + lane / W;
    route_token_ranked<LP>(logits + t * rs, t < tokens, p, ti + t * p.top, tw + t * p.top, lds + lane / W * p.lds_words(), lane % W);
  }
}

template <int LP>
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, int64_t rs,
                                                        int32_t* __restrict__ idx, float* __restrict__ wt, int64_t T_,
                                                        RouteArgs p) {
  extern __shared__ float4 lds4[];                                   // p.lds_words() per token
  constexpr int TW = tokens_per_wave<LP>();
  const int wv = threadIdx.x >> 6;
  const int64_t t = ((int64_t)blockIdx.x * 4 + wv) * TW;
  if (t >= T_) return;
  route_wave<LP>(logits, rs, t, T_, p, idx, wt, reinterpret_cast<float*>(lds4) + wv * TW * p.lds_words(), threadIdx.x & 63);
}

struct SortArgs {
  const int32_t* idx;        // [tokens, top]
  const float* wt;           // [tokens, top]
  int64_t tokens;
  int E, top, shared;        // shared 1: every token also has choice `top`, expert E with weight 1
  float* self_weight;        // [tokens] sum of the weights of choices >= E (identity experts: no rows, slot -1), or null
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
  const int tokens = (int)p.tokens, pairs = tokens * p.top;        // fit 32 bits, checked by the launcher
  const int C = p.top + p.shared;
  if (p.self_weight) {
    for (int t = threadIdx.x; t < tokens; t += blockDim.x) {
      float w = 0.0f;
      for (int j = 0; j < p.top; ++j)
        if (idx[t * p.top + j] >= p.E) w += p.wt[t * p.top + j];
      p.self_weight[t] = w;
    }
  }
  constexpr int AHEAD = 8;             // pairs of a thread whose loads, then counters, are on their way together
  for (int base = threadIdx.x; base < pairs; base += AHEAD * blockDim.x) {
    int e[AHEAD], slot[AHEAD];
    float w[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const int i = base + k * blockDim.x;
      e[k] = i < pairs ? idx[i] : p.E;
      w[k] = i < pairs && p.sorted_weight ? p.wt[i] : 0.0f;
    }
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) slot[k] = e[k] < p.E ? atomicAdd(&cnt[e[k]], 1) : -1;
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const int i = base + k * blockDim.x, t = i / p.top;
      if (i >= pairs) break;
      p.slot_of[t * C + (i - t * p.top)] = slot[k];
      if (slot[k] < 0) continue;
      p.sorted_token[slot[k]] = t;
      if (p.sorted_weight) p.sorted_weight[slot[k]] = w[k];
    }
  }
  if (!p.shared) return;
  const int routed = p.offsets[p.E];                 // written before the barrier ahead of this call
  for (int t = threadIdx.x; t < tokens; t += blockDim.x) {
    const int slot = routed + t;
    p.sorted_token[slot] = t;
    if (p.sorted_weight) p.sorted_weight[slot] = 1.0f;
    p.slot_of[t * C + p.top] = slot;
  }
}

__global__ __launch_bounds__(1024) void moe_sort_kernel(SortArgs p) {
  extern __shared__ int32_t cnt[];   // [E] counts, then cursors
  const int pairs = (int)(p.tokens * p.top);
  for (int e = threadIdx.x; e < p.E; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  for (int base = threadIdx.x; base < pairs; base += 8 * blockDim.x) {
    int e[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) e[k] = base + k * blockDim.x < pairs ? p.idx[base + k * blockDim.x] : p.E;
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (e[k] < p.E) atomicAdd(&cnt[e[k]], 1);
  }
  __syncthreads();
  counts_to_starts(cnt, p);
  __syncthreads();
  scatter_pairs(cnt, p.idx, p);
}

// routing and ordering of a short step in one launch: sixteen wavefronts route the tokens, then sort together
template <int LP>
__global__ __launch_bounds__(1024) void moe_plan_kernel(const float* __restrict__ logits, int64_t rs, int32_t* idx_out,
                                                        float* wt_out, SortArgs p, RouteArgs r) {
  constexpr int TW = tokens_per_wave<LP>();
  extern __shared__ float4 lds4[];                  // 16 x TW x r.lds_words() | [E] | choices [tokens * top] | their weights
  const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
  float* scores = reinterpret_cast<float*>(lds4) + wv * TW * r.lds_words();
  int32_t* cnt = reinterpret_cast<int32_t*>(lds4) + 16 * TW * r.lds_words();
  int32_t* choice = cnt + p.E;
  const int tokens = (int)p.tokens, pairs = tokens * p.top;
  float* weight = reinterpret_cast<float*>(choice + pairs);
  for (int e = threadIdx.x; e < p.E; e += blockDim.x) cnt[e] = 0;
#pragma unroll 1
  for (int t = wv * TW; t < tokens; t += 16 * TW) route_wave<LP>(logits, rs, t, tokens, r, choice, weight, scores, lane);
  __syncthreads();
  for (int i = threadIdx.x; i < pairs; i += blockDim.x) {
    if (choice[i] < p.E) atomicAdd(&cnt[choice[i]], 1);
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
    for (int j = 0; j < top; ++j) {
      const int slot = slot_of[t * top + j];
      if (slot >= 0) a += wt[t * top + j] * y[(int64_t)slot * width + c];
    }
    if (shared) a += gate * shared[t * width + c];
    out[t * width + c] = a;
  }
}

// the kernels' lanes per token for n outputs
template <typename F>
void with_lanes(int n, F f) {
  if (n <= 16) f(std::integral_constant<int, 16>());
  else if (n <= 32) f(std::integral_constant<int, 32>());
  else if (n <= 64) f(std::integral_constant<int, 64>());
  else if (n <= ROUTE_RANKED) f(std::integral_constant<int, 128>());
  else f(std::integral_constant<int, 0>());
}

void launch_route(const float* logits, int64_t rs, int32_t* idx, float* weights, int64_t tokens, const RouteArgs& r, hipStream_t s) {
  with_lanes(r.n, [&](auto lp) {
    constexpr int LP = decltype(lp)::value, per = 4 * tokens_per_wave<LP>();
    moe_route_kernel<LP><<<dim3((unsigned)((tokens + per - 1) / per)), dim3(256), per * r.lds_words() * sizeof(float), s>>>(
        logits, rs, idx, weights, tokens, r);
  });
}

}  // namespace

extern "C" int nv_moe_route(const float* logits, int64_t row_stride, int32_t* idx, float* weights, int64_t tokens,
                            int experts, int top, int mode, nv_stream_t stream) {
  NV_CHECK_ARG(logits && idx && weights, "nv_moe_route: null pointer");
  NV_CHECK_ARG(mode >= 0 && mode <= 3, "nv_moe_route: bad mode %d", mode);
  NV_CHECK_ARG(tokens >= 0 && experts > 0 && top > 0 && top <= experts, "nv_moe_route: bad shape experts=%d top=%d",
               experts, top);
  if (tokens == 0) return NV_OK;
  const RouteArgs r{experts, top, mode, nullptr, 0, 0, 1.0f};
  launch_route(logits, row_stride, idx, weights, tokens, r, (hipStream_t)stream);
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_moe_sort(const int32_t* idx, int64_t tokens, int experts, int top, int32_t* offsets,
                           int32_t* sorted_token, int32_t* slot_of, nv_stream_t stream) {
  NV_CHECK_ARG(idx && offsets && sorted_token && slot_of, "nv_moe_sort: null pointer");
  NV_CHECK_ARG(tokens >= 0 && experts > 0 && experts <= 8192 && top > 0 && tokens * (top + 1) < (1ll << 31),
               "nv_moe_sort: bad shape");
  SortArgs p{idx, nullptr, tokens, experts, top, 0, nullptr, offsets, sorted_token, nullptr, slot_of};
  moe_sort_kernel<<<dim3(1), dim3(1024), (size_t)experts * sizeof(int32_t), (hipStream_t)stream>>>(p);
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_moe_plan(const float* logits, int64_t row_stride, int64_t tokens, int experts, int top, int mode, int shared,
                           int identity, const float* correction, int groups, int keep_groups, float scale, int32_t* idx,
                           float* weights, int32_t* offsets, int32_t* sorted_token, float* sorted_weight, int32_t* slot_of,
                           float* self_weight, nv_stream_t stream) {
  NV_CHECK_ARG(logits && idx && weights && offsets && sorted_token && slot_of, "nv_moe_plan: null pointer");
  NV_CHECK_ARG(mode >= 0 && mode <= 3 && (shared == 0 || shared == 1), "nv_moe_plan: bad mode %d / %d", mode, shared);
  NV_CHECK_ARG(tokens >= 0 && tokens * (top + 1) < (1ll << 31) && experts > 0 && identity >= 0 && experts + identity <= 8192 &&
                   top > 0 && top <= experts + identity,
               "nv_moe_plan: bad shape experts=%d identity=%d top=%d", experts, identity, top);
  NV_CHECK_ARG((identity == 0) == (self_weight == nullptr), "nv_moe_plan: identity experts need self_weight");
  const RouteArgs r{experts + identity, top, mode, correction, groups, keep_groups, scale};
  NV_CHECK_ARG(!r.scored() || mode != 0, "nv_moe_plan: mode 0 has no scores to correct or group");
  NV_CHECK_ARG(groups >= 0 && (groups == 0 || (r.n % groups == 0 && keep_groups > 0 && keep_groups <= groups &&
                                               keep_groups * (r.n / groups) >= top)),
               "nv_moe_plan: bad groups %d / %d", groups, keep_groups);
  if (tokens == 0) return NV_OK;
  hipStream_t s = (hipStream_t)stream;
  SortArgs p{idx, weights, tokens, experts, top, shared, self_weight, offsets, sorted_token, sorted_weight, slot_of};
  const size_t scores = (size_t)r.lds_words() * sizeof(float);      // per token that a wavefront works on
  bool done = false;
  if (tokens <= 64 && tokens * top <= 2048) {
    with_lanes(r.n, [&](auto lp) {
      constexpr int LP = decltype(lp)::value;
      const size_t lds = (experts + 2 * tokens * top) * sizeof(int32_t) + 16 * tokens_per_wave<LP>() * scores;
      if (lds > 64 * 1024) return;
      moe_plan_kernel<LP><<<dim3(1), dim3(1024), lds, s>>>(logits, row_stride, idx, weights, p, r);
      done = true;
    });
  }
  if (done) {
    NV_CHECK_LAUNCH();
    return NV_OK;
  }
  NV_CHECK_ARG(4 * scores <= 64 * 1024, "nv_moe_plan: the scores of %d outputs exceed the LDS", r.n);
  launch_route(logits, row_stride, idx, weights, tokens, r, s);
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
