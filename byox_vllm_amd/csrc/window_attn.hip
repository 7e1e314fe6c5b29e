// Softmax attention over a paged cache with grouped key/value heads, key and value sizes that may differ, and a score
// that is shaped before the softmax:
//     s_ij = cap(q_i . k_j) - slope_h (i - j),   cap(z) = c tanh(z / c) (or z without a cap),
// over the keys 0 <= i - j < window (window 0: every earlier key).  q arrives already normalised and multiplied by its
// scale and per-head temperature (qk_norm_store below), so the kernel's own arithmetic is the dot product, the cap,
// the distance term and the softmax, all in fp32.  Options of a design: no distance term; a sink, one learned logit per
// query head that joins the softmax's denominator without a key or a value; kept first keys, which every later query sees
// beside its window (0 <= i - j < window or j < keep_first); values that ARE the keys (rows [k: G * d]
// only, read twice); a sigmoid output gate from fp32 logits laid out like the output, or one logit per head; chunks, in
// which a query sees the keys j <= i of its own chunk only (floor(i / chunk) == floor(j / chunk), counted from the
// sequence's first position).
//
// qk_norm_store: per token, RMS norm over each query and key head (one weight vector shared by the heads), the query
// scaled by scale * temp[h] and left in fp32, the normalised key and the value written to the token's cache row
// [k: G * d | v: G * dv] in the storage type.  The norms may be absent (null weights: the projection as it is), and
// the query may carry a temperature that grows with the position p: 1 + coef * ln(floor((p + 1) / every) + 1).
// Further options: one root mean square over all heads of q (and of k) with a weight per number; a rotation of the first
// rot_dims numbers of every head after the norm (dimension i with i + rot_dims / 2, or interleaved 2i with 2i + 1, angle
// position * inv_freq[i]); values
// blended with another layer's values of the same token, v <- (1 - lam) v + lam v_first, before they are stored.
//
// qk_pairs_store_kernel: the same where a number depends on itself and its neighbour only.
//
// qk_conv_store_kernel: the same behind a short causal convolution over time on every channel of q, k and v.
//
// window_attn_kernel: a workgroup owns TQ consecutive tokens of the packed batch and one key/value head, i.e. up to
// TQ * (H / G) query rows that read the same keys; tokens of different requests inside the tile are served one request
// after the other.  Keys go through LDS in tiles of TK rows; online softmax per row.
#include "anyt.h"

namespace {

struct QkArgs {
  const float* proj;      // [tokens, proj_rs]: q | k | v at the given column offsets (fp32 projections)
  const void* bias;       // [proj columns] added to the projections (same column offsets), or null
  int64_t proj_rs;
  int q_off, k_off, v_off;
  const void* qn;         // query norm weight: [d] shared by the heads, or [H * d] when norm_whole
  const void* kn;         // [d] or [G * d]
  const void* temp;       // [H] or null
  const int64_t* positions;   // [tokens], read when temp_every > 0 or rot_dims > 0
  float temp_coef;
  int temp_every;         // 0: no position temperature
  const int32_t* slot_mapping;   // [tokens] cache row of each token, -1: none
  void* cache;            // [rows, G * (d + dv)]
  float* q_out;           // [tokens, H * d]
  int H, G, d, dv;
  float scale, eps;
  int norm_whole;         // 1: one root mean square over all H * d query numbers (and over all G * d key numbers);
                          // 2: one per head, without weights
  const float* inv_freq;  // [rot_dims / 2] rotation frequencies, read when rot_dims > 0
  int rot_dims;           // the first rot_dims numbers of every head are rotated, dimension i with i + rot_dims / 2
  float mscale;           // multiplies cosine and sine
  const float* v_first;   // [tokens, v_first_rs] values to blend in, or null
  int64_t v_first_rs;
  const void* vmix;       // one number lam: v <- (1 - lam) v + lam v_first
  int interleaved;        // 1: dimension 2i is rotated with 2i + 1 instead of i with i + rot_dims / 2
};

template <typename T>
__global__ __launch_bounds__(256) void qk_norm_store_kernel(QkArgs p) {
  __shared__ float red[32];
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const float* row = p.proj + t * p.proj_rs;
  const int64_t slot = p.slot_mapping[t];
  const int cw = p.G * (p.d + p.dv);       // dv 0: the values are the keys, rows hold keys only
  T* crow = slot >= 0 ? reinterpret_cast<T*>(p.cache) + slot * cw : nullptr;
  float pos_temp = 1.0f;
  if (p.temp_every > 0) pos_temp = 1.0f + p.temp_coef * logf((float)((p.positions[t] + 1) / p.temp_every) + 1.0f);
  const T* qn = reinterpret_cast<const T*>(p.qn);
  const T* kn = reinterpret_cast<const T*>(p.kn);
  const T* temp = reinterpret_cast<const T*>(p.temp);
  const T* bias = reinterpret_cast<const T*>(p.bias);
  const int half = p.rot_dims / 2;
  const float pos = p.rot_dims > 0 ? (float)p.positions[t] : 0.0f;
  // cosine and sine of the token's angles once for all heads (rotations over more than 256 numbers evaluate them in place)
  __shared__ float s_cs[128], s_sn[128];
  const bool trig_shared = half > 0 && half <= 128;
  if (trig_shared) {
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
      const float a = pos * p.inv_freq[i];
      s_cs[i] = cosf(a) * p.mscale;
      s_sn[i] = sinf(a) * p.mscale;
    }
    __syncthreads();
  }
  float inv_q = 1.0f, inv_k = 1.0f;
  if (qn && p.norm_whole == 1) {
    float sq = 0.0f, sk = 0.0f;
    for (int e = threadIdx.x; e < p.H * p.d; e += blockDim.x) {
      const float x = row[p.q_off + e] + (bias ? ld_f32<T>(bias + p.q_off + e) : 0.0f);
      sq += x * x;
    }
    for (int e = threadIdx.x; e < p.G * p.d; e += blockDim.x) {
      const float x = row[p.k_off + e] + (bias ? ld_f32<T>(bias + p.k_off + e) : 0.0f);
      sk += x * x;
    }
    inv_q = 1.0f / sqrtf(block_sum(sq, red) / (float)(p.H * p.d) + p.eps);
    inv_k = 1.0f / sqrtf(block_sum(sk, red) / (float)(p.G * p.d) + p.eps);
  }
  for (int v = wv; v < p.H + p.G; v += nw) {
    const bool is_q = v < p.H;
    const int hv = is_q ? v : v - p.H;
    const int col = is_q ? p.q_off + hv * p.d : p.k_off + hv * p.d;
    const float* src = row + col;
    float inv = is_q ? inv_q : inv_k;
    if (p.norm_whole == 2 || (qn && p.norm_whole == 0)) {
      float ss = 0.0f;
      for (int e = lane; e < p.d; e += 64) {
        const float x = src[e] + (bias ? ld_f32<T>(bias + col + e) : 0.0f);
        ss += x * x;
      }
      ss = wave_sum(ss);
      inv = 1.0f / sqrtf(ss / (float)p.d + p.eps);
    }
    const T* nw_ = is_q ? qn : kn;
    if (nw_ && p.norm_whole == 1) nw_ += hv * p.d;
    auto normed = [&](int e) {
      const float x = src[e] + (bias ? ld_f32<T>(bias + col + e) : 0.0f);
      return x * inv * (nw_ ? ld_f32<T>(nw_ + e) : 1.0f);
    };
    auto value = [&](int e) {      // normalised, then rotated
      float x = normed(e);
      if (e < p.rot_dims) {
        const bool first = p.interleaved ? !(e & 1) : e < half;
        const int fi = p.interleaved ? e >> 1 : first ? e : e - half;
        float cs, sn;
        if (trig_shared) {
          cs = s_cs[fi];
          sn = s_sn[fi];
        } else {
          const float a = pos * p.inv_freq[fi];
          cs = cosf(a) * p.mscale;
          sn = sinf(a) * p.mscale;
        }
        const int pair = p.interleaved ? e ^ 1 : first ? e + half : e - half;
        const float other = normed(pair);
        x = first ? x * cs - other * sn : x * cs + other * sn;
      }
      return x;
    };
    if (is_q) {
      const float f = p.scale * (temp ? ld_f32<T>(temp + v) : 1.0f) * pos_temp;
      for (int e = lane; e < p.d; e += 64) p.q_out[t * p.H * p.d + v * p.d + e] = value(e) * f;
    } else if (crow) {
      for (int e = lane; e < p.d; e += 64) st_f32<T>(crow + hv * p.d + e, value(e));
    }
  }
  if (crow && p.dv > 0) {
    const float lam = p.v_first ? ld_f32<T>(reinterpret_cast<const T*>(p.vmix)) : 0.0f;
    for (int e = threadIdx.x; e < p.G * p.dv; e += blockDim.x) {
      float x = row[p.v_off + e] + (bias ? ld_f32<T>(bias + p.v_off + e) : 0.0f);
      if (p.v_first) x = (1.0f - lam) * x + lam * p.v_first[t * p.v_first_rs + e];
      st_f32<T>(crow + p.G * p.d + e, x);
    }
  }
}

// The case without norms, temperatures, biases and blended values whose rotation (if any) is interleaved: every output
// depends on a pair of neighbouring inputs, so a thread takes four consecutive numbers of q | k | v per access.
template <typename T>
__global__ __launch_bounds__(256) void qk_pairs_store_kernel(QkArgs p) {
  typedef typename Pack4<T>::type P;
  __shared__ float s_cs[128], s_sn[128];
  const int64_t t = blockIdx.x;
  const float* row = p.proj + t * p.proj_rs;
  const int64_t slot = p.slot_mapping[t];
  const int nq = p.H * p.d, nk = p.G * p.d, nv = p.G * p.dv, half = p.rot_dims / 2;
  T* crow = slot >= 0 ? reinterpret_cast<T*>(p.cache) + slot * (nk + nv) : nullptr;
  if (half > 0) {
    const float pos = (float)p.positions[t];
    for (int i = threadIdx.x; i < half; i += 256) {
      const float a = pos * p.inv_freq[i];
      s_cs[i] = cosf(a) * p.mscale;
      s_sn[i] = sinf(a) * p.mscale;
    }
    __syncthreads();
  }
  for (int c = threadIdx.x * 4; c < nq + nk + nv; c += 1024) {
    const bool is_q = c < nq, is_v = c >= nq + nk;
    const int rel = is_q ? c : is_v ? c - nq - nk : c - nq;
    f32x4 x = *reinterpret_cast<const f32x4*>(row + (is_q ? p.q_off : is_v ? p.v_off : p.k_off) + rel);
    if (!is_v) {
      const int e = rel % p.d;
#pragma unroll
      for (int j = 0; j < 4; j += 2) {
        if (e + j < p.rot_dims) {
          const float cs = s_cs[(e + j) >> 1], sn = s_sn[(e + j) >> 1], u = x[j], v = x[j + 1];
          x[j] = u * cs - v * sn;
          x[j + 1] = v * cs + u * sn;
        }
      }
    }
    if (is_q) {
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] *= p.scale;
      *reinterpret_cast<f32x4*>(p.q_out + t * nq + rel) = x;
    } else if (crow) {
      *reinterpret_cast<P*>(crow + (is_v ? nk : 0) + rel) = Pack4<T>::narrow(x);
    }
  }
}

// A short causal convolution per channel of q | k | v, y_t = sum_j w[c][j] x_(t - taps + 1 + j) with zeros ahead of the
// sequence, then (optionally) every query and key head divided by its root mean square, then query scale and page store.
// The last taps - 1 inputs of a request are its state.
struct QkConvArgs {
  const float* proj;      // [tokens, proj_rs]: q | k | v at the column offsets
  int64_t proj_rs;
  int q_off, k_off, v_off;
  const void* w;          // [H d + G d + G dv, taps] in the storage type
  int taps;
  float* state;           // [slots, taps - 1, H d + G d + G dv]
  const int32_t* cu_q;    // [B + 1]
  const int32_t* past;    // [B]
  const int32_t* slots;   // [B]
  const int32_t* seq_of;  // [tokens]
  const int32_t* slot_mapping;   // [tokens] cache row or -1
  void* cache;            // [rows, G (d + dv)]
  float* q_out;           // [tokens, H d]
  int64_t tokens;
  int H, G, d, dv, norm;
  float scale, eps;
  int L, v_units;         // lanes that share a head (a power of two, 4 L >= d); units of 4 L value channels
};

constexpr int QC_MAX_TAPS = 8;

// d % 4 == 0 and dv % 4 == 0.  A unit of L lanes owns a query head, a key head or a run of value channels, four channels
// per lane, and walks TT consecutive tokens with the last taps rows of its channels in registers.  The tokens that reach
// back over their portion's start (its first taps - 1) are all served by the workgroup of the portion's FIRST token, which
// reads the slot there and at once writes its new contents: a channel's accesses to the slot come from one thread.
template <typename T, int MAXT>
__global__ __launch_bounds__(256) void qk_conv_store_kernel(QkConvArgs p, int TT) {
  typedef typename Pack4<T>::type P;
  const int L = p.L, unit = blockIdx.y * (256 / L) + threadIdx.x / L, e = (threadIdx.x % L) * 4;
  const int taps = p.taps, keep = taps - 1;
  const int nq = p.H * p.d, nk = p.G * p.d, nv = p.G * p.dv, C = nq + nk + nv;
  const bool is_q = unit < p.H, is_v = unit >= p.H + p.G;
  const int rel = is_v ? (unit - p.H - p.G) * 4 * L + e : (is_q ? unit : unit - p.H) * p.d + e;   // within q, k or v
  const bool on = unit < p.H + p.G + p.v_units && (is_v ? rel < nv : e < p.d);
  const int col = on ? (is_q ? p.q_off : is_v ? p.v_off : p.k_off) + rel : p.q_off;
  const int ch = on ? (is_q ? 0 : is_v ? nq + nk : nq) + rel : 0;
  const int64_t t_begin = (int64_t)blockIdx.x * TT, t_end = min(p.tokens, t_begin + TT);
  f32x4 wt[MAXT], win[MAXT];        // inside the walk win[MAXT - 1 - m] is the row m tokens back
  const T* w = reinterpret_cast<const T*>(p.w) + (int64_t)ch * taps;
  if (taps == 4) {                  // wt[MAXT - 1 - m] multiplies the row m tokens back
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4 v = Pack4<T>::widen(*reinterpret_cast<const P*>(w + i * 4));
#pragma unroll
      for (int m = 0; m < MAXT; ++m) wt[MAXT - 1 - m][i] = m < 4 ? v[3 - (m & 3)] : 0.0f;
    }
  } else {
#pragma unroll
    for (int m = 0; m < MAXT; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) wt[MAXT - 1 - m][i] = m < taps ? ld_f32<T>(w + i * taps + keep - m) : 0.0f;
  }
  auto row = [&](int64_t t) { return *reinterpret_cast<const f32x4*>(p.proj + max(t, (int64_t)0) * p.proj_rs + col); };
  const f32x4 zero = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  // before the walk the window stands one token earlier
  const int64_t t_first = p.cu_q[p.seq_of[t_begin]];
#pragma unroll
  for (int m = 1; m < MAXT; ++m) win[MAXT - m] = (m <= keep && t_begin - m >= t_first) ? row(t_begin - m) : zero;
  win[0] = zero;
  int b = 0;
  int64_t t0 = 0, t1 = 0;           // the request of token t and its tokens of this step
  f32x4 x_next = row(t_begin);      // a token's row is on the way while the one before it is worked on
  for (int64_t t = t_begin; t < p.tokens; ++t) {
    if (t >= t1) {
      b = p.seq_of[t];
      t0 = p.cu_q[b];
      t1 = p.cu_q[b + 1];
    }
    // past the tile: only the first tokens of a portion that began inside it
    if (t >= t_end && !(t0 >= t_begin && t0 < t_end && t - t0 < keep)) break;
    const f32x4 x = x_next;
    if (TT > 1) x_next = row(min(t + 1, p.tokens - 1));
    if (t == t0 && keep > 0) {
      float* slot = p.state + (int64_t)p.slots[b] * keep * C + ch;
      const bool fresh = p.past[b] == 0;
#pragma unroll
      for (int m = 1; m < MAXT; ++m)       // slot row keep - m holds the input m tokens ahead of the portion
        win[MAXT - m] = (m <= keep && on && !fresh) ? *reinterpret_cast<const f32x4*>(slot + (int64_t)(keep - m) * C) : zero;
      if (on) {
        const int n = (int)(t1 - t0);
#pragma unroll
        for (int m = 1; m < MAXT; ++m) {   // the new row keep - m: the input m - 1 tokens ahead of the portion's last one
          if (m > keep) continue;
          f32x4 v = zero;
          if (n - m >= 0) {
            v = row(t0 + n - m);
          } else {
#pragma unroll
            for (int o = 1; o < MAXT; ++o)
              if (o == m - n) v = win[MAXT - o];
          }
          *reinterpret_cast<f32x4*>(slot + (int64_t)(keep - m) * C) = v;
        }
      }
    }
#pragma unroll
    for (int m = 0; m + 1 < MAXT; ++m) win[m] = win[m + 1];
    win[MAXT - 1] = x;
    if (t0 < t_begin && t - t0 < keep) continue;          // served by the workgroup of the portion's first token
    f32x4 y = zero;
#pragma unroll
    for (int m = 0; m < MAXT; ++m) {
      if (MAXT - 1 - m >= taps) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] += wt[m][i] * win[m][i];
    }
    float f = 1.0f;
    if (p.norm) {                                          // every lane of the wavefront takes part
      float ss = on ? y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3] : 0.0f;
      for (int o = 1; o < L; o <<= 1) ss += __shfl_xor(ss, o, 64);
      if (!is_v) f = 1.0f / sqrtf(ss / (float)p.d + p.eps);
    }
    if (!on) continue;
    if (is_q) f *= p.scale;
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] *= f;
    if (is_q) {
      *reinterpret_cast<f32x4*>(p.q_out + t * nq + rel) = y;
    } else {
      const int64_t slot = p.slot_mapping[t];
      if (slot >= 0)
        *reinterpret_cast<P*>(reinterpret_cast<T*>(p.cache) + slot * (nk + nv) + (is_v ? nk : 0) + rel) = Pack4<T>::narrow(y);
    }
  }
}

struct WAttnArgs {
  const float* q;          // [tokens, H * d]
  const void* cache;       // [rows, G * (d + dv)]
  const int32_t* tables;   // [B, table_cols]
  int table_cols;
  const int32_t* cu_q;     // [B + 1]
  const int32_t* past;     // [B]
  const int32_t* seq_of;   // [tokens]
  void* out;               // [tokens, out_rs]: head h at columns h * dv
  int64_t out_rs;
  int64_t tokens;
  int H, G, d, dv, block_size, window, TQ, TK;
  float softcap, out_scale;
  int cw, v_col;           // numbers per cache row; column where the values of key/value head 0 begin (0: the keys)
  int slope_on;            // the distance term 2^(-8 (h + 1) / H) (i - j)
  const void* sink;        // [H] logits that join the denominator, or null
  const float* gate;       // [tokens, gate_rs] logits whose sigmoid multiplies the output (head h at h * dv), or null
  int64_t gate_rs;
  int gate_head;           // 1: one logit per head (head h at column h)
  int chunk;               // > 0: a query sees only the keys of its own chunk, floor(i / chunk) == floor(j / chunk)
  int keep;                // the first `keep` keys stay visible behind the window (0: none; not together with chunk)
  int ksplit;              // SPLIT only: workgroups that share a token's keys (blockIdx.z); > 1: results go to `partial`
  float* partial;          // [tokens, H, ksplit, dv + 2]: unnormalised output, then maximum and sum
};

// (factor for the accumulated values, denominator) once the walk over the keys is over: the sink joins the sum
__device__ __forceinline__ void close_softmax(float m, float l, bool has_sink, float sink, float& f, float& den) {
  if (!has_sink) {
    f = 1.0f;
    den = l;
    return;
  }
  const float top = fmaxf(m, sink);
  f = m == -INFINITY ? 0.0f : expf(m - top);
  den = l * f + expf(sink - top);
}

template <typename T>
__global__ __launch_bounds__(256) void window_attn_kernel(WAttnArgs p) {
  extern __shared__ float lds[];
  const int R = p.H / p.G, d = p.d, dv = p.dv, TK = p.TK, dp = d + 1;
  const int maxrows = p.TQ * R;
  float* sq = lds;                       // [rows][d]
  float* sk = sq + maxrows * d;          // [TK][d + 1]
  float* sv = sk + TK * dp;              // [TK][dv]
  float* sc = sv + TK * dv;              // [rows][TK]
  float* acc = sc + maxrows * TK;        // [rows][dv]
  float* sm = acc + maxrows * dv;        // [rows] running maximum
  float* sl = sm + maxrows;              // [rows] running sum
  float* scorr = sl + maxrows;           // [rows]
  const int g = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int64_t t_begin = (int64_t)blockIdx.x * p.TQ;
  const int64_t t_end = min(p.tokens, t_begin + p.TQ);
  const T* cache = reinterpret_cast<const T*>(p.cache);
  const int cw = p.cw;
  T* out = reinterpret_cast<T*>(p.out);
  const T* sink = reinterpret_cast<const T*>(p.sink);

  for (int64_t ts = t_begin; ts < t_end;) {
    const int b = p.seq_of[ts];
    const int64_t te = min(t_end, (int64_t)p.cu_q[b + 1]);
    const int nq = (int)(te - ts), rows = nq * R;
    const int p0 = p.past[b] + (int)(ts - p.cu_q[b]);
    const int32_t* table = p.tables + (int64_t)b * p.table_cols;
    for (int i = tid; i < rows * d; i += 256) {
      const int rr = i / d, e = i % d;
      sq[i] = p.q[(ts + rr / R) * p.H * d + (g * R + rr % R) * d + e];
    }
    for (int i = tid; i < rows * dv; i += 256) acc[i] = 0.0f;
    if (tid < rows) {
      sm[tid] = -INFINITY;
      sl[tid] = 0.0f;
    }
    __syncthreads();
    int lo = p.window > 0 ? max(0, p0 - p.window + 1) : 0;
    if (p.chunk > 0) lo = max(lo, p0 / p.chunk * p.chunk);      // the tile's first token has the earliest chunk
    const int hi = p0 + nq - 1;
    // the walk is over c = c_first .. hi: the kept keys ahead of lo come first (c < lo: key c - c_first), then key c itself
    const int c_first = lo - min(p.keep, lo);
    for (int j0 = c_first; j0 <= hi; j0 += TK) {
      const int nk = min(TK, hi + 1 - j0);
      for (int i = tid; i < nk * (d + dv); i += 256) {
        const int j = i / (d + dv), e = i % (d + dv);
        const int kp = j0 + j < lo ? j0 + j - c_first : j0 + j;
        const int64_t crow = (int64_t)table[kp / p.block_size] * p.block_size + kp % p.block_size;
        if (e < d) sk[j * dp + e] = ld_f32<T>(cache + crow * cw + g * d + e);
        else sv[j * dv + e - d] = ld_f32<T>(cache + crow * cw + p.v_col + g * dv + e - d);
      }
      __syncthreads();
      for (int i = tid; i < rows * TK; i += 256) {
        const int rr = i / TK, j = i % TK;
        const int pos = p0 + rr / R, kp = j0 + j < lo ? j0 + j - c_first : j0 + j;
        float s = -INFINITY;
        if (j < nk && kp <= pos && (p.window <= 0 || pos - kp < p.window || kp < p.keep) &&
            (p.chunk <= 0 || kp >= pos / p.chunk * p.chunk)) {
          s = 0.0f;
          const float* qv = sq + rr * d;
          const float* kv = sk + j * dp;
          for (int e = 0; e < d; ++e) s += qv[e] * kv[e];
          if (p.softcap > 0.0f) s = p.softcap * tanhf(s / p.softcap);
          const int h = g * R + rr % R;
          if (p.slope_on) s -= exp2f(-8.0f * (float)(h + 1) / (float)p.H) * (float)(pos - kp);
        }
        sc[i] = s;
      }
      __syncthreads();
      for (int rr = wv; rr < rows; rr += 4) {
        float m = -INFINITY;
        for (int j = lane; j < TK; j += 64) m = fmaxf(m, sc[rr * TK + j]);
        m = wave_max(m);
        const float m_old = sm[rr];
        const float m_new = fmaxf(m_old, m);
        float sum = 0.0f;
        for (int j = lane; j < TK; j += 64) {
          const float s = sc[rr * TK + j];
          const float e = s == -INFINITY ? 0.0f : expf(s - m_new);
          sc[rr * TK + j] = e;
          sum += e;
        }
        sum = wave_sum(sum);
        if (lane == 0) {
          const float corr = m_new == -INFINITY ? 1.0f : expf(m_old - m_new);   // exp(-inf) = 0 at the first tile
          scorr[rr] = corr;
          sm[rr] = m_new;
          sl[rr] = sl[rr] * corr + sum;
        }
      }
      __syncthreads();
      for (int i = tid; i < rows * dv; i += 256) {
        const int rr = i / dv, e = i % dv;
        float a = acc[i] * scorr[rr];
        const float* pv = sc + rr * TK;
        for (int j = 0; j < nk; ++j) a += pv[j] * sv[j * dv + e];
        acc[i] = a;
      }
      __syncthreads();
    }
    for (int i = tid; i < rows * dv; i += 256) {
      const int rr = i / dv, e = i % dv, h = g * R + rr % R;
      float f, den;
      close_softmax(sm[rr], sl[rr], sink != nullptr, sink ? ld_f32<T>(sink + h) : 0.0f, f, den);
      float v = acc[i] * f / den * p.out_scale;
      if (p.gate) v *= sigmoid_f32(p.gate[(ts + rr / R) * p.gate_rs + (p.gate_head ? h : h * dv + e)]);
      st_f32<T>(out + (ts + rr / R) * p.out_rs + h * dv + e, v);
    }
    __syncthreads();
    ts = te;
  }
}

// ---- the same attention on the matrix cores (bf16 cache) ----
// A workgroup of four wavefronts owns up to 64 query rows, 16 per wavefront: TQ consecutive tokens times the R heads
// that share key/value head g.  Per tile of 64 keys the K rows are staged row-major and the V rows transposed (both
// bf16, zero-filled past the last key); every wavefront computes S = Q K^T for its rows with the queries held as
// register fragments, shapes and masks the scores in the accumulator layout (a lane owns four rows of one key column),
// keeps running maxima and sums per row with 16-lane reductions, passes P through a private LDS patch to turn it into an
// A operand, and accumulates O += P V.  Scores, maxima, sums and rescaling are fp32; Q and P enter the MFMAs as bf16.
//
// SPLIT (steps of one token per request, at most 16 heads per key head): the four wavefronts hold the SAME rows and
// walk different key tiles, each with its own staging area and no workgroup barrier inside the walk; their partial
// (maximum, sum, output) triples meet in LDS at the end.  A decoded token's window is thus read four tiles at a time.
constexpr int MA_KEYS = 64, MA_VST = MA_KEYS + 8, MA_PST = MA_KEYS + 8;

constexpr size_t ma_stage_bytes(int ks, int ct) {     // one staging area: K tile, transposed V tile
  return ((size_t)MA_KEYS * (ks * 32 + 8) + (size_t)ct * 16 * MA_VST) * 2;
}
constexpr size_t ma_lds_bytes(int ks, int ct, bool split) {
  return split ? 4 * (ma_stage_bytes(ks, ct) + 16 * MA_PST * 2) : ma_stage_bytes(ks, ct) + 4 * 16 * MA_PST * 2;
}

// EXT: chunks, kept first keys and the gate of one logit per head are compiled in; launches that use none of them take
// the kernel without
template <int KS, int CT, bool SPLIT, bool EXT>
__global__ __launch_bounds__(256, (!SPLIT && KS <= 4 && CT <= 8) ? 2 : 1) void window_attn_mfma_kernel(WAttnArgs p) {
  constexpr int DK = KS * 32, KST = DK + 8, DVP = CT * 16;
  constexpr int STAGE = (int)(ma_stage_bytes(KS, CT) / 2);                 // bf16 elements of one staging area
  extern __shared__ u32x4 lds_raw[];
  __shared__ int64_t sRowAll[SPLIT ? 4 : 1][2][MA_KEYS];
  const int R = p.H / p.G, d = p.d, dv = p.dv;
  const int g = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int lc = lane & 15, lg = lane >> 4;
  bf16_t* base = reinterpret_cast<bf16_t*>(lds_raw);
  bf16_t* sK = base + (SPLIT ? wv * STAGE : 0);              // [64][KST]
  bf16_t* sVt = sK + MA_KEYS * KST;                          // [DVP][MA_VST]
  bf16_t* sPw = base + (SPLIT ? 4 : 1) * STAGE + wv * 16 * MA_PST;   // [16][MA_PST] of this wavefront
  int64_t (*sRows)[MA_KEYS] = sRowAll[SPLIT ? wv : 0];     // cache rows of this tile's keys and of the next one's
  constexpr int ST = SPLIT ? 64 : 256;                                    // threads that stage a tile together
  constexpr int NKC = MA_KEYS * (DK / 8) / ST, NVC = MA_KEYS * (DVP / 8) / ST;   // 16-byte pieces per thread
  const int stid = SPLIT ? lane : tid;
  const int row0 = SPLIT ? 0 : wv * 16;                                   // first query row of this wavefront
  auto sync = [&]() {
    if constexpr (SPLIT) {      // the area is private to this wavefront: its own LDS accesses complete in order
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    } else {
      __syncthreads();
    }
  };
  const int64_t t_begin = (int64_t)blockIdx.x * p.TQ;
  const int64_t t_end = min(p.tokens, t_begin + p.TQ);
  const bf16_t* cache = reinterpret_cast<const bf16_t*>(p.cache);
  const int cw = p.cw;
  bf16_t* out = reinterpret_cast<bf16_t*>(p.out);
  const bf16_t* sink = reinterpret_cast<const bf16_t*>(p.sink);

  for (int64_t ts = t_begin; ts < t_end;) {
    const int b = p.seq_of[ts];
    const int64_t te = min(t_end, (int64_t)p.cu_q[b + 1]);
    const int nq = (int)(te - ts), rows = nq * R;
    const int p0 = p.past[b] + (int)(ts - p.cu_q[b]);
    const int32_t* table = p.tables + (int64_t)b * p.table_cols;
    const bool wave_on = row0 < rows;
    // query fragments of this wavefront's 16 rows (A operand: lane holds row lc, features 8 lg .. 8 lg + 7 of each step)
    bf16x8 qf[KS];
    {
      const int rr = row0 + lc;
      const bool ok = rr < rows;
      const float* qrow = ok ? p.q + ((ts + rr / R) * p.H + g * R + rr % R) * d : nullptr;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int e = ks * 32 + lg * 8 + i;
          qf[ks][i] = (bf16_t)((ok && e < d) ? qrow[e] : 0.0f);
        }
      }
    }
    // the four accumulator rows of this lane
    int pos[4], kmin[EXT ? 4 : 1];      // kmin: first key of the row's chunk
    float slope[4], m_run[4], l_run[4];
    bool valid[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int rr = row0 + lg * 4 + r;
      valid[r] = rr < rows;
      pos[r] = p0 + rr / R;
      if constexpr (EXT) kmin[r] = p.chunk > 0 ? pos[r] / p.chunk * p.chunk : 0;
      slope[r] = p.slope_on ? exp2f(-8.0f * (float)(g * R + rr % R + 1) / (float)p.H) : 0.0f;
      m_run[r] = -INFINITY;
      l_run[r] = 0.0f;
    }
    f32x4 acc_o[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) acc_o[ct] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    const int wpos_lo = p0 + row0 / R, wpos_hi = p0 + min(rows - 1, row0 + 15) / R;

    const int lo_w = p.window > 0 ? max(0, p0 - p.window + 1) : 0;
    // the tile's first token has the earliest chunk
    const int lo = (EXT && p.chunk > 0) ? max(lo_w, p0 / p.chunk * p.chunk) : lo_w, hi = p0 + nq - 1;
    // kept keys: the walk is over c = c_first .. hi; c < lo means key c - c_first (those ahead of the window), else key c
    const int c_first = EXT ? lo - min(p.keep, lo) : lo;
    auto key_of = [&](int c) { return EXT && c < lo ? c - c_first : c; };
    const int walkers = SPLIT ? 4 * p.ksplit : 1;          // wavefronts (of all workgroups) that share this token's keys
    const int j_first = c_first + (SPLIT ? ((int)blockIdx.z * 4 + wv) * MA_KEYS : 0);
    auto row_of = [&](int c) {
      const int kp = key_of(c);
      return c <= hi ? (int64_t)table[kp / p.block_size] * p.block_size + kp % p.block_size : (int64_t)-1;
    };
    int turn = 0;
    if (stid < MA_KEYS) sRows[0][stid] = row_of(j_first + stid);
    sync();
    for (int j0 = j_first; j0 <= hi; j0 += walkers * MA_KEYS) {
      const int64_t* sRow = sRows[turn];
      turn ^= 1;
      // all of a thread's loads are issued before the first LDS store: one round trip to memory per tile
      u32x4 kreg[NKC], vreg[NVC];
#pragma unroll
      for (int i = 0; i < NKC; ++i) {
        const int c = stid + i * ST, key = c / (DK / 8), part = c % (DK / 8);
        const int64_t row = sRow[key];
        kreg[i] = u32x4{0u, 0u, 0u, 0u};
        if (row >= 0 && part * 8 < d) kreg[i] = *reinterpret_cast<const u32x4*>(cache + row * cw + g * d + part * 8);
      }
#pragma unroll
      for (int i = 0; i < NVC; ++i) {
        const int c = stid + i * ST, key = c % MA_KEYS, part = c / MA_KEYS;
        const int64_t row = sRow[key];
        vreg[i] = u32x4{0u, 0u, 0u, 0u};
        if (row >= 0 && part * 8 < dv)
          vreg[i] = *reinterpret_cast<const u32x4*>(cache + row * cw + p.v_col + g * dv + part * 8);
      }
      if (stid < MA_KEYS) sRows[turn][stid] = row_of(j0 + walkers * MA_KEYS + stid);      // its table entry is on the way with them
#pragma unroll
      for (int i = 0; i < NKC; ++i) {
        const int c = stid + i * ST, key = c / (DK / 8), part = c % (DK / 8);
        *reinterpret_cast<u32x4*>(sK + key * KST + part * 8) = kreg[i];
      }
#pragma unroll
      for (int i = 0; i < NVC; ++i) {
        const int c = stid + i * ST, key = c % MA_KEYS, part = c / MA_KEYS;
        uint16_t* dst = reinterpret_cast<uint16_t*>(sVt) + (part * 8) * MA_VST + key;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          dst[(2 * w) * MA_VST] = (uint16_t)(vreg[i][w] & 0xffffu);
          dst[(2 * w + 1) * MA_VST] = (uint16_t)(vreg[i][w] >> 16);
        }
      }
      sync();
      // keys this wavefront's rows can see: [wpos_lo - window + 1, wpos_hi]
      bool need = wave_on && j0 <= wpos_hi && (p.window <= 0 || j0 + MA_KEYS - 1 > wpos_lo - p.window);
      if constexpr (EXT)
        need = wave_on && key_of(j0) <= wpos_hi && (need || key_of(j0) < p.keep) &&
               (p.chunk <= 0 || j0 + MA_KEYS - 1 >= wpos_lo / p.chunk * p.chunk);
      if (need) {
        f32x4 acc_s[4];
#pragma unroll
        for (int sub = 0; sub < 4; ++sub) {
          acc_s[sub] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
          for (int ks = 0; ks < KS; ++ks) {
            const bf16x8 kf = *reinterpret_cast<const bf16x8*>(sK + (sub * 16 + lc) * KST + ks * 32 + lg * 8);
            acc_s[sub] = mfma16(qf[ks], kf, acc_s[sub]);
          }
        }
        float corr[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float mt = -INFINITY;
#pragma unroll
          for (int sub = 0; sub < 4; ++sub) {
            const int kp = key_of(j0 + sub * 16 + lc);
            const int dist = pos[r] - kp;
            float sc = acc_s[sub][r];
            if (p.softcap > 0.0f) sc = p.softcap * tanhf(sc / p.softcap);
            sc -= slope[r] * (float)dist;
            bool vis = valid[r] && dist >= 0 && (p.window <= 0 || dist < p.window || (EXT && kp < p.keep));
            if constexpr (EXT) vis = vis && kp >= kmin[r];
            sc = vis ? sc : -INFINITY;
            acc_s[sub][r] = sc;
            mt = fmaxf(mt, sc);
          }
          mt = lanes_max<16>(mt);
          const float m_new = fmaxf(m_run[r], mt);
          corr[r] = m_new == -INFINITY ? 1.0f : __expf(m_run[r] - m_new);
          float sum = 0.0f;
#pragma unroll
          for (int sub = 0; sub < 4; ++sub) {
            const float sc = acc_s[sub][r];
            const float e = sc == -INFINITY ? 0.0f : __expf(sc - m_new);
            sum += e;
            sPw[(lg * 4 + r) * MA_PST + sub * 16 + lc] = (bf16_t)e;
          }
          sum = lanes_sum<16>(sum);
          l_run[r] = l_run[r] * corr[r] + sum;
          m_run[r] = m_new;
        }
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc_o[ct][r] *= corr[r];
        // the patch is private to this wavefront: its own LDS accesses complete in order
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
        for (int ks = 0; ks < MA_KEYS / 32; ++ks) {
          const bf16x8 pf = *reinterpret_cast<const bf16x8*>(sPw + lc * MA_PST + ks * 32 + lg * 8);
#pragma unroll
          for (int ct = 0; ct < CT; ++ct) {
            const bf16x8 vf = *reinterpret_cast<const bf16x8*>(sVt + (ct * 16 + lc) * MA_VST + ks * 32 + lg * 8);
            acc_o[ct] = mfma16(pf, vf, acc_o[ct]);
          }
        }
      }
      sync();
    }
    if constexpr (SPLIT) {
      // partial results of the four wavefronts: rows of DVP outputs, the maximum and the sum, in each one's V area
      constexpr int PW = DVP + 2;
      float* part = reinterpret_cast<float*>(sVt);
      static_assert((size_t)16 * PW * 4 <= (size_t)DVP * MA_VST * 2, "partials fit the V area");
#pragma unroll
      for (int r = 0; r < 4; ++r) {
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) part[(lg * 4 + r) * PW + ct * 16 + lc] = acc_o[ct][r];
        if (lc == 0) {
          part[(lg * 4 + r) * PW + DVP] = m_run[r];
          part[(lg * 4 + r) * PW + DVP + 1] = l_run[r];
        }
      }
      __syncthreads();
      for (int idx = tid; idx < 16 * DVP; idx += 256) {
        const int rr = idx / DVP, e = idx % DVP;
        if (rr >= rows || e >= dv) continue;
        float m = -INFINITY;
#pragma unroll
        for (int w = 0; w < 4; ++w)
          m = fmaxf(m, reinterpret_cast<const float*>(base + w * STAGE + MA_KEYS * KST)[rr * PW + DVP]);
        float l = 0.0f, o = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          const float* pw = reinterpret_cast<const float*>(base + w * STAGE + MA_KEYS * KST);
          const float mw = pw[rr * PW + DVP];
          const float f = mw == -INFINITY ? 0.0f : __expf(mw - m);
          l += pw[rr * PW + DVP + 1] * f;
          o += pw[rr * PW + e] * f;
        }
        const int h = g * R + rr % R;
        if (p.ksplit > 1) {      // another launch joins the workgroups' shares (and the sink, and the gate)
          float* dst = p.partial + (((ts + rr / R) * p.H + h) * p.ksplit + blockIdx.z) * (dv + 2);
          dst[e] = o;
          if (e == 0) {
            dst[dv] = m;
            dst[dv + 1] = l;
          }
          continue;
        }
        float f, den;
        close_softmax(m, l, sink != nullptr, sink ? ld_f32<bf16_t>(sink + h) : 0.0f, f, den);
        float v = o * f * p.out_scale / den;
        if (p.gate) v *= sigmoid_f32(p.gate[(ts + rr / R) * p.gate_rs + ((EXT && p.gate_head) ? h : h * dv + e)]);
        out[(ts + rr / R) * p.out_rs + h * dv + e] = (bf16_t)v;
      }
      __syncthreads();
    } else if (wave_on) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int rr = row0 + lg * 4 + r;
        if (!valid[r]) continue;
        const int h = g * R + rr % R;
        float fs, den;
        close_softmax(m_run[r], l_run[r], sink != nullptr, sink ? ld_f32<bf16_t>(sink + h) : 0.0f, fs, den);
        const float f = p.out_scale * fs / den;
        bf16_t* orow = out + (ts + rr / R) * p.out_rs + h * dv;
        const float* grow = p.gate ? p.gate + (ts + rr / R) * p.gate_rs + ((EXT && p.gate_head) ? h : h * dv) : nullptr;
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          const int e = ct * 16 + lc;
          if (e < dv) orow[e] = (bf16_t)(acc_o[ct][r] * f * (grow ? sigmoid_f32(grow[(EXT && p.gate_head) ? 0 : e]) : 1.0f));
        }
      }
    }
    ts = te;
  }
}

// ---- one token per request, few query heads per key head (bf16 cache) ----
// A decoded token's R query rows are far too few for a matrix-core tile to pay for its staging, so the keys stay in
// registers: LPK lanes share a key, eight numbers (16 bytes) each, a wavefront reads KPW = 64 / LPK keys per access and U
// such accesses of keys and of values are in flight before the first is used.  Scores are reduced over the LPK lanes; every
// group of LPK lanes keeps its own running maximum, sum and weighted values, which meet by shuffles, then in LDS.  All of it
// is fp32.  Workgroups (blockIdx.z) and their wavefronts take every 4 * ksplit-th batch of KPW * U keys.
template <int LPK, int RP, int U>
__global__ __launch_bounds__(256) void window_attn_rows_kernel(WAttnArgs p) {
  constexpr int KPW = 64 / LPK, KB = KPW * U;
  static_assert(KB <= 64, "one lane looks up one key of a batch");
  __shared__ float part[4][RP][LPK * 8 + 2];
  const int R = p.H / p.G, d = p.d, dv = p.dv;
  const int64_t t = blockIdx.x;
  const int g = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int li = lane % LPK, sub = lane / LPK;
  const int b = p.seq_of[t];
  const int pos = p.past[b] + (int)(t - p.cu_q[b]);
  const int32_t* table = p.tables + (int64_t)b * p.table_cols;
  const bf16_t* cache = reinterpret_cast<const bf16_t*>(p.cache);
  const int cw = p.cw;
  const bool k_on = li * 8 < d, v_on = li * 8 < dv;
  float q[RP][8], acc[RP][8], m[RP], l[RP];
#pragma unroll
  for (int r = 0; r < RP; ++r) {
    const float* qr = p.q + (t * p.H + g * R + r) * d + li * 8;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      q[r][e] = (r < R && k_on) ? qr[e] : 0.0f;
      acc[r][e] = 0.0f;
    }
    m[r] = -INFINITY;
    l[r] = 0.0f;
  }
  int lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  if (p.chunk > 0) lo = max(lo, pos / p.chunk * p.chunk);
  const int c_first = lo - min(p.keep, lo);               // kept keys ahead of the window, as in the other kernels
  for (int c0 = c_first + ((int)blockIdx.z * 4 + wv) * KB; c0 <= pos; c0 += 4 * p.ksplit * KB) {
    int64_t row_of = -1;
    {
      const int c = c0 + lane;
      if (lane < KB && c <= pos) {
        const int kp = c < lo ? c - c_first : c;
        row_of = (int64_t)table[kp / p.block_size] * p.block_size + kp % p.block_size;
      }
    }
    u32x4 kr[U], vr[U];
    bool seen[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int64_t row = __shfl(row_of, u * KPW + sub, 64);
      seen[u] = row >= 0;
      kr[u] = vr[u] = u32x4{0u, 0u, 0u, 0u};
      if (seen[u] && k_on) kr[u] = *reinterpret_cast<const u32x4*>(cache + row * cw + g * d + li * 8);
      if (seen[u] && v_on) vr[u] = *reinterpret_cast<const u32x4*>(cache + row * cw + p.v_col + g * dv + li * 8);
    }
    float s[RP][U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int r = 0; r < RP; ++r) {
        float a = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w)
          a += q[r][2 * w] * lo_f32<bf16_t>(kr[u][w]) + q[r][2 * w + 1] * hi_f32<bf16_t>(kr[u][w]);
        s[r][u] = a;
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int r = 0; r < RP; ++r) {
        s[r][u] = lanes_sum<LPK == 8 ? 8 : 16>(s[r][u]);
        if constexpr (LPK == 32) s[r][u] += __shfl_xor(s[r][u], 16, 64);
      }
    }
#pragma unroll
    for (int r = 0; r < RP; ++r) {
      const float slope = p.slope_on ? exp2f(-8.0f * (float)(g * R + r + 1) / (float)p.H) : 0.0f;
      float mt = m[r];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int c = c0 + u * KPW + sub, kp = c < lo ? c - c_first : c;
        float a = s[r][u];
        if (p.softcap > 0.0f) a = p.softcap * tanhf(a / p.softcap);
        a -= slope * (float)(pos - kp);
        s[r][u] = seen[u] ? a : -INFINITY;
        mt = fmaxf(mt, s[r][u]);
      }
      const float corr = mt == -INFINITY ? 1.0f : __expf(m[r] - mt);
      m[r] = mt;
      l[r] *= corr;
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[r][e] *= corr;
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float e_ = s[r][u] == -INFINITY ? 0.0f : __expf(s[r][u] - mt);
        l[r] += e_;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          acc[r][2 * w] += e_ * lo_f32<bf16_t>(vr[u][w]);
          acc[r][2 * w + 1] += e_ * hi_f32<bf16_t>(vr[u][w]);
        }
      }
    }
  }
  // the KPW groups of a wavefront
#pragma unroll
  for (int o = LPK; o < 64; o <<= 1) {
#pragma unroll
    for (int r = 0; r < RP; ++r) {
      const float m2 = __shfl_xor(m[r], o, 64), l2 = __shfl_xor(l[r], o, 64);
      const float mt = fmaxf(m[r], m2);
      const float f1 = m[r] == -INFINITY ? 0.0f : __expf(m[r] - mt), f2 = m2 == -INFINITY ? 0.0f : __expf(m2 - mt);
      l[r] = l[r] * f1 + l2 * f2;
      m[r] = mt;
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[r][e] = acc[r][e] * f1 + __shfl_xor(acc[r][e], o, 64) * f2;
    }
  }
  if (sub == 0) {
#pragma unroll
    for (int r = 0; r < RP; ++r) {
#pragma unroll
      for (int e = 0; e < 8; ++e) part[wv][r][li * 8 + e] = acc[r][e];
      if (li == 0) {
        part[wv][r][LPK * 8] = m[r];
        part[wv][r][LPK * 8 + 1] = l[r];
      }
    }
  }
  __syncthreads();
  const bf16_t* sink = reinterpret_cast<const bf16_t*>(p.sink);
  bf16_t* out = reinterpret_cast<bf16_t*>(p.out);
  for (int i = tid; i < R * dv; i += 256) {
    const int r = i / dv, e = i % dv, h = g * R + r;
    float mt = -INFINITY, sum = 0.0f, o = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) mt = fmaxf(mt, part[w][r][LPK * 8]);
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float mw = part[w][r][LPK * 8];
      const float f = mw == -INFINITY ? 0.0f : __expf(mw - mt);
      sum += part[w][r][LPK * 8 + 1] * f;
      o += part[w][r][e] * f;
    }
    if (p.ksplit > 1) {
      float* dst = p.partial + ((t * p.H + h) * p.ksplit + blockIdx.z) * (dv + 2);
      dst[e] = o;
      if (e == 0) {
        dst[dv] = mt;
        dst[dv + 1] = sum;
      }
      continue;
    }
    float f, den;
    close_softmax(mt, sum, sink != nullptr, sink ? ld_f32<bf16_t>(sink + h) : 0.0f, f, den);
    float v = o * f * p.out_scale / den;
    if (p.gate) v *= sigmoid_f32(p.gate[t * p.gate_rs + (p.gate_head ? h : h * dv + e)]);
    out[t * p.out_rs + h * dv + e] = (bf16_t)v;
  }
}

template <int LPK>
void launch_window_rows(const WAttnArgs& p, int R, dim3 grid, hipStream_t s) {
  if (R == 1) window_attn_rows_kernel<LPK, 1, LPK == 8 ? 4 : 8><<<grid, dim3(256), 0, s>>>(p);
  else if (R == 2) window_attn_rows_kernel<LPK, 2, LPK == 8 ? 4 : 8><<<grid, dim3(256), 0, s>>>(p);
  else window_attn_rows_kernel<LPK, 4, 4><<<grid, dim3(256), 0, s>>>(p);
}

// joins the shares of the ksplit workgroups that walked one token's keys: one wavefront per (token, head)
__global__ __launch_bounds__(256) void window_attn_join_kernel(WAttnArgs p) {
  const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= p.tokens * p.H) return;
  const int lane = threadIdx.x & 63, dv = p.dv, h = (int)(row % p.H);
  const int64_t t = row / p.H;
  const float* src = p.partial + row * p.ksplit * (dv + 2);
  // all maxima and sums first (at most 8 shares: the loads go out together), then one weight per share
  float mz[8], wz[8];
  float m = -INFINITY, l = 0.0f;
#pragma unroll
  for (int z = 0; z < 8; ++z) {
    mz[z] = z < p.ksplit ? src[z * (dv + 2) + dv] : -INFINITY;
    wz[z] = z < p.ksplit ? src[z * (dv + 2) + dv + 1] : 0.0f;
    m = fmaxf(m, mz[z]);
  }
#pragma unroll
  for (int z = 0; z < 8; ++z) {
    const float f = mz[z] == -INFINITY ? 0.0f : __expf(mz[z] - m);
    l += wz[z] * f;
    wz[z] = f;
  }
  const bf16_t* sink = reinterpret_cast<const bf16_t*>(p.sink);
  float f, den;
  close_softmax(m, l, sink != nullptr, sink ? ld_f32<bf16_t>(sink + h) : 0.0f, f, den);
  bf16_t* out = reinterpret_cast<bf16_t*>(p.out) + t * p.out_rs + h * dv;
  for (int e = lane; e < dv; e += 64) {
    float o = 0.0f;
#pragma unroll
    for (int z = 0; z < 8; ++z)
      if (z < p.ksplit) o += src[z * (dv + 2) + e] * wz[z];
    float v = o * f * p.out_scale / den;
    if (p.gate) v *= sigmoid_f32(p.gate[t * p.gate_rs + (p.gate_head ? h : h * dv + e)]);
    out[e] = (bf16_t)v;
  }
}

template <int KS, int CT, bool SPLIT, bool EXT>
hipError_t launch_window_mfma4(const WAttnArgs& p, dim3 grid, hipStream_t s) {
  constexpr size_t lds = ma_lds_bytes(KS, CT, SPLIT);
  static size_t allowed = 64 * 1024;
  if (lds > allowed) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&window_attn_mfma_kernel<KS, CT, SPLIT, EXT>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    allowed = lds;
  }
  window_attn_mfma_kernel<KS, CT, SPLIT, EXT><<<grid, dim3(256), lds, s>>>(p);
  return hipGetLastError();
}

template <int KS, int CT, bool SPLIT>
hipError_t launch_window_mfma3(const WAttnArgs& p, dim3 grid, hipStream_t s) {
  if (p.chunk > 0 || p.keep > 0 || (p.gate && p.gate_head)) return launch_window_mfma4<KS, CT, SPLIT, true>(p, grid, s);
  return launch_window_mfma4<KS, CT, SPLIT, false>(p, grid, s);
}

template <int KS, int CT>
hipError_t launch_window_mfma2(const WAttnArgs& p, bool split, dim3 grid, hipStream_t s) {
  if constexpr (ma_lds_bytes(KS, CT, true) <= 156 * 1024) {
    if (split) return launch_window_mfma3<KS, CT, true>(p, grid, s);
  }
  return launch_window_mfma3<KS, CT, false>(p, grid, s);
}

template <int KS>
hipError_t launch_window_mfma(const WAttnArgs& p, int ct, bool split, dim3 grid, hipStream_t s) {
  switch (ct) {
    case 2: return launch_window_mfma2<KS, 2>(p, split, grid, s);
    case 4: return launch_window_mfma2<KS, 4>(p, split, grid, s);
    case 8: return launch_window_mfma2<KS, 8>(p, split, grid, s);
    default: return launch_window_mfma2<KS, 16>(p, split, grid, s);
  }
}

}  // namespace

// Workgroups that share one decoded token's keys: enough to put about 256 workgroups on the chip, at most 8.  A
// function of the launch shape alone (not of the contexts), so a captured launch stays valid as contexts grow.
static int window_attn_key_splits(int64_t tokens, int kv_heads) {
  const int64_t groups = tokens * kv_heads;
  int k = 1;
  while (k < 8 && groups * k * 2 <= 256) k *= 2;
  return k;
}

extern "C" size_t nv_paged_softmax_attn_workspace_bytes(int64_t tokens, int max_q, int heads, int kv_heads, int vdim) {
  if (max_q > 1 || tokens <= 0 || heads / kv_heads > 16) return 0;
  const int k = window_attn_key_splits(tokens, kv_heads);
  return k > 1 ? (size_t)tokens * heads * k * (vdim + 2) * sizeof(float) : 0;
}

extern "C" int nv_qk_store(const float* proj, const void* bias, int64_t proj_row_stride, int q_off, int k_off, int v_off,
                           const void* q_norm, const void* k_norm, const void* temp, const int64_t* positions,
                           float temp_coef, int temp_every, float scale, float eps, const int32_t* slot_mapping,
                           void* cache, float* q_out, int64_t tokens, int heads, int kv_heads, int dim, int vdim, int dtype,
                           nv_stream_t stream) {
  return nv_qk_rotate_store(proj, bias, proj_row_stride, q_off, k_off, v_off, q_norm, k_norm, 0, temp, positions, temp_coef,
                            temp_every, nullptr, 0, 0, 1.0f, nullptr, 0, nullptr, scale, eps, slot_mapping, cache, q_out,
                            tokens, heads, kv_heads, dim, vdim, dtype, stream);
}

extern "C" int nv_qk_rotate_store(const float* proj, const void* bias, int64_t proj_row_stride, int q_off, int k_off,
                                  int v_off, const void* q_norm, const void* k_norm, int norm_whole, const void* temp,
                                  const int64_t* positions, float temp_coef, int temp_every, const float* inv_freq,
                                  int rot_dims, int interleaved, float mscale, const float* v_first,
                                  int64_t v_first_row_stride,
                                  const void* vmix, float scale, float eps, const int32_t* slot_mapping, void* cache,
                                  float* q_out, int64_t tokens, int heads, int kv_heads, int dim, int vdim, int dtype,
                                  nv_stream_t stream) {
  NV_CHECK_ARG(proj && slot_mapping && cache && q_out, "nv_qk_store: null pointer");
  NV_CHECK_ARG((q_norm == nullptr) == (k_norm == nullptr), "nv_qk_store: both norm weights or none");
  NV_CHECK_ARG(dtype == NV_BF16 || dtype == NV_F32, "nv_qk_store: bad dtype %d", dtype);
  NV_CHECK_ARG(tokens >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim >= 0,
               "nv_qk_store: bad shape");
  NV_CHECK_ARG(temp_every >= 0 && (temp_every == 0 || positions), "nv_qk_store: the position temperature needs positions");
  NV_CHECK_ARG(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || (positions && inv_freq)),
               "nv_qk_store: a rotation over %d of %d numbers needs positions and frequencies", rot_dims, dim);
  NV_CHECK_ARG(!v_first || (vmix && vdim > 0), "nv_qk_store: blending values needs its weight");
  if (tokens == 0) return NV_OK;
  auto al = [](const void* q, size_t n) { return (uintptr_t)q % n == 0; };
  NV_CHECK_ARG(norm_whole >= 0 && norm_whole <= 2 && (norm_whole != 2 || !q_norm), "nv_qk_store: bad norm %d", norm_whole);
  const bool pairs = !q_norm && norm_whole != 2 && !temp && !bias && !v_first && temp_every == 0 && (rot_dims == 0 || (interleaved && rot_dims <= 256)) &&
                     dim % 4 == 0 && vdim % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 &&
                     proj_row_stride % 4 == 0 && al(proj, 16) && al(q_out, 16) && al(cache, 16);
  QkArgs p{proj, bias, proj_row_stride, q_off, k_off, v_off, q_norm, k_norm, temp, positions, temp_coef, temp_every,
           slot_mapping, cache, q_out, heads, kv_heads, dim, vdim, scale, eps, norm_whole, inv_freq, rot_dims, mscale,
           v_first, v_first_row_stride, vmix, interleaved};
  if (pairs)
    NV_DISPATCH_T(dtype, qk_pairs_store_kernel<T><<<dim3((unsigned)tokens), dim3(256), 0, (hipStream_t)stream>>>(p));
  else
    NV_DISPATCH_T(dtype, qk_norm_store_kernel<T><<<dim3((unsigned)tokens), dim3(256), 0, (hipStream_t)stream>>>(p));
  NV_CHECK_LAUNCH();
  return NV_OK;
}

// lanes per head of qk_conv_store_kernel
static int qk_conv_lanes(int dim) {
  int L = 8;
  while (4 * L < dim) L *= 2;
  return L;
}

extern "C" int nv_qk_conv_store_ok(const void* proj, int64_t proj_row_stride, int q_off, int k_off, int v_off,
                                   const void* cache, const void* q_out, const void* state, int dim, int vdim, int taps) {
  auto al = [](const void* q) { return (uintptr_t)q % 16 == 0; };
  return dim % 4 == 0 && vdim % 4 == 0 && dim <= 256 && taps >= 1 && taps <= QC_MAX_TAPS && q_off % 4 == 0 && k_off % 4 == 0 &&
         v_off % 4 == 0 && proj_row_stride % 4 == 0 && al(proj) && al(cache) && al(q_out) && al(state);
}

extern "C" int nv_qk_conv_store(const float* proj, int64_t proj_row_stride, int q_off, int k_off, int v_off, const void* w,
                                int taps, float* state, const int32_t* cu_q, const int32_t* past_lens,
                                const int32_t* state_slots, const int32_t* seq_of_token, const int32_t* slot_mapping,
                                void* cache, float* q_out, int64_t tokens, int max_q, int heads, int kv_heads, int dim,
                                int vdim, int norm, float scale, float eps, int dtype, nv_stream_t stream) {
  NV_CHECK_ARG(proj && w && cu_q && past_lens && state_slots && seq_of_token && slot_mapping && cache && q_out &&
                   (state || taps == 1),
               "nv_qk_conv_store: null pointer");
  NV_CHECK_ARG(dtype == NV_BF16 || dtype == NV_F32, "nv_qk_conv_store: bad dtype %d", dtype);
  NV_CHECK_ARG(tokens >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0,
               "nv_qk_conv_store: bad shape");
  NV_CHECK_ARG(nv_qk_conv_store_ok(proj, proj_row_stride, q_off, k_off, v_off, cache, q_out, state, dim, vdim, taps),
               "nv_qk_conv_store: heads of %d + %d numbers, %d taps or an alignment this launch does not serve", dim, vdim, taps);
  if (tokens == 0) return NV_OK;
  const int L = qk_conv_lanes(dim), v_units = (kv_heads * vdim + 4 * L - 1) / (4 * L);
  const int units = heads + kv_heads + v_units, per = 256 / L, TT = max_q <= 1 ? 1 : 8;
  QkConvArgs p{proj, proj_row_stride, q_off, k_off, v_off, w, taps, state, cu_q, past_lens, state_slots, seq_of_token,
               slot_mapping, cache, q_out, tokens, heads, kv_heads, dim, vdim, norm, scale, eps, L, v_units};
  const dim3 grid((unsigned)((tokens + TT - 1) / TT), (unsigned)((units + per - 1) / per));
  hipStream_t s = (hipStream_t)stream;
  if (taps <= 4) NV_DISPATCH_T(dtype, qk_conv_store_kernel<T, 4><<<grid, dim3(256), 0, s>>>(p, TT));
  else NV_DISPATCH_T(dtype, qk_conv_store_kernel<T, QC_MAX_TAPS><<<grid, dim3(256), 0, s>>>(p, TT));
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_qk_norm_store(const float* proj, const void* bias, int64_t proj_row_stride, int q_off, int k_off,
                                int v_off, const void* q_norm, const void* k_norm, const void* temp, float scale, float eps,
                                const int32_t* slot_mapping, void* cache, float* q_out, int64_t tokens, int heads,
                                int kv_heads, int dim, int vdim, int dtype, nv_stream_t stream) {
  NV_CHECK_ARG(q_norm && k_norm && vdim > 0, "nv_qk_norm_store: null pointer");
  return nv_qk_store(proj, bias, proj_row_stride, q_off, k_off, v_off, q_norm, k_norm, temp, nullptr, 0.0f, 0, scale, eps,
                     slot_mapping, cache, q_out, tokens, heads, kv_heads, dim, vdim, dtype, stream);
}

extern "C" int nv_window_attn(const float* q, const void* cache, const int32_t* block_tables, int table_cols,
                              const int32_t* cu_q, const int32_t* past_lens, const int32_t* seq_of_token, void* out,
                              int64_t out_row_stride, int64_t tokens, int max_q, int heads, int kv_heads, int dim, int vdim,
                              int block_size, int window, float softcap, float out_scale, int dtype, nv_stream_t stream) {
  return nv_paged_softmax_attn(q, cache, block_tables, table_cols, cu_q, past_lens, seq_of_token, out, out_row_stride,
                               tokens, max_q, heads, kv_heads, dim, vdim, block_size, window, 0, 0, softcap, out_scale, 1, 0,
                               nullptr, nullptr, 0, 0, nullptr, 0, dtype, stream);
}

extern "C" int nv_paged_softmax_attn(const float* q, const void* cache, const int32_t* block_tables, int table_cols,
                                     const int32_t* cu_q, const int32_t* past_lens, const int32_t* seq_of_token, void* out,
                                     int64_t out_row_stride, int64_t tokens, int max_q, int heads, int kv_heads, int dim,
                                     int vdim, int block_size, int window, int chunk, int keep_first, float softcap,
                                     float out_scale,
                                     int distance_term, int values_are_keys, const void* sink, const float* gate,
                                     int64_t gate_row_stride, int gate_per_head, void* workspace, size_t workspace_bytes,
                                     int dtype, nv_stream_t stream) {
  NV_CHECK_ARG(q && cache && block_tables && cu_q && past_lens && seq_of_token && out, "nv_window_attn: null pointer");
  NV_CHECK_ARG(!values_are_keys || vdim == dim, "nv_window_attn: values that are the keys have the keys' size");
  const int cw = values_are_keys ? kv_heads * dim : kv_heads * (dim + vdim), v_col = values_are_keys ? 0 : kv_heads * dim;
  NV_CHECK_ARG(dtype == NV_BF16 || dtype == NV_F32, "nv_window_attn: bad dtype %d", dtype);
  NV_CHECK_ARG(tokens >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0 &&
                   block_size > 0 && window >= 0 && chunk >= 0 && keep_first >= 0 && table_cols > 0,
               "nv_window_attn: bad shape");
  NV_CHECK_ARG(chunk == 0 || keep_first == 0, "nv_window_attn: chunks and kept first keys exclude each other");
  if (tokens == 0) return NV_OK;
  const int R = heads / kv_heads;
  // bf16 caches with 16-byte-aligned heads of up to 256 numbers: the matrix-core kernel
  if (dtype == NV_BF16 && dim % 8 == 0 && vdim % 8 == 0 && dim <= 256 && vdim <= 256 && R <= 64 && kv_heads <= 65535 &&
      (uintptr_t)cache % 16 == 0 && cw % 8 == 0 && v_col % 8 == 0 && getenv("NV_WINDOW_ATTN_MFMA_OFF") == nullptr) {
    const int ks = dim <= 64 ? 2 : dim <= 128 ? 4 : 8;
    const int ct = vdim <= 32 ? 2 : vdim <= 64 ? 4 : vdim <= 128 ? 8 : 16;
    if (ma_lds_bytes(ks, ct, false) <= 160 * 1024) {
      // one token per request: the wavefronts split the window (where four staging areas fit the LDS)
      const bool split = max_q <= 1 && R <= 16 && ma_lds_bytes(ks, ct, true) <= 156 * 1024;
      const bool rows = max_q <= 1 && R <= 4 && getenv("NV_WINDOW_ATTN_ROWS_OFF") == nullptr;   // keys in registers
      const int TQm = max_q <= 1 ? 1 : 64 / R;
      // ... and with few requests several workgroups do, when the caller brought room for their shares
      int ksplit = split || rows ? window_attn_key_splits(tokens, kv_heads) : 1;
      if (ksplit > 1 && (!workspace || workspace_bytes < (size_t)tokens * heads * ksplit * (vdim + 2) * sizeof(float)))
        ksplit = 1;
      WAttnArgs pm{q, cache, block_tables, table_cols, cu_q, past_lens, seq_of_token, out, out_row_stride, tokens, heads,
                   kv_heads, dim, vdim, block_size, window, TQm, MA_KEYS, softcap, out_scale, cw, v_col, distance_term, sink,
                   gate, gate_row_stride, gate_per_head, chunk, keep_first, ksplit, reinterpret_cast<float*>(workspace)};
      dim3 gridm((unsigned)((tokens + TQm - 1) / TQm), (unsigned)kv_heads, (unsigned)ksplit);
      hipStream_t st = (hipStream_t)stream;
      const int wide = dim > vdim ? dim : vdim;
      if (rows && wide <= 64) launch_window_rows<8>(pm, R, gridm, st);
      else if (rows && wide <= 128) launch_window_rows<16>(pm, R, gridm, st);
      else if (rows) launch_window_rows<32>(pm, R, gridm, st);
      const hipError_t e = rows ? hipGetLastError() : ks == 2 ? launch_window_mfma<2>(pm, ct, split, gridm, st)
                           : ks == 4 ? launch_window_mfma<4>(pm, ct, split, gridm, st)
                                     : launch_window_mfma<8>(pm, ct, split, gridm, st);
      if (e != hipSuccess) {
        nv_set_error("nv_window_attn: %s", hipGetErrorString(e));
        return NV_ERR_LAUNCH;
      }
      if (ksplit > 1) {
        window_attn_join_kernel<<<dim3((unsigned)((tokens * heads + 3) / 4)), dim3(256), 0, st>>>(pm);
        NV_CHECK_LAUNCH();
      }
      return NV_OK;
    }
  }
  const size_t budget = 64 * 1024;
  auto need = [&](int tq, int tk) {
    const size_t rows = (size_t)tq * R;
    return (rows * dim + (size_t)tk * (dim + 1) + (size_t)tk * vdim + rows * tk + rows * vdim + 3 * rows) * sizeof(float);
  };
  int TQ = max_q <= 1 ? 1 : 16, TK = 64;
  while (TK > 8 && need(1, TK) > budget) TK /= 2;
  NV_CHECK_ARG(need(1, TK) <= budget, "nv_window_attn: heads of %d + %d numbers do not fit the LDS plan", dim, vdim);
  while (TQ > 1 && (need(TQ, TK) > budget || TQ * R > 256)) TQ /= 2;
  NV_CHECK_ARG(R <= 256 && kv_heads <= 65535, "nv_window_attn: %d query heads per key head exceed a workgroup", R);
  const int64_t tiles = (tokens + TQ - 1) / TQ;
  WAttnArgs p{q, cache, block_tables, table_cols, cu_q, past_lens, seq_of_token, out, out_row_stride, tokens, heads,
              kv_heads, dim, vdim, block_size, window, TQ, TK, softcap, out_scale, cw, v_col, distance_term, sink, gate,
              gate_row_stride, gate_per_head, chunk, keep_first, 1, nullptr};
  dim3 grid((unsigned)tiles, (unsigned)kv_heads);
  NV_DISPATCH_T(dtype, window_attn_kernel<T><<<grid, dim3(256), need(TQ, TK), (hipStream_t)stream>>>(p));
  NV_CHECK_LAUNCH();
  return NV_OK;
}
