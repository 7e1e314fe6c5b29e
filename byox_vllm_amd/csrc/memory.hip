// Matrix memories with one decay per head and token: a per-head state S [dim, vdim] in fp32,
//   S_t = keep_t S_(t-1) + take_t k_t v_t^T,   o_t = S_t^T q_t,
// in two forms.
//   MEM_CONST  (lightning attention, retention): keep_t = decay[h], a constant of the head, take_t = 1; q, k, v may pass
//              through SiLU first, q and k may be rotated by their position; o_t leaves as it is.
//   MEM_EXPGATE (the matrix memory of xLSTM): log gates i_t = cap tanh(zi / cap) and f_t = logsigmoid(cap tanh(zf / cap))
//              from one logit each per head, a running maximum m_t = max(f_t + m_(t-1), i_t) that starts at 0,
//              keep_t = exp(f_t + m_(t-1) - m_t), take_t = exp(i_t - m_t); a normaliser n_t = keep_t n_(t-1) + take_t k_t
//              runs beside S, and o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).
// A request's slot holds, per head, S (dim x vdim), then in the second form n (dim) and m (1) once per slice of 64 value
// columns.  One workgroup owns one (request, head, slice of 64 state columns) triple - columns are independent of each
// other, so slices need nothing from each other but each keeps its own copy of the normaliser and the maximum; launches
// of many requests give a workgroup all slices of a head instead - and walks the request's tokens of this step in order, starting from the slot (or from zero when
// the request has no tokens behind it) and leaving the state there: a prompt portion, the next portion and single
// decoded tokens can all go through this one kernel (states that do not fit a workgroup's registers: a slow general kernel
// that keeps the state in its slot).  The results are fp32 rows; the norm and gate that follow them span
// heads or not, depending on the design, and run in nv_group_rmsnorm_f32.
//
// Thread (cs, v) keeps the entries S[cs * DC .. cs * DC + DC - 1][v] of state column v of its slice in registers (the key channels
// of a column are split over CS threads; their partial o_t meet in LDS once per chunk of tokens).  Tokens are staged
// sixteen at a time: k and q rows in LDS (padded to DMAX with zeros), the thread's own v values in registers; the gates
// of the chunk are a scalar recurrence that one thread walks while the others stage.  Thread d < dim also carries n[d];
// the sixteen n . q meet through wavefront sums.
//
// Single tokens in the first form can take their head's norm and gate along in one launch (retention_step_kernel).
// Prompts in the first form take retention_chunk_kernel where sizes and alignments allow: with ONE constant decay per head, C tokens at once are
// matrix products on the fp32 matrix cores (v_mfma_f32_16x16x4_f32, true fp32),
//   o_i = decay^(i+1) S^T q_i + sum_(j <= i) decay^(i-j) (q_i . k_j) v_j,
//   S  <- decay^n S + sum_j decay^(n-1-j) k_j v_j^T,
// so a chunk costs three short phases instead of C dependent steps.  Each power of the decay is formed on its own (no
// quotients of powers: nothing overflows or cancels, however small the decay).
#include "anyt.h"

namespace {

enum { MEM_CONST = 0, MEM_EXPGATE = 1 };
constexpr int MM_TC = 16;

struct MemArgs {
  const float* proj;     // [tokens, proj_rs]: q | k | v (and the gate logits zi | zf, one per head) at column offsets
  int64_t proj_rs;
  int q_off, k_off, v_off, i_off, f_off;
  const void* bias;      // [proj columns] in the storage type, added to the gate logits; or null
  const float* decay;    // [H] (MEM_CONST)
  float* state;          // [slots, H, per_head]
  const int32_t* cu_q;   // [B + 1] token ranges of the requests in this step
  const int32_t* past;   // [B] tokens each request already holds
  const int32_t* slots;  // [B] state slot of each request
  float* out;            // [tokens, out_rs]: head h at columns h * vdim
  int64_t out_rs;
  int H, dim, vdim, per_head, silu;
  float q_scale, k_scale, cap;
  const float* rot;      // [tokens, rot_dims]: cosines then sines of the tokens' angles, read when rot_dims > 0
  int rot_dims;          // the first rot_dims numbers of q and k turn, number i with i + rot_dims / 2
};

__device__ __forceinline__ float maybe_silu(float z, int on) { return on ? silu_f32(z) : z; }

// number i of the q or k vector at src (activated), turned by the token's angles
__device__ __forceinline__ float turned(const MemArgs& p, const float* src, int i, const float* rot_row) {
  const float x = maybe_silu(src[i], p.silu);
  if (i >= p.rot_dims) return x;
  const int half = p.rot_dims >> 1;
  const bool first = i < half;
  const int f = first ? i : i - half;
  const float other = maybe_silu(src[first ? i + half : f], p.silu), c = rot_row[f], s = rot_row[half + f];
  return first ? x * c - other * s : x * c + other * s;
}

constexpr int MEM_SLICE = 64;      // state columns that share one copy of n | m

template <typename T, int DMAX, int CS, int MODE>
__global__ __launch_bounds__(256) void matrix_memory_kernel(MemArgs p) {
  constexpr int DC = DMAX / CS;
  extern __shared__ float4 lds4[];
  float* lds = reinterpret_cast<float*>(lds4);
  const int vd = p.vdim;
  // the workgroup covers vdp state columns (a multiple of 64: one slice, or several when the launch has workgroups enough)
  const int tid = threadIdx.x, nthr = blockDim.x, vdp = nthr / CS, nwt = nthr >> 6;
  float* sk = lds;                       // [TC][DMAX]
  float* sq = sk + MM_TC * DMAX;         // [TC][DMAX]
  float* sg = sq + MM_TC * DMAX;         // [3][TC] keep, take, exp(-m)
  float* sred = sg + 3 * MM_TC;          // [TC][wavefronts] partial n . q
  float* so = sred + MM_TC * nwt;        // [CS][TC][vdp] partial outputs (CS > 1)
  const int h = blockIdx.x, b = blockIdx.y;
  const int vl = tid % vdp, cs = tid / vdp;          // column inside the slice, split of the key channels
  const int v = blockIdx.z * vdp + vl;
  const int cb = cs * DC;
  const bool active = v < vd;
  const int col = active ? v : 0;
  const int t0 = p.cu_q[b], t1 = p.cu_q[b + 1];
  if (t1 <= t0) return;
  float* S_g = p.state + ((int64_t)p.slots[b] * p.H + h) * p.per_head;
  const int copy0 = blockIdx.z * (vdp / MEM_SLICE);                     // first of the n | m copies this workgroup owns
  const int ncopies = min(vdp / MEM_SLICE, (vd + MEM_SLICE - 1) / MEM_SLICE - copy0);
  float* n_g = S_g + (int64_t)p.dim * vd + (int64_t)copy0 * (p.dim + 1);
  const bool fresh = p.past[b] == 0;
  float S[DC];
#pragma unroll
  for (int i = 0; i < DC; ++i) S[i] = (active && cb + i < p.dim && !fresh) ? S_g[(int64_t)(cb + i) * vd + v] : 0.0f;
  const bool has_n = MODE == MEM_EXPGATE && tid < p.dim;
  float nreg = (has_n && !fresh) ? n_g[tid] : 0.0f;
  float m_run = (MODE == MEM_EXPGATE && tid == 0 && !fresh) ? n_g[p.dim] : 0.0f;   // walked by thread 0 only
  const float decay = MODE == MEM_CONST ? p.decay[h] : 0.0f;
  const T* bias = reinterpret_cast<const T*>(p.bias);
  for (int c0 = t0; c0 < t1; c0 += MM_TC) {
    const int nt = min(MM_TC, t1 - c0);
    float vreg[MM_TC];
#pragma unroll
    for (int j = 0; j < MM_TC; ++j) {
      vreg[j] = 0.0f;
      if (j < nt) vreg[j] = maybe_silu(p.proj[(int64_t)(c0 + j) * p.proj_rs + p.v_off + h * vd + col], p.silu);
    }
    __syncthreads();                     // the previous chunk's rows are no longer read
    for (int base = tid * 4; base < nt * DMAX; base += nthr * 4) {
      const int j = base / DMAX, i = base % DMAX;          // DMAX is a multiple of 4: the four share a token
      float k4[4], q4[4];
      const float* row = p.proj + (int64_t)(c0 + j) * p.proj_rs + h * p.dim;
      const float* rot_row = p.rot + (int64_t)(c0 + j) * p.rot_dims;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const bool in = i + e < p.dim;
        k4[e] = in ? turned(p, row + p.k_off, i + e, rot_row) * p.k_scale : 0.0f;
        q4[e] = in ? turned(p, row + p.q_off, i + e, rot_row) * p.q_scale : 0.0f;
      }
      *reinterpret_cast<float4*>(sk + base) = make_float4(k4[0], k4[1], k4[2], k4[3]);
      *reinterpret_cast<float4*>(sq + base) = make_float4(q4[0], q4[1], q4[2], q4[3]);
    }
    // the chunk's gates are a scalar chain: one thread walks it while the others stage
    if (MODE == MEM_EXPGATE && tid == 0) {
      for (int j = 0; j < nt; ++j) {
        const float* row = p.proj + (int64_t)(c0 + j) * p.proj_rs;
        float zi = row[p.i_off + h], zf = row[p.f_off + h];
        if (bias) {
          zi += ld_f32<T>(bias + p.i_off + h);
          zf += ld_f32<T>(bias + p.f_off + h);
        }
        const float ig = p.cap * tanhf(zi / p.cap);
        const float fg = log_sigmoid_f32(p.cap * tanhf(zf / p.cap));
        const float m_new = fmaxf(fg + m_run, ig);
        sg[j] = expf(fg + m_run - m_new);
        sg[MM_TC + j] = expf(ig - m_new);
        sg[2 * MM_TC + j] = expf(-m_new);
        m_run = m_new;
      }
    }
    __syncthreads();
    float o[MM_TC], pn[MM_TC];
#pragma unroll
    for (int j = 0; j < MM_TC; ++j) {
      float acc0 = 0.0f, acc1 = 0.0f;
      pn[j] = 0.0f;
      if (j < nt) {
        const float keep = MODE == MEM_CONST ? decay : sg[j];
        const float take = MODE == MEM_CONST ? 1.0f : sg[MM_TC + j];
        const float vv = vreg[j] * take;
        const float4* k4 = reinterpret_cast<const float4*>(sk + j * DMAX + cb);
        const float4* q4 = reinterpret_cast<const float4*>(sq + j * DMAX + cb);
#pragma unroll
        for (int i = 0; i < DC / 4; ++i) {
          const float4 k = k4[i], q = q4[i];
          S[4 * i + 0] = keep * S[4 * i + 0] + k.x * vv;
          S[4 * i + 1] = keep * S[4 * i + 1] + k.y * vv;
          S[4 * i + 2] = keep * S[4 * i + 2] + k.z * vv;
          S[4 * i + 3] = keep * S[4 * i + 3] + k.w * vv;
          acc0 += S[4 * i + 0] * q.x;
          acc1 += S[4 * i + 1] * q.y;
          acc0 += S[4 * i + 2] * q.z;
          acc1 += S[4 * i + 3] * q.w;
        }
        if (has_n) {
          nreg = keep * nreg + take * sk[j * DMAX + tid];
          pn[j] = nreg * sq[j * DMAX + tid];
        }
      }
      o[j] = acc0 + acc1;
    }
    if constexpr (CS > 1) {
#pragma unroll
      for (int j = 0; j < MM_TC; ++j) so[(cs * MM_TC + j) * vdp + vl] = o[j];
    }
    if constexpr (MODE == MEM_EXPGATE) {
#pragma unroll
      for (int j = 0; j < MM_TC; ++j) {
        const float s = wave_sum(pn[j]);
        if ((tid & 63) == 0) sred[j * nwt + (tid >> 6)] = s;
      }
    }
    if constexpr (CS > 1 || MODE == MEM_EXPGATE) __syncthreads();
    if (cs == 0 && active) {
#pragma unroll
      for (int j = 0; j < MM_TC; ++j) {
        if (j < nt) {
          float r = o[j];
          if constexpr (CS > 1) {
            r = 0.0f;
#pragma unroll
            for (int q = 0; q < CS; ++q) r += so[(q * MM_TC + j) * vdp + vl];
          }
          if constexpr (MODE == MEM_EXPGATE) {
            float nq = 0.0f;
            for (int w = 0; w < nwt; ++w) nq += sred[j * nwt + w];
            r /= fmaxf(fabsf(nq), sg[2 * MM_TC + j]) + 1e-6f;
          }
          p.out[(int64_t)(c0 + j) * p.out_rs + h * vd + v] = r;
        }
      }
    }
  }
  if (active) {
#pragma unroll
    for (int i = 0; i < DC; ++i)
      if (cb + i < p.dim) S_g[(int64_t)(cb + i) * vd + v] = S[i];
  }
  for (int c = 0; c < ncopies; ++c) {
    if (has_n) n_g[c * (p.dim + 1) + tid] = nreg;
    if (MODE == MEM_EXPGATE && tid == 0) n_g[c * (p.dim + 1) + p.dim] = m_run;
  }
}

// States too large for a workgroup's registers: the state stays in its slot (fp32, through the caches) and is read and
// written once per token; thread v owns column v, so no two threads touch the same entry.  Slow and general.
template <typename T, int MODE>
__global__ __launch_bounds__(256) void matrix_memory_generic_kernel(MemArgs p) {
  extern __shared__ float4 lds4[];
  float* sk = reinterpret_cast<float*>(lds4);   // [dim]
  float* sq = sk + p.dim;                       // [dim]
  float* sg = sq + p.dim;                       // keep, take, exp(-m), then 32 floats for sums
  float* red = sg + 4;
  const int vd = p.vdim, tid = threadIdx.x, nthr = blockDim.x;
  const int h = blockIdx.x, b = blockIdx.y;
  const int t0 = p.cu_q[b], t1 = p.cu_q[b + 1];
  if (t1 <= t0) return;
  float* S_g = p.state + ((int64_t)p.slots[b] * p.H + h) * p.per_head;
  float* n_g = S_g + (int64_t)p.dim * vd;           // copies of n | m, one per 64 value columns, all kept equal
  const int copies = (vd + MEM_SLICE - 1) / MEM_SLICE;
  if (p.past[b] == 0)
    for (int i = tid; i < p.per_head; i += nthr) S_g[i] = 0.0f;
  float m_run = (MODE == MEM_EXPGATE && tid == 0 && p.past[b] != 0) ? n_g[p.dim] : 0.0f;
  const float decay = MODE == MEM_CONST ? p.decay[h] : 0.0f;
  const T* bias = reinterpret_cast<const T*>(p.bias);
  __syncthreads();
  for (int t = t0; t < t1; ++t) {
    const float* row = p.proj + (int64_t)t * p.proj_rs;
    for (int i = tid; i < p.dim; i += nthr) {
      const float* rot_row = p.rot + (int64_t)t * p.rot_dims;
      sk[i] = turned(p, row + p.k_off + h * p.dim, i, rot_row) * p.k_scale;
      sq[i] = turned(p, row + p.q_off + h * p.dim, i, rot_row) * p.q_scale;
    }
    if (tid == 0) {
      if constexpr (MODE == MEM_EXPGATE) {
        float zi = row[p.i_off + h], zf = row[p.f_off + h];
        if (bias) {
          zi += ld_f32<T>(bias + p.i_off + h);
          zf += ld_f32<T>(bias + p.f_off + h);
        }
        const float ig = p.cap * tanhf(zi / p.cap);
        const float fg = log_sigmoid_f32(p.cap * tanhf(zf / p.cap));
        const float m_new = fmaxf(fg + m_run, ig);
        sg[0] = expf(fg + m_run - m_new);
        sg[1] = expf(ig - m_new);
        sg[2] = expf(-m_new);
        m_run = m_new;
      } else {
        sg[0] = decay;
        sg[1] = 1.0f;
        sg[2] = 0.0f;
      }
    }
    __syncthreads();
    const float keep = sg[0], take = sg[1];
    float den = 1.0f;
    if constexpr (MODE == MEM_EXPGATE) {
      float pn = 0.0f;
      for (int i = tid; i < p.dim; i += nthr) {
        const float n = keep * n_g[i] + take * sk[i];
        for (int c = 0; c < copies; ++c) n_g[c * (p.dim + 1) + i] = n;
        pn += n * sq[i];
      }
      den = fmaxf(fabsf(block_sum(pn, red)), sg[2]) + 1e-6f;
    }
    for (int v = tid; v < vd; v += nthr) {
      const float vv = maybe_silu(row[p.v_off + h * vd + v], p.silu) * take;
      float acc = 0.0f;
      for (int i = 0; i < p.dim; ++i) {
        const float sv = keep * S_g[(int64_t)i * vd + v] + sk[i] * vv;
        S_g[(int64_t)i * vd + v] = sv;
        acc += sv * sq[i];
      }
      p.out[(int64_t)t * p.out_rs + h * vd + v] = acc / den;
    }
    __syncthreads();   // sk / sq / sg are rewritten by the next token
  }
  if (MODE == MEM_EXPGATE && tid == 0)
    for (int c = 0; c < copies; ++c) n_g[c * (p.dim + 1) + p.dim] = m_run;
}

// One token per request in the first form, with what follows it per head: o = S^T q after the update, divided by its root
// mean square, times silu (or sigmoid) of the gate.  A workgroup owns one (head, request): lanes take four state columns
// each, the key rows are dealt to the row groups of CG = vdim / 4 lanes, eight rows of state per thread in flight; the row
// groups' partial o meet in LDS.
constexpr int RS_THREADS = 512, RS_ROWS = 8;

struct StepArgs {
  MemArgs m;
  int g_off, gate_silu;
  float eps;
  void* out;             // [tokens, out_rs] in the storage type
  int64_t out_rs;
};

template <typename T>
__global__ __launch_bounds__(RS_THREADS) void retention_step_kernel(StepArgs a) {
  const MemArgs& p = a.m;
  typedef typename Pack4<T>::type P;
  extern __shared__ float4 lds4[];
  __shared__ float red[32];
  const int d = p.dim, vd = p.vdim, CG = vd >> 2, RG = RS_THREADS / CG;
  float* so = reinterpret_cast<float*>(lds4);     // [RG][vd]
  float* sq = so + RG * vd;                       // [d]
  float* sk = sq + d;                             // [d]
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int t = p.cu_q[b];
  if (p.cu_q[b + 1] <= t) return;
  const int rg = tid / CG, c = (tid - rg * CG) * 4;
  const bool on = rg < RG;
  const bool fresh = p.past[b] == 0;
  float* S_g = p.state + ((int64_t)p.slots[b] * p.H + h) * p.per_head;
  const float* row = p.proj + (int64_t)t * p.proj_rs;
  f32x4 s[RS_ROWS];
  auto load = [&](int first) {
#pragma unroll
    for (int i = 0; i < RS_ROWS; ++i) {
      const int r = first + i * RG;
      s[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
      if (on && !fresh && r < d) s[i] = *reinterpret_cast<const f32x4*>(S_g + (int64_t)r * vd + c);
    }
  };
  load(rg);
  const f32x4 v = on ? *reinterpret_cast<const f32x4*>(row + p.v_off + h * vd + c) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  const f32x4 z = on && rg == 0 ? *reinterpret_cast<const f32x4*>(row + a.g_off + h * vd + c) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  const float decay = p.decay[h];
  const float* rot_row = p.rot + (int64_t)t * p.rot_dims;
  for (int i = tid; i < d; i += RS_THREADS) {
    sk[i] = turned(p, row + p.k_off + h * d, i, rot_row) * p.k_scale;
    sq[i] = turned(p, row + p.q_off + h * d, i, rot_row) * p.q_scale;
  }
  __syncthreads();
  f32x4 o = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  for (int first = rg; on && first < d; first += RS_ROWS * RG) {
    if (first != rg) load(first);
#pragma unroll
    for (int i = 0; i < RS_ROWS; ++i) {
      const int r = first + i * RG;
      if (r >= d) continue;
      const float k = sk[r], q = sq[r];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s[i][e] = decay * s[i][e] + k * v[e];
        o[e] += s[i][e] * q;
      }
      *reinterpret_cast<f32x4*>(S_g + (int64_t)r * vd + c) = s[i];
    }
  }
  if (on) *reinterpret_cast<f32x4*>(so + rg * vd + c) = o;
  __syncthreads();
  float ss = 0.0f;
  if (rg == 0) {
    for (int g = 1; g < RG; ++g) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(so + g * vd + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += x[e];
    }
    ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)vd + a.eps);
  if (rg != 0) return;
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] *= inv * (a.gate_silu ? silu_f32(z[e]) : sigmoid_f32(z[e]));
  *reinterpret_cast<P*>(reinterpret_cast<T*>(a.out) + (int64_t)t * a.out_rs + h * vd + c) = Pack4<T>::narrow(o);
}

// A workgroup of eight wavefronts owns one (head, request, slice of 64 state columns) and walks the request's tokens of this
// step in chunks of C.  In LDS: the chunk's q and k rows (rotated, scaled), its values and the state TRANSPOSED (column
// major: the products read four consecutive k numbers of a row or column per access), the decayed scores.  The state itself
// stays in the wavefronts' accumulators from chunk to chunk; its LDS copy serves the products with q.  Matrix steps of four
// numbers take the numbers {16 kk + 4 g + m : g = 0 .. 3} of a sum in step m, so one 16-byte access feeds four of them.
// The next chunk's rows are on their way from memory while a chunk is worked on.
constexpr int RC_WAVES = 8, RC_COLS = 64;

constexpr size_t rc_lds_floats(int dmax, int c) {
  return (size_t)(2 * c + RC_COLS) * (dmax + 4) + (size_t)(RC_COLS + c) * (c + 4) + c + 4;
}

template <int DMAX, int C>
__global__ __launch_bounds__(64 * RC_WAVES) void retention_chunk_kernel(MemArgs p) {
  constexpr int DP = DMAX + 4, CP = C + 4, DT = DMAX / 16, CT = C / 16, NTHR = 64 * RC_WAVES;
  constexpr int UNITS = C * (DMAX / 8) / NTHR, VUNITS = C * (RC_COLS / 4) / NTHR;       // staged pieces per thread
  constexpr int OT = CT * 4 / RC_WAVES, ST = DT * 4 / RC_WAVES;                         // 16 x 16 tiles per wavefront
  static_assert(UNITS >= 1 && VUNITS >= 1 && OT >= 1 && ST >= 1 && (ST <= 4 || ST % 4 == 0), "tiles fit the wavefronts");
  extern __shared__ float4 lds4[];
  float* sq = reinterpret_cast<float*>(lds4);     // [C][DP]
  float* sk = sq + C * DP;                        // [C][DP]
  float* st = sk + C * DP;                        // [64][DP] state, transposed
  float* sv = st + RC_COLS * DP;                  // [64][CP] values, transposed
  float* sp = sv + RC_COLS * CP;                  // [C][CP] decayed scores
  float* pw = sp + C * CP;                        // [C + 1] powers of the decay
  const int h = blockIdx.x, b = blockIdx.y, col0 = blockIdx.z * RC_COLS;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lc = lane & 15, lg = lane >> 4;
  const int d = p.dim, vd = p.vdim, half = p.rot_dims >> 1;
  const int t0 = p.cu_q[b], t1 = p.cu_q[b + 1];
  if (t1 <= t0) return;
  float* S_g = p.state + ((int64_t)p.slots[b] * p.H + h) * p.per_head;
  const bool fresh = p.past[b] == 0;
  for (int i = tid; i <= C; i += NTHR) pw[i] = (float)pow((double)p.decay[h], (double)i);

  // staging: unit u of a token is a pair of four-number pieces of q and k that turn together (or two that do not turn)
  const f32x4 zero = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  f32x4 q_a[UNITS], q_b[UNITS], k_a[UNITS], k_b[UNITS], cs[UNITS], sn[UNITS], vv[VUNITS];
  auto places = [&](int i, int& j, int& a, int& c) {
    const int u = tid + i * NTHR, pu = u % (DMAX / 8);
    j = u / (DMAX / 8);
    a = pu * 4 < half ? pu * 4 : p.rot_dims + (pu * 4 - half) * 2;
    c = pu * 4 < half ? a + half : a + 4;
  };
  auto fetch = [&](int c0) {
    const int n = min(C, t1 - c0);
#pragma unroll
    for (int i = 0; i < UNITS; ++i) {
      int j, a, c;
      places(i, j, a, c);
      q_a[i] = q_b[i] = k_a[i] = k_b[i] = cs[i] = sn[i] = zero;
      if (j < n && a < d) {
        const float* row = p.proj + (int64_t)(c0 + j) * p.proj_rs + h * d;
        q_a[i] = *reinterpret_cast<const f32x4*>(row + p.q_off + a);
        q_b[i] = *reinterpret_cast<const f32x4*>(row + p.q_off + c);
        k_a[i] = *reinterpret_cast<const f32x4*>(row + p.k_off + a);
        k_b[i] = *reinterpret_cast<const f32x4*>(row + p.k_off + c);
        if (a < half) {
          const float* rot = p.rot + (int64_t)(c0 + j) * p.rot_dims;
          cs[i] = *reinterpret_cast<const f32x4*>(rot + a);
          sn[i] = *reinterpret_cast<const f32x4*>(rot + half + a);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < VUNITS; ++i) {
      const int u = tid + i * NTHR, j = (u & 15) + 16 * (u / 256), c = col0 + ((u >> 4) & 15) * 4;
      vv[i] = zero;
      if (j < n && c < vd) vv[i] = *reinterpret_cast<const f32x4*>(p.proj + (int64_t)(c0 + j) * p.proj_rs + p.v_off + h * vd + c);
    }
  };
  auto store = [&]() {
#pragma unroll
    for (int i = 0; i < UNITS; ++i) {
      int j, a, c;
      places(i, j, a, c);
      const bool turn = a < half;
      f32x4 qa = q_a[i], qb = q_b[i], ka = k_a[i], kb = k_b[i];
      if (p.silu) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          qa[e] = silu_f32(qa[e]);
          qb[e] = silu_f32(qb[e]);
          ka[e] = silu_f32(ka[e]);
          kb[e] = silu_f32(kb[e]);
        }
      }
      if (turn) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float u = qa[e], v = qb[e], x = ka[e], y = kb[e];
          qa[e] = u * cs[i][e] - v * sn[i][e];
          qb[e] = v * cs[i][e] + u * sn[i][e];
          ka[e] = x * cs[i][e] - y * sn[i][e];
          kb[e] = y * cs[i][e] + x * sn[i][e];
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        qa[e] *= p.q_scale;
        qb[e] *= p.q_scale;
        ka[e] *= p.k_scale;
        kb[e] *= p.k_scale;
      }
      *reinterpret_cast<f32x4*>(sq + j * DP + a) = qa;
      *reinterpret_cast<f32x4*>(sq + j * DP + c) = qb;
      *reinterpret_cast<f32x4*>(sk + j * DP + a) = ka;
      *reinterpret_cast<f32x4*>(sk + j * DP + c) = kb;
    }
#pragma unroll
    for (int i = 0; i < VUNITS; ++i) {
      const int u = tid + i * NTHR, j = (u & 15) + 16 * (u / 256), c = ((u >> 4) & 15) * 4;
#pragma unroll
      for (int e = 0; e < 4; ++e) sv[(c + e) * CP + j] = maybe_silu(vv[i][e], p.silu);
    }
  };
  auto at4 = [](const float* q) { return *reinterpret_cast<const f32x4*>(q); };
  auto step4 = [](const f32x4& a, const f32x4& x, f32x4 acc) {
#pragma unroll
    for (int m = 0; m < 4; ++m) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[m], x[m], acc, 0, 0, 0);
    return acc;
  };

  // this wavefront's tiles: outputs (row tile o_row, column tiles o_col ..), state (tiles s0 .. in row-major order of 4 columns)
  const int o_row = wv * OT / 4, o_col = wv * OT % 4, s0 = wv * ST;
  f32x4 acc_s[ST];
#pragma unroll
  for (int i = 0; i < ST; ++i) {
    const int row = (s0 + i) / 4 * 16 + lg * 4, c = (s0 + i) % 4 * 16 + lc;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc_s[i][r] = (!fresh && row + r < d && col0 + c < vd) ? S_g[(int64_t)(row + r) * vd + col0 + c] : 0.0f;
    *reinterpret_cast<f32x4*>(st + c * DP + row) = acc_s[i];
  }
  fetch(t0);
  for (int c0 = t0; c0 < t1; c0 += C) {
    const int n = min(C, t1 - c0), nt = (n + 15) / 16;
    store();
    __syncthreads();
    if (c0 + C < t1) fetch(c0 + C);
    // scores of the tiles on and below the diagonal, decayed
    for (int idx = wv; idx < nt * (nt + 1) / 2; idx += RC_WAVES) {
      int ti = 0;
      while ((ti + 1) * (ti + 2) / 2 <= idx) ++ti;
      const int tj = idx - ti * (ti + 1) / 2;
      f32x4 acc0 = zero, acc1 = zero;
#pragma unroll
      for (int kk = 0; kk < DT; kk += 2) {
        acc0 = step4(at4(sq + (ti * 16 + lc) * DP + kk * 16 + lg * 4), at4(sk + (tj * 16 + lc) * DP + kk * 16 + lg * 4), acc0);
        acc1 = step4(at4(sq + (ti * 16 + lc) * DP + kk * 16 + 16 + lg * 4), at4(sk + (tj * 16 + lc) * DP + kk * 16 + 16 + lg * 4),
                     acc1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = ti * 16 + lg * 4 + r, j = tj * 16 + lc;
        sp[i * CP + j] = j <= i ? (acc0[r] + acc1[r]) * pw[i - j] : 0.0f;
      }
    }
    // what the state ahead of the chunk contributes
    f32x4 acc_o[OT];
#pragma unroll
    for (int o = 0; o < OT; ++o) acc_o[o] = zero;
    if (o_row < nt) {
#pragma unroll
      for (int kk = 0; kk < DT; ++kk) {
        const f32x4 a = at4(sq + (o_row * 16 + lc) * DP + kk * 16 + lg * 4);
#pragma unroll
        for (int o = 0; o < OT; ++o) acc_o[o] = step4(a, at4(st + ((o_col + o) * 16 + lc) * DP + kk * 16 + lg * 4), acc_o[o]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float f = pw[o_row * 16 + lg * 4 + r + 1];
#pragma unroll
        for (int o = 0; o < OT; ++o) acc_o[o][r] *= f;
      }
    }
    __syncthreads();
    if (o_row < nt) {
      for (int kk = 0; kk <= o_row; ++kk) {
        const f32x4 a = at4(sp + (o_row * 16 + lc) * CP + kk * 16 + lg * 4);
#pragma unroll
        for (int o = 0; o < OT; ++o) acc_o[o] = step4(a, at4(sv + ((o_col + o) * 16 + lc) * CP + kk * 16 + lg * 4), acc_o[o]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = o_row * 16 + lg * 4 + r;
        if (i >= n) continue;
        float* orow = p.out + (int64_t)(c0 + i) * p.out_rs + h * vd + col0;
#pragma unroll
        for (int o = 0; o < OT; ++o) {
          const int c = (o_col + o) * 16 + lc;
          if (col0 + c < vd) orow[c] = acc_o[o][r];
        }
      }
    }
    // the state behind the chunk
    const float keep = pw[n];
#pragma unroll
    for (int i = 0; i < ST; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc_s[i][r] *= keep;
    for (int kk = 0; kk < nt; ++kk) {
      float f[4];
#pragma unroll
      for (int m = 0; m < 4; ++m) f[m] = pw[max(n - 1 - (kk * 16 + lg * 4 + m), 0)];       // rows past n are zero
      constexpr int COLS = ST < 4 ? ST : 4;                        // column tiles that share a piece of k
      f32x4 x[COLS];
#pragma unroll
      for (int c = 0; c < COLS; ++c) x[c] = at4(sv + ((s0 + c) % 4 * 16 + lc) * CP + kk * 16 + lg * 4);
#pragma unroll
      for (int rt = 0; rt < ST / COLS; ++rt) {
        const int row = (s0 / 4 + rt) * 16 + lc;
        f32x4 a;
#pragma unroll
        for (int m = 0; m < 4; ++m) a[m] = sk[(kk * 16 + lg * 4 + m) * DP + row] * f[m];
#pragma unroll
        for (int c = 0; c < COLS; ++c) acc_s[rt * COLS + c] = step4(a, x[c], acc_s[rt * COLS + c]);
      }
    }
    if (c0 + C < t1) {
#pragma unroll
      for (int i = 0; i < ST; ++i)
        *reinterpret_cast<f32x4*>(st + ((s0 + i) % 4 * 16 + lc) * DP + (s0 + i) / 4 * 16 + lg * 4) = acc_s[i];
      __syncthreads();                 // q, k, v and scores of this chunk are no longer read
    }
  }
#pragma unroll
  for (int i = 0; i < ST; ++i) {
    const int row = (s0 + i) / 4 * 16 + lg * 4, c = (s0 + i) % 4 * 16 + lc;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (row + r < d && col0 + c < vd) S_g[(int64_t)(row + r) * vd + col0 + c] = acc_s[i][r];
  }
}

template <int DMAX, int C>
hipError_t launch_retention_chunk(const MemArgs& p, dim3 grid, hipStream_t s) {
  constexpr size_t lds = rc_lds_floats(DMAX, C) * sizeof(float);
  static_assert(lds <= 160 * 1024, "the chunk fits the LDS");
  static bool allowed = false;
  if (!allowed) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_chunk_kernel<DMAX, C>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    allowed = true;
  }
  retention_chunk_kernel<DMAX, C><<<grid, dim3(64 * RC_WAVES), lds, s>>>(p);
  return hipGetLastError();
}

template <typename T, int DMAX, int CS>
void launch_mem_mode(const MemArgs& p, int mode, dim3 grid, int threads, size_t lds, hipStream_t s) {
  if (mode == MEM_CONST) matrix_memory_kernel<T, DMAX, CS, MEM_CONST><<<grid, dim3(threads), lds, s>>>(p);
  else matrix_memory_kernel<T, DMAX, CS, MEM_EXPGATE><<<grid, dim3(threads), lds, s>>>(p);
}

template <typename T, int DMAX>
void launch_mem_cs(const MemArgs& p, int mode, int cs, dim3 grid, int threads, size_t lds, hipStream_t s) {
  if constexpr (DMAX >= 64) {
    if (cs == 4) return launch_mem_mode<T, DMAX, 4>(p, mode, grid, threads, lds, s);
  }
  if constexpr (DMAX >= 32 && DMAX <= 128) {
    if (cs == 2) return launch_mem_mode<T, DMAX, 2>(p, mode, grid, threads, lds, s);
  }
  if constexpr (DMAX <= 64) launch_mem_mode<T, DMAX, 1>(p, mode, grid, threads, lds, s);
}

template <typename T>
void launch_mem(const MemArgs& p, int mode, int dmax, int cs, dim3 grid, int threads, size_t lds, hipStream_t s) {
  switch (dmax) {
    case 16: return launch_mem_cs<T, 16>(p, mode, cs, grid, threads, lds, s);
    case 32: return launch_mem_cs<T, 32>(p, mode, cs, grid, threads, lds, s);
    case 64: return launch_mem_cs<T, 64>(p, mode, cs, grid, threads, lds, s);
    case 128: return launch_mem_cs<T, 128>(p, mode, cs, grid, threads, lds, s);
    default: return launch_mem_cs<T, 256>(p, mode, cs, grid, threads, lds, s);
  }
}

}  // namespace

extern "C" int64_t nv_matrix_memory_state_size(int mode, int dim, int vdim) {
  return (int64_t)dim * vdim + (mode == MEM_EXPGATE ? (int64_t)((vdim + MEM_SLICE - 1) / MEM_SLICE) * (dim + 1) : 0);
}

extern "C" int nv_matrix_memory(const float* proj, int64_t proj_row_stride, int q_off, int k_off, int v_off, int i_off,
                                int f_off, const void* bias, const float* decay, float* state, const int32_t* cu_q,
                                const int32_t* past_lens, const int32_t* state_slots, float* out, int64_t out_row_stride,
                                int num_seqs, int heads, int dim, int vdim, int mode, int silu, float q_scale,
                                float k_scale, const float* rot, int rot_dims, float cap, int max_q, int dtype,
                                nv_stream_t stream) {
  NV_CHECK_ARG(proj && state && cu_q && past_lens && state_slots && out, "nv_matrix_memory: null pointer");
  NV_CHECK_ARG(dtype == NV_BF16 || dtype == NV_F32, "nv_matrix_memory: bad dtype %d", dtype);
  NV_CHECK_ARG(mode == MEM_CONST || mode == MEM_EXPGATE, "nv_matrix_memory: bad mode %d", mode);
  NV_CHECK_ARG(mode != MEM_CONST || decay, "nv_matrix_memory: constant decays are missing");
  NV_CHECK_ARG(mode != MEM_EXPGATE || cap > 0.0f, "nv_matrix_memory: the gate cap must be positive");
  NV_CHECK_ARG(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || rot),
               "nv_matrix_memory: a rotation over %d of %d numbers needs its cosines and sines", rot_dims, dim);
  NV_CHECK_ARG(heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && num_seqs >= 0 && num_seqs <= 65535,
               "nv_matrix_memory: bad shape heads=%d dim=%d vdim=%d seqs=%d", heads, dim, vdim, num_seqs);
  if (num_seqs == 0) return NV_OK;
  int dmax = 16;
  while (dmax < dim) dmax *= 2;
  // One workgroup per slice of 64 state columns, the key channels of a column split over as many threads as leave each
  // at least 16 of them ...
  int slices = (vdim + MEM_SLICE - 1) / MEM_SLICE, cs = dmax >= 64 ? 4 : dmax / 16, vdp = MEM_SLICE;
  // ... unless the launch fills the chip anyway (many requests): then one workgroup walks all columns, if that fits 256
  // threads with at most 64 state registers each (shared staging and fewer, fuller workgroups win there)
  if (slices > 1 && (int64_t)heads * num_seqs >= 512) {
    const int vround = slices * MEM_SLICE;
    int cu = 1;
    while (cu < 4 && vround * cu * 2 <= 256 && dmax / (cu * 2) >= 16) cu *= 2;
    if (vround * cu <= 256 && dmax / cu <= 64 && vround * cu >= dim) {
      cs = cu;
      vdp = vround;
      slices = 1;
    }
  }
  const int threads = vdp * cs;
  MemArgs p{proj, proj_row_stride, q_off, k_off, v_off, i_off, f_off, bias, decay, state, cu_q, past_lens, state_slots,
            out, out_row_stride, heads, dim, vdim, (int)nv_matrix_memory_state_size(mode, dim, vdim), silu, q_scale, k_scale, cap,
            rot, rot_dims};
  // prompts with one constant decay per head: chunks on the matrix cores
  auto al16 = [](const void* q) { return (uintptr_t)q % 16 == 0; };
  const int vslices = (vdim + RC_COLS - 1) / RC_COLS;
  if (mode == MEM_CONST && max_q >= MM_TC && dim % 8 == 0 && dim <= 256 && vdim % 4 == 0 && rot_dims % 8 == 0 &&
      q_off % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 && proj_row_stride % 4 == 0 && al16(proj) && al16(rot) &&
      vslices <= 65535 && getenv("NV_MATRIX_MEMORY_STEPS") == nullptr && getenv("NV_MATRIX_MEMORY_GENERIC") == nullptr) {
    const dim3 grid(heads, num_seqs, vslices);
    const hipError_t e = dim <= 64    ? launch_retention_chunk<64, 64>(p, grid, (hipStream_t)stream)
                         : dim <= 128 ? launch_retention_chunk<128, 64>(p, grid, (hipStream_t)stream)
                                      : launch_retention_chunk<256, 32>(p, grid, (hipStream_t)stream);
    if (e != hipSuccess) {
      nv_set_error("nv_matrix_memory: %s", hipGetErrorString(e));
      return NV_ERR_LAUNCH;
    }
    return NV_OK;
  }
  if (dmax > 256 || slices > 65535 || getenv("NV_MATRIX_MEMORY_GENERIC") != nullptr) {
    const size_t glds = ((size_t)2 * dim + 4 + 32) * sizeof(float);
    NV_CHECK_ARG(glds <= 64 * 1024, "nv_matrix_memory: keys of %d numbers exceed the LDS", dim);
    dim3 grid(heads, num_seqs);
    if (mode == MEM_CONST) {
      NV_DISPATCH_T(dtype, matrix_memory_generic_kernel<T, MEM_CONST><<<grid, dim3(256), glds, (hipStream_t)stream>>>(p));
    } else {
      NV_DISPATCH_T(dtype, matrix_memory_generic_kernel<T, MEM_EXPGATE><<<grid, dim3(256), glds, (hipStream_t)stream>>>(p));
    }
    NV_CHECK_LAUNCH();
    return NV_OK;
  }
  const size_t lds =
      (size_t)(MM_TC * 2 * dmax + 3 * MM_TC + MM_TC * (threads / 64) + (cs > 1 ? cs * MM_TC * vdp : 0)) * sizeof(float);
  NV_CHECK_ARG(lds <= 64 * 1024 && threads <= 256, "nv_matrix_memory: launch plan out of range");
  NV_DISPATCH_T(dtype, launch_mem<T>(p, mode, dmax, cs, dim3(heads, num_seqs, slices), threads, lds, (hipStream_t)stream));
  NV_CHECK_LAUNCH();
  return NV_OK;
}

extern "C" int nv_retention_step_ok(const float* proj, int64_t proj_row_stride, int q_off, int k_off, int v_off, int g_off,
                                    const float* state, const void* out, int64_t out_row_stride, int dim, int vdim) {
  auto al16 = [](const void* q) { return (uintptr_t)q % 16 == 0; };
  const size_t rg = RS_THREADS / (vdim >= 4 ? vdim / 4 : 1);
  return vdim % 4 == 0 && vdim <= 1024 && (rg * vdim + 2 * (size_t)dim) * sizeof(float) <= 60 * 1024 && v_off % 4 == 0 &&
         g_off % 4 == 0 && proj_row_stride % 4 == 0 && out_row_stride % 4 == 0 && al16(proj) && al16(state) && al16(out);
}

extern "C" int nv_retention_step(const float* proj, int64_t proj_row_stride, int q_off, int k_off, int v_off, int g_off,
                                 const float* decay, float* state, const int32_t* cu_q, const int32_t* past_lens,
                                 const int32_t* state_slots, const float* rot, int rot_dims, float q_scale, float k_scale,
                                 float eps, int gate_silu, void* out, int64_t out_row_stride, int num_seqs, int heads, int dim,
                                 int vdim, int dtype, nv_stream_t stream) {
  NV_CHECK_ARG(proj && decay && state && cu_q && past_lens && state_slots && out, "nv_retention_step: null pointer");
  NV_CHECK_ARG(dtype == NV_BF16 || dtype == NV_F32, "nv_retention_step: bad dtype %d", dtype);
  NV_CHECK_ARG(heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && num_seqs >= 0 && num_seqs <= 65535 &&
                   nv_retention_step_ok(proj, proj_row_stride, q_off, k_off, v_off, g_off, state, out, out_row_stride, dim, vdim),
               "nv_retention_step: heads=%d dim=%d vdim=%d seqs=%d or an alignment this launch does not serve", heads, dim, vdim,
               num_seqs);
  NV_CHECK_ARG(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || rot),
               "nv_retention_step: a rotation over %d of %d numbers needs its cosines and sines", rot_dims, dim);
  if (num_seqs == 0) return NV_OK;
  StepArgs a{{proj, proj_row_stride, q_off, k_off, v_off, 0, 0, nullptr, decay, state, cu_q, past_lens, state_slots, nullptr, 0,
              heads, dim, vdim, dim * vdim, 0, q_scale, k_scale, 0.0f, rot, rot_dims},
             g_off, gate_silu, eps, out, out_row_stride};
  const size_t lds = ((size_t)(RS_THREADS / (vdim / 4)) * vdim + 2 * (size_t)dim) * sizeof(float);
  NV_DISPATCH_T(dtype, retention_step_kernel<T><<<dim3(heads, num_seqs), dim3(RS_THREADS), lds, (hipStream_t)stream>>>(a));
  NV_CHECK_LAUNCH();
  return NV_OK;
}
