// Gated delta rule over RAGGED steps: per head an fp32 state S [dk, dv] that forgets per key entry and is corrected towards the
// token's value along the token's key,
//
//     S <- diag(g_t) S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t,
//
// with k and q unit vectors (q times a constant), beta = sigmoid of a projected number per head and
// g = exp(-exp(A_log_h) softplus(z + dt_bias)) per key entry from projected rows z.
//
//   ll_delta_scan   the whole recurrence: unit norms, decays, step sizes, walk over the state, read-out (fp32)
//
// Both reductions over the key entries are taken from the state BEFORE the token -- S^T (g k) gives the correction, and
// o = S^T (g q) + (k . q) u -- so a token costs one round of cross-lane sums instead of two, and the four products per state
// entry (two sums, the decay, the write) are independent of each other up to u.
//
// Storage dtype DT = LL_F16 / LL_BF16 / LL_F32 for the projected rows.  fp32 whatever DT: decays, their logarithms and
// exponentials, step sizes, unit norms, the state and its read-out.  A sequence whose run starts at position 0 starts from a
// zero state whatever an earlier owner of its slot left; state is never cleared on release.
#include "common.h"

#include <math.h>

namespace {

template <int DT>
__device__ __forceinline__ float ldv(const void* p, int64_t i) {
  if constexpr (DT == LL_F32) return ((const float*)p)[i];
  else return to_f32<DT>(((const uint16_t*)p)[i]);
}

constexpr int kMaxPer = 4;   // key entries a lane holds: dk <= 256

struct DeltaArgs {
  const void* q;   // [n, q_ld]: head j's entries at columns j dk ..
  const void* k;
  const void* v;   // [n, v_ld]: head h's entries at columns h dv ..
  int64_t q_ld, k_ld, v_ld;
  int heads, dk, dv;
  int qk_rep;      // value head h reads query / key head h / qk_rep
  float q_scale, unit_eps;
  const void* gate;          // rows [n, gate_ld] of heads dk raw decay logits; dt_bias [heads dk]; a_log [heads]
  int64_t gate_ld;
  const void* dt_bias;
  const void* a_log;
  const void* beta;          // rows [n, beta_ld] of one raw step size per head
  int64_t beta_ld;
  float* pre_g;              // decays of the step [n, heads, dk] and scalars [n, heads] evaluated ahead of the walk (or NULL)
  f32x4* pre_s;
  float* o;                  // fp32 [n, heads dv]
  const int32_t* seq_start;
  const int32_t* seq_first_pos;
  const int32_t* seq_slot;
  float* state;              // fp32 [slots, heads, dk, dv]
};

// fp32 storage: libm; 16-bit storage: the hardware exp2 / log2 / reciprocal (1 ulp each), log1p by the ratio t / (w - 1) that undoes
// the rounding of w = 1 + t
template <int DT>
__device__ __forceinline__ float softplus(float z) {
  if constexpr (DT == LL_F32) {
    return z > 20.f ? z : log1pf(expf(z));
  } else {
    const float t = __builtin_amdgcn_exp2f(fabsf(z) * -1.44269504088896341f);
    const float w = 1.0f + t;
    const float l = w == 1.0f ? t : __builtin_amdgcn_logf(w) * 0.693147180559945309f * t * __builtin_amdgcn_rcpf(w - 1.0f);
    return fmaxf(z, 0.f) + l;
  }
}
template <int DT>
__device__ __forceinline__ float decay_exp(float x) {
  if constexpr (DT == LL_F32) return expf(x);
  else return __builtin_amdgcn_exp2f(x * 1.44269504088896341f);
}

// Everything a (token, head) contributes besides its values, by one wave: lane l holds key entries l, l + 64, ..
// s = (factor of k, factor of q, beta, unit k . scaled unit q).  ONE definition for the walk and for the pass ahead of it.
template <int DT>
__device__ __forceinline__ f32x4 token_scalars(const DeltaArgs& a, int64_t row, int head, int lane, float (&qv)[kMaxPer], float (&kv)[kMaxPer]) {
  const int c0 = head / a.qk_rep * a.dk;
  float qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
  for (int j = 0; j < kMaxPer; ++j) {
    const int e = lane + 64 * j;
    qv[j] = kv[j] = 0.f;
    if (e < a.dk) {
      qv[j] = ldv<DT>(a.q, row * a.q_ld + c0 + e);
      kv[j] = ldv<DT>(a.k, row * a.k_ld + c0 + e);
    }
    qq += qv[j] * qv[j];
    kk += kv[j] * kv[j];
    qk += qv[j] * kv[j];
  }
  qq = wave_sum(qq);
  kk = wave_sum(kk);
  qk = wave_sum(qk);
  const float fk = 1.0f / sqrtf(kk + a.unit_eps);
  const float fq = 1.0f / sqrtf(qq + a.unit_eps) * a.q_scale;
  const float b = ldv<DT>(a.beta, row * a.beta_ld + head);
  return f32x4{fk, fq, 1.0f / (1.0f + expf(-b)), qk * fk * fq};
}

template <int DT>
__device__ __forceinline__ float entry_decay(const DeltaArgs& a, int64_t row, int head, int e, float rate) {
  const int c = head * a.dk + e;
  return decay_exp<DT>(-rate * softplus<DT>(ldv<DT>(a.gate, row * a.gate_ld + c) + ldv<DT>(a.dt_bias, c)));
}

// One wave per (token, head): decays and scalars of a step, once, ahead of the walk (whose column workgroups would each
// evaluate them again).
template <int DT>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const DeltaArgs a, int64_t items) {
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int lane = threadIdx.x & 63;
  const int64_t row = item / a.heads;
  const int head = (int)(item - row * a.heads);
  float qv[kMaxPer], kv[kMaxPer];
  const f32x4 s = token_scalars<DT>(a, row, head, lane, qv, kv);
  const float rate = expf(ldv<DT>(a.a_log, head));
#pragma unroll
  for (int j = 0; j < kMaxPer; ++j) {
    const int e = lane + 64 * j;
    if (e < a.dk) a.pre_g[item * a.dk + e] = entry_decay<DT>(a, row, head, e, rate);
  }
  if (lane == 0) a.pre_s[item] = s;
}

// sum over the 16 lanes of a DPP row (every lane of the row active); the result is in every lane of the row
__device__ __forceinline__ float row16_sum(float v) {
  float t;
  t = ll_dpp_f32<0xB1>(v); v += t;   // quad_perm [1,0,3,2]
  t = ll_dpp_f32<0x4E>(v); v += t;   // quad_perm [2,3,0,1]
  t = ll_dpp_f32<0x124>(v); v += t;  // row_ror:4
  t = ll_dpp_f32<0x128>(v); v += t;  // row_ror:8
  return v;
}

// C neighbouring state columns of one row; rows and the first column are such that a row's C columns lie inside it together when
// vec is set (dv a multiple of C, aligned state)
template <int C>
__device__ __forceinline__ void load_cols(const float* p, int col, int dv, bool on, bool vec, float (&o)[C]) {
#pragma unroll
  for (int c = 0; c < C; ++c) o[c] = 0.f;
  if (!on) return;
  if constexpr (C == 4) {
    if (vec) {
      if (col < dv) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(p + col);
        o[0] = v[0]; o[1] = v[1]; o[2] = v[2]; o[3] = v[3];
      }
      return;
    }
  }
#pragma unroll
  for (int c = 0; c < C; ++c)
    if (col + c < dv) o[c] = p[col + c];
}
template <int C>
__device__ __forceinline__ void store_cols(float* p, int col, int dv, bool on, bool vec, const float (&o)[C]) {
  if (!on) return;
  if constexpr (C == 4) {
    if (vec) {
      if (col < dv) *reinterpret_cast<f32x4*>(p + col) = f32x4{o[0], o[1], o[2], o[3]};
      return;
    }
  }
#pragma unroll
  for (int c = 0; c < C; ++c)
    if (col + c < dv) p[col + c] = o[c];
}

// One workgroup of four waves per (sequence of the step, head, 16 C columns of the state).  A lane owns C neighbouring columns
// and the key entries rg, rg + 16, .. (R of them), rg = its place in its 16-lane row: the sums over key entries are one row
// reduction.  Tokens are taken TB at a time: (decay, g k, g q, k) of every key entry is staged in LDS as one 16-byte record
// (entries past dk are zero records: their state stays zero), values and scalars beside them.  PRE: decays and scalars were
// evaluated ahead; what the next pass stages is fetched into registers under the walk of the current one.  Else (a decoded token
// per sequence) TB is 1 and one wave evaluates them here.  A column's arithmetic does not depend on C or PRE, so every form
// leaves the same bits; the walk is the same token-by-token expression whatever the step's cut.
template <int DT, int R, int C, bool PRE>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaArgs a) {
  constexpr int DKP = 16 * R, COLS = 16 * C, TB = PRE ? (R <= 8 ? 16 : 8) : 1;
  constexpr int RPT = PRE ? TB * DKP / 256 : 1, VPT = TB * COLS > 256 ? TB * COLS / 256 : 1;   // records / values a thread stages
  __shared__ f32x4 sg[TB * DKP];     // (decay, g k, g q, k)
  __shared__ float2 sf[TB];          // factors of the raw k and q
  __shared__ float2 ss[TB];          // beta, k . q
  __shared__ __attribute__((aligned(16))) float sv[TB * COLS];    // values
  __shared__ __attribute__((aligned(16))) float so[TB * COLS];    // read-outs
  const int b = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * COLS;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, rg = lane & 15;
  const int mine = wave * 4 * C + (lane >> 4) * C;   // this lane's first column inside the workgroup's slice
  const int dk = a.dk, dv = a.dv, heads = a.heads;
  const int t0 = a.seq_start[b], t1 = a.seq_start[b + 1];
  if (t1 <= t0) return;
  float* st = a.state + ((int64_t)a.seq_slot[b] * heads + head) * dk * dv;
  const bool carry = a.seq_first_pos[b] > 0;
  const bool vec = dv % 4 == 0;      // (the state is 16-byte aligned: the host checks)
  const int qh0 = head / a.qk_rep * dk;
  float S[R][C];
#pragma unroll
  for (int r = 0; r < R; ++r) load_cols<C>(st + (int64_t)(rg + 16 * r) * dv, c0 + mine, dv, carry && rg + 16 * r < dk, vec, S[r]);

  float pg[RPT], pk[RPT], pq[RPT], pv[VPT];
  f32x4 ps = {0.f, 0.f, 0.f, 0.f};
  auto fetch = [&](int base) {       // what the pass at `base` stages: global -> registers
    const int nt = t1 - base < TB ? t1 - base : TB;
    if (PRE) {
      if (tid < nt) ps = a.pre_s[(int64_t)(base + tid) * heads + head];
#pragma unroll
      for (int u = 0; u < RPT; ++u) {
        const int i = tid + 256 * u, tt = i / DKP, e = i - tt * DKP;
        pg[u] = pk[u] = pq[u] = 0.f;
        if (tt < nt && e < dk) {
          const int64_t row = base + tt;
          pg[u] = a.pre_g[(row * heads + head) * dk + e];
          pk[u] = ldv<DT>(a.k, row * a.k_ld + qh0 + e);
          pq[u] = ldv<DT>(a.q, row * a.q_ld + qh0 + e);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < VPT; ++u) {
      const int i = tid + 256 * u, tt = i / COLS, cc = i - tt * COLS;
      pv[u] = (tt < nt && c0 + cc < dv) ? ldv<DT>(a.v, (int64_t)(base + tt) * a.v_ld + head * dv + c0 + cc) : 0.f;
    }
  };
  fetch(t0);
  for (int base = t0; base < t1; base += TB) {
    const int nt = t1 - base < TB ? t1 - base : TB;
    __syncthreads();                 // the previous pass has been read
    if (PRE) {
      if (tid < nt) {
        sf[tid] = make_float2(ps[0], ps[1]);
        ss[tid] = make_float2(ps[2], ps[3]);
      }
      __syncthreads();               // (a record needs its token's factors)
#pragma unroll
      for (int u = 0; u < RPT; ++u) {
        const int i = tid + 256 * u;
        const float2 f = sf[i / DKP];
        const float k = pk[u] * f.x;
        sg[i] = f32x4{pg[u], pg[u] * k, pg[u] * (pq[u] * f.y), k};
      }
    } else if (wave == 0) {
      float qv[kMaxPer], kv[kMaxPer];
      const float rate = expf(ldv<DT>(a.a_log, head));
      const f32x4 s = token_scalars<DT>(a, base, head, lane, qv, kv);
      if (lane == 0) ss[0] = make_float2(s[2], s[3]);
#pragma unroll
      for (int j = 0; j < kMaxPer; ++j) {
        const int e = lane + 64 * j;
        if (e < DKP) {
          f32x4 rec = {0.f, 0.f, 0.f, 0.f};
          if (e < dk) {
            const float g = entry_decay<DT>(a, base, head, e, rate);
            const float k = kv[j] * s[0];
            rec = f32x4{g, g * k, g * (qv[j] * s[1]), k};
          }
          sg[e] = rec;
        }
      }
    }
#pragma unroll
    for (int u = 0; u < VPT; ++u)
      if (tid + 256 * u < TB * COLS) sv[tid + 256 * u] = pv[u];
    __syncthreads();
    if (base + TB < t1) fetch(base + TB);
    // everything a token needs is read one token ahead (LDS answers in order: a scalar asked for behind the next token's records
    // would wait for all of them)
    struct Ahead {
      f32x4 rec[R];
      float2 s;
      float val[C];
    };
    auto read = [&](int tt, Ahead& x) {
      x.s = ss[tt];
#pragma unroll
      for (int c = 0; c < C; ++c) x.val[c] = sv[tt * COLS + mine + c];
#pragma unroll
      for (int r = 0; r < R; ++r) x.rec[r] = sg[tt * DKP + rg + 16 * r];
    };
    auto token = [&](int tt, const Ahead& x) {
      float p[C], w[C];
#pragma unroll
      for (int c = 0; c < C; ++c) {
        p[c] = w[c] = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
          p[c] = __builtin_fmaf(S[r][c], x.rec[r][1], p[c]);
          w[c] = __builtin_fmaf(S[r][c], x.rec[r][2], w[c]);
        }
      }
#pragma unroll
      for (int c = 0; c < C; ++c) {
        p[c] = row16_sum(p[c]);
        w[c] = row16_sum(w[c]);
      }
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const float u = x.s.x * (x.val[c] - p[c]);
#pragma unroll
        for (int r = 0; r < R; ++r) S[r][c] = __builtin_fmaf(x.rec[r][0], S[r][c], x.rec[r][3] * u);
        w[c] = __builtin_fmaf(x.s.y, u, w[c]);
      }
      if (rg == 0) {
#pragma unroll
        for (int c = 0; c < C; ++c) so[tt * COLS + mine + c] = w[c];
      }
    };
    Ahead xa, xb;
    read(0, xa);
    for (int tt = 0; tt < nt; tt += 2) {
      if (TB > 1) read(tt + 1 < nt ? tt + 1 : tt, xb);
      token(tt, xa);
      if (TB > 1) {
        read(tt + 2 < nt ? tt + 2 : tt, xa);
        if (tt + 1 < nt) token(tt + 1, xb);
      }
    }
    __syncthreads();
    for (int i = tid; i < nt * COLS; i += 256) {
      const int tt = i / COLS, cc = i - tt * COLS;
      if (c0 + cc < dv) a.o[((int64_t)(base + tt) * heads + head) * dv + c0 + cc] = so[i];
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) store_cols<C>(st + (int64_t)(rg + 16 * r) * dv, c0 + mine, dv, rg + 16 * r < dk, vec, S[r]);
}

}  // namespace

#define LL_BY_DTYPE(dtype, CALL)                  \
  do {                                            \
    if (dtype == LL_F16) { CALL(LL_F16); }        \
    else if (dtype == LL_BF16) { CALL(LL_BF16); } \
    else { CALL(LL_F32); }                        \
  } while (0)

extern "C" int ll_delta_scan_supported(int64_t dk, int64_t dv) { return dk >= 1 && dk <= 64 * kMaxPer && dv >= 1 ? 1 : 0; }

// fp32 floats of the scratch that lets a step's decays and scalars be evaluated once, ahead of the walk
extern "C" int64_t ll_delta_scan_scratch_floats(int64_t n, int64_t heads, int64_t dk) { return n * heads * (dk + 4); }

extern "C" int ll_delta_scan(const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, int64_t heads,
                             int64_t dk, int64_t dv, int64_t qk_rep, float q_scale, float unit_eps, const void* gate, int64_t gate_ld,
                             const void* dt_bias, const void* a_log, const void* beta, int64_t beta_ld, float* o, int64_t batch,
                             const int32_t* seq_start, const int32_t* seq_first_pos, const int32_t* seq_slot, float* state,
                             float* scratch, int64_t n, int dtype, void* stream) {
  if (dtype != LL_F16 && dtype != LL_BF16 && dtype != LL_F32) return LL_ERR_DTYPE;
  if (batch < 0 || n < 0 || heads < 1 || heads > 65535 || !ll_delta_scan_supported(dk, dv) || qk_rep < 1 || heads % qk_rep ||
      (dv + 15) / 16 > 65535)
    return LL_ERR_SHAPE;
  const int64_t qk_cols = heads / qk_rep * dk;
  if (q_ld < qk_cols || k_ld < qk_cols || v_ld < heads * dv || gate_ld < heads * dk || beta_ld < heads) return LL_ERR_SHAPE;
  if (batch == 0 || n == 0) return LL_OK;
  if (!q || !k || !v || !gate || !dt_bias || !a_log || !beta || !o || !seq_start || !seq_first_pos || !seq_slot || !state) return LL_ERR_ARG;
  if ((scratch && !ll_aligned16(scratch)) || !ll_aligned16(state)) return LL_ERR_ARG;
  DeltaArgs a;
  a.q = q; a.k = k; a.v = v; a.q_ld = q_ld; a.k_ld = k_ld; a.v_ld = v_ld;
  a.heads = (int)heads; a.dk = (int)dk; a.dv = (int)dv; a.qk_rep = (int)qk_rep; a.q_scale = q_scale; a.unit_eps = unit_eps;
  a.gate = gate; a.gate_ld = gate_ld; a.dt_bias = dt_bias; a.a_log = a_log; a.beta = beta; a.beta_ld = beta_ld;
  a.pre_s = reinterpret_cast<f32x4*>(scratch);
  a.pre_g = scratch ? scratch + n * heads * 4 : nullptr;
  a.o = o; a.seq_start = seq_start; a.seq_first_pos = seq_first_pos; a.seq_slot = seq_slot; a.state = state;
  hipStream_t st = (hipStream_t)stream;
  if (scratch) {
    const int64_t items = n * heads;
    if ((items + 3) / 4 > 0x7fffffffll) return LL_ERR_SHAPE;
#define CALL(DT) delta_prepare_kernel<DT><<<dim3((unsigned)((items + 3) / 4)), 256, 0, st>>>(a, items)
    LL_BY_DTYPE(dtype, CALL);
#undef CALL
  }
  const int rmax = (int)((dk + 15) / 16);
  const int R = rmax <= 4 ? 4 : rmax <= 8 ? 8 : 16;
  // Columns per lane.  LDS records are read once per 4 C columns of a wave, so more columns cost fewer reads; a walk over many
  // tokens needs two waves per SIMD to hide one wave's reduction behind the other's sums (heads of more than 128 key entries are
  // bound by the records: one is enough).  A decoded token moves the state once: widest accesses.
  static const int forced = getenv("LL_DELTA_COLS") ? atoi(getenv("LL_DELTA_COLS")) : 0;   // A/B knob, read once
  auto waves = [&](int c) { return batch * heads * ((dv + 16 * c - 1) / (16 * c)) * 4; };
  int C;
  if (!scratch) C = dv > 32 ? 4 : dv > 16 ? 2 : 1;
  else if (dv > 32 && waves(4) >= (R == 16 ? 1024 : 2048)) C = 4;
  else C = (dv > 16 && waves(2) >= 2048) ? 2 : 1;
  if (forced == 1 || forced == 2 || forced == 4) C = forced;
  const dim3 grid((unsigned)batch, (unsigned)heads, (unsigned)((dv + 16 * C - 1) / (16 * C)));
#define CALL_P(DT, RR, CC)                                                       \
  if (scratch) delta_scan_kernel<DT, RR, CC, true><<<grid, 256, 0, st>>>(a);     \
  else delta_scan_kernel<DT, RR, CC, false><<<grid, 256, 0, st>>>(a)
#define CALL_C(DT, RR)                 \
  if (C == 4) { CALL_P(DT, RR, 4); }   \
  else if (C == 2) { CALL_P(DT, RR, 2); } \
  else { CALL_P(DT, RR, 1); }
#define CALL(DT)                      \
  if (R == 4) { CALL_C(DT, 4); }      \
  else if (R == 8) { CALL_C(DT, 8); } \
  else { CALL_C(DT, 16); }
  LL_BY_DTYPE(dtype, CALL);
#undef CALL
#undef CALL_C
#undef CALL_P
  return LL_LAUNCH_CHECK();
}
