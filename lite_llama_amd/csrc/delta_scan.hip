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
  int tb;                    // tokens staged per pass
  const int32_t* seq_start;
  const int32_t* seq_first_pos;
  const int32_t* seq_slot;
  float* state;              // fp32 [slots, heads, dk, dv]
};

__device__ __forceinline__ float softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

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
  return expf(-rate * softplus(ldv<DT>(a.gate, row * a.gate_ld + c) + ldv<DT>(a.dt_bias, c)));
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

// One workgroup of four waves per (sequence of the step, head, 16 C columns of the state).  A lane owns C neighbouring columns
// and the key entries rg, rg + 16, .. (R of them), rg = its place in its 16-lane row: the sums over key entries are one row
// reduction.  Tokens are taken tb at a time: (decay, g k, g q, k) of every key entry is staged in LDS as one 16-byte record
// (entries past dk are zero records: their state stays zero), values and scalars beside them.  A column's arithmetic does not
// depend on C, so every form leaves the same bits; the walk is the same token-by-token expression whatever the step's cut.
template <int DT, int R, int C>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaArgs a) {
  extern __shared__ float lds[];
  constexpr int DKP = 16 * R, COLS = 16 * C;
  const int b = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * COLS;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, rg = lane & 15;
  const int mine = wave * 4 * C + (lane >> 4) * C;   // this lane's first column inside the workgroup's slice
  const int dk = a.dk, dv = a.dv, tb = a.tb, heads = a.heads;
  f32x4* sg = reinterpret_cast<f32x4*>(lds);          // [tb][DKP] (decay, g k, g q, k)
  f32x4* ss = sg + tb * DKP;                          // [tb] (-, -, beta, k . q)
  float* sv = reinterpret_cast<float*>(ss + tb);      // [tb][COLS] values
  float* so = sv + tb * COLS;                         // [tb][COLS] read-outs
  const int t0 = a.seq_start[b], t1 = a.seq_start[b + 1];
  float* st = a.state + ((int64_t)a.seq_slot[b] * heads + head) * dk * dv;
  const bool carry = a.seq_first_pos[b] > 0;
  const int qh0 = head / a.qk_rep * dk;
  const float rate = a.pre_g ? 0.f : expf(ldv<DT>(a.a_log, head));
  float S[R][C];
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int c = 0; c < C; ++c) {
      const int e = rg + 16 * r, col = c0 + mine + c;
      S[r][c] = (carry && e < dk && col < dv) ? st[(int64_t)e * dv + col] : 0.f;
    }
  for (int base = t0; base < t1; base += tb) {
    const int nt = t1 - base < tb ? t1 - base : tb;
    __syncthreads();   // the previous pass has been read
    if (a.pre_g) {
      if (tid < nt) ss[tid] = a.pre_s[(int64_t)(base + tid) * heads + head];
      for (int i = tid; i < nt * DKP; i += 256) {
        const int tt = i / DKP, e = i - tt * DKP;
        f32x4 rec = {0.f, 0.f, 0.f, 0.f};
        if (e < dk) {
          const int64_t row = base + tt;
          const f32x4 s = a.pre_s[row * heads + head];
          const float g = a.pre_g[(row * heads + head) * dk + e];
          const float k = ldv<DT>(a.k, row * a.k_ld + qh0 + e) * s[0];
          rec = f32x4{g, g * k, g * (ldv<DT>(a.q, row * a.q_ld + qh0 + e) * s[1]), k};
        }
        sg[i] = rec;
      }
    } else {
      for (int tt = wave; tt < nt; tt += 4) {
        float qv[kMaxPer], kv[kMaxPer];
        const f32x4 s = token_scalars<DT>(a, base + tt, head, lane, qv, kv);
        if (lane == 0) ss[tt] = s;
#pragma unroll
        for (int j = 0; j < kMaxPer; ++j) {
          const int e = lane + 64 * j;
          if (e < DKP) {
            f32x4 rec = {0.f, 0.f, 0.f, 0.f};
            if (e < dk) {
              const float g = entry_decay<DT>(a, base + tt, head, e, rate);
              const float k = kv[j] * s[0];
              rec = f32x4{g, g * k, g * (qv[j] * s[1]), k};
            }
            sg[tt * DKP + e] = rec;
          }
        }
      }
    }
    for (int i = tid; i < nt * COLS; i += 256) {
      const int tt = i / COLS, cc = i - tt * COLS;
      sv[i] = c0 + cc < dv ? ldv<DT>(a.v, (int64_t)(base + tt) * a.v_ld + head * dv + c0 + cc) : 0.f;
    }
    __syncthreads();
    f32x4 rec[R], nxt[R];
#pragma unroll
    for (int r = 0; r < R; ++r) rec[r] = sg[rg + 16 * r];
    for (int tt = 0; tt < nt; ++tt) {
      const int at = tt + 1 < nt ? tt + 1 : tt;   // the next token's records are read under this token's sums
#pragma unroll
      for (int r = 0; r < R; ++r) nxt[r] = sg[at * DKP + rg + 16 * r];
      float p[C], w[C], u[C];
#pragma unroll
      for (int c = 0; c < C; ++c) {
        p[c] = w[c] = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
          p[c] = __builtin_fmaf(S[r][c], rec[r][1], p[c]);
          w[c] = __builtin_fmaf(S[r][c], rec[r][2], w[c]);
        }
      }
      const f32x4 s = ss[tt];
#pragma unroll
      for (int c = 0; c < C; ++c) {
        p[c] = row16_sum(p[c]);
        w[c] = row16_sum(w[c]);
      }
#pragma unroll
      for (int c = 0; c < C; ++c) {
        u[c] = s[2] * (sv[tt * COLS + mine + c] - p[c]);
#pragma unroll
        for (int r = 0; r < R; ++r) S[r][c] = __builtin_fmaf(rec[r][0], S[r][c], rec[r][3] * u[c]);
      }
      if (rg == 0) {
#pragma unroll
        for (int c = 0; c < C; ++c) so[tt * COLS + mine + c] = __builtin_fmaf(s[3], u[c], w[c]);
      }
#pragma unroll
      for (int r = 0; r < R; ++r) rec[r] = nxt[r];
    }
    __syncthreads();
    for (int i = tid; i < nt * COLS; i += 256) {
      const int tt = i / COLS, cc = i - tt * COLS;
      if (c0 + cc < dv) a.o[((int64_t)(base + tt) * heads + head) * dv + c0 + cc] = so[i];
    }
  }
  if (t1 > t0) {
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const int e = rg + 16 * r, col = c0 + mine + c;
        if (e < dk && col < dv) st[(int64_t)e * dv + col] = S[r][c];
      }
  }
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
                             float* scratch, int64_t n, int64_t longest_run, int dtype, void* stream) {
  if (dtype != LL_F16 && dtype != LL_BF16 && dtype != LL_F32) return LL_ERR_DTYPE;
  if (batch < 0 || n < 0 || heads < 1 || heads > 65535 || !ll_delta_scan_supported(dk, dv) || qk_rep < 1 || heads % qk_rep ||
      (dv + 15) / 16 > 65535)
    return LL_ERR_SHAPE;
  const int64_t qk_cols = heads / qk_rep * dk;
  if (q_ld < qk_cols || k_ld < qk_cols || v_ld < heads * dv || gate_ld < heads * dk || beta_ld < heads) return LL_ERR_SHAPE;
  if (batch == 0 || n == 0) return LL_OK;
  if (!q || !k || !v || !gate || !dt_bias || !a_log || !beta || !o || !seq_start || !seq_first_pos || !seq_slot || !state) return LL_ERR_ARG;
  if (scratch && !ll_aligned16(scratch)) return LL_ERR_ARG;
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
  a.tb = R <= 8 ? 16 : 8;
  if (longest_run > 0 && longest_run < a.tb) a.tb = (int)longest_run;
  // columns per lane: as many as still leave two waves per SIMD (LDS records are read once per 4 C columns of a wave)
  static const int forced = getenv("LL_DELTA_COLS") ? atoi(getenv("LL_DELTA_COLS")) : 0;   // A/B knob, read once
  auto waves = [&](int c) { return batch * heads * ((dv + 16 * c - 1) / (16 * c)) * 4; };
  int C = (dv > 32 && waves(4) >= 1024) ? 4 : (dv > 16 && waves(2) >= 1024) ? 2 : 1;
  if (forced == 1 || forced == 2 || forced == 4) C = forced;
  const size_t lds = sizeof(float) * (size_t)(a.tb * (4 * 16 * R + 4 + 2 * 16 * C));
  const dim3 grid((unsigned)batch, (unsigned)heads, (unsigned)((dv + 16 * C - 1) / (16 * C)));
#define CALL_C(DT, RR)                                                    \
  if (C == 4) delta_scan_kernel<DT, RR, 4><<<grid, 256, lds, st>>>(a);    \
  else if (C == 2) delta_scan_kernel<DT, RR, 2><<<grid, 256, lds, st>>>(a); \
  else delta_scan_kernel<DT, RR, 1><<<grid, 256, lds, st>>>(a)
#define CALL(DT)                    \
  if (R == 4) { CALL_C(DT, 4); }    \
  else if (R == 8) { CALL_C(DT, 8); } \
  else { CALL_C(DT, 16); }
  LL_BY_DTYPE(dtype, CALL);
#undef CALL
#undef CALL_C
  return LL_LAUNCH_CHECK();
}
