// Retention over RAGGED steps (several sequences, each bringing a run of consecutive tokens against the state its earlier steps
// left): per head, with ONE fixed decay,
//
//   q, k <- rotated (entry i with entry i + half of the first 2 half entries, by the token's cos / sin), k times a constant
//   S_t = decay_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t
//
// over an fp32 state [dk, dv] per (sequence slot, head).  Because the decay is a constant of the head, a run of C tokens is three
// matrix products: with t, u counted inside the chunk and S the state in front of it
//
//   o_t = decay^(t + 1) S^T q_t + sum_(u <= t) decay^(t - u) (q_t . k_u) v_u
//   S  <- decay^C S + sum_u decay^(C - 1 - u) k_u v_u^T
//
//   retention_chunk_kernel    runs of several tokens: a workgroup per (sequence, head, 32 state columns) walks the run in chunks of
//                             32 tokens on the fp32 matrix cores (v_mfma_f32_16x16x4: operands, scores, state are fp32, for
//                             every storage dtype); the read-out goes to an fp32 scratch, normed and gated by ll_gated_out_norm
//   retention_decode_kernel   one decoded token per sequence: a workgroup per (sequence, head) rotates, updates the state, reads
//                             it out, norms the head, gates and stores -- one launch
//
// A run that starts at position 0 starts from zeros whatever an earlier owner of the slot left.
#include "common.h"

#include <math.h>

namespace {

template <int DT>
__device__ __forceinline__ float ldv(const void* p, int64_t i) {
  if constexpr (DT == LL_F32) return ((const float*)p)[i];
  else return to_f32<DT>(((const uint16_t*)p)[i]);
}
template <int DT>
__device__ __forceinline__ void stv(void* p, int64_t i, float v) {
  if constexpr (DT == LL_F32) ((float*)p)[i] = v;
  else ((uint16_t*)p)[i] = from_f32<DT>(v);
}

struct RetentionArgs {
  const void* q;   // [n, q_ld]: head h's entries at columns h dk ..
  const void* k;
  const void* v;   // [n, v_ld]: head h's entries at columns h dv ..
  int64_t q_ld, k_ld, v_ld;
  int heads, dk, dv;
  const float* rot;   // fp32 [n][rot_ld]: (cos, sin) of pair i at 2 i; read for i < half
  int64_t rot_ld;
  int half;
  float k_scale;
  const float* decay;   // fp32 [heads]
  const int32_t* seq_start;
  const int32_t* seq_first_pos;
  const int32_t* seq_slot;
  float* state;   // fp32 [slots, heads, dk, dv]
  float* o;       // chunk form: fp32 [n, heads dv]
  const void* gate;   // decode form: rows [n, gate_ld] of heads dv gate logits (NULL: no gate), RMS epsilon, result rows
  int64_t gate_ld;
  float eps;
  void* out;
  int64_t out_ld;
};

// entry i of a rotated head at row element `at` (the head's first element)
template <int DT>
__device__ __forceinline__ float rotated_entry(const void* p, int64_t at, int i, int half, const float* cs) {
  const float x = ldv<DT>(p, at + i);
  if (i >= 2 * half) return x;
  if (i < half) return x * cs[2 * i] - ldv<DT>(p, at + i + half) * cs[2 * i + 1];
  return x * cs[2 * (i - half)] + ldv<DT>(p, at + i - half) * cs[2 * (i - half) + 1];
}

// ------------------------------------------------------------------------------------------------------------------------
// decoded tokens.  Thread (row group g, piece): CV neighbouring state columns, key entries g, g + groups, ..
// ------------------------------------------------------------------------------------------------------------------------
constexpr int kRows = 8;   // state rows in flight per thread

template <int DT, int CV>
__global__ __launch_bounds__(256) void retention_decode_kernel(const RetentionArgs a) {
  extern __shared__ float lds[];
  __shared__ float red[4];
  const int b = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int dk = a.dk, dv = a.dv;
  const int pieces = dv / CV, per_pass = pieces < 256 ? pieces : 256;
  const int groups = 256 / per_pass;
  float* sq = lds;          // [dk]
  float* sk = sq + dk;      // [dk]
  float* so = sk + dk;      // [groups][dv]
  const int64_t t = a.seq_start[b];
  const bool carry = a.seq_first_pos[b] > 0;
  const float dec = a.decay[head];
  float* st = a.state + ((int64_t)a.seq_slot[b] * a.heads + head) * dk * dv;
  const float* cs = a.rot + t * a.rot_ld;
  for (int i = tid; i < dk; i += 256) {
    sq[i] = rotated_entry<DT>(a.q, t * a.q_ld + (int64_t)head * dk, i, a.half, cs);
    sk[i] = rotated_entry<DT>(a.k, t * a.k_ld + (int64_t)head * dk, i, a.half, cs) * a.k_scale;
  }
  __syncthreads();
  const int g = tid / per_pass;
  if (g < groups) {
    for (int pc = tid - g * per_pass; pc < pieces; pc += per_pass) {
      float val[CV], acc[CV];
#pragma unroll
      for (int e = 0; e < CV; ++e) {
        val[e] = ldv<DT>(a.v, t * a.v_ld + (int64_t)head * dv + pc * CV + e);
        acc[e] = 0.f;
      }
      // eight rows of the state at a time: all of them are requested before the first is written back
      for (int r0 = g; r0 < dk; r0 += kRows * groups) {
        float S[kRows][CV];
#pragma unroll
        for (int j = 0; j < kRows; ++j) {
          const int r = r0 + j * groups;
          const float* sp = st + (int64_t)r * dv + pc * CV;
          const bool in = carry && r < dk;
          if constexpr (CV == 4) {
            f32x4 old = {0.f, 0.f, 0.f, 0.f};
            if (in) old = *reinterpret_cast<const f32x4*>(sp);
#pragma unroll
            for (int e = 0; e < 4; ++e) S[j][e] = old[e];
          } else {
            S[j][0] = in ? sp[0] : 0.f;
          }
        }
#pragma unroll
        for (int j = 0; j < kRows; ++j) {
          const int r = r0 + j * groups;
          if (r >= dk) break;
          float* sp = st + (int64_t)r * dv + pc * CV;
          const float kr = sk[r], qr = sq[r];
#pragma unroll
          for (int e = 0; e < CV; ++e) {
            S[j][e] = __builtin_fmaf(dec, S[j][e], kr * val[e]);
            acc[e] = __builtin_fmaf(S[j][e], qr, acc[e]);
          }
          if constexpr (CV == 4) *reinterpret_cast<f32x4*>(sp) = f32x4{S[j][0], S[j][1], S[j][2], S[j][3]};
          else sp[0] = S[j][0];
        }
      }
#pragma unroll
      for (int e = 0; e < CV; ++e) so[g * dv + pc * CV + e] = acc[e];
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < dv; c += 256) {   // (a thread keeps its own columns through both passes)
    float o = so[c];
    for (int j = 1; j < groups; ++j) o += so[j * dv + c];
    so[c] = o;
    ss += o * o;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  ss = ((red[0] + red[1]) + red[2]) + red[3];
  const float inv = 1.0f / sqrtf(ss / (float)dv + a.eps);
  for (int c = tid; c < dv; c += 256) {
    float y = so[c] * inv;
    if (a.gate) {
      const float z = ldv<DT>(a.gate, t * a.gate_ld + (int64_t)head * dv + c);
      if constexpr (DT == LL_F32) y *= z / (1.0f + expf(-z));
      else y *= z * ll_sigmoidf(z);
    }
    stv<DT>(a.out, t * a.out_ld + (int64_t)head * dv + c, y);
  }
}

// ------------------------------------------------------------------------------------------------------------------------
// runs of several tokens
// ------------------------------------------------------------------------------------------------------------------------
constexpr int kC = 32;    // tokens per chunk
constexpr int kCols = 32;   // state columns per workgroup
constexpr int kVS = kCols + 4;
constexpr int kPS = kC + 4;

template <int KT>
constexpr size_t chunk_lds_floats() {   // q, k [kC][16 KT + 4], state^T [kCols][16 KT + 4], values twice, scores, powers
  return (size_t)(2 * kC + kCols) * (16 * KT + 4) + 2 * kC * kVS + kC * kPS + kC + 4;
}

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// Four waves.  Operands of v_mfma_f32_16x16x4: lane (t = lane & 15, c = lane >> 4) holds A[t][c], B[c][t]; result element r of the
// lane is D[4 c + r][t].  The contraction may run in any order both operands share: a lane takes four CONSECUTIVE entries
// 16 s + 4 c .. of a row with one 16-byte LDS read and feeds them to four products.
//   scores     wave (tt, ct): K[16 ct ..] Q[16 tt ..]^T, so a lane ends with four neighbouring keys u of one query t: times
//              decay^(t - u), one 16-byte write into the score matrix
//   read-out   wave (tt, ct): queries 16 tt .., columns 16 ct ..: Q S, rows times decay^(t + 1), plus scores V
//   state      wave w owns key-entry tiles w, w + 4, .. of all 32 columns in registers
// VEC (16-bit storage, widths and strides multiples of 8): the next chunk's rows are fetched into registers under this chunk's
// products, in items of (token, 8 rotated pairs) or (token, 8 unrotated entries).
template <int DT, int KT, bool VEC>
__global__ __launch_bounds__(256) void retention_chunk_kernel(const RetentionArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int KS = 16 * KT + 4;
  constexpr int NI = KT / 4;   // items per thread and chunk
  constexpr int NS = KT / 4;   // key-entry tiles per wave
  float* sq = lds;                  // [kC][KS]
  float* sk = sq + kC * KS;         // [kC][KS]
  float* ss = sk + kC * KS;         // [kCols][KS]  state in front of the chunk, transposed
  float* sv = ss + kCols * KS;      // [kC][kVS]
  float* sd = sv + kC * kVS;        // [kC][kVS]    values times decay^(n - 1 - u)
  float* sp = sd + kC * kVS;        // [kC][kPS]    scores
  float* pw = sp + kC * kPS;        // [kC + 1]     powers of the decay
  const int b = blockIdx.x / a.heads, head = blockIdx.x - b * a.heads, c0 = blockIdx.y * kCols;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, t = lane & 15, c = lane >> 4;
  const int tt = wave & 1, ct = wave >> 1;
  const int dk = a.dk, dv = a.dv, half = a.half;
  const int t0 = a.seq_start[b], t1 = a.seq_start[b + 1];
  if (t0 >= t1) return;
  const bool carry = a.seq_first_pos[b] > 0;
  float* st = a.state + ((int64_t)a.seq_slot[b] * a.heads + head) * dk * dv;
  for (int i = tid; i < (int)chunk_lds_floats<KT>() / 4; i += 256) reinterpret_cast<f32x4*>(lds)[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 S[NS][2];
#pragma unroll
  for (int i = 0; i < NS; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * (wave + 4 * i) + 4 * c + r, col = c0 + 16 * j + t;
        S[i][j][r] = (carry && kk < dk && col < dv) ? st[(int64_t)kk * dv + col] : 0.f;
      }
  __syncthreads();
  if (tid <= kC) pw[tid] = powf(a.decay[head], (float)tid);

  // what a thread fetches of a chunk (VEC)
  U16x8 rq[VEC ? NI : 1][2], rk[VEC ? NI : 1][2], rv;
  f32x4 rc[VEC ? NI : 1][4];
  const int pairs8 = half >> 3, per_row = pairs8 + ((dk - 2 * half) >> 3);
  auto fetch = [&](int base) {
    if constexpr (VEC) {
      const uint16_t* qp = (const uint16_t*)a.q;
      const uint16_t* kp = (const uint16_t*)a.k;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int item = tid + 256 * i, row = item / per_row, pc = item - row * per_row;
        const int64_t tok = base + row;
        if (row < kC && tok < t1) {
          const int64_t qa = tok * a.q_ld + (int64_t)head * dk, ka = tok * a.k_ld + (int64_t)head * dk;
          const int lo = pc < pairs8 ? 8 * pc : 2 * half + 8 * (pc - pairs8);
          rq[i][0] = *reinterpret_cast<const U16x8*>(qp + qa + lo);
          rk[i][0] = *reinterpret_cast<const U16x8*>(kp + ka + lo);
          if (pc < pairs8) {
            rq[i][1] = *reinterpret_cast<const U16x8*>(qp + qa + lo + half);
            rk[i][1] = *reinterpret_cast<const U16x8*>(kp + ka + lo + half);
            const f32x4* cs = reinterpret_cast<const f32x4*>(a.rot + tok * a.rot_ld + 2 * lo);
#pragma unroll
            for (int e = 0; e < 4; ++e) rc[i][e] = cs[e];
          }
        }
      }
      const int row = tid >> 2, pc = tid & 3;
      if (row < kC && base + row < t1 && c0 + 8 * pc < dv)
        rv = *reinterpret_cast<const U16x8*>((const uint16_t*)a.v + (int64_t)(base + row) * a.v_ld + (int64_t)head * dv + c0 + 8 * pc);
    }
  };
  // rows of a chunk of n tokens into LDS (rows past the run are zeros)
  auto stage = [&](int base, int n) {
    if constexpr (VEC) {
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int item = tid + 256 * i, row = item / per_row, pc = item - row * per_row;
        if (row >= kC) continue;
        const bool in = row < n;
        if (pc < pairs8) {
          float* qd = sq + row * KS + 8 * pc;
          float* kd = sk + row * KS + 8 * pc;
#pragma unroll
          for (int h4 = 0; h4 < 2; ++h4) {
            f32x4 q0, q1, k0, k1;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const int j = 4 * h4 + e;
              const float cs = rc[i][j >> 1][(j & 1) * 2], sn = rc[i][j >> 1][(j & 1) * 2 + 1];
              const float qa = to_f32<DT>(rq[i][0].v[j]), qb = to_f32<DT>(rq[i][1].v[j]);
              const float ka = to_f32<DT>(rk[i][0].v[j]), kb = to_f32<DT>(rk[i][1].v[j]);
              q0[e] = in ? qa * cs - qb * sn : 0.f;
              q1[e] = in ? qb * cs + qa * sn : 0.f;
              k0[e] = in ? (ka * cs - kb * sn) * a.k_scale : 0.f;
              k1[e] = in ? (kb * cs + ka * sn) * a.k_scale : 0.f;
            }
            *reinterpret_cast<f32x4*>(qd + 4 * h4) = q0;
            *reinterpret_cast<f32x4*>(qd + half + 4 * h4) = q1;
            *reinterpret_cast<f32x4*>(kd + 4 * h4) = k0;
            *reinterpret_cast<f32x4*>(kd + half + 4 * h4) = k1;
          }
        } else {
          const int lo = 2 * half + 8 * (pc - pairs8);
#pragma unroll
          for (int h4 = 0; h4 < 2; ++h4) {
            f32x4 q0, k0;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              q0[e] = in ? to_f32<DT>(rq[i][0].v[4 * h4 + e]) : 0.f;
              k0[e] = in ? to_f32<DT>(rk[i][0].v[4 * h4 + e]) * a.k_scale : 0.f;
            }
            *reinterpret_cast<f32x4*>(sq + row * KS + lo + 4 * h4) = q0;
            *reinterpret_cast<f32x4*>(sk + row * KS + lo + 4 * h4) = k0;
          }
        }
      }
      const int row = tid >> 2, pc = tid & 3;
      if (row < kC) {
        const bool in = row < n && c0 + 8 * pc < dv;
        const float w = row < n ? pw[n - 1 - row] : 0.f;
#pragma unroll
        for (int h4 = 0; h4 < 2; ++h4) {
          f32x4 x, d;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            x[e] = in ? to_f32<DT>(rv.v[4 * h4 + e]) : 0.f;
            d[e] = x[e] * w;
          }
          *reinterpret_cast<f32x4*>(sv + row * kVS + 8 * pc + 4 * h4) = x;
          *reinterpret_cast<f32x4*>(sd + row * kVS + 8 * pc + 4 * h4) = d;
        }
      }
    } else {
      for (int i = tid; i < kC * dk; i += 256) {
        const int row = i / dk, e = i - row * dk;
        float qv = 0.f, kv = 0.f;
        if (row < n) {
          const int64_t tok = base + row;
          const float* cs = a.rot + tok * a.rot_ld;
          qv = rotated_entry<DT>(a.q, tok * a.q_ld + (int64_t)head * dk, e, half, cs);
          kv = rotated_entry<DT>(a.k, tok * a.k_ld + (int64_t)head * dk, e, half, cs) * a.k_scale;
        }
        sq[row * KS + e] = qv;
        sk[row * KS + e] = kv;
      }
      for (int i = tid; i < kC * kCols; i += 256) {
        const int row = i / kCols, e = i - row * kCols;
        const float x = (row < n && c0 + e < dv) ? ldv<DT>(a.v, (int64_t)(base + row) * a.v_ld + (int64_t)head * dv + c0 + e) : 0.f;
        sv[row * kVS + e] = x;
        sd[row * kVS + e] = row < n ? x * pw[n - 1 - row] : 0.f;
      }
    }
  };

  fetch(t0);
  for (int base = t0; base < t1; base += kC) {
    const int n = t1 - base < kC ? t1 - base : kC;
    __syncthreads();   // the powers are there; everybody has read the previous chunk
    stage(base, n);
#pragma unroll
    for (int i = 0; i < NS; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) *reinterpret_cast<f32x4*>(ss + (16 * j + t) * KS + 16 * (wave + 4 * i) + 4 * c) = S[i][j];
    __syncthreads();
    if (base + kC < t1) fetch(base + kC);
    // scores of keys 16 ct .. against queries 16 tt .. (keys behind every query of the tile: zeros), and the read-out of the state
    // in front of the chunk: one query fragment feeds both products
    f32x4 p = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f};
    {
      const float* qp = sq + (16 * tt + t) * KS + 4 * c;
      const float* kp = sk + (16 * ct + t) * KS + 4 * c;
      const float* op = ss + (16 * ct + t) * KS + 4 * c;
      if (ct <= tt) {
#pragma unroll
        for (int s = 0; s < KT; ++s) {
          const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + 16 * s), kf = *reinterpret_cast<const f32x4*>(kp + 16 * s),
                      sf = *reinterpret_cast<const f32x4*>(op + 16 * s);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            p = mfma4(kf[e], qf[e], p);
            o = mfma4(qf[e], sf[e], o);
          }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int gap = 16 * (tt - ct) + t - 4 * c - r;
          p[r] = gap >= 0 ? p[r] * pw[gap] : 0.f;
        }
      } else {
#pragma unroll
        for (int s = 0; s < KT; ++s) {
          const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + 16 * s), sf = *reinterpret_cast<const f32x4*>(op + 16 * s);
#pragma unroll
          for (int e = 0; e < 4; ++e) o = mfma4(qf[e], sf[e], o);
        }
      }
    }
    *reinterpret_cast<f32x4*>(sp + (16 * tt + t) * kPS + 16 * ct + 4 * c) = p;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] *= pw[16 * tt + 4 * c + r + 1];
    __syncthreads();   // the scores are there
#pragma unroll
    for (int s = 0; s < kC / 16; ++s) {
      const f32x4 pa = *reinterpret_cast<const f32x4*>(sp + (16 * tt + t) * kPS + 16 * s + 4 * c);
#pragma unroll
      for (int e = 0; e < 4; ++e) o = mfma4(pa[e], sv[(16 * s + 4 * c + e) * kVS + 16 * ct + t], o);
    }
    const float dn = pw[n];
#pragma unroll
    for (int i = 0; i < NS; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][j][r] *= dn;
#pragma unroll
    for (int s = 0; s < kC / 16; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int u = 16 * s + 4 * c + e;
        const float v0 = sd[u * kVS + t], v1 = sd[u * kVS + 16 + t];
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          const float kk = sk[u * KS + 16 * (wave + 4 * i) + t];
          S[i][0] = mfma4(kk, v0, S[i][0]);
          S[i][1] = mfma4(kk, v1, S[i][1]);
        }
      }
    const int col = c0 + 16 * ct + t;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 16 * tt + 4 * c + r;
      if (row < n && col < dv) a.o[((int64_t)(base + row) * a.heads + head) * dv + col] = o[r];
    }
  }
#pragma unroll
  for (int i = 0; i < NS; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * (wave + 4 * i) + 4 * c + r, col = c0 + 16 * j + t;
        if (kk < dk && col < dv) st[(int64_t)kk * dv + col] = S[i][j][r];
      }
}

template <int DT, int KT, bool VEC>
int launch_chunk(const RetentionArgs& a, dim3 grid, hipStream_t st) {
  constexpr size_t bytes = chunk_lds_floats<KT>() * sizeof(float);
  if (bytes > 64 * 1024) {
    static const hipError_t once = hipFuncSetAttribute((const void*)retention_chunk_kernel<DT, KT, VEC>,
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    if (once != hipSuccess) return LL_ERR_LAUNCH;
  }
  retention_chunk_kernel<DT, KT, VEC><<<grid, 256, bytes, st>>>(a);
  return LL_LAUNCH_CHECK();
}

}  // namespace

extern "C" int ll_retention_supported(int64_t dk, int64_t dv) { return dk >= 1 && dk <= 256 && dv >= 1 && dv <= 8192 ? 1 : 0; }

// o (fp32 [n, heads dv]) given: runs of any length, read-out only (norm and gate are ll_gated_out_norm's).  o NULL: every sequence
// brings ONE token; out rows = RMS-normed heads times silu(gate).
extern "C" int ll_retention(const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, int64_t heads,
                            int64_t dk, int64_t dv, const float* rot, int64_t rot_ld, int64_t half, float k_scale, const float* decay,
                            const int32_t* seq_start, const int32_t* seq_first_pos, const int32_t* seq_slot, float* state, float* o,
                            const void* gate, int64_t gate_ld, float eps, void* out, int64_t out_ld, int64_t n, int64_t batch,
                            int dtype, void* stream) {
  if (dtype != LL_F16 && dtype != LL_BF16 && dtype != LL_F32) return LL_ERR_DTYPE;
  if (n < 0 || batch < 0 || heads < 1 || heads > 65535 || !ll_retention_supported(dk, dv) || half < 0 || 2 * half > dk ||
      (half > 0 && rot_ld < 2 * half) || q_ld < heads * dk || k_ld < heads * dk || v_ld < heads * dv || batch * heads > 0x7fffffffll)
    return LL_ERR_SHAPE;
  if (!o && (n != batch || out_ld < heads * dv || (gate && gate_ld < heads * dv))) return LL_ERR_SHAPE;
  if (n == 0 || batch == 0) return LL_OK;
  if (!q || !k || !v || !decay || !seq_start || !seq_first_pos || !seq_slot || !state || (half > 0 && !rot) || (!o && !out)) return LL_ERR_ARG;
  RetentionArgs a;
  a.q = q; a.k = k; a.v = v; a.q_ld = q_ld; a.k_ld = k_ld; a.v_ld = v_ld;
  a.heads = (int)heads; a.dk = (int)dk; a.dv = (int)dv;
  a.rot = rot; a.rot_ld = half > 0 ? rot_ld : 0; a.half = (int)half; a.k_scale = k_scale; a.decay = decay;
  a.seq_start = seq_start; a.seq_first_pos = seq_first_pos; a.seq_slot = seq_slot; a.state = state; a.o = o;
  a.gate = gate; a.gate_ld = gate_ld; a.eps = eps; a.out = out; a.out_ld = out_ld;
  hipStream_t st = (hipStream_t)stream;
  if (!o) {
    const bool wide = dv % 4 == 0 && ll_aligned16(state);
    const int64_t pieces = wide ? dv / 4 : dv, per_pass = pieces < 256 ? pieces : 256;
    const size_t lds = sizeof(float) * (size_t)(2 * dk + (256 / per_pass) * dv);
    const dim3 grid((unsigned)batch, (unsigned)heads);
#define LL_RD(DT)                                                               \
  if (wide) retention_decode_kernel<DT, 4><<<grid, 256, lds, st>>>(a);          \
  else retention_decode_kernel<DT, 1><<<grid, 256, lds, st>>>(a)
    if (dtype == LL_F16) { LL_RD(LL_F16); }
    else if (dtype == LL_BF16) { LL_RD(LL_BF16); }
    else { LL_RD(LL_F32); }
#undef LL_RD
    return LL_LAUNCH_CHECK();
  }
  // the column slices of a (sequence, head) are batch * heads workgroups apart: with a multiple of 8 of those they share an XCD's L2
  const dim3 grid((unsigned)(batch * heads), (unsigned)((dv + kCols - 1) / kCols));
  const bool vec = dtype != LL_F32 && dk % 8 == 0 && dv % 8 == 0 && half % 8 == 0 && q_ld % 8 == 0 && k_ld % 8 == 0 && v_ld % 8 == 0 &&
                   rot_ld % 4 == 0 && ll_aligned16(q) && ll_aligned16(k) && ll_aligned16(v) && (half == 0 || ll_aligned16(rot));
#define LL_RC(DT, V)                                                            \
  return dk <= 64 ? launch_chunk<DT, 4, V>(a, grid, st) : dk <= 128 ? launch_chunk<DT, 8, V>(a, grid, st) : launch_chunk<DT, 16, V>(a, grid, st)
  if (dtype == LL_F32) { LL_RC(LL_F32, false); }
  if (dtype == LL_F16) {
    if (vec) { LL_RC(LL_F16, true); }
    LL_RC(LL_F16, false);
  }
  if (vec) { LL_RC(LL_BF16, true); }
  LL_RC(LL_BF16, false);
#undef LL_RC
}
