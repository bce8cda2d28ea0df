// Several residual STREAMS that a learned matrix mixes at every sublayer (hyper-connections).  A sublayer f with vectors
// in [P], out [P] and a matrix mix [from P][to P] reads and updates the streams x_1 .. x_P (fp32) as
//
//     u = sum_s in_s x_s,   y = scale * f(norm(u)),   x_t <- sum_s mix[s][t] x_s + out_t y     (all t from the old x)
//
//   ll_stream_norm   closes one sublayer and opens the next in ONE launch: the sublayer's result (the sum of several rows per
//                    token, plus a shared row times a per-token factor) times an element-wise scale enters all streams, the
//                    streams are mixed, the next sublayer's input is gathered from the new streams and RMS-normed with a weight
//                    stored around one or around zero.  Without a pending result the streams are only read.
//
// The streams of a token are neighbours, [n][P][width]; right after the embedding they are one row per token that every
// stream reads (stream stride 0).  Storage dtype DT = LL_F16 / LL_BF16 / LL_F32 for activations and weights; streams, mixing,
// sums and norms are fp32.
#include "common.h"

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
template <int DT>
__device__ __forceinline__ f32x4 ld4(const void* p, int64_t i) {  // four storage-dtype values at element i (multiple of 4)
  if constexpr (DT == LL_F32) {
    return *reinterpret_cast<const f32x4*>((const float*)p + i);
  } else {
    const uint2 u = *reinterpret_cast<const uint2*>((const uint16_t*)p + i);
    return f32x4{to_f32<DT>((uint16_t)(u.x & 0xffff)), to_f32<DT>((uint16_t)(u.x >> 16)), to_f32<DT>((uint16_t)(u.y & 0xffff)),
                 to_f32<DT>((uint16_t)(u.y >> 16))};
  }
}
template <int DT>
__device__ __forceinline__ void st4(void* p, int64_t i, f32x4 v) {
  if constexpr (DT == LL_F32) {
    *reinterpret_cast<f32x4*>((float*)p + i) = v;
  } else {
    uint2 u;
    u.x = (uint32_t)from_f32<DT>(v[0]) | ((uint32_t)from_f32<DT>(v[1]) << 16);
    u.y = (uint32_t)from_f32<DT>(v[2]) | ((uint32_t)from_f32<DT>(v[3]) << 16);
    *reinterpret_cast<uint2*>((uint16_t*)p + i) = u;
  }
}

// sum over a 256-thread workgroup in a fixed order (wave sums, then the four waves in order)
__device__ __forceinline__ float block_sum256(float v, float* lds4) {
  v = wave_sum(v);
  const int wave = threadIdx.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) lds4[wave] = v;
  __syncthreads();
  return ((lds4[0] + lds4[1]) + lds4[2]) + lds4[3];
}

struct StreamArgs {
  const float* x_in;
  int64_t in_tok, in_stream;   // strides of x_in (elements); in_stream 0: one row that every stream reads
  float* x_out;                // [n][P][width]
  const void* y;               // [n][parts][width] or NULL: nothing is pending
  int parts;
  const void* shared;          // [n][width] or NULL
  const float* shared_scale;   // [n]
  const void* scale;           // [width] or NULL
  const void* mix;             // [P][P] from, to
  const void* out_w;           // [P]
  const void* in_w;            // [P] or NULL: ones (the sum of the streams)
  const void* norm_w;          // [width]
  float weight_base;           // added to the norm weight (1: a weight stored around zero)
  float eps;
  void* h;                     // [n][width] or NULL
  int width, streams;
};

// Any number of streams and any width.  Thread i owns channels i, i + 256, ..; the old values of a channel's streams wait in
// LDS while the new ones are formed (x_out may be x_in).
template <int DT>
__global__ __launch_bounds__(256) void stream_norm_kernel(const StreamArgs a) {
  extern __shared__ float old[];   // [streams][256]
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x, W = a.width, P = a.streams;
  const float* xi = a.x_in + t * a.in_tok;
  float* xo = a.x_out + t * (int64_t)P * W;
  const float sscale = a.shared ? a.shared_scale[t] : 0.f;
  auto gathered = [&](int i) -> float {   // (after the update: the streams this thread wrote itself)
    float u = 0.f;
    for (int s = 0; s < P; ++s) {
      const float x = a.y ? xo[(int64_t)s * W + i] : xi[s * a.in_stream + i];
      u += (a.in_w ? ldv<DT>(a.in_w, s) : 1.0f) * x;
    }
    return u;
  };
  float ssq = 0.f;
  for (int i = tid; i < W; i += 256) {
    if (a.y) {
      float d = 0.f;
      for (int p = 0; p < a.parts; ++p) d += ldv<DT>(a.y, (t * a.parts + p) * (int64_t)W + i);
      if (a.shared) d += sscale * ldv<DT>(a.shared, t * (int64_t)W + i);
      if (a.scale) d *= ldv<DT>(a.scale, i);
      for (int s = 0; s < P; ++s) old[s * 256 + tid] = xi[s * a.in_stream + i];
      for (int to = 0; to < P; ++to) {
        float v = 0.f;
        for (int s = 0; s < P; ++s) v += ldv<DT>(a.mix, s * P + to) * old[s * 256 + tid];
        xo[(int64_t)to * W + i] = v + ldv<DT>(a.out_w, to) * d;
      }
    }
    if (a.h) {
      const float u = gathered(i);
      ssq += u * u;
    }
  }
  if (!a.h) return;
  ssq = block_sum256(ssq, red);
  const float inv = 1.0f / sqrtf(ssq / (float)W + a.eps);
  for (int i = tid; i < W; i += 256) stv<DT>(a.h, t * (int64_t)W + i, gathered(i) * inv * (a.weight_base + ldv<DT>(a.norm_w, i)));
}

// Register form: pieces of four channels, up to PM streams (EXACT: exactly PM), the gathered input kept in registers between
// the passes.  One pass over the streams.
template <int DT, int PM, bool EXACT, int NV>
__global__ __launch_bounds__(256) void stream_norm_vec_kernel(const StreamArgs a) {
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x, W = a.width;
  const int P = EXACT ? PM : a.streams;
  const float* xi = a.x_in + t * a.in_tok;
  float* xo = a.x_out + t * (int64_t)P * W;
  const float sscale = a.shared ? a.shared_scale[t] : 0.f;
  float mx[PM][PM], ow[PM], iw[PM];
#pragma unroll
  for (int s = 0; s < PM; ++s) {
    iw[s] = s < P ? (a.in_w ? ldv<DT>(a.in_w, s) : 1.0f) : 0.f;
    ow[s] = (a.y && s < P) ? ldv<DT>(a.out_w, s) : 0.f;
#pragma unroll
    for (int to = 0; to < PM; ++to) mx[s][to] = (a.y && s < P && to < P) ? ldv<DT>(a.mix, s * P + to) : 0.f;
  }
  f32x4 u[NV];
  float ssq = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int i = 4 * (tid + 256 * k);
    u[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (i < W) {
      f32x4 x[PM];
#pragma unroll
      for (int s = 0; s < PM; ++s)
        x[s] = (EXACT || s < P) ? *reinterpret_cast<const f32x4*>(xi + s * a.in_stream + i) : f32x4{0.f, 0.f, 0.f, 0.f};
      if (a.y) {
        f32x4 d = {0.f, 0.f, 0.f, 0.f};
        for (int p = 0; p < a.parts; ++p) d += ld4<DT>(a.y, (t * a.parts + p) * (int64_t)W + i);
        if (a.shared) d += sscale * ld4<DT>(a.shared, t * (int64_t)W + i);
        if (a.scale) d *= ld4<DT>(a.scale, i);
#pragma unroll
        for (int to = 0; to < PM; ++to) {
          if (EXACT || to < P) {
            f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < PM; ++s) v += mx[s][to] * x[s];
            v += ow[to] * d;
            *reinterpret_cast<f32x4*>(xo + (int64_t)to * W + i) = v;
            u[k] += iw[to] * v;
          }
        }
      } else {
#pragma unroll
        for (int s = 0; s < PM; ++s) u[k] += iw[s] * x[s];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ssq += u[k][e] * u[k][e];
    }
  }
  if (!a.h) return;
  ssq = block_sum256(ssq, red);
  const float inv = 1.0f / sqrtf(ssq / (float)W + a.eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int i = 4 * (tid + 256 * k);
    if (i < W) {
      const f32x4 w = ld4<DT>(a.norm_w, i);
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = u[k][e] * inv * (a.weight_base + w[e]);
      st4<DT>(a.h, t * (int64_t)W + i, o);
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

extern "C" int ll_stream_norm(const float* x_in, int64_t in_tok, int64_t in_stream, float* x_out, const void* y, int64_t parts,
                              const void* shared, const float* shared_scale, const void* scale, const void* mix, const void* out_w,
                              const void* in_w, const void* norm_w, float weight_base, float eps, void* h, int64_t n, int64_t width,
                              int64_t streams, int dtype, void* stream) {
  if (dtype != LL_F16 && dtype != LL_BF16 && dtype != LL_F32) return LL_ERR_DTYPE;
  if (n < 0 || n > 0x7fffffffll || width < 1 || width > (1 << 20) || streams < 1 || streams > 32 || parts < 0 || parts > 64) return LL_ERR_SHAPE;
  if (in_stream != 0 && in_stream < width) return LL_ERR_SHAPE;
  if (in_tok < (in_stream ? (streams - 1) * in_stream + width : width)) return LL_ERR_SHAPE;
  if (n == 0) return LL_OK;
  if (!x_in || (h && !norm_w) || (!y && !h)) return LL_ERR_ARG;
  if (y && (!x_out || !mix || !out_w || parts < 1 || (shared && !shared_scale))) return LL_ERR_ARG;
  // in place only where a token's streams are read and written at the same places
  if (y && x_out == x_in && !(in_tok == streams * width && (in_stream == width || streams == 1))) return LL_ERR_ARG;
  StreamArgs a;
  a.x_in = x_in; a.in_tok = in_tok; a.in_stream = in_stream; a.x_out = x_out; a.y = y; a.parts = (int)parts; a.shared = shared;
  a.shared_scale = shared_scale; a.scale = scale; a.mix = mix; a.out_w = out_w; a.in_w = in_w; a.norm_w = norm_w;
  a.weight_base = weight_base; a.eps = eps; a.h = h; a.width = (int)width; a.streams = (int)streams;
  const dim3 grid((unsigned)n);
  hipStream_t st = (hipStream_t)stream;
  const int al = dtype == LL_F32 ? 16 : 8;   // bytes a four-channel piece of a storage-dtype row must be aligned to
  auto ok = [&](const void* p) { return !p || (reinterpret_cast<uintptr_t>(p) % al) == 0; };
  const bool vec = width % 4 == 0 && width <= 4096 && streams <= 8 && in_tok % 4 == 0 && in_stream % 4 == 0 && ll_aligned16(x_in) &&
                   (!y || ll_aligned16(x_out)) && ok(y) && ok(shared) && ok(scale) && ok(norm_w) && ok(h);
  if (!vec) {
    const size_t lds = sizeof(float) * 256 * (size_t)streams;
#define CALL(DT) stream_norm_kernel<DT><<<grid, 256, lds, st>>>(a)
    LL_BY_DTYPE(dtype, CALL);
#undef CALL
    return LL_LAUNCH_CHECK();
  }
#define CALL_V(DT, PM, E)                                                            \
  if (width <= 1024) stream_norm_vec_kernel<DT, PM, E, 1><<<grid, 256, 0, st>>>(a);  \
  else if (width <= 2048) stream_norm_vec_kernel<DT, PM, E, 2><<<grid, 256, 0, st>>>(a); \
  else stream_norm_vec_kernel<DT, PM, E, 4><<<grid, 256, 0, st>>>(a)
#define CALL(DT)                                    \
  if (streams == 1) { CALL_V(DT, 1, true); }        \
  else if (streams == 2) { CALL_V(DT, 2, true); }   \
  else if (streams == 3) { CALL_V(DT, 3, true); }   \
  else if (streams == 4) { CALL_V(DT, 4, true); }   \
  else { CALL_V(DT, 8, false); }
  LL_BY_DTYPE(dtype, CALL);
#undef CALL
#undef CALL_V
  return LL_LAUNCH_CHECK();
}
