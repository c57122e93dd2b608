// A residual stream that is kept in float32 whatever the engine's dtype, and the norms that read
// and feed it:
//
//   Dynamic Tanh          y = tanh(alpha * x) * w + b            (elementwise, nothing of the row)
//   RMS norm              y = x * rsqrt(mean(x^2) + eps) * w
//
// ptl_stream_add_dyt: stream += post(y) and out = pre(stream) in one pass over the rows: the norm
//   behind a sublayer, the residual sum and the norm in front of the next sublayer. Every piece
//   is optional: no y (only the norm in front), no post norm (a plain sum), no out, and a copy
//   of the new stream in the engine's dtype for a product that reads the stream itself.
// ptl_stream_add_rmsnorm: stream += rmsnorm(y) * w, the same with a norm that needs the row.
// ptl_stream_add_rmsnorm_sum: the same for a result that is a weighted sum of two and a bias.
// ptl_stream_postnorm: stream = rmsnorm(alpha stream + y) * w, the norm behind the residual sum, with y a
//   weighted sum of up to two results each of which may be RMS-normed first (where it stands, below).
// ptl_stream_scaled_sum: stream += s1 (y1 + bias) + s2 y2 with a scale an entry, and the RMS norm in front
//   of what reads the stream next: two sublayers side by side on one input (where it stands, below).
// ptl_stream_rmsnorm: the RMS norm of rows of the stream, in the engine's type.
// ptl_dyt: the norm alone, for rows that are no stream (the rows picked for the head).
// ptl_embedding_scaled: stream[t] = table[ids[t]] * scale, in float32 (``copies`` times side by side in
//   a row, for a model that keeps several streams). ptl_embedding_positions: the same with a sinusoidal
//   vector of the token's position added.
// ptl_softcap: cap * tanh(x / cap) on float32 logits.
// ptl_hyper_mix: several residual streams a token (hyper-connections): the streams' update behind a
//   sublayer and the read-out with its RMS norm in front of the next one (where it stands, below).
// ptl_gelu_gather_mul: out[t, j] = gelu_tanh(z[t, j]) * table[ids[t], col0 + j]: a gate on a
//   per-token vector looked up in a table that several layers share.
//
// All arithmetic is float32; tanhf / expf are the accurate ones.
#include "common.h"
#include <math.h>
#include <type_traits>

struct DytArgs {
  const float* w;     // [H]; null: the norm is absent
  const float* b;     // [H] or null
  float alpha;
};

__device__ __forceinline__ float dyt_apply(const DytArgs& n, float x, int c) {
  const float y = tanhf(n.alpha * x) * n.w[c];
  return n.b ? y + n.b[c] : y;
}

template <typename TY, typename TO>
__global__ void __launch_bounds__(256)
stream_add_dyt_kernel(float* __restrict__ stream, const TY* __restrict__ y, DytArgs post,
                      TO* __restrict__ out, DytArgs pre, TO* __restrict__ copy, size_t total, int H) {
  size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  const size_t step = (size_t)gridDim.x * 256;
  for (; i < total; i += step) {
    const int c = (int)(i % H);
    float s = stream[i];
    if (y) {
      const float v = to_float<TY>(y[i]);
      s += post.w ? dyt_apply(post, v, c) : v;
      stream[i] = s;
    }
    if (out) out[i] = from_float<TO>(dyt_apply(pre, s, c));
    if (copy) copy[i] = from_float<TO>(s);
  }
}

template <typename TY, typename TO>
static int launch_add_dyt(float* stream, const void* y, DytArgs post, void* out, DytArgs pre, void* copy,
                          size_t total, int H, hipStream_t st) {
  size_t blocks = (total + 255) / 256;
  if (blocks > 65536) blocks = 65536;
  stream_add_dyt_kernel<TY, TO><<<(int)blocks, 256, 0, st>>>(stream, (const TY*)y, post, (TO*)out, pre,
                                                            (TO*)copy, total, H);
  return ptl_launch_status();
}

// y_dtype: of y; out_dtype: of out and copy. Null pointers switch the pieces off (see above).
extern "C" int ptl_stream_add_dyt(float* stream, const void* y, int y_dtype, const float* post_w,
                                  const float* post_b, float post_alpha, void* out, int out_dtype,
                                  const float* pre_w, const float* pre_b, float pre_alpha, void* copy,
                                  int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !stream || (out && !pre_w)) return PTL_ERR_ARG;
  const DytArgs post{post_w, post_b, post_alpha}, pre{pre_w, pre_b, pre_alpha};
  const size_t total = (size_t)T_ * H;
#define GO(TY, TO) return launch_add_dyt<TY, TO>(stream, y, post, out, pre, copy, total, H, st)
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) GO(float, float);
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) GO(float, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) GO(bf16_t, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) GO(bf16_t, float);
#undef GO
  return PTL_ERR_ARG;
}

template <typename TX, typename TO>
__global__ void __launch_bounds__(256)
dyt_kernel(TO* __restrict__ out, const TX* __restrict__ x, DytArgs n, size_t total, int H) {
  size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  const size_t step = (size_t)gridDim.x * 256;
  for (; i < total; i += step) out[i] = from_float<TO>(dyt_apply(n, to_float<TX>(x[i]), (int)(i % H)));
}

extern "C" int ptl_dyt(void* out, int out_dtype, const void* x, int x_dtype, const float* w,
                       const float* b, float alpha, int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !w) return PTL_ERR_ARG;
  const DytArgs n{w, b, alpha};
  const size_t total = (size_t)T_ * H;
  size_t blocks = (total + 255) / 256;
  if (blocks > 65536) blocks = 65536;
#define GO(TX, TO)                                                                                   \
  {                                                                                                  \
    dyt_kernel<TX, TO><<<(int)blocks, 256, 0, st>>>((TO*)out, (const TX*)x, n, total, H);            \
    return ptl_launch_status();                                                                      \
  }
  if (x_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) GO(float, float);
  if (x_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) GO(float, bf16_t);
  if (x_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) GO(bf16_t, bf16_t);
  if (x_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) GO(bf16_t, float);
#undef GO
  return PTL_ERR_ARG;
}

// One workgroup a row: the sum of squares of y, then stream += y * rsqrt(mean + eps) * w and, when
// asked for, out = pre(stream) and the copy of the new stream.
template <typename TY, typename TO>
__global__ void __launch_bounds__(256)
stream_add_rmsnorm_kernel(float* __restrict__ stream, const TY* __restrict__ y, const float* __restrict__ w,
                          float eps, TO* __restrict__ out, DytArgs pre, TO* __restrict__ copy, int H) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * H;
  float ss = 0.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    const float v = to_float<TY>(y[row + c]);
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)H + eps);
  for (int c = threadIdx.x; c < H; c += 256) {
    const float s = stream[row + c] + to_float<TY>(y[row + c]) * r * w[c];
    stream[row + c] = s;
    if (out) out[row + c] = from_float<TO>(dyt_apply(pre, s, c));
    if (copy) copy[row + c] = from_float<TO>(s);
  }
}

extern "C" int ptl_stream_add_rmsnorm(float* stream, const void* y, int y_dtype, const float* w, float eps,
                                      void* out, int out_dtype, const float* pre_w, const float* pre_b,
                                      float pre_alpha, void* copy, int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !stream || !y || !w || (out && !pre_w)) return PTL_ERR_ARG;
  const DytArgs pre{pre_w, pre_b, pre_alpha};
#define GO(TY, TO)                                                                                   \
  {                                                                                                  \
    stream_add_rmsnorm_kernel<TY, TO><<<T_, 256, 0, st>>>(stream, (const TY*)y, w, eps, (TO*)out, pre, \
                                                          (TO*)copy, H);                             \
    return ptl_launch_status();                                                                      \
  }
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) GO(float, float);
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) GO(float, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) GO(bf16_t, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) GO(bf16_t, float);
#undef GO
  return PTL_ERR_ARG;
}

// The same for a sublayer whose result is a weighted sum that has not been added up yet:
// y = a y1 + b y2 + c bias (y2 and bias optional), stream += rmsnorm(y) * w. The sum is float32.
template <typename TY, typename TO>
__global__ void __launch_bounds__(256)
stream_add_rmsnorm_sum_kernel(float* __restrict__ stream, const TY* __restrict__ y1, float a,
                              const TY* __restrict__ y2, float b, const float* __restrict__ bias, float c,
                              const float* __restrict__ w, float eps, TO* __restrict__ copy, int H) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * H;
  float ss = 0.f;
  for (int j = threadIdx.x; j < H; j += 256) {
    float v = a * to_float<TY>(y1[row + j]);
    if (y2) v = fmaf(b, to_float<TY>(y2[row + j]), v);
    if (bias) v = fmaf(c, bias[j], v);
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)H + eps);
  for (int j = threadIdx.x; j < H; j += 256) {
    float v = a * to_float<TY>(y1[row + j]);
    if (y2) v = fmaf(b, to_float<TY>(y2[row + j]), v);
    if (bias) v = fmaf(c, bias[j], v);
    const float s = stream[row + j] + v * r * w[j];
    stream[row + j] = s;
    if (copy) copy[row + j] = from_float<TO>(s);
  }
}

extern "C" int ptl_stream_add_rmsnorm_sum(float* stream, const void* y1, float a, const void* y2, float b,
                                          int y_dtype, const float* bias, float c, const float* w, float eps,
                                          void* copy, int out_dtype, int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !stream || !y1 || !w) return PTL_ERR_ARG;
#define GO(TY, TO)                                                                                    \
  {                                                                                                   \
    stream_add_rmsnorm_sum_kernel<TY, TO><<<T_, 256, 0, st>>>(stream, (const TY*)y1, a, (const TY*)y2, b, \
                                                              bias, c, w, eps, (TO*)copy, H);         \
    return ptl_launch_status();                                                                       \
  }
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) GO(float, float);
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) GO(float, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) GO(bf16_t, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) GO(bf16_t, float);
#undef GO
  return PTL_ERR_ARG;
}

// The norm behind the residual sum: stream <- u * rsqrt(mean(u^2) + eps) * w with
//   u = alpha stream + a n1(y1) + b n2(y2) + c bias,    n(y) = y * rsqrt(mean(y^2) + n_eps) * nw, or y
// (y2, the bias and both inner norms are optional), and a copy of the new stream in the engine's
// type. One workgroup a row; a thread keeps its VPT groups of VEC neighbouring entries of y1, y2 and
// the stream in registers from the one pass over memory to the last use.
struct PostNormArgs {
  float* stream; float alpha;
  const void* y1; float a; const float* n1;
  const void* y2; float b; const float* n2;
  const float* bias; float c;
  float n_eps;
  const float* w; float eps;
  void* copy;
  int H;
};

template <int NT, int VPT, int VEC, typename TY, typename TO>
__global__ void __launch_bounds__(NT) stream_postnorm_kernel(PostNormArgs A) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * A.H;
  const TY* y1 = (const TY*)A.y1 + row;
  const TY* y2 = A.y2 ? (const TY*)A.y2 + row : nullptr;
  float* stream = A.stream + row;
  float v1[VPT][VEC], v2[VPT][VEC], u[VPT][VEC];
  float s1 = 0.f, s2 = 0.f;
  auto read = [&](const auto* p, int i0, float (&v)[VEC]) {
    typedef typename std::remove_cv<typename std::remove_pointer<decltype(p)>::type>::type T;
    if (VEC == 1) {
      v[0] = to_float<T>(p[i0]);
    } else if (sizeof(T) == 4) {
      const float4 x = *reinterpret_cast<const float4*>(p + i0);
      v[0] = x.x; v[VEC > 1 ? 1 : 0] = x.y; v[VEC > 2 ? 2 : 0] = x.z; v[VEC > 3 ? 3 : 0] = x.w;
    } else {
      const uint2 x = *reinterpret_cast<const uint2*>(p + i0);
      v[0] = __uint_as_float(x.x << 16); v[VEC > 1 ? 1 : 0] = __uint_as_float(x.x & 0xffff0000u);
      v[VEC > 2 ? 2 : 0] = __uint_as_float(x.y << 16); v[VEC > 3 ? 3 : 0] = __uint_as_float(x.y & 0xffff0000u);
    }
  };
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (k * NT + threadIdx.x) * VEC;
    if (i >= A.H) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v1[k][j] = v2[k][j] = u[k][j] = 0.f;
      continue;
    }
    read(y1, i, v1[k]);
    if (y2) read(y2, i, v2[k]);
    read((const float*)stream, i, u[k]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      if (!y2) v2[k][j] = 0.f;
      s1 = fmaf(v1[k][j], v1[k][j], s1);
      s2 = fmaf(v2[k][j], v2[k][j], s2);
    }
  }
  float f1 = A.a, f2 = A.b;
  if (A.n1) f1 *= 1.0f / sqrtf(block_sum(s1, scratch) / (float)A.H + A.n_eps);
  if (A.n2) f2 *= 1.0f / sqrtf(block_sum(s2, scratch) / (float)A.H + A.n_eps);
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (k * NT + threadIdx.x) * VEC;
    if (i >= A.H) continue;
    float w1[VEC], w2[VEC], bs[VEC];
    if (A.n1) read(A.n1, i, w1);
    if (A.n2) read(A.n2, i, w2);
    if (A.bias) read(A.bias, i, bs);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      float x = A.alpha * u[k][j];
      x = fmaf(f1, A.n1 ? v1[k][j] * w1[j] : v1[k][j], x);
      if (y2) x = fmaf(f2, A.n2 ? v2[k][j] * w2[j] : v2[k][j], x);
      if (A.bias) x = fmaf(A.c, bs[j], x);
      u[k][j] = x;
      ss = fmaf(x, x, ss);
    }
  }
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)A.H + A.eps);
  TO* copy = A.copy ? (TO*)A.copy + row : nullptr;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (k * NT + threadIdx.x) * VEC;
    if (i >= A.H) continue;
    float w[VEC];
    read(A.w, i, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[k][j] = u[k][j] * r * w[j];
    if (VEC == 1) {
      stream[i] = u[k][0];
      if (copy) copy[i] = from_float<TO>(u[k][0]);
    } else {
      *reinterpret_cast<float4*>(stream + i) = make_float4(u[k][0], u[k][VEC > 1 ? 1 : 0], u[k][VEC > 2 ? 2 : 0], u[k][VEC > 3 ? 3 : 0]);
      if (copy) {
        TO e[VEC];
#pragma unroll
        for (int j = 0; j < VEC; ++j) e[j] = from_float<TO>(u[k][j]);
        if (sizeof(TO) == 2) *reinterpret_cast<uint2*>(copy + i) = *reinterpret_cast<const uint2*>(e);
        else *reinterpret_cast<float4*>(copy + i) = *reinterpret_cast<const float4*>(e);
      }
    }
  }
}

template <typename TY, typename TO>
static int launch_postnorm(const PostNormArgs& A, int T_, hipStream_t st) {
  auto odd = [](const void* p) { return ((uintptr_t)p & 15) != 0; };
  const bool vec = A.H % 4 == 0 && !odd(A.stream) && !odd(A.y1) && !odd(A.y2) && !odd(A.n1) && !odd(A.n2) &&
                   !odd(A.bias) && !odd(A.w) && !odd(A.copy);
  const int n = vec ? A.H / 4 : A.H;         // groups of entries of a row
  // few rows: a row over 1,024 threads, so that a thread's loads are one or two deep
  const bool few = T_ <= 512 && n > 256;
#define GO(NT, VPT)                                                                  \
  if (n <= NT * VPT) {                                                               \
    if (vec) stream_postnorm_kernel<NT, VPT, 4, TY, TO><<<T_, NT, 0, st>>>(A);       \
    else stream_postnorm_kernel<NT, VPT, 1, TY, TO><<<T_, NT, 0, st>>>(A);           \
    return ptl_launch_status();                                                      \
  }
  if (!few) { GO(256, 1) GO(256, 2) GO(256, 4) }
  GO(1024, 1) GO(1024, 2) GO(1024, 4)
  if (!vec) { GO(1024, 16) }
#undef GO
  return PTL_ERR_ARG;
}

// stream float32 [T, H], in place; y1, y2 [T, H] of y_dtype; n1, n2, bias, w float32 [H]; copy [T, H] of
// out_dtype or null. H up to 16,384.
extern "C" int ptl_stream_postnorm(float* stream, float alpha, const void* y1, float a, const float* n1,
                                   const void* y2, float b, const float* n2, int y_dtype, const float* bias, float c,
                                   float n_eps, const float* w, float eps, void* copy, int out_dtype, int T_, int H,
                                   hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !stream || !y1 || !w || (n2 && !y2)) return PTL_ERR_ARG;
  const PostNormArgs A{stream, alpha, y1, a, n1, y2, b, n2, bias, c, n_eps, w, eps, copy, H};
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) return launch_postnorm<float, float>(A, T_, st);
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) return launch_postnorm<float, bf16_t>(A, T_, st);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) return launch_postnorm<bf16_t, bf16_t>(A, T_, st);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) return launch_postnorm<bf16_t, float>(A, T_, st);
  return PTL_ERR_ARG;
}

// The residual sum of sublayers whose results are scaled entry by entry, and the norm that follows:
//   stream += s1 * (y1 + bias) + s2 * y2;    out = stream * rsqrt(mean(stream^2) + eps) * w
// (y1, y2, bias and both scales are optional: no y1 and no y2 leaves the stream as it is; w null: no
// norm, no out). y2 may also come as routed experts leave it: the rows of a token's choices times
// their weights, and a shared expert's row (RoutedArgs). Behind the norm a time mixer's inputs can be made as
// well, for rows that are sequences of one token (MixArgs): out_m = h + (h' - h) mu_m, h' the row kept in
// the sequence's state slot. One workgroup a row; a thread keeps its VPT groups of VEC neighbouring entries in
// registers from the one pass over memory to the last use.
struct RoutedArgs {
  const void* rows; long ldr;               // the experts' results, sorted by expert; null: none
  const int32_t* pos_of; const float* wgt; int top;      // [T * top]; wgt null: ones
  const void* shared;                       // [T, H] or null
};
struct MixArgs {
  void* out; long mix_stride;               // [n, T, H]; null: none
  const float* mu; int n;                   // [n, H]
  const float* state; long slot_stride; long off; const int32_t* slots;
};
struct ScaledSumArgs {
  float* stream;
  const void* y1; const float* s1; const float* bias;
  const void* y2; const float* s2;
  const float* w; float eps;
  void* out;
  int H;
  RoutedArgs routed;
  MixArgs mix;
};

template <int VEC, typename T>
__device__ __forceinline__ void read_vec(const T* p, float (&v)[VEC]) {
  if (VEC == 1) {
    v[0] = to_float<T>(p[0]);
  } else if (sizeof(T) == 4) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[VEC > 1 ? 1 : 0] = x.y; v[VEC > 2 ? 2 : 0] = x.z; v[VEC > 3 ? 3 : 0] = x.w;
  } else {
    const uint2 x = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(x.x << 16); v[VEC > 1 ? 1 : 0] = __uint_as_float(x.x & 0xffff0000u);
    v[VEC > 2 ? 2 : 0] = __uint_as_float(x.y << 16); v[VEC > 3 ? 3 : 0] = __uint_as_float(x.y & 0xffff0000u);
  }
}

template <int NT, int VPT, int VEC, typename T1, typename T2, typename TO>
__global__ void __launch_bounds__(NT) stream_scaled_sum_kernel(ScaledSumArgs A) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * A.H;
  float* stream = A.stream + row;
  float u[VPT][VEC], d[VPT][VEC];          // d: the kept row, asked for long before it is needed
  const float* kept = A.mix.out ? A.mix.state + (size_t)A.mix.slots[blockIdx.x] * A.mix.slot_stride + A.mix.off : nullptr;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (k * NT + threadIdx.x) * VEC;
    if (i >= A.H) continue;
    read_vec<VEC>((const float*)stream + i, u[k]);
    if (kept) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) d[k][j] = kept[i + j];
    }
    if (A.y1) {
      float y[VEC], f[VEC];
      read_vec<VEC>((const T1*)A.y1 + row + i, y);
      if (A.bias) {
        read_vec<VEC>(A.bias + i, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[j] += f[j];
      }
      if (A.s1) read_vec<VEC>(A.s1 + i, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[k][j] = fmaf(A.s1 ? f[j] : 1.f, y[j], u[k][j]);
    }
    if (A.y2 || A.routed.rows) {
      float y[VEC], f[VEC];
      if (A.routed.rows) {
        const RoutedArgs& R = A.routed;
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[j] = 0.f;
#pragma unroll 4
        for (int c = 0; c < R.top; ++c) {
          const size_t pair = (size_t)blockIdx.x * R.top + c;
          const int p = R.pos_of[pair];
          if (p < 0) continue;
          const float g = R.wgt ? R.wgt[pair] : 1.f;
          read_vec<VEC>((const T2*)R.rows + (size_t)p * R.ldr + i, f);
#pragma unroll
          for (int j = 0; j < VEC; ++j) y[j] = fmaf(f[j], g, y[j]);
        }
        if (R.shared) {
          read_vec<VEC>((const T2*)R.shared + row + i, f);
#pragma unroll
          for (int j = 0; j < VEC; ++j) y[j] += f[j];
        }
      } else {
        read_vec<VEC>((const T2*)A.y2 + row + i, y);
      }
      if (A.s2) read_vec<VEC>(A.s2 + i, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[k][j] = fmaf(A.s2 ? f[j] : 1.f, y[j], u[k][j]);
    }
    if (A.y1 || A.y2 || A.routed.rows) {
      if (VEC == 1) stream[i] = u[k][0];
      else *reinterpret_cast<float4*>(stream + i) = make_float4(u[k][0], u[k][VEC > 1 ? 1 : 0], u[k][VEC > 2 ? 2 : 0], u[k][VEC > 3 ? 3 : 0]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(u[k][j], u[k][j], ss);
  }
  if (!A.w) return;
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)A.H + A.eps);
  TO* out = (TO*)A.out + row;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (k * NT + threadIdx.x) * VEC;
    if (i >= A.H) continue;
    float w[VEC];
    read_vec<VEC>(A.w + i, w);
    TO e[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) e[j] = from_float<TO>(u[k][j] * r * w[j]);
    auto put = [](TO* at, const TO (&v)[VEC]) {
      if (VEC == 1) at[0] = v[0];
      else if (sizeof(TO) == 2) *reinterpret_cast<uint2*>(at) = *reinterpret_cast<const uint2*>(v);
      else *reinterpret_cast<float4*>(at) = *reinterpret_cast<const float4*>(v);
    };
    put(out + i, e);
    if (A.mix.out) {
      const MixArgs& M = A.mix;
      float h[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        h[j] = to_float<TO>(e[j]);
        d[k][j] -= h[j];
      }
      constexpr int AT_ONCE = 5;            // the factors of so many mixes are asked for together
      for (int m0 = 0; m0 < M.n; m0 += AT_ONCE) {
        float f[AT_ONCE][VEC];
#pragma unroll
        for (int m = 0; m < AT_ONCE; ++m)
          if (m0 + m < M.n) read_vec<VEC>(M.mu + (size_t)(m0 + m) * A.H + i, f[m]);
#pragma unroll
        for (int m = 0; m < AT_ONCE; ++m) {
          if (m0 + m >= M.n) continue;
#pragma unroll
          for (int j = 0; j < VEC; ++j) e[j] = from_float<TO>(fmaf(d[k][j], f[m][j], h[j]));
          put((TO*)M.out + (size_t)(m0 + m) * M.mix_stride + row + i, e);
        }
      }
    }
  }
}

template <typename T1, typename T2, typename TO>
static int launch_scaled_sum(const ScaledSumArgs& A, int T_, hipStream_t st) {
  auto odd = [](const void* p) { return ((uintptr_t)p & 15) != 0; };
  const bool vec = A.H % 4 == 0 && !odd(A.stream) && !odd(A.y1) && !odd(A.s1) && !odd(A.bias) && !odd(A.y2) &&
                   !odd(A.s2) && !odd(A.w) && !odd(A.out) && !odd(A.routed.rows) && !odd(A.routed.shared) &&
                   A.routed.ldr % 4 == 0 && !odd(A.mix.out) && !odd(A.mix.mu) && A.mix.mix_stride % 4 == 0;
  const int n = vec ? A.H / 4 : A.H;         // groups of entries of a row
  // few rows: a row over 1,024 threads, so that a thread's loads are one or two deep
  const bool few = T_ <= 512 && n > 256;
#define GO(NT, VPT)                                                                      \
  if (n <= NT * VPT) {                                                                   \
    if (vec) stream_scaled_sum_kernel<NT, VPT, 4, T1, T2, TO><<<T_, NT, 0, st>>>(A);     \
    else stream_scaled_sum_kernel<NT, VPT, 1, T1, T2, TO><<<T_, NT, 0, st>>>(A);         \
    return ptl_launch_status();                                                          \
  }
  if (!few) { GO(256, 1) GO(256, 2) GO(256, 4) }
  GO(1024, 1) GO(1024, 2) GO(1024, 4)
  if (!vec) { GO(1024, 16) }
#undef GO
  return PTL_ERR_ARG;
}

// stream float32 [T, H], in place; y1 [T, H] float32 or null; y2 [T, H] of y2_dtype or null, or in its place rows
// (ldr), pos_of, wgt, top and shared of y2_dtype (RoutedArgs); s1, s2, bias, w float32 [H] or null; out [T, H] of
// out_dtype (with w); mix_out [n_mix, T, H] of out_dtype or null, with mu float32 [n_mix, H] and row t's kept
// row at state + slots[t] * slot_stride + off (MixArgs). H up to 16,384.
extern "C" int ptl_stream_scaled_sum(float* stream, const float* y1, const float* s1, const float* bias,
                                     const void* y2, int y2_dtype, const float* s2, const void* rows, long ldr,
                                     const int32_t* pos_of, const float* wgt, int top, const void* shared,
                                     const float* w, float eps, void* out, int out_dtype, void* mix_out,
                                     long mix_stride, const float* mu, int n_mix, const float* state,
                                     long slot_stride, long off, const int32_t* slots, int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !stream || (bias && !y1) || (w && !out) || (!y1 && !y2 && !rows && !w) || (y2 && rows) ||
      (rows && (!pos_of || top <= 0 || ldr < H)) || (shared && !rows) ||
      (mix_out && (!w || !mu || n_mix <= 0 || !state || !slots || mix_stride < (long)T_ * H || off < 0 ||
                   off + H > slot_stride)))
    return PTL_ERR_ARG;
  const ScaledSumArgs A{stream, y1, s1, bias, y2, s2, w, eps, out, H, RoutedArgs{rows, ldr, pos_of, wgt, top, shared},
                        MixArgs{mix_out, mix_stride, mu, n_mix, state, slot_stride, off, slots}};
  if (y2_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) return launch_scaled_sum<float, float, float>(A, T_, st);
  if (y2_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) return launch_scaled_sum<float, float, bf16_t>(A, T_, st);
  if (y2_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) return launch_scaled_sum<float, bf16_t, bf16_t>(A, T_, st);
  return PTL_ERR_ARG;
}

// out = x * rsqrt(mean(x^2) + eps) * w for rows of a float32 stream, in the engine's type (the rows
// picked for the head).
template <typename TO>
__global__ void __launch_bounds__(256)
stream_rmsnorm_kernel(TO* __restrict__ out, const float* __restrict__ x, const float* __restrict__ w,
                      float eps, int H) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * H;
  float ss = 0.f;
  for (int j = threadIdx.x; j < H; j += 256) ss = fmaf(x[row + j], x[row + j], ss);
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)H + eps);
  for (int j = threadIdx.x; j < H; j += 256) out[row + j] = from_float<TO>(x[row + j] * r * w[j]);
}

extern "C" int ptl_stream_rmsnorm(void* out, int out_dtype, const float* x, const float* w, float eps,
                                  int T_, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || !x || !w) return PTL_ERR_ARG;
  if (out_dtype == PTL_DTYPE_F32)
    stream_rmsnorm_kernel<float><<<T_, 256, 0, st>>>((float*)out, x, w, eps, H);
  else if (out_dtype == PTL_DTYPE_BF16)
    stream_rmsnorm_kernel<bf16_t><<<T_, 256, 0, st>>>((bf16_t*)out, x, w, eps, H);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}

template <typename T>
__global__ void embedding_scaled_kernel(float* __restrict__ out, const T* __restrict__ table,
                                        const int32_t* __restrict__ ids, int H, int V, float scale,
                                        int copies) {
  const int t = blockIdx.x;
  int id = ids[t];
  if (id < 0 || id >= V) id = 0;          // checked on the host; never read out of bounds
  const T* src = table + (size_t)id * H;
  float* dst = out + (size_t)t * H * copies;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = to_float<T>(src[i]) * scale;
    for (int s = 0; s < copies; ++s) dst[(size_t)s * H + i] = v;
  }
}

extern "C" int ptl_embedding_scaled(float* out, const void* table, const int32_t* ids, int T_, int H,
                                    int V, float scale, int copies, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || V <= 0 || copies < 1) return PTL_ERR_ARG;
  const int threads = H >= 1024 ? 256 : (H >= 256 ? 128 : 64);
  if (dtype == PTL_DTYPE_F32)
    embedding_scaled_kernel<float><<<T_, threads, 0, st>>>(out, (const float*)table, ids, H, V, scale, copies);
  else if (dtype == PTL_DTYPE_BF16)
    embedding_scaled_kernel<bf16_t><<<T_, threads, 0, st>>>(out, (const bf16_t*)table, ids, H, V, scale, copies);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}

// out[t, j] = table[ids[t], j] * scale + sin or cos (j even or odd) of positions[t] * freq[j / 2]
template <typename T>
__global__ void __launch_bounds__(256)
embedding_positions_kernel(float* __restrict__ out, const T* __restrict__ table, const int32_t* __restrict__ ids,
                           const int32_t* __restrict__ positions, const float* __restrict__ freq, int H, int V,
                           float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  if (id < 0 || id >= V) id = 0;          // checked on the host; never read out of bounds
  const T* src = table + (size_t)id * H;
  float* dst = out + (size_t)t * H;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; 2 * i < H; i += blockDim.x) {
    float s, c;
    sincosf(pos * freq[i], &s, &c);
    dst[2 * i] = fmaf(to_float<T>(src[2 * i]), scale, s);
    if (2 * i + 1 < H) dst[2 * i + 1] = fmaf(to_float<T>(src[2 * i + 1]), scale, c);
  }
}

extern "C" int ptl_embedding_positions(float* out, const void* table, const int32_t* ids, const int32_t* positions,
                                       const float* freq, int T_, int H, int V, float scale, int dtype,
                                       hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || V <= 0 || !positions || !freq) return PTL_ERR_ARG;
  const int threads = H >= 512 ? 256 : (H >= 256 ? 128 : 64);
  if (dtype == PTL_DTYPE_F32)
    embedding_positions_kernel<float><<<T_, threads, 0, st>>>(out, (const float*)table, ids, positions, freq, H, V, scale);
  else if (dtype == PTL_DTYPE_BF16)
    embedding_positions_kernel<bf16_t><<<T_, threads, 0, st>>>(out, (const bf16_t*)table, ids, positions, freq, H, V,
                                                               scale);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}

// logits <- cap * tanh(logits / cap), in place
__global__ void __launch_bounds__(256) softcap_kernel(float* __restrict__ x, float cap, size_t total) {
  size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  const size_t step = (size_t)gridDim.x * 256;
  for (; i < total; i += step) x[i] = cap * tanhf(x[i] / cap);
}

extern "C" int ptl_softcap(float* x, float cap, long total, hipStream_t st) {
  if (total <= 0) return PTL_OK;
  if (!x || !(cap > 0.f)) return PTL_ERR_ARG;
  long blocks = (total + 255) / 256;
  if (blocks > 16384) blocks = 16384;
  softcap_kernel<<<(int)blocks, 256, 0, st>>>(x, cap, (size_t)total);
  return ptl_launch_status();
}

// out[t] = e * rsqrt(mean(e^2) + eps) * w with e = table[ids[t]] * scale, as float32: a residual
// stream that starts from the normed embedding, in one pass over the row.
template <typename T>
__global__ void __launch_bounds__(256)
embedding_rmsnorm_kernel(float* __restrict__ out, const T* __restrict__ table, const int32_t* __restrict__ ids,
                         const float* __restrict__ w, float eps, int H, int V, float scale) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  int id = ids[t];
  if (id < 0 || id >= V) id = 0;          // checked on the host; never read out of bounds
  const T* src = table + (size_t)id * H;
  float* dst = out + (size_t)t * H;
  float ss = 0.f;
  for (int j = threadIdx.x; j < H; j += 256) {
    const float v = to_float<T>(src[j]) * scale;
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)H + eps);
  for (int j = threadIdx.x; j < H; j += 256) dst[j] = to_float<T>(src[j]) * scale * r * w[j];
}

extern "C" int ptl_embedding_rmsnorm(float* out, const void* table, const int32_t* ids, const float* w,
                                     float eps, int T_, int H, int V, float scale, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || V <= 0 || !w) return PTL_ERR_ARG;
  if (dtype == PTL_DTYPE_F32)
    embedding_rmsnorm_kernel<float><<<T_, 256, 0, st>>>(out, (const float*)table, ids, w, eps, H, V, scale);
  else if (dtype == PTL_DTYPE_BF16)
    embedding_rmsnorm_kernel<bf16_t><<<T_, 256, 0, st>>>(out, (const bf16_t*)table, ids, w, eps, H, V, scale);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}

template <typename T>
__global__ void __launch_bounds__(256)
gelu_gather_mul_kernel(T* __restrict__ out, const T* __restrict__ z, const T* __restrict__ table,
                       const int32_t* __restrict__ ids, int n, int ld, int col0, int V, size_t total) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const size_t t = i / n;
  const int j = (int)(i - t * n);
  int id = ids[t];
  if (id < 0 || id >= V) id = 0;
  const float e = to_float<T>(table[(size_t)id * ld + col0 + j]);
  out[i] = from_float<T>(gelu_tanh(to_float<T>(z[i])) * e);
}

// z, out [T, n] dense; table [V, ld]; the token's vector is table[id, col0 : col0 + n]
extern "C" int ptl_gelu_gather_mul(void* out, const void* z, const void* table, const int32_t* ids,
                                   int T_, int n, int ld, int col0, int V, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (n <= 0 || V <= 0 || col0 < 0 || col0 + n > ld) return PTL_ERR_ARG;
  const size_t total = (size_t)T_ * n;
  const size_t blocks = (total + 255) / 256;
  if (blocks > 0x7fffffff) return PTL_ERR_ARG;
  if (dtype == PTL_DTYPE_F32)
    gelu_gather_mul_kernel<float><<<(int)blocks, 256, 0, st>>>((float*)out, (const float*)z,
                                                               (const float*)table, ids, n, ld, col0, V, total);
  else if (dtype == PTL_DTYPE_BF16)
    gelu_gather_mul_kernel<bf16_t><<<(int)blocks, 256, 0, st>>>((bf16_t*)out, (const bf16_t*)z,
                                                                (const bf16_t*)table, ids, n, ld, col0, V, total);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}

// Hyper-connections: a token has S residual streams x_1 .. x_S, [T, S, H] float32. Around a sublayer
//
//   u = sum_s in[s] x_s;   y = sublayer(rmsnorm(u) w);   x_t <- sum_s mix[s, t] x_s + out[t] y
//
// (all streams at once from the old ones). One kernel makes the update behind a sublayer and the
// read-out in front of the next one: with y, the streams are updated in place; with nw, u is read
// from the (new) streams and normed into ``out``. Either half may be absent. Null coefficients
// stand for a single plain stream: in = ones, mix = the identity, out = ones (then S = 1 is the
// residual sum in front of a norm, and in = ones alone is the sum of the streams). One workgroup
// a token (of 1,024 threads when the rows are few, else 256); u waits in LDS between the pass that makes it and the one that scales it.
#define HYPER_MAX_S 16

template <int SM, int NT, typename TY, typename TO>
__global__ void __launch_bounds__(NT)
hyper_mix_kernel(float* __restrict__ streams, const TY* __restrict__ y, const float* __restrict__ mix,
                 const float* __restrict__ outc, const float* __restrict__ inc, const float* __restrict__ nw,
                 float eps, TO* __restrict__ out, int S, int H) {
  extern __shared__ float us[];            // [H]
  __shared__ float scratch[16];
  __shared__ float cm[HYPER_MAX_S * HYPER_MAX_S], co[HYPER_MAX_S], ci[HYPER_MAX_S];
  const int tid = threadIdx.x;
  if (tid < S * S) cm[tid] = mix ? mix[tid] : (tid / S == tid % S ? 1.f : 0.f);
  if (tid < S) {
    co[tid] = outc ? outc[tid] : 1.f;
    ci[tid] = inc ? inc[tid] : 1.f;
  }
  __syncthreads();
  float* row = streams + (size_t)blockIdx.x * S * H;
  float ss = 0.f;
  for (int c = tid; c < H; c += NT) {
    float x[SM];
#pragma unroll
    for (int s = 0; s < SM; ++s) x[s] = s < S ? row[(size_t)s * H + c] : 0.f;
    if (y) {
      const float v = to_float<TY>(y[(size_t)blockIdx.x * H + c]);
      float nx[SM];
#pragma unroll
      for (int t = 0; t < SM; ++t) {
        float a = t < S ? co[t] * v : 0.f;         // (entries from S on are not there: never read)
#pragma unroll
        for (int s = 0; s < SM; ++s) a = fmaf(s < S && t < S ? cm[s * S + t] : 0.f, x[s], a);
        nx[t] = t < S ? a : 0.f;
      }
#pragma unroll
      for (int t = 0; t < SM; ++t) {
        x[t] = nx[t];
        if (t < S) row[(size_t)t * H + c] = nx[t];
      }
    }
    if (nw) {
      float u = 0.f;
#pragma unroll
      for (int s = 0; s < SM; ++s) u = fmaf(s < S ? ci[s] : 0.f, x[s], u);
      us[c] = u;
      ss = fmaf(u, u, ss);
    }
  }
  if (!nw) return;
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)H + eps);
  for (int c = tid; c < H; c += NT) out[(size_t)blockIdx.x * H + c] = from_float<TO>(us[c] * r * nw[c]);
}

template <typename TY, typename TO>
static int launch_hyper(float* streams, const void* y, const float* mix, const float* outc, const float* inc,
                        const float* nw, float eps, void* out, int T_, int S, int H, hipStream_t st) {
  const size_t lds = nw ? (size_t)H * sizeof(float) : 0;
  // few rows: a row's entries over 1,024 threads, so that a thread's loads are one or two deep
  const bool few = T_ <= 512 && H > 256;
#define GO(SM)                                                                                       \
  {                                                                                                  \
    if (lds > 48 * 1024 &&                                                                           \
        (hipFuncSetAttribute((const void*)hyper_mix_kernel<SM, 256, TY, TO>,                         \
                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess ||  \
         hipFuncSetAttribute((const void*)hyper_mix_kernel<SM, 1024, TY, TO>,                        \
                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess))   \
      return PTL_ERR_LAUNCH;                                                                         \
    if (few)                                                                                         \
      hyper_mix_kernel<SM, 1024, TY, TO><<<T_, 1024, lds, st>>>(streams, (const TY*)y, mix, outc, inc, nw, \
                                                                eps, (TO*)out, S, H);                \
    else                                                                                             \
      hyper_mix_kernel<SM, 256, TY, TO><<<T_, 256, lds, st>>>(streams, (const TY*)y, mix, outc, inc, nw,   \
                                                              eps, (TO*)out, S, H);                  \
    return ptl_launch_status();                                                                      \
  }
  if (S <= 1) GO(1)
  if (S <= 2) GO(2)
  if (S <= 4) GO(4)
  if (S <= 8) GO(8)
  GO(16)
#undef GO
}

// streams [T, S, H] float32 (updated in place when y is given); y [T, H] of y_dtype or null; mix
// [S, S] (from, to), outc [S], inc [S] float32 or null; nw [H] float32 or null: no read-out; out
// [T, H] of out_dtype.
extern "C" int ptl_hyper_mix(float* streams, const void* y, int y_dtype, const float* mix, const float* outc,
                             const float* inc, const float* nw, float eps, void* out, int out_dtype, int T_,
                             int S, int H, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || S < 1 || S > HYPER_MAX_S || !streams || (nw && !out) || (!y && !nw) ||
      (size_t)H * sizeof(float) > 150 * 1024)
    return PTL_ERR_ARG;
#define GO(TY, TO) return launch_hyper<TY, TO>(streams, y, mix, outc, inc, nw, eps, out, T_, S, H, st)
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_F32) GO(float, float);
  if (y_dtype == PTL_DTYPE_F32 && out_dtype == PTL_DTYPE_BF16) GO(float, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_BF16) GO(bf16_t, bf16_t);
  if (y_dtype == PTL_DTYPE_BF16 && out_dtype == PTL_DTYPE_F32) GO(bf16_t, float);
#undef GO
  return PTL_ERR_ARG;
}
