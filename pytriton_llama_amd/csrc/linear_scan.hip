// Linear recurrences: per head a matrix S [D, Dv] (keys x values) that decays and takes outer products,
//
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,     o_t = S_t^T q_t
//
// in three forms:
//   MODE_SCALAR   one decay a head and token, a_t = exp(-exp(A_log) dt_t) with dt_t = softplus(raw +
//                 bias); the value is dt_t v_t and skip v_t is added to the result: the state-space
//                 duality of Mamba-2 (Dao, Gu: "Transformers are SSMs: Generalized Models and
//                 Efficient Algorithms Through Structured State Space Duality") with S = state^T
//   MODE_CHANNEL  a decay a key channel, a_t[d] in (0, 1]: gated linear attention (Yang, Wang, Shen,
//                 Panda, Kim: "Gated Linear Attention Transformers with Hardware-Efficient Training")
//   MODE_BONUS    the same decays, with a read-out in front of the update and a factor on the current
//                 token's own product: o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t, u [H, D]: the time
//                 mixer of RWKV-6 (Peng et al.: "Eagle and Finch: RWKV with Matrix-Valued States and
//                 Dynamic Recurrence")
// Everything is float32. Query head h uses q/k head h / heads_per_qk. S lives in the request's state
// slot as [H][Dv][DS] floats (a column of S after the other, DS = D rounded up to a multiple of 4).
//
// ptl_linear_decode_conv, ptl_linear_decode_lowrank, ptl_linear_decode_bonus: sequences of one token. A workgroup takes 16 to 64
//   columns of a head of a sequence, a column in 16 lanes (one row of a wave for the data-parallel lane moves); what is in front of the
//   recurrence is done by the workgroup itself: the short causal convolution with SiLU (scalar form)
//   or the low-rank decays (channel and bonus forms). Bound by reading and writing S once.
// ptl_linear_scan: portions. The rows of a sequence are walked in chunks of 32 tokens whose products
//   run on the matrix cores in float32 (v_mfma_f32_16x16x4_f32):
//     P[t, s] = sum_d q_t[d] k_s[d] a(s, t)[d]      s <= t, a(s, t) the decays of tokens s + 1 .. t
//     O[t, :] = sum_s P[t, s] v_s + sum_d q_t[d] a(start, t)[d] S[d, :]
//     S[d, :] = a(start, end)[d] S[d, :] + sum_s a(s, end)[d] k_s[d] v_s
//   (bonus form: the read-outs of token t take the decays up to t - 1 only, and P[t, t] takes u)
//   A workgroup of four waves takes 64 columns of a head; a wave keeps its 16 columns of S in the
//   accumulators of the last product, which is also how the middle product wants them as an operand.
//   Long sequences are cut into segments that are walked side by side: a local pass (what every
//   segment makes of a zero state), a combine (the segments' start states) and the final pass.
// ptl_lowrank_decay: the decays of all rows of a step, with z = W2[c, :] . f(r_t) + b[c]:
//   DECAY_SIGMOID   a[t, c] = sigmoid(z)^(1 / tau), f the identity
//   DECAY_EXP       a[t, c] = exp(-exp(z)), f = tanh
// ptl_time_shift: the inputs of a time mixer, out[j, t, :] = x_t + (x_(t-1) - x_t) mu[j, :] for several
//   mu at once; the row before a portion's first lies in the state slot (the scan and decode kernels
//   that follow leave the portion's last row there: ShiftArgs).
//
// Decays between tokens are never formed as quotients or differences of large numbers: in the scalar
// form the logarithms are summed in double, in the channel form products of decays are taken inside
// blocks of 16 tokens, so decays that vanish do no harm.
#include "common.h"
#include <math.h>

#define MODE_SCALAR 0
#define MODE_CHANNEL 1
#define MODE_BONUS 2
#define DECAY_SIGMOID 0
#define DECAY_EXP 1
#define QC 32                // tokens of a chunk
#define XLD 68               // row stride of the values in LDS
#define PLD 36               // row stride of P in LDS

typedef float f32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float row16_sum(float v) {
  // the sum over the 16 lanes of a row, in every lane: rotations by 8, 4, 2 and 1 inside the row
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, false));
  return v;
}
__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
// sigmoid(z)^p = 2^(-p log2(1 + e^-z)), with log2(1 + e^-z) = log2(1 + e^-|z|) + max(-z, 0) log2 e: the
// logarithm's argument lies in [1, 2], where the sum's rounding moves the logarithm by no more than
// the result's own last place (p up to about 1)
__device__ __forceinline__ float sigmoid_power(float z, float p) {
  const float zl = z * 1.4426950408889634f;
  const float l = __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(zl))) + fmaxf(-zl, 0.f);
  return __builtin_amdgcn_exp2f(-p * l);
}

// The hardware's exponential in base 2 and reciprocal: tanh to a few 1e-7 (it enters a sum of R such terms),
// e^z to a few 1e-7 of itself, which is what the decay's logarithm is known to.
__device__ __forceinline__ float decay_in(int form, float r) {
  return form == DECAY_EXP
             ? fmaf(-2.0f, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.885390081777927f * r)), 1.0f)
             : r;
}
__device__ __forceinline__ float decay_of(int form, float z, float inv_tau) {
  const float log2e = 1.4426950408889634f;
  return form == DECAY_EXP ? __builtin_amdgcn_exp2f(-log2e * __builtin_amdgcn_exp2f(log2e * z)) : sigmoid_power(z, inv_tau);
}

// The last row of x that a sequence brings, kept as float32 [W] at ``off`` of its state slot (x null:
// nothing is kept). Part ``part`` of ``parts`` of the row, 256 threads.
struct ShiftArgs {
  const void* x; long ldx; int dtype;
  long off;
  int W;
};
__device__ __forceinline__ void keep_row(const ShiftArgs& s, float* slot, size_t row, int part, int parts) {
  const int per = (s.W + parts - 1) / parts;
  for (int c = part * per + threadIdx.x; c < min(s.W, (part + 1) * per); c += 256)
    slot[s.off + c] = s.dtype == PTL_DTYPE_F32 ? ((const float*)s.x)[row * s.ldx + c]
                                               : bf16_to_float(((const bf16_t*)s.x)[row * s.ldx + c]);
}

struct LinArgs {
  float* out;                                     // [T, H, Dv]
  const float* q; long ldq;                       // q[t * ldq + g * D + d]
  const float* k; long ldk;
  const float* v; long ldv;                       // v[t * ldv + h * Dv + c]
  float qscale;
  const float* dt; long ldt;                      // scalar: raw step sizes [t * ldt + h]
  const float* A_log; const float* dt_bias; const float* skip;     // [H]
  const float* decay; long lda;                   // channel: [t * lda + h * D + d]
  float* state; long slot_stride;
  float* work;                                    // per (sequence, segment): [H][Dv][DS], then the decays
  const int32_t* q_start; const int32_t* state_slots;
  int H, heads_per_qk, D, DS, Dv;
  int P, seg_len;                                 // segments a sequence at most, tokens of one
  const float* bonus;                             // bonus: [H, D]
  ShiftArgs shift;
};

// floats of one segment's work area: S, and its decays (one a head, or one a key channel)
__host__ __device__ static inline size_t work_floats(const LinArgs& A, int mode) {
  return (size_t)A.H * A.Dv * A.DS + (mode == MODE_SCALAR ? (size_t)(A.H + 3) / 4 * 4 : (size_t)A.H * A.DS);
}

// ---- chunks of 32 tokens on the matrix cores -----------------------------------------------------
template <int NDT, int MODE, bool FINAL>
constexpr size_t chunk_lds_floats() {
  constexpr size_t rows = (size_t)QC * (16 * NDT + 4);
  return rows * (1 + (FINAL ? 1 : 0) + (MODE != MODE_SCALAR ? 1 : 0)) + (size_t)QC * XLD +
         (FINAL ? (size_t)QC * PLD : 0) + (MODE != MODE_SCALAR && FINAL ? (size_t)QC * 20 : 0) +
         (MODE != MODE_SCALAR ? 2 * 16 * NDT : 2 * 5 * QC) + (MODE == MODE_BONUS ? 16 * NDT : 0);
}

// workgroups a compute unit that the registers are shared out for (one where S takes many of them)
constexpr int chunk_workgroups(int ndt, bool final) { return ndt > 8 && final ? 1 : 2; }

template <int NDT, int MODE, bool FINAL>
__global__ void __launch_bounds__(256, chunk_workgroups(NDT, FINAL)) linear_chunk_kernel(LinArgs A, int vec) {
  constexpr bool CHANNEL = MODE != MODE_SCALAR;      // a decay a key channel
  constexpr bool BONUS = MODE == MODE_BONUS;
  constexpr int DP = 16 * NDT;              // key channels, padded
  constexpr int LD = DP + 4;                // row stride of q, k and the decays in LDS
  constexpr int NQ = DP / 4;                // float4 of a row
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* Ks = lds;                                              // [QC][LD]
  float* Qs = Ks + QC * LD;                                     // FINAL: [QC][LD]
  float* As = Qs + (FINAL ? QC * LD : 0);                       // channel: [QC][LD]
  float* Xs = As + (CHANNEL ? QC * LD : 0);        // [QC][XLD]
  float* Ps = Xs + QC * XLD;                                    // FINAL: [QC][PLD]
  float* Pd = Ps + (FINAL ? QC * PLD : 0);                      // channel, FINAL: [QC][20], second halves of the
                                                                // sums over d of the two diagonal tiles
  float* tot = Pd + (CHANNEL && FINAL ? QC * 20 : 0);   // channel: [2][DP]
  // scalar, twice (this chunk's and the next one's): [QC] each of the sums of the log decays from the
  // chunk's start, the step sizes, the decays from the chunk's start, the step sizes x decays to its end
  double* cums = reinterpret_cast<double*>(tot);
  float* bon = tot + 2 * DP;                                    // bonus: [DP]
  float* dtss = reinterpret_cast<float*>(cums + 2 * QC);
  float* ess = dtss + 2 * QC;
  float* wss = ess + 2 * QC;

  const int tid = threadIdx.x, lane = tid & 63, ln = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y;
  const int seq = blockIdx.z / A.P, seg = blockIdx.z % A.P;
  const int row0 = A.q_start[seq];
  const int qlen = A.q_start[seq + 1] - row0;
  const int nseg = (qlen + A.seg_len - 1) / A.seg_len;
  if (qlen <= 0 || seg >= nseg || (!FINAL && seg == nseg - 1)) return;
  const int t_begin = seg * A.seg_len, t_end = min(qlen, t_begin + A.seg_len);
  const int D = A.D, DS = A.DS, Dv = A.Dv, g = h / A.heads_per_qk;
  const int c0 = blockIdx.x * 64;
  const int c = c0 + 16 * wave + ln;                            // this lane's column
  const bool wave_live = c0 + 16 * wave < Dv, live = c < Dv;
  const size_t wsize = work_floats(A, MODE);
  auto work_at = [&](int p) { return A.work + ((size_t)seq * A.P + p) * wsize; };
  auto column = [&](float* base) { return base + ((size_t)h * Dv + c) * DS; };
  float* slot = A.state + (size_t)A.state_slots[seq] * A.slot_stride;

  f32x4_t S[NDT];                           // S[dt][i]: key channel 16 dt + 4 lg + i of column c
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt) {
    S[dt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int d = 16 * dt + 4 * lg;
    if (FINAL && live && d < DS) S[dt] = *reinterpret_cast<const f32x4_t*>(column(A.P > 1 ? work_at(seg) : slot) + d);
  }
  double log_total = 0.0;                   // scalar, local pass: the segment's decay
  float my_total = 1.f;                     // channel, local pass: of key channel tid
  float neg_A = 0.f, dt_bias = 0.f, skip = 0.f;
  if (MODE == MODE_SCALAR) {
    neg_A = -expf(A.A_log[h]);
    dt_bias = A.dt_bias[h];
    skip = A.skip[h];
  }

  // The rows of the next chunk are on their way from global memory into registers while the current
  // one is worked on from LDS: a thread holds NR float4 of k (and of q and the decays) and two of v.
  constexpr int NR = (QC * NQ + 255) / 256;
  f32x4_t fk[NR], fq[FINAL ? NR : 1], fa[CHANNEL ? NR : 1], fv[2];
  float fdt = 0.f;                          // scalar: a token's raw step size
  auto fetch4 = [&](const float* p, int col, int most) {
    f32x4_t x = {0.f, 0.f, 0.f, 0.f};
    if (vec) {
      x = *reinterpret_cast<const f32x4_t*>(p + col);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = col + j < most ? p[col + j] : 0.f;
    }
    return x;
  };
  auto fetch = [&](int t0) {
    const int steps = min(QC, t_end - t0);
#pragma unroll
    for (int n = 0; n < NR; ++n) {
      const int i = tid + 256 * n, r = i / NQ, d = (i - r * NQ) * 4;
      const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
      const size_t row = (size_t)(row0 + t0 + r);
      const bool in = r < steps && d < D;
      fk[n] = in ? fetch4(A.k + row * A.ldk + g * D, d, D) : zero;
      if (FINAL) fq[n] = in ? fetch4(A.q + row * A.ldq + g * D, d, D) : zero;
      if (CHANNEL) fa[n] = in ? fetch4(A.decay + row * A.lda + h * D, d, D) : zero;
    }
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int i = tid + 256 * n, r = i >> 4, x0 = (i & 15) * 4;
      fv[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (r < steps && c0 + x0 < Dv) fv[n] = fetch4(A.v + (size_t)(row0 + t0 + r) * A.ldv + (size_t)h * Dv, c0 + x0, Dv);
    }
  };
  auto put = [&]() {
#pragma unroll
    for (int n = 0; n < NR; ++n) {
      const int i = tid + 256 * n, r = i / NQ, d = (i - r * NQ) * 4;
      if (QC * NQ % 256 != 0 && i >= QC * NQ) break;
      *reinterpret_cast<f32x4_t*>(Ks + r * LD + d) = fk[n];
      if (FINAL) *reinterpret_cast<f32x4_t*>(Qs + r * LD + d) = fq[n] * A.qscale;
      // (rows past the end: zeros; their decay is taken as one where it matters, below)
      if (CHANNEL) *reinterpret_cast<f32x4_t*>(As + r * LD + d) = fa[n];
    }
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int i = tid + 256 * n;
      *reinterpret_cast<f32x4_t*>(Xs + (i >> 4) * XLD + (i & 15) * 4) = fv[n];
    }
  };

  // Scalar: the last wave, a lane a token, works the next chunk's scalars out while the others make P;
  // the raw step sizes are read a chunk earlier still.
  const bool scalar_wave = MODE == MODE_SCALAR && wave == 3;
  auto fetch_dt = [&](int t0) {
    if (scalar_wave && t0 + lane < t_end && lane < QC) fdt = A.dt[(size_t)(row0 + t0 + lane) * A.ldt + h];
  };
  auto scalars = [&](int t0, int buf) {
    const float step = t0 + lane < t_end && lane < QC ? softplus_f(fdt + dt_bias) : 0.f;
    double s = (double)(neg_A * step);
#pragma unroll
    for (int o = 1; o < QC; o <<= 1) {
      const double up = __shfl_up(s, o, 64);
      if (lane >= o) s += up;
    }
    const double all = __shfl(s, QC - 1, 64);
    if (lane < QC) {
      cums[buf * QC + lane] = s;
      dtss[buf * QC + lane] = step;
      ess[buf * QC + lane] = expf((float)s);
      wss[buf * QC + lane] = step * expf((float)(all - s));
    }
  };

  if (BONUS) {
    for (int d = tid; d < DP; d += 256) bon[d] = d < D ? A.bonus[(size_t)h * D + d] : 0.f;
  }
  fetch(t_begin);
  fetch_dt(t_begin);
  if (scalar_wave) scalars(t_begin, 0);
  fetch_dt(t_begin + QC);
  int buf = 0;
  for (int t0 = t_begin; t0 < t_end; t0 += QC, buf ^= 1) {
    const int steps = min(QC, t_end - t0);
    const double* cum = cums + buf * QC;
    const float *dts = dtss + buf * QC, *es = ess + buf * QC, *ws = wss + buf * QC;
    __syncthreads();                        // the chunk before is done with
    put();
    __syncthreads();
    if (t0 + QC < t_end) fetch(t0 + QC);
    if (scalar_wave) {
      if (t0 + QC < t_end) scalars(t0 + QC, buf ^ 1);
      fetch_dt(t0 + 2 * QC);
    }

    if (CHANNEL) {
      // The two diagonal tiles: lane (t, lg) walks s from t down, w = q_t times the decays of
      // s + 1 .. t (bonus: of s + 1 .. t - 1 from s = t - 1 on, and q_t times u at s = t); wave w takes tile
      // w % 2 and half of the key channels, a lane every fourth float4.
      if (FINAL) {
        const int base = 16 * (wave & 1), half = wave >> 1;
        float acc[16];
#pragma unroll
        for (int s = 0; s < 16; ++s) acc[s] = 0.f;
        for (int qd = half * (NQ / 2) + lg; qd < (half + 1) * (NQ / 2); qd += 4) {
          const f32x4_t qt = *reinterpret_cast<const f32x4_t*>(Qs + (base + ln) * LD + 4 * qd);
          f32x4_t w = {0.f, 0.f, 0.f, 0.f}, own = w;
          if (BONUS) own = qt * *reinterpret_cast<const f32x4_t*>(bon + 4 * qd);
#pragma unroll
          for (int s = 15; s >= 0; --s) {
            if (s < 15) w *= *reinterpret_cast<const f32x4_t*>(As + (base + s + 1) * LD + 4 * qd);
            if (s + (BONUS ? 1 : 0) == ln) w = qt;
            const f32x4_t x = BONUS && s == ln ? own : w;
            const f32x4_t ks = *reinterpret_cast<const f32x4_t*>(Ks + (base + s) * LD + 4 * qd);
            acc[s] += (x[0] * ks[0] + x[1] * ks[1]) + (x[2] * ks[2] + x[3] * ks[3]);
          }
        }
#pragma unroll
        for (int s = 0; s < 16; ++s) {
          acc[s] += __shfl_xor(acc[s], 16, 64);
          acc[s] += __shfl_xor(acc[s], 32, 64);
        }
        // lane (t, lg) keeps columns 4 lg .. 4 lg + 3 (zero right of the diagonal: w was zero there)
        f32x4_t mine;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          mine[i] = lg == 0 ? acc[i] : (lg == 1 ? acc[4 + i] : (lg == 2 ? acc[8 + i] : acc[12 + i]));
        if (half == 0) *reinterpret_cast<f32x4_t*>(Ps + (base + ln) * PLD + base + 4 * lg) = mine;
        else *reinterpret_cast<f32x4_t*>(Pd + (base + ln) * 20 + 4 * lg) = mine;
        __syncthreads();
      }
      // q_t times the decays from the start of its block of 16 (bonus: without its own), k_s times those
      // to the block's end
      for (int i = tid; i < 2 * DP; i += 256) {
        const int b = i / DP, d = i - b * DP;
        float* a = As + 16 * b * LD + d;
        if (FINAL) {
          float e = 1.f;
          float* q = Qs + 16 * b * LD + d;
#pragma unroll
          for (int t = 0; t < 16; ++t) {
            if (BONUS) q[t * LD] *= e;
            e *= 16 * b + t < steps ? a[t * LD] : 1.f;
            if (!BONUS) q[t * LD] *= e;
          }
        }
        float f = 1.f;
        float* k = Ks + 16 * b * LD + d;
#pragma unroll
        for (int t = 15; t >= 0; --t) {
          k[t * LD] *= f;
          f *= 16 * b + t < steps ? a[t * LD] : 1.f;
        }
        tot[i] = f;
      }
      __syncthreads();
    }

    if (FINAL) {
      // P: tiles (t, s) = (0, 0), (1, 0), (1, 1), one a wave (channel: the second one is left)
      if (MODE == MODE_SCALAR ? wave < 3 : wave == 3) {
        const int tt = MODE == MODE_SCALAR ? (wave > 0) : 1, ts = MODE == MODE_SCALAR ? (wave == 2) : 0;
        f32x4_t p = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
          const f32x4_t ka = *reinterpret_cast<const f32x4_t*>(Ks + (16 * ts + ln) * LD + 16 * dt + 4 * lg);
          const f32x4_t qb = *reinterpret_cast<const f32x4_t*>(Qs + (16 * tt + ln) * LD + 16 * dt + 4 * lg);
#pragma unroll
          for (int m = 0; m < 4; ++m) p = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[m], qb[m], p, 0, 0, 0);
        }
        if (MODE == MODE_SCALAR) {
          const int t = 16 * tt + ln;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int s = 16 * ts + 4 * lg + i;
            p[i] = s <= t ? p[i] * (dts[s] * expf((float)(cum[t] - cum[s]))) : 0.f;
          }
        }
        *reinterpret_cast<f32x4_t*>(Ps + (16 * tt + ln) * PLD + 16 * ts + 4 * lg) = p;
      }
      f32x4_t O[2];
      if (wave_live) {
        O[0] = O[1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
          const f32x4_t q0 = *reinterpret_cast<const f32x4_t*>(Qs + ln * LD + 16 * dt + 4 * lg);
          f32x4_t q1 = *reinterpret_cast<const f32x4_t*>(Qs + (16 + ln) * LD + 16 * dt + 4 * lg);
          if (CHANNEL) q1 *= *reinterpret_cast<const f32x4_t*>(tot + 16 * dt + 4 * lg);
#pragma unroll
          for (int m = 0; m < 4; ++m) {
            O[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(q0[m], S[dt][m], O[0], 0, 0, 0);
            O[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q1[m], S[dt][m], O[1], 0, 0, 0);
          }
        }
        if (MODE == MODE_SCALAR) {
          O[0] *= *reinterpret_cast<const f32x4_t*>(es + 4 * lg);
          O[1] *= *reinterpret_cast<const f32x4_t*>(es + 16 + 4 * lg);
        }
      }
      __syncthreads();                      // P is there
      if (wave_live) {
#pragma unroll
        for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
          for (int ts = 0; ts <= tt; ++ts) {
            f32x4_t pa = *reinterpret_cast<const f32x4_t*>(Ps + (16 * tt + ln) * PLD + 16 * ts + 4 * lg);
            if (CHANNEL && ts == tt) pa += *reinterpret_cast<const f32x4_t*>(Pd + (16 * tt + ln) * 20 + 4 * lg);
#pragma unroll
            for (int m = 0; m < 4; ++m)
              O[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(pa[m], Xs[(16 * ts + 4 * lg + m) * XLD + 16 * wave + ln], O[tt], 0, 0, 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int t = 16 * tt + 4 * lg + i;
            float o = O[tt][i];
            if (MODE == MODE_SCALAR) o = fmaf(skip, Xs[t * XLD + 16 * wave + ln], o);
            if (live && t < steps) A.out[((size_t)(row0 + t0 + t) * A.H + h) * Dv + c] = o;
          }
        }
      }
    }
    // S
    if (wave_live) {
      if (MODE == MODE_SCALAR) {
        const float e = es[QC - 1];
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) S[dt] *= e;
      } else {
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt)
          S[dt] *= *reinterpret_cast<const f32x4_t*>(tot + 16 * dt + 4 * lg) *
                   *reinterpret_cast<const f32x4_t*>(tot + DP + 16 * dt + 4 * lg);
      }
#pragma unroll
      for (int ts = 0; ts < 2; ++ts) {
        float x[4];
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          const int s = 16 * ts + 4 * lg + m;
          x[m] = Xs[s * XLD + 16 * wave + ln];
          if (MODE == MODE_SCALAR) x[m] *= ws[s];
        }
        float f[NDT];                       // channel: the second block's decays on top of the first's
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) f[dt] = CHANNEL && ts == 0 ? tot[DP + 16 * dt + ln] : 1.f;
#pragma unroll
        for (int m = 0; m < 4; ++m) {
#pragma unroll
          for (int dt = 0; dt < NDT; ++dt) {
            float ka = Ks[(16 * ts + 4 * lg + m) * LD + 16 * dt + ln];
            if (CHANNEL && ts == 0) ka *= f[dt];
            S[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka, x[m], S[dt], 0, 0, 0);
          }
        }
      }
    }
    if (!FINAL) {
      if (MODE == MODE_SCALAR) log_total += cum[QC - 1];
      else if (tid < DP) my_total *= tot[tid] * tot[DP + tid];
    }
  }

  float* to = !FINAL ? work_at(seg + 1) : (seg == nseg - 1 ? slot : nullptr);
  if (to) {
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
      const int d = 16 * dt + 4 * lg;
      if (live && d < DS) *reinterpret_cast<f32x4_t*>(column(to) + d) = S[dt];
    }
  }
  // (the rows' inputs were made from the old kept row by a kernel in front of this one)
  if (FINAL && seg == nseg - 1 && A.shift.x)
    keep_row(A.shift, slot, (size_t)(row0 + qlen - 1), blockIdx.y * gridDim.x + blockIdx.x, gridDim.x * gridDim.y);
  if (!FINAL && blockIdx.x == 0) {
    float* decays = work_at(seg + 1) + (size_t)A.H * Dv * DS;
    if (MODE == MODE_SCALAR) {
      if (tid == 0) decays[h] = expf((float)log_total);
    } else if (tid < DS) {
      decays[(size_t)h * DS + tid] = my_total;
    }
  }
}

// start(0) = the slot's state; start(p + 1) = decays(p) start(p) + what segment p added. A thread takes
// four key channels of one column through the sequence's segments.
template <int MODE>
__global__ void __launch_bounds__(256) linear_combine_kernel(LinArgs A) {
  const int seq = blockIdx.y;
  const int qlen = A.q_start[seq + 1] - A.q_start[seq];
  if (qlen <= 0) return;
  const int nseg = (qlen + A.seg_len - 1) / A.seg_len;
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  const int nq = A.DS / 4;
  if (i >= (size_t)A.H * A.Dv * nq) return;
  const int dq = (int)(i % nq), h = (int)(i / nq / A.Dv);
  const size_t wsize = work_floats(A, MODE), decays = (size_t)A.H * A.Dv * A.DS;
  float* w = A.work + (size_t)seq * A.P * wsize;
  f32x4_t cur = *reinterpret_cast<const f32x4_t*>(A.state + (size_t)A.state_slots[seq] * A.slot_stride + 4 * i);
  *reinterpret_cast<f32x4_t*>(w + 4 * i) = cur;
  constexpr int AHEAD = 8;                  // segments whose loads are under way together
  for (int p0 = 1; p0 < nseg; p0 += AHEAD) {
    f32x4_t u[AHEAD], f[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (p0 + j < nseg) {
        const float* at = w + (size_t)(p0 + j) * wsize;
        u[j] = *reinterpret_cast<const f32x4_t*>(at + 4 * i);
        if (MODE == MODE_SCALAR) {
          const float e = at[decays + h];
          f[j] = f32x4_t{e, e, e, e};
        } else {
          f[j] = *reinterpret_cast<const f32x4_t*>(at + decays + (size_t)h * A.DS + 4 * dq);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (p0 + j < nseg) {
        cur = f[j] * cur + u[j];
        *reinterpret_cast<f32x4_t*>(w + (size_t)(p0 + j) * wsize + 4 * i) = cur;
      }
    }
  }
}

template <int NDT, int MODE, bool FINAL>
static int launch_chunks(const LinArgs& A, int vec, int n_seqs, hipStream_t st) {
  constexpr size_t lds = chunk_lds_floats<NDT, MODE, FINAL>() * sizeof(float);
  static bool raised = false;               // (per instantiation)
  if (lds > 48 * 1024 && !raised) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(&linear_chunk_kernel<NDT, MODE, FINAL>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) {
      (void)hipGetLastError();
      return PTL_ERR_LAUNCH;
    }
    raised = true;
  }
  linear_chunk_kernel<NDT, MODE, FINAL><<<dim3((A.Dv + 63) / 64, A.H, n_seqs * A.P), 256, lds, st>>>(A, vec);
  return ptl_launch_status();
}

template <int MODE>
static int launch_scan(const LinArgs& A, int n_seqs, hipStream_t st) {
  constexpr int LOCAL = MODE == MODE_SCALAR ? MODE_SCALAR : MODE_CHANNEL;      // (what does not read out)
  if (A.D <= 0 || A.D > 256 || A.Dv <= 0 || A.H <= 0 || A.H > 65535 || A.heads_per_qk <= 0 ||
      A.H % A.heads_per_qk || A.P < 1 || (long)n_seqs * A.P > 65535 || A.seg_len < 1 || (A.P > 1 && !A.work) ||
      A.slot_stride < (long)A.H * A.Dv * A.DS || A.slot_stride % 4 || ((uintptr_t)A.state & 15) ||
      ((uintptr_t)A.work & 15))
    return PTL_ERR_ARG;
  auto aligned = [](const float* p, long ld) { return ld % 4 == 0 && ((uintptr_t)p & 15) == 0; };
  if (A.shift.x && (A.shift.W <= 0 || A.shift.off < (long)A.H * A.Dv * A.DS || A.shift.off + A.shift.W > A.slot_stride))
    return PTL_ERR_ARG;
  const int vec = A.D % 4 == 0 && A.Dv % 4 == 0 && aligned(A.q, A.ldq) && aligned(A.k, A.ldk) && aligned(A.v, A.ldv) &&
                  (MODE == MODE_SCALAR || aligned(A.decay, A.lda));
  const int tiles = (A.D + 15) / 16;
#define GO(N)                                                                                      \
  if (tiles <= N) {                                                                                \
    if (A.P > 1) {                                                                                 \
      if (int e = launch_chunks<N, LOCAL, false>(A, vec, n_seqs, st)) return e;                    \
      const size_t quads = (size_t)A.H * A.Dv * (A.DS / 4);                                        \
      linear_combine_kernel<LOCAL><<<dim3((unsigned)((quads + 255) / 256), n_seqs), 256, 0, st>>>(A); \
      if (int e = ptl_launch_status()) return e;                                                   \
    }                                                                                              \
    return launch_chunks<N, MODE, true>(A, vec, n_seqs, st);                                       \
  }
  GO(1) GO(2) GO(3) GO(4) GO(6) GO(8) GO(12) GO(16)
#undef GO
  return PTL_ERR_ARG;
}

// Floats of the workspace that ptl_linear_scan wants when P > 1.
extern "C" long ptl_linear_work_floats(int mode, int n_seqs, int P, int H, int D, int Dv) {
  LinArgs A{};
  A.H = H; A.Dv = Dv; A.DS = (D + 3) / 4 * 4;
  return (long)(work_floats(A, mode) * n_seqs * P);
}

// Portions of n_seqs sequences. mode 0 (scalar): dt, A_log, dt_bias, skip; mode 1
// (channel): decay; mode 2 (bonus): decay and bonus. P: the most segments of seg_len rows that one of the
// sequences has. shift_x (or null): [T, ldx] of shift_dtype, whose row of every sequence's last token is
// left in the sequence's slot (ShiftArgs).
extern "C" int ptl_linear_scan(int mode, float* out, const float* q, long ldq, const float* k, long ldk,
                               const float* v, long ldv, float qscale, const float* dt, long ldt,
                               const float* A_log, const float* dt_bias, const float* skip, const float* decay,
                               long lda, const float* bonus, const void* shift_x, long shift_ldx, int shift_dtype,
                               long shift_off, int shift_W, float* state, long slot_stride, float* work, int P,
                               int seg_len, const int32_t* q_start, const int32_t* state_slots, int n_seqs, int H,
                               int G, int D, int Dv, hipStream_t st) {
  if (n_seqs <= 0) return PTL_OK;
  if (G <= 0 || H % G) return PTL_ERR_ARG;
  LinArgs A{out, q, ldq, k, ldk, v, ldv, qscale, dt, ldt, A_log, dt_bias, skip, decay, lda, state, slot_stride, work,
            q_start, state_slots, H, H / G, D, (D + 3) / 4 * 4, Dv, P, seg_len, bonus,
            ShiftArgs{shift_x, shift_ldx, shift_dtype, shift_off, shift_W}};
  if (mode == MODE_SCALAR) {
    if (!dt || !A_log || !dt_bias || !skip) return PTL_ERR_ARG;
    return launch_scan<MODE_SCALAR>(A, n_seqs, st);
  }
  if (!decay) return PTL_ERR_ARG;
  if (mode == MODE_BONUS) return bonus ? launch_scan<MODE_BONUS>(A, n_seqs, st) : PTL_ERR_ARG;
  if (mode != MODE_CHANNEL) return PTL_ERR_ARG;
  return launch_scan<MODE_CHANNEL>(A, n_seqs, st);
}

// ---- the low-rank decays of all rows ---------------------------------------------------------------
// grid (blocks of 64 channels, blocks of 64 rows), a wave 16 of the channels: z^T = W2 f(r)^T as
// v_mfma_f32_16x16x4_f32. A lane holds its channel's entries 16 k + 4 lg .. + 3 of W2 as one float4 a
// chunk of 16 (in the same order as those of r, which is all a sum needs), f(r) lies in LDS.
template <int RC>
__global__ void __launch_bounds__(256)
lowrank_decay_kernel(float* __restrict__ out, const float* __restrict__ r, long ldr, const float* __restrict__ w,
                     const float* __restrict__ b, int form, float inv_tau, int T, int C, int R) {
  constexpr int RP = 16 * RC, LD = RP + 4;
  __shared__ __attribute__((aligned(16))) float rs[64 * LD];
  const int tid = threadIdx.x, lane = tid & 63, ln = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int t0 = blockIdx.y * 64, rows = min(64, T - t0), c0 = blockIdx.x * 64 + 16 * wave;
  f32x4_t wf[RC];
  const float* wr = w + (size_t)min(c0 + ln, C - 1) * R;
#pragma unroll
  for (int k = 0; k < RC; ++k)
#pragma unroll
    for (int m = 0; m < 4; ++m) wf[k][m] = 16 * k + 4 * lg + m < R ? wr[16 * k + 4 * lg + m] : 0.f;
  for (int i = tid; i < 64 * RP; i += 256) {
    const int t = i / RP, j = i - t * RP;
    rs[t * LD + j] = t < rows && j < R ? decay_in(form, r[(size_t)(t0 + t) * ldr + j]) : 0.f;
  }
  f32x4_t bias;
#pragma unroll
  for (int i = 0; i < 4; ++i) bias[i] = b[min(c0 + 4 * lg + i, C - 1)];
  __syncthreads();
  const bool four = C % 4 == 0 && ((uintptr_t)out & 15) == 0;
  for (int tt = 0; tt < rows; tt += 16) {
    f32x4_t z = bias;
#pragma unroll
    for (int k = 0; k < RC; ++k) {
      const f32x4_t x = *reinterpret_cast<const f32x4_t*>(rs + (tt + ln) * LD + 16 * k + 4 * lg);
#pragma unroll
      for (int m = 0; m < 4; ++m) z = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[k][m], x[m], z, 0, 0, 0);
    }
    // lane (ln, lg): channels c0 + 4 lg .. + 3 of row tt + ln
    if (tt + ln >= rows) continue;
    float* o = out + (size_t)(t0 + tt + ln) * C + c0 + 4 * lg;
#pragma unroll
    for (int i = 0; i < 4; ++i) z[i] = decay_of(form, z[i], inv_tau);
    if (four) {
      if (c0 + 4 * lg < C) *reinterpret_cast<f32x4_t*>(o) = z;
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (c0 + 4 * lg + i < C) o[i] = z[i];
    }
  }
}

// ranks above 128: a thread a channel, its row of W2 read again for every row
#define DECAY_ROWS 8
__global__ void __launch_bounds__(256)
lowrank_decay_wide_kernel(float* __restrict__ out, const float* __restrict__ r, long ldr, const float* __restrict__ w,
                          const float* __restrict__ b, int form, float inv_tau, int T, int C, int R) {
  extern __shared__ __attribute__((aligned(16))) float rw[];       // [DECAY_ROWS][R]
  const int t0 = blockIdx.y * DECAY_ROWS, rows = min(DECAY_ROWS, T - t0);
  const int c = blockIdx.x * 256 + threadIdx.x;
  for (int i = threadIdx.x; i < rows * R; i += 256) rw[i] = decay_in(form, r[(size_t)(t0 + i / R) * ldr + i % R]);
  __syncthreads();
  if (c >= C) return;
  const float* wr = w + (size_t)c * R;
  float z[DECAY_ROWS];
#pragma unroll
  for (int t = 0; t < DECAY_ROWS; ++t) z[t] = b[c];
  for (int j = 0; j < R; ++j) {
    const float x = wr[j];
#pragma unroll
    for (int t = 0; t < DECAY_ROWS; ++t) z[t] = fmaf(x, t < rows ? rw[t * R + j] : 0.f, z[t]);
  }
#pragma unroll
  for (int t = 0; t < DECAY_ROWS; ++t)
    if (t < rows) out[(size_t)(t0 + t) * C + c] = decay_of(form, z[t], inv_tau);
}

extern "C" int ptl_lowrank_decay(float* out, const float* r, long ldr, const float* w, const float* b,
                                 int form, float inv_tau, int T_, int C, int R, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  const size_t lds = (size_t)DECAY_ROWS * R * sizeof(float);
  if (C <= 0 || R <= 0 || lds > 48 * 1024 || (form != DECAY_SIGMOID && form != DECAY_EXP) ||
      (T_ + DECAY_ROWS - 1) / DECAY_ROWS > 65535)
    return PTL_ERR_ARG;
  const dim3 grid((C + 63) / 64, (T_ + 63) / 64);
#define GO(RC) lowrank_decay_kernel<RC><<<grid, 256, 0, st>>>(out, r, ldr, w, b, form, inv_tau, T_, C, R)
  if (R <= 16) GO(1);
  else if (R <= 32) GO(2);
  else if (R <= 64) GO(4);
  else if (R <= 128) GO(8);
  else
    lowrank_decay_wide_kernel<<<dim3((C + 255) / 256, (T_ + DECAY_ROWS - 1) / DECAY_ROWS), 256, lds, st>>>(
        out, r, ldr, w, b, form, inv_tau, T_, C, R);
#undef GO
  return ptl_launch_status();
}

// ---- one token -------------------------------------------------------------------------------------
// What follows the recurrence head by head: y = o / sqrt(mean(o^2) + eps) * w * silu(gate), [T, H * Dv] in
// the engine's type (y null: the kernel leaves o). One workgroup has the whole head then.
struct HeadArgs {
  void* y; int dtype;
  const float* w;                           // [H, Dv]
  int gate_off;                             // column of p
  float eps;
};

struct DecodeArgs {
  float* out;                               // [T, H, Dv]
  const float* p; long ldp;                 // the float32 projection
  int q_off, k_off, v_off;                  // columns of q [G, D], k [G, D] and v [H, Dv] (before the convolution)
  float qscale;
  // scalar form
  int dt_off;
  const float* A_log; const float* dt_bias; const float* skip;     // [H]
  const float* cw; const float* cb; int taps; long tail_off;       // convolution [C, taps], [C]; channel of a
  int conv_off, C;                                                 // column: column - conv_off; tail [taps - 1, C]
  // channel form
  int a_off;
  const float* w2; const float* b2; int R; float inv_tau;          // [H * D, R], [H * D]
  int form;                                 // DECAY_SIGMOID, DECAY_EXP
  float* state; long slot_stride;
  const int32_t* q_start; const int32_t* state_slots;
  int H, heads_per_qk, D, DS, Dv;
  const float* bonus;                       // bonus form: [H, D]
  ShiftArgs shift;
  HeadArgs head;
};

// NB: blocks of 16 columns a workgroup takes (what is in front of the recurrence is then done less often)
template <int J, int NB, int MODE>
__global__ void __launch_bounds__(256) linear_decode_kernel(DecodeArgs A) {
  constexpr bool CHANNEL = MODE != MODE_SCALAR, BONUS = MODE == MODE_BONUS;
  __shared__ __attribute__((aligned(16))) float ks[64 * J], qs[64 * J], as[CHANNEL ? 64 * J : 4], xs[16 * NB];
  __shared__ __attribute__((aligned(16))) float us[BONUS ? 64 * J : 4];
  extern __shared__ float rs[];             // channel: [R], the decays' low-rank input
  const int tid = threadIdx.x, cg = tid >> 4, l = tid & 15;
  const int h = blockIdx.y, seq = blockIdx.z, g = h / A.heads_per_qk;
  const int row = A.q_start[seq];
  if (A.q_start[seq + 1] <= row) return;
  const int D = A.D, DS = A.DS, Dv = A.Dv;
  const int c0 = blockIdx.x * 16 * NB;
  float* slot = A.state + (size_t)A.state_slots[seq] * A.slot_stride;
  auto column = [&](int b) { return slot + ((size_t)h * Dv + c0 + 16 * b + cg) * DS; };
  f32x4_t S[NB][J];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const int d = 4 * (l + 16 * j);
      S[b][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (c0 + 16 * b + cg < Dv && d < DS)
        S[b][j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(column(b) + d));
    }
  const float* p = A.p + (size_t)row * A.ldp;
  // what the columns of the projection hold for this workgroup: k and q of the head (group), its values
  auto value = [&](int col) {
    float x = p[col];
    if (MODE == MODE_SCALAR) {
      const int ch = col - A.conv_off;
      float s = A.cb ? A.cb[ch] : 0.f;
      const float* w = A.cw + (size_t)ch * A.taps;
      const float* tail = slot + A.tail_off + ch;
      for (int j = 0; j < A.taps - 1; ++j) s = fmaf(w[j], tail[(size_t)j * A.C], s);
      x = silu_f(fmaf(w[A.taps - 1], x, s));
    }
    return x;
  };
  const int DP = 64 * J;
  for (int i = tid; i < 2 * DP + 16 * NB; i += 256) {
    if (i < DP) {
      ks[i] = i < D ? value(A.k_off + g * D + i) : 0.f;
    } else if (i < 2 * DP) {
      const int d = i - DP;
      qs[d] = d < D ? value(A.q_off + g * D + d) * A.qscale : 0.f;
      if (BONUS) us[d] = d < D ? A.bonus[h * D + d] : 0.f;
    } else {
      const int cc = c0 + i - 2 * DP;
      xs[i - 2 * DP] = cc < Dv ? value(A.v_off + h * Dv + cc) : 0.f;
    }
  }
  float decay = 1.f, step = 1.f;
  if (MODE == MODE_SCALAR) {
    step = softplus_f(p[A.dt_off + h] + A.dt_bias[h]);
    decay = expf(-expf(A.A_log[h]) * step);
  } else {
    for (int j = tid; j < A.R; j += 256) rs[j] = decay_in(A.form, p[A.a_off + j]);
    __syncthreads();
    // 256 / (64 J) lanes a key channel share its row of W2
    constexpr int LPC = J == 1 ? 4 : (J == 2 ? 2 : 1);
    for (int i = tid; i < DP * LPC; i += 256) {
      const int d = i / LPC, ch = h * D + min(d, D - 1);
      const float* w = A.w2 + (size_t)ch * A.R;
      float z = 0.f;
      for (int j = i % LPC; j < A.R; j += LPC) z = fmaf(w[j], rs[j], z);
#pragma unroll
      for (int o = 1; o < LPC; o <<= 1) z += __shfl_xor(z, o, 64);
      if (i % LPC == 0) as[d] = d < D ? decay_of(A.form, z + A.b2[ch], A.inv_tau) : 1.f;
    }
  }
  __syncthreads();
  const float skip = MODE == MODE_SCALAR ? A.skip[h] : 0.f;
  __shared__ float os[BONUS ? 16 * NB : 1];
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const bool live = c0 + 16 * b + cg < Dv;
    const float x = xs[16 * b + cg], v = x * step;
    float o = 0.f;
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const int d = 4 * (l + 16 * j);
      const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(ks + d), q4 = *reinterpret_cast<const f32x4_t*>(qs + d);
      f32x4_t s = S[b][j], read;
      if (BONUS) read = s + *reinterpret_cast<const f32x4_t*>(us + d) * k4 * v;
      if (CHANNEL) s *= *reinterpret_cast<const f32x4_t*>(as + d);
      else s *= decay;
      s += k4 * v;
      if (!BONUS) read = s;
      o += (read[0] * q4[0] + read[1] * q4[1]) + (read[2] * q4[2] + read[3] * q4[3]);
      if (live && d < DS) __builtin_nontemporal_store(s, reinterpret_cast<f32x4_t*>(column(b) + d));
    }
    o = row16_sum(o);
    if (BONUS && A.head.y) {
      if (l == 0) os[16 * b + cg] = live ? o : 0.f;
    } else if (live && l == 0) {
      A.out[((size_t)row * A.H + h) * Dv + c0 + 16 * b + cg] = fmaf(skip, x, o);
    }
  }
  if (BONUS && A.head.y) {
    __syncthreads();
    if (tid < 64) {                         // (Dv <= 16 NB <= 64: a lane a value)
      const float o = tid < 16 * NB ? os[tid] : 0.f;
      const float r = 1.0f / sqrtf(wave_sum(o * o) / (float)Dv + A.head.eps);
      if (tid < Dv) {
        const float y = o * r * A.head.w[h * Dv + tid] * silu_f(p[A.head.gate_off + h * Dv + tid]);
        const size_t at = ((size_t)row * A.H + h) * Dv + tid;
        if (A.head.dtype == PTL_DTYPE_F32) ((float*)A.head.y)[at] = y;
        else ((bf16_t*)A.head.y)[at] = float_to_bf16(y);
      }
    }
  }
  if (A.shift.x) keep_row(A.shift, slot, (size_t)row, blockIdx.y * gridDim.x + blockIdx.x, gridDim.x * gridDim.y);
}

template <int MODE>
static int launch_decode(const DecodeArgs& A, int n_seqs, hipStream_t st) {
  if (A.D <= 0 || A.D > 256 || A.Dv <= 0 || A.H <= 0 || A.H > 65535 || n_seqs > 65535 || A.heads_per_qk <= 0 ||
      A.slot_stride < (long)A.H * A.Dv * A.DS || A.slot_stride % 4 || ((uintptr_t)A.state & 15) || A.R > 8192 ||
      (A.shift.x && (A.shift.W <= 0 || A.shift.off < (long)A.H * A.Dv * A.DS || A.shift.off + A.shift.W > A.slot_stride)))
    return PTL_ERR_ARG;
  const size_t lds = MODE == MODE_SCALAR ? 0 : (size_t)A.R * sizeof(float);
  // as many columns a workgroup as leave about two workgroups a compute unit (of 256)
  const int blocks = (A.Dv + 15) / 16;
  const long all = (long)blocks * A.H * n_seqs;
  int nb = blocks >= 4 && all >= 4 * 512 ? 4 : (blocks >= 2 && all >= 2 * 512 ? 2 : 1);
  if (A.head.y) {                           // the heads are finished here: whole heads
    if (blocks > 4) return PTL_ERR_ARG;
    nb = blocks > 2 ? 4 : blocks;
  }
  const dim3 grid((blocks + nb - 1) / nb, A.H, n_seqs);
#define GO(J)                                                                       \
  {                                                                                 \
    if (nb == 4) linear_decode_kernel<J, 4, MODE><<<grid, 256, lds, st>>>(A);       \
    else if (nb == 2) linear_decode_kernel<J, 2, MODE><<<grid, 256, lds, st>>>(A);  \
    else linear_decode_kernel<J, 1, MODE><<<grid, 256, lds, st>>>(A);                \
    return ptl_launch_status();                                                     \
  }
  switch ((A.DS + 63) / 64) {
    case 1: GO(1)
    case 2: GO(2)
    case 3: GO(3)
    default: GO(4)
  }
#undef GO
}

// Sequences 0 .. n_seqs - 1, one token each, scalar form behind a short convolution. p float32 [T,
// ldp] with the raw x (H heads of Dv), B and C (G groups of D) and step sizes at their columns;
// conv_off: the column of the convolution's channel 0. The tails are read, not advanced.
extern "C" int ptl_linear_decode_conv(float* out, const float* p, long ldp, int x_off, int b_off, int c_off,
                                      int dt_off, const float* A_log, const float* dt_bias, const float* skip,
                                      const float* cw, const float* cb, int taps, int conv_off, int C,
                                      long tail_off, float* state, long slot_stride, const int32_t* q_start,
                                      const int32_t* state_slots, int n_seqs, int H, int G, int D, int Dv,
                                      hipStream_t st) {
  if (n_seqs <= 0) return PTL_OK;
  if (G <= 0 || H % G || taps < 1 || !cw || tail_off < (long)H * Dv * ((D + 3) / 4 * 4)) return PTL_ERR_ARG;
  DecodeArgs A{};
  A.out = out; A.p = p; A.ldp = ldp; A.q_off = c_off; A.k_off = b_off; A.v_off = x_off; A.qscale = 1.f;
  A.dt_off = dt_off; A.A_log = A_log; A.dt_bias = dt_bias; A.skip = skip;
  A.cw = cw; A.cb = cb; A.taps = taps; A.tail_off = tail_off; A.conv_off = conv_off; A.C = C;
  A.state = state; A.slot_stride = slot_stride; A.q_start = q_start; A.state_slots = state_slots;
  A.H = H; A.heads_per_qk = H / G; A.D = D; A.DS = (D + 3) / 4 * 4; A.Dv = Dv;
  return launch_decode<MODE_SCALAR>(A, n_seqs, st);
}

static DecodeArgs lowrank_args(float* out, const float* p, long ldp, int q_off, int k_off, int v_off, int a_off,
                               float qscale, const float* w2, const float* b2, int R, int form, float inv_tau,
                               float* state, long slot_stride, const int32_t* q_start, const int32_t* state_slots,
                               int H, int D, int Dv) {
  DecodeArgs A{};
  A.out = out; A.p = p; A.ldp = ldp; A.q_off = q_off; A.k_off = k_off; A.v_off = v_off; A.qscale = qscale;
  A.a_off = a_off; A.w2 = w2; A.b2 = b2; A.R = R; A.form = form; A.inv_tau = inv_tau;
  A.state = state; A.slot_stride = slot_stride; A.q_start = q_start; A.state_slots = state_slots;
  A.H = H; A.heads_per_qk = 1; A.D = D; A.DS = (D + 3) / 4 * 4; A.Dv = Dv;
  return A;
}

// The channel form: q, k (H heads of D), v (H of Dv) and the decays' low-rank input r [R] at columns of p;
// w2 [H * D, R], b2 [H * D].
extern "C" int ptl_linear_decode_lowrank(float* out, const float* p, long ldp, int q_off, int k_off, int v_off,
                                         int a_off, float qscale, const float* w2, const float* b2, int R,
                                         float inv_tau, float* state, long slot_stride, const int32_t* q_start,
                                         const int32_t* state_slots, int n_seqs, int H, int D, int Dv,
                                         hipStream_t st) {
  if (n_seqs <= 0) return PTL_OK;
  if (R <= 0 || !w2 || !b2) return PTL_ERR_ARG;
  return launch_decode<MODE_CHANNEL>(lowrank_args(out, p, ldp, q_off, k_off, v_off, a_off, qscale, w2, b2, R,
                                                  DECAY_SIGMOID, inv_tau, state, slot_stride, q_start, state_slots,
                                                  H, D, Dv), n_seqs, st);
}

// The bonus form: as above with decays exp(-exp(w2 . tanh(r) + b2)), bonus [H, D]; the sequences' rows of
// shift_x [T, ldx] are left in their slots (ShiftArgs). y (or null; Dv up to 64): the heads are normed, weighted
// and gated (HeadArgs) into y, and out is not written.
extern "C" int ptl_linear_decode_bonus(float* out, void* y, int y_dtype, const float* head_w, int gate_off, float eps,
                                       const float* p, long ldp, int q_off, int k_off, int v_off,
                                       int a_off, const float* w2, const float* b2, int R, const float* bonus,
                                       const void* shift_x, long shift_ldx, int shift_dtype, long shift_off,
                                       int shift_W, float* state, long slot_stride, const int32_t* q_start,
                                       const int32_t* state_slots, int n_seqs, int H, int D, int Dv, hipStream_t st) {
  if (n_seqs <= 0) return PTL_OK;
  if (R <= 0 || !w2 || !b2 || !bonus || (y && (!head_w || gate_off < 0)) || (!y && !out)) return PTL_ERR_ARG;
  DecodeArgs A = lowrank_args(out, p, ldp, q_off, k_off, v_off, a_off, 1.f, w2, b2, R, DECAY_EXP, 0.f, state,
                              slot_stride, q_start, state_slots, H, D, Dv);
  A.bonus = bonus;
  A.shift = ShiftArgs{shift_x, shift_ldx, shift_dtype, shift_off, shift_W};
  A.head = HeadArgs{y, y_dtype, head_w, gate_off, eps};
  return launch_decode<MODE_BONUS>(A, n_seqs, st);
}

// ---- the inputs of a time mixer ----------------------------------------------------------------------
// One workgroup a (row, block of 256 x VEC columns); a thread makes all n_mix results of its columns.
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
time_shift_kernel(T* __restrict__ out, long mix_stride, const T* __restrict__ x, long ldx, const float* __restrict__ mu,
                  int n_mix, const float* __restrict__ state, long slot_stride, long off,
                  const int32_t* __restrict__ q_start, const int32_t* __restrict__ state_slots, int n_seqs, int W) {
  const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (c >= W) return;
  // the sequence of the row (the last one whose first row is not beyond t); a row behind all of them: none
  int lo = 0, hi = n_seqs;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (q_start[mid] <= t) lo = mid; else hi = mid - 1;
  }
  float a[VEC], d[VEC];
  auto read = [&](const T* p, float (&v)[VEC]) {
    if (VEC == 1) {
      v[0] = to_float<T>(p[0]);
    } else if (sizeof(T) == 2) {
      union { uint4 u; bf16_t e[8]; } r;
      r.u = *reinterpret_cast<const uint4*>(p);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = bf16_to_float(r.e[j]);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; j += 4) {
        const float4 r = *reinterpret_cast<const float4*>(p + j);
        v[j] = r.x; v[j + (VEC > 1)] = r.y; v[j + 2 * (VEC > 1)] = r.z; v[j + 3 * (VEC > 1)] = r.w;
      }
    }
  };
  read(x + (size_t)t * ldx + c, a);
  if (lo < n_seqs && q_start[lo] < t) {
    read(x + (size_t)(t - 1) * ldx + c, d);
  } else {
    const float* kept = lo < n_seqs ? state + (size_t)state_slots[lo] * slot_stride + off + c : nullptr;
#pragma unroll
    for (int j = 0; j < VEC; ++j) d[j] = kept ? kept[j] : 0.f;
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) d[j] -= a[j];
  for (int m = 0; m < n_mix; ++m) {
    const float* f = mu + (size_t)m * W + c;
    T* o = out + (size_t)m * mix_stride + (size_t)t * W + c;
    if (VEC == 1) {
      o[0] = from_float<T>(fmaf(d[0], f[0], a[0]));
    } else {
      float ff[VEC];
#pragma unroll
      for (int j = 0; j < VEC; j += 4) {
        const float4 r = *reinterpret_cast<const float4*>(f + j);
        ff[j] = r.x; ff[j + (VEC > 1)] = r.y; ff[j + 2 * (VEC > 1)] = r.z; ff[j + 3 * (VEC > 1)] = r.w;
      }
      if (sizeof(T) == 2) {
        union { uint4 u; bf16_t e[8]; } r;
#pragma unroll
        for (int j = 0; j < VEC; ++j) r.e[j] = float_to_bf16(fmaf(d[j], ff[j], a[j]));
        *reinterpret_cast<uint4*>(o) = r.u;
      } else {
#pragma unroll
        for (int j = 0; j < VEC; j += 4)
          *reinterpret_cast<float4*>(o + j) =
              make_float4(fmaf(d[j], ff[j], a[j]), fmaf(d[j + (VEC > 1)], ff[j + (VEC > 1)], a[j + (VEC > 1)]),
                          fmaf(d[j + 2 * (VEC > 1)], ff[j + 2 * (VEC > 1)], a[j + 2 * (VEC > 1)]),
                          fmaf(d[j + 3 * (VEC > 1)], ff[j + 3 * (VEC > 1)], a[j + 3 * (VEC > 1)]));
      }
    }
  }
}

// out [n_mix, T, W] (mix_stride elements from one mix to the next, rows dense), x [T, ldx] of dtype, mu
// float32 [n_mix, W]; the kept rows float32 [W] at off of the slots.
extern "C" int ptl_time_shift(void* out, long mix_stride, const void* x, long ldx, const float* mu, int n_mix,
                              const float* state, long slot_stride, long off, const int32_t* q_start,
                              const int32_t* state_slots, int n_seqs, int T_, int W, int dtype, hipStream_t st) {
  if (T_ <= 0 || n_mix <= 0) return PTL_OK;
  if (W <= 0 || ldx < W || mix_stride < (long)T_ * W || off < 0 || off + W > slot_stride) return PTL_ERR_ARG;
  const bool even = W % 8 == 0 && ldx % 8 == 0 && mix_stride % 8 == 0 &&
                    (((uintptr_t)out | (uintptr_t)x | (uintptr_t)mu) & 15) == 0;
  auto grid = [&](int vec) { return dim3(T_, (W + 256 * vec - 1) / (256 * vec)); };
#define GO(T, VEC)                                                                                               \
  time_shift_kernel<T, VEC><<<grid(VEC), 256, 0, st>>>((T*)out, mix_stride, (const T*)x, ldx, mu, n_mix, state,    \
                                                       slot_stride, off, q_start, state_slots, n_seqs, W)
  if (dtype == PTL_DTYPE_F32) {
    if (even) GO(float, 4); else GO(float, 1);
  } else if (dtype == PTL_DTYPE_BF16) {
    if (even) GO(bf16_t, 8); else GO(bf16_t, 1);
  } else {
    return PTL_ERR_ARG;
  }
#undef GO
  return ptl_launch_status();
}
