// What lies between a mixer's first projection and its attention, and between its attention (or
// recurrence) and its output projection, for mixers whose queries and keys are normed:
//
// ptl_qkv_prepare: one workgroup a token, or several that share its heads when the tokens are few.
//   Reads the float32 row of the projection (q | k | v at
//   given columns), adds the biases, norms queries and keys (RMS norm over every head on its own
//   with one weight for all heads, or over the whole of q and the whole of k with a weight of that
//   size, or not at all), turns the first rot_dims entries of every head by the token's position
//   (entry i with entry i + rot_dims / 2; sine and cosine times ``mag``), writes the queries
//   [T, Hq, Dk] in the engine's type and the keys and values into the token's cache slot
//   (k_cache [pages, Hk, page_size, Dk], v_cache [pages, Hv, page_size, Dv]). A layer that reads
//   another's keys and values has none of its own: k_off < 0.
//
// ptl_conv_qkv_prepare: the same place of a mixer whose queries, keys and values pass a short causal
//   convolution over time first and whose queries and keys are normed after the rotation. A wave
//   takes one head of a run of neighbouring rows (where it stands, below).
//
// ptl_head_norm_gate: one wave a (token, head). From float32 results a [T, HA, Dv]:
//   o = a[h * maps] - lam * a[h * maps + 1] (maps 2) or a[h] (maps 1); o / sqrt(mean(o^2) + eps)
//   over the head's Dv values, times a weight (one for all heads, or one a head, or none), times a
//   constant, times act(gate) with the gate read from a float32 matrix at given columns
//   (sigmoid, SiLU, or none). The result [T, H * Dv] is in the engine's type.
//
// ptl_gate_group_norm: one workgroup a (token, group of columns), or one wave where a group's columns
//   fit its registers. y float32 [T, n] times silu(gate),
//   then every one of the equal groups of neighbouring columns divided by its own root mean square,
//   times a weight [n]; the result is in the engine's type. For the leading rows of a step that are
//   sequences of one token it also advances the inputs that a short convolution keeps in the state
//   slot (the recurrence in front of it has read the old ones).
//
// All arithmetic is float32: the angle is float(position) * frequency (behind a convolution with the
// product's rounding put back), sinf / cosf / expf are the accurate ones.
#include "common.h"
#include <math.h>

#define NORM_NONE 0
#define NORM_HEAD 1
#define NORM_WHOLE 2

// A token's work is cut into ``gridDim.y`` slices of whole heads (queries, then keys, then values),
// so that the few tokens of a decode step still fill the chip. Every slice reads the whole row of
// q and k when the norm is over the whole of them, else only its heads.
template <typename TO>
__global__ void __launch_bounds__(256)
qkv_prepare_kernel(TO* __restrict__ q_out, const float* __restrict__ p, long ldp, int q_off, int k_off,
                   int v_off, const float* __restrict__ qb, const float* __restrict__ kb,
                   const float* __restrict__ vb, int norm_mode, const float* __restrict__ qw,
                   const float* __restrict__ kw, float eps, int rot_dims,
                   const float* __restrict__ inv_freq, float mag, const int32_t* __restrict__ positions,
                   const int32_t* __restrict__ slots, TO* __restrict__ k_cache, TO* __restrict__ v_cache,
                   int Hq, int Hk, int Hv, int Dk, int Dv, int page_size, int heads_per_slice) {
  extern __shared__ float lds[];
  const bool own = k_off >= 0;
  const int nq = Hq * Dk, nk = own ? Hk * Dk : 0;
  const int heads_qk = Hq + (own ? Hk : 0);
  float* raw = lds;                       // [nq + nk]: q then k, bias added (this slice's heads, or all)
  float* rs = raw + nq + nk;              // [Hq + Hk] (per head) or [2] (whole): 1 / rms
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  // this slice: heads h_lo .. h_hi of q | k | v counted in one row
  const int h_lo = blockIdx.y * heads_per_slice;
  const int h_hi = min(h_lo + heads_per_slice, heads_qk + (own ? Hv : 0));
  const int qk_lo = min(h_lo, heads_qk), qk_hi = min(h_hi, heads_qk);      // its q and k heads
  const float* row = p + (size_t)t * ldp;
  if (qk_lo < qk_hi) {
    const int e_lo = norm_mode == NORM_WHOLE ? 0 : qk_lo * Dk;
    const int e_hi = norm_mode == NORM_WHOLE ? nq + nk : qk_hi * Dk;
    for (int e = e_lo + tid; e < e_hi; e += 256)
      raw[e] = e < nq ? row[q_off + e] + (qb ? qb[e] : 0.f) : row[k_off + e - nq] + (kb ? kb[e - nq] : 0.f);
    __syncthreads();
    if (norm_mode == NORM_HEAD) {
      const int wave = tid >> 6, lane = tid & 63;
      for (int h = qk_lo + wave; h < qk_hi; h += 4) {
        const float* x = raw + (size_t)h * Dk;          // (k heads follow the q heads, same size)
        float ss = 0.f;
        for (int d = lane; d < Dk; d += 64) ss = fmaf(x[d], x[d], ss);
        ss = wave_sum(ss);
        if (lane == 0) rs[h] = 1.0f / sqrtf(ss / (float)Dk + eps);
      }
      __syncthreads();
    } else if (norm_mode == NORM_WHOLE) {
      float ss = 0.f;
      for (int e = tid; e < nq; e += 256) ss = fmaf(raw[e], raw[e], ss);
      ss = block_sum(ss, scratch);
      float sk = 0.f;
      for (int e = tid; e < nk; e += 256) sk = fmaf(raw[nq + e], raw[nq + e], sk);
      sk = block_sum(sk, scratch);
      if (tid == 0) {
        rs[0] = 1.0f / sqrtf(ss / (float)nq + eps);
        rs[1] = nk ? 1.0f / sqrtf(sk / (float)nk + eps) : 0.f;
      }
      __syncthreads();
    }
  }
  const int half = rot_dims >> 1;
  const float pos = (float)positions[t];
  const int slot = slots ? slots[t] : -1;
  const int page = slot >= 0 ? slot / page_size : 0, in_page = slot >= 0 ? slot % page_size : 0;
  for (int e = qk_lo * Dk + tid; e < qk_hi * Dk; e += 256) {
    const bool is_k = e >= nq;
    const int i = is_k ? e - nq : e;                  // index inside q or inside k
    const int h = i / Dk, d = i - h * Dk;
    const float* w = is_k ? kw : qw;
    float r = 1.f;
    if (norm_mode == NORM_HEAD) r = rs[is_k ? Hq + h : h];
    else if (norm_mode == NORM_WHOLE) r = rs[is_k ? 1 : 0];
    const int wi = norm_mode == NORM_WHOLE ? i : d;
    float val = raw[e] * r;
    if (norm_mode != NORM_NONE) val *= w[wi];
    if (d < rot_dims) {
      const int dp = d < half ? d + half : d - half;
      float other = raw[e + dp - d] * r;
      if (norm_mode != NORM_NONE) other *= w[wi + dp - d];
      const float a = pos * inv_freq[d < half ? d : d - half];
      const float c = cosf(a) * mag, s = sinf(a) * mag;
      val = d < half ? val * c - other * s : val * c + other * s;
    }
    if (!is_k) {
      q_out[(size_t)t * nq + i] = from_float<TO>(val);
    } else if (slot >= 0) {
      k_cache[(((size_t)page * Hk + h) * page_size + in_page) * Dk + d] = from_float<TO>(val);
    }
  }
  if (own && slot >= 0 && h_hi > heads_qk) {
    const int v_lo = max(h_lo, heads_qk) - heads_qk, v_hi = h_hi - heads_qk;
    for (int e = v_lo * Dv + tid; e < v_hi * Dv; e += 256) {
      const int h = e / Dv, d = e - h * Dv;
      v_cache[(((size_t)page * Hv + h) * page_size + in_page) * Dv + d] =
          from_float<TO>(row[v_off + e] + (vb ? vb[e] : 0.f));
    }
  }
}

extern "C" int ptl_qkv_prepare(void* q_out, const float* p, long ldp, int q_off, int k_off, int v_off,
                               const float* qb, const float* kb, const float* vb, int norm_mode,
                               const float* qw, const float* kw, float eps, int rot_dims,
                               const float* inv_freq, float mag, const int32_t* positions,
                               const int32_t* slots, void* k_cache, void* v_cache, int T_, int Hq, int Hk,
                               int Hv, int Dk, int Dv, int page_size, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (Hq <= 0 || Dk <= 0 || rot_dims < 0 || rot_dims > Dk || (rot_dims & 1) || (rot_dims && !inv_freq) ||
      norm_mode < 0 || norm_mode > 2 || (norm_mode && !qw) || !positions)
    return PTL_ERR_ARG;
  if (k_off >= 0 && (Hk <= 0 || Hv <= 0 || Dv <= 0 || page_size <= 0 || (norm_mode && !kw) ||
                     (slots && (!k_cache || !v_cache))))
    return PTL_ERR_ARG;
  const size_t floats = (size_t)Hq * Dk + (k_off >= 0 ? (size_t)Hk * Dk : 0) + Hq + (k_off >= 0 ? Hk : 0) + 2;
  const size_t lds = floats * sizeof(float);
  if (lds > 60 * 1024) return PTL_ERR_ARG;
  // slices of whole heads: about 512 workgroups in all when the tokens are few, one a token when
  // they are many
  const int heads = Hq + (k_off >= 0 ? Hk + Hv : 0);
  int slices = (512 + T_ - 1) / T_;
  if (slices > heads) slices = heads;
  if (slices < 1) slices = 1;
  const int heads_per_slice = (heads + slices - 1) / slices;
  slices = (heads + heads_per_slice - 1) / heads_per_slice;
  dim3 grid(T_, slices);
#define GO(TO)                                                                                        \
  {                                                                                                   \
    qkv_prepare_kernel<TO><<<grid, 256, lds, st>>>((TO*)q_out, p, ldp, q_off, k_off, v_off, qb, kb,   \
                                                   vb, norm_mode, qw, kw, eps, rot_dims, inv_freq,    \
                                                   mag, positions, slots, (TO*)k_cache,               \
                                                   (TO*)v_cache, Hq, Hk, Hv, Dk, Dv, page_size,       \
                                                   heads_per_slice);                                  \
    return ptl_launch_status();                                                                       \
  }
  if (dtype == PTL_DTYPE_F32) GO(float)
  if (dtype == PTL_DTYPE_BF16) GO(bf16_t)
#undef GO
  return PTL_ERR_ARG;
}

// ---- a short convolution, a rotation and then a norm ---------------------------------------------
// u_t = p_t + bias (the columns of q, k and v: one row of channels q | k | v);
// y_t = sum_j cw[:, j] u_(t - taps + 1 + j), inputs in front of the step's rows from the slot's kept
//   ones [taps - 1, C] (bias included; zeros where a sequence starts);
// q and k: the first rot_dims entries of a head turn by the row's position (pairs of neighbours, or
//   entry i with entry i + rot_dims / 2), then, when ``norm``, the head is divided by its root mean square.
// A wave takes one head for RUN rows one after the other, a lane NP pairs of its entries; the rows' inputs
// are asked for before the first is worked on, and the four waves of a workgroup (four heads of the
// same rows) share the rows' sines and cosines through LDS. With
// TAPS > 0 the last TAPS - 1 inputs of a lane's entries stay in registers from row to row (TAPS = 0: any
// number of taps, read again for every row). The first n_single sequences bring one row each: their
// lanes also advance the kept inputs they have just read (those of longer portions are advanced
// behind this kernel, when no wave reads them any more).

// Sine and cosine of pos * f, with what the product's rounding loses put back: at position 1,000 the
// rounded angle of a fast entry is off by some 1e-5, and by another amount for a query than for its keys.
__device__ __forceinline__ void turn_of(float pos, float f, float& sn, float& cs) {
  const float a = pos * f, rest = fmaf(pos, f, -a);
  float s, c;
  sincosf(a, &s, &c);
  sn = fmaf(rest, c, s);
  cs = fmaf(-rest, s, c);
}

#define PAIRS_NEIGHBOURS 0
#define PAIRS_HALF 1

struct ConvQkvArgs {
  const float* p; long ldp; int off[3];
  const float* bias;                        // [C] or null
  const float* cw; int taps;                // [C, taps]; null with taps 1: no convolution
  float* state; long slot_stride; long tail_off;
  const int32_t* q_start; const int32_t* state_slots; int n_seqs, n_single;
  const int32_t* positions; const int32_t* slots;
  int rot_dims, layout; const float* inv_freq;
  int norm; float eps;
  int T, Hq, Hk, Hv, Dk, Dv, page_size;
};

template <int NP, int TAPS, int RUN, typename TO>
__global__ void __launch_bounds__(256)
conv_qkv_prepare_kernel(TO* __restrict__ q_out, TO* __restrict__ k_cache, TO* __restrict__ v_cache, ConvQkvArgs A) {
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int head = blockIdx.y * 4 + wave;
  const int t_begin = blockIdx.x * RUN, t_end = min(A.T, t_begin + RUN);
  __shared__ float2 turns[RUN][64 * NP];    // (sine, cosine) of every row and pair
  if (A.rot_dims > 0 && (int)blockIdx.y * 4 < A.Hq + A.Hk) {
    const int pairs = A.rot_dims / 2;
    for (int i = threadIdx.x; i < RUN * pairs; i += 256) {
      const int r = i / pairs, j = i - r * pairs;
      if (t_begin + r < t_end) {
        float2 v;
        turn_of((float)A.positions[t_begin + r], A.inv_freq[j], v.x, v.y);
        turns[r][j] = v;
      }
    }
  }
  __syncthreads();
  if (head >= A.Hq + A.Hk + A.Hv) return;
  const int part = head < A.Hq ? 0 : (head < A.Hq + A.Hk ? 1 : 2);
  const int h = head - (part == 0 ? 0 : (part == 1 ? A.Hq : A.Hq + A.Hk));
  const int D = part == 2 ? A.Dv : A.Dk;
  const int C = (A.Hq + A.Hk) * A.Dk + A.Hv * A.Dv;
  const int c0 = (part == 0 ? 0 : (part == 1 ? A.Hq * A.Dk : (A.Hq + A.Hk) * A.Dk)) + h * D;      // channel of entry 0
  const int col0 = A.off[part] + h * D;
  const int rot = part == 2 ? 0 : A.rot_dims;
  const int taps = TAPS > 0 ? TAPS : A.taps;
  // the entries of this lane's pairs (-1: none)
  int e[NP][2];
#pragma unroll
  for (int n = 0; n < NP; ++n) {
    const int j = lane + 64 * n;
    if (A.layout == PAIRS_HALF && 2 * j < rot) { e[n][0] = j; e[n][1] = j + rot / 2; }
    else { e[n][0] = 2 * j; e[n][1] = 2 * j + 1; }
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (e[n][i] >= D) e[n][i] = -1;
  }
  // two neighbouring entries at an even column, rows of an even length: one 8-byte load
  const bool two = ((A.ldp | col0) & 1) == 0 && ((uintptr_t)A.p & 7) == 0 && !(A.layout == PAIRS_HALF && rot > 0) && D % 2 == 0;
  float2 ahead[RUN][NP];                    // the rows' columns
#pragma unroll
  for (int r = 0; r < RUN; ++r)
#pragma unroll
    for (int n = 0; n < NP; ++n) {
      float2 x = make_float2(0.f, 0.f);
      const float* at = A.p + (size_t)(t_begin + r) * A.ldp + col0;
      if (t_begin + r < t_end) {
        if (two) {
          if (e[n][0] >= 0) x = *reinterpret_cast<const float2*>(at + e[n][0]);
        } else {
          if (e[n][0] >= 0) x.x = at[e[n][0]];
          if (e[n][1] >= 0) x.y = at[e[n][1]];
        }
      }
      ahead[r][n] = x;
    }
  float w[NP][2][TAPS > 0 ? TAPS : 1], b[NP][2];
#pragma unroll
  for (int n = 0; n < NP; ++n) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      b[n][i] = A.bias && e[n][i] >= 0 ? A.bias[c0 + e[n][i]] : 0.f;
      if (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[n][i][j] = e[n][i] >= 0 ? (A.cw ? A.cw[(size_t)(c0 + e[n][i]) * TAPS + j] : 1.f) : 0.f;
      }
    }
  }
  auto input = [&](int row, int n, int i) {
    return e[n][i] >= 0 ? A.p[(size_t)row * A.ldp + col0 + e[n][i]] + b[n][i] : 0.f;
  };
  // the sequence of the first row: the last one whose first row is not beyond it
  int seq = 0, hi = A.n_seqs;
  while (seq < hi) {
    const int mid = (seq + hi + 1) >> 1;
    if (A.q_start[mid] <= t_begin) seq = mid; else hi = mid - 1;
  }
  if (seq >= A.n_seqs) return;              // rows that belong to no sequence
  const int my_slot = A.slots && lane < RUN && t_begin + lane < t_end ? A.slots[t_begin + lane] : -1;
  bool fresh = true;                        // the window in registers is not of this sequence yet
  int row0 = 0, seq_end = A.q_start[seq + 1];
  float* kept = nullptr;
  float win[NP][2][TAPS > 1 ? TAPS - 1 : 1];
#pragma unroll
  for (int q = 0; q < RUN; ++q) {
    const int t = t_begin + q;
    if (t >= t_end) return;
    if (q == 0 || t >= seq_end) {           // (sequences without rows are skipped)
      while (seq < A.n_seqs && A.q_start[seq + 1] <= t) ++seq;
      if (seq >= A.n_seqs) return;
      row0 = A.q_start[seq];
      seq_end = A.q_start[seq + 1];
      if (taps > 1) kept = A.state + (size_t)A.state_slots[seq] * A.slot_stride + A.tail_off;
      fresh = true;
    }
    auto before = [&](int r, int n, int i) {                   // the input of row r of the sequence (r < 0: a kept one)
      if (r >= 0) return input(row0 + r, n, i);
      return e[n][i] >= 0 ? kept[(size_t)(taps - 1 + r) * C + c0 + e[n][i]] : 0.f;
    };
    const int r = t - row0;
    float y[NP][2];
#pragma unroll
    for (int n = 0; n < NP; ++n)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const float x = (i == 0 ? ahead[q][n].x : ahead[q][n].y) + b[n][i];
        if (TAPS > 0) {
          if (fresh) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) win[n][i][j] = before(r - (TAPS - 1) + j, n, i);
          }
          float s = 0.f;
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) s = fmaf(w[n][i][j], win[n][i][j], s);
          y[n][i] = fmaf(w[n][i][TAPS - 1], x, s);
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) win[n][i][j] = j + 1 < TAPS - 1 ? win[n][i][j + 1] : x;
          if (seq < A.n_single && e[n][i] >= 0) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) kept[(size_t)j * C + c0 + e[n][i]] = win[n][i][j];
          }
        } else {
          const float* wr = A.cw + (size_t)(c0 + max(e[n][i], 0)) * taps;
          float s = 0.f;
          for (int j = 0; j < taps - 1; ++j) s = fmaf(wr[j], before(r - (taps - 1) + j, n, i), s);
          y[n][i] = fmaf(wr[taps - 1], x, s);
          if (seq < A.n_single && e[n][i] >= 0) {
            float* k = kept + c0 + e[n][i];
            for (int j = 0; j < taps - 1; ++j) k[(size_t)j * C] = j + 1 < taps - 1 ? k[(size_t)(j + 1) * C] : x;
          }
        }
      }
    fresh = false;
    float scale = 1.f;
    if (part < 2) {
      if (rot > 0) {
#pragma unroll
        for (int n = 0; n < NP; ++n) {
          if (2 * (lane + 64 * n) >= rot) continue;
          const float sn = turns[q][lane + 64 * n].x, cs = turns[q][lane + 64 * n].y;
          const float u = y[n][0], v = y[n][1];
          y[n][0] = u * cs - v * sn;
          y[n][1] = v * cs + u * sn;
        }
      }
      if (A.norm) {
        float ss = 0.f;
#pragma unroll
        for (int n = 0; n < NP; ++n)
#pragma unroll
          for (int i = 0; i < 2; ++i)
            if (e[n][i] >= 0) ss = fmaf(y[n][i], y[n][i], ss);
        scale = 1.0f / sqrtf(wave_sum(ss) / (float)D + A.eps);
      }
    }
    TO* dst = nullptr;
    if (part == 0) {
      dst = q_out + ((size_t)t * A.Hq + h) * D;
    } else {
      const int slot = __builtin_amdgcn_readlane(my_slot, q);
      const int page = max(slot, 0) / A.page_size, at = max(slot, 0) % A.page_size;
      if (slot >= 0) dst = part == 1 ? k_cache + (((size_t)page * A.Hk + h) * A.page_size + at) * D
                      : v_cache + (((size_t)page * A.Hv + h) * A.page_size + at) * D;
    }
    if (dst == nullptr) continue;
#pragma unroll
    for (int n = 0; n < NP; ++n) {
      if (sizeof(TO) == 2 && D % 2 == 0 && e[n][0] >= 0 && e[n][1] == e[n][0] + 1 && e[n][0] % 2 == 0) {
        union { uint32_t u; bf16_t x[2]; } two;
        two.x[0] = float_to_bf16(y[n][0] * scale);
        two.x[1] = float_to_bf16(y[n][1] * scale);
        *reinterpret_cast<uint32_t*>(dst + e[n][0]) = two.u;
      } else {
#pragma unroll
        for (int i = 0; i < 2; ++i)
          if (e[n][i] >= 0) dst[e[n][i]] = from_float<TO>(y[n][i] * scale);
      }
    }
  }
}

// p float32 [T, ldp] with q (Hq heads of Dk), k (Hk of Dk) and v (Hv of Dv) at their columns; bias, cw: of the
// channels q | k | v. q_out [T, Hq, Dk] and the caches of dtype; slots null: nothing is written to the caches.
extern "C" int ptl_conv_qkv_prepare(void* q_out, const float* p, long ldp, int q_off, int k_off, int v_off,
                                    const float* bias, const float* cw, int taps, float* state, long slot_stride,
                                    long tail_off, const int32_t* q_start, const int32_t* state_slots, int n_seqs,
                                    int n_single, const int32_t* positions, const int32_t* slots, int rot_dims,
                                    int layout, const float* inv_freq, int norm, float eps, void* k_cache,
                                    void* v_cache, int T_, int Hq, int Hk, int Hv, int Dk, int Dv, int page_size,
                                    int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (Hq <= 0 || Hk <= 0 || Hv <= 0 || Dk <= 0 || Dv <= 0 || Dk > 640 || Dv > 640 || page_size <= 0 || taps < 1 ||
      (!cw && taps != 1) || rot_dims < 0 || rot_dims > Dk || (rot_dims & 1) || (rot_dims && !inv_freq) || n_seqs <= 0 ||
      n_single < 0 || n_single > n_seqs || (layout != PAIRS_NEIGHBOURS && layout != PAIRS_HALF) || !positions ||
      (slots && (!k_cache || !v_cache)) || (Hq + Hk + Hv + 3) / 4 > 65535 ||
      (taps > 1 && (!state || tail_off < 0 ||
                    tail_off + (long)(taps - 1) * ((Hq + Hk) * Dk + Hv * Dv) > slot_stride)))
    return PTL_ERR_ARG;
  ConvQkvArgs A{p, ldp, {q_off, k_off, v_off}, bias, cw, taps, state, slot_stride, tail_off, q_start, state_slots,
                n_seqs, n_single, positions, slots, rot_dims, layout, inv_freq, norm, eps, T_, Hq, Hk, Hv, Dk, Dv,
                page_size};
  // runs of rows that share their inputs where the chip stays filled
  const bool wide = (Dk > Dv ? Dk : Dv) > 128;
  const int run = !wide && (long)T_ * (Hq + Hk + Hv) >= 16384 ? 8 : 1;
  const dim3 grid((T_ + run - 1) / run, (Hq + Hk + Hv + 3) / 4);
#define GO(NP, TAPS, RUN, TO)                                                                                       \
  conv_qkv_prepare_kernel<NP, TAPS, RUN, TO><<<grid, 256, 0, st>>>((TO*)q_out, (TO*)k_cache, (TO*)v_cache, A)
#define BY_TAPS(NP, RUN, TO)                                     \
  if (taps == 4) GO(NP, 4, RUN, TO);                             \
  else if (taps == 1) GO(NP, 1, RUN, TO);                        \
  else GO(NP, 0, RUN, TO)
#define BY_SIZE(TO)                                                             \
  if (wide) { BY_TAPS(5, 1, TO); }                                              \
  else if (run == 8) { BY_TAPS(1, 8, TO); }                                     \
  else { BY_TAPS(1, 1, TO); }
  if (dtype == PTL_DTYPE_F32) { BY_SIZE(float) }
  else if (dtype == PTL_DTYPE_BF16) { BY_SIZE(bf16_t) }
  else return PTL_ERR_ARG;
#undef BY_SIZE
#undef BY_TAPS
#undef GO
  return ptl_launch_status();
}

#define ACT_NONE 0
#define ACT_SIGMOID 1
#define ACT_SILU 2

template <typename TO>
__global__ void __launch_bounds__(256)
head_norm_gate_kernel(TO* __restrict__ out, long ldo, const float* __restrict__ a, int maps, float lam,
                      const float* __restrict__ w, int w_stride, float mult, const float* __restrict__ gate,
                      long ldg, int g_off, int act, float eps, int T_, int H, int Dv) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const long item = (long)blockIdx.x * 4 + wave;
  if (item >= (long)T_ * H) return;
  const int t = (int)(item / H), h = (int)(item - (long)t * H);
  const float* a1 = a + ((size_t)t * H * maps + (size_t)h * maps) * Dv;
  const float* a2 = a1 + Dv;
  float ss = 0.f;
  for (int d = lane; d < Dv; d += 64) {
    const float o = maps == 2 ? a1[d] - lam * a2[d] : a1[d];
    ss = fmaf(o, o, ss);
  }
  ss = wave_sum(ss);
  const float r = mult / sqrtf(ss / (float)Dv + eps);
  const float* g = gate ? gate + (size_t)t * ldg + g_off + (size_t)h * Dv : nullptr;
  TO* dst = out + (size_t)t * ldo + (size_t)h * Dv;
  for (int d = lane; d < Dv; d += 64) {
    float o = (maps == 2 ? a1[d] - lam * a2[d] : a1[d]) * r;
    if (w) o *= w[(size_t)h * w_stride + d];
    if (g) {
      const float z = g[d];
      const float sg = 1.0f / (1.0f + expf(-z));
      o *= act == ACT_SILU ? z * sg : sg;
    }
    dst[d] = from_float<TO>(o);
  }
}

// One map, heads of up to 256 values that divide by 4: LPH lanes a head with a float4 each, 64 / LPH heads
// (neighbours of one row after the other) a wave.
template <int LPH, typename TO>
__global__ void __launch_bounds__(256)
head_norm_gate_vec_kernel(TO* __restrict__ out, long ldo, const float* __restrict__ a, const float* __restrict__ w,
                          int w_stride, float mult, const float* __restrict__ gate, long ldg, int g_off, int act, float eps,
                          long items, int H, int Dv) {
  const long item = ((long)blockIdx.x * 256 + threadIdx.x) / LPH;
  const int d = 4 * (threadIdx.x % LPH);
  const bool in = item < items && d < Dv;
  const long t = item / H;
  const int h = (int)(item - t * H);
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f), g = o;
  if (in) {
    o = *reinterpret_cast<const float4*>(a + (size_t)item * Dv + d);
    if (gate) g = *reinterpret_cast<const float4*>(gate + (size_t)t * ldg + g_off + (size_t)h * Dv + d);
  }
  float ss = fmaf(o.x, o.x, fmaf(o.y, o.y, fmaf(o.z, o.z, o.w * o.w)));
#pragma unroll
  for (int s = 1; s < LPH; s <<= 1) ss += __shfl_xor(ss, s, 64);
  if (!in) return;
  const float r = mult / sqrtf(ss / (float)Dv + eps);
  float v[4] = {o.x * r, o.y * r, o.z * r, o.w * r};
  const float z[4] = {g.x, g.y, g.z, g.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (w) v[i] *= w[(size_t)h * w_stride + d + i];
    if (gate) {
      const float sg = 1.0f / (1.0f + expf(-z[i]));
      v[i] *= act == ACT_SILU ? z[i] * sg : sg;
    }
  }
  TO* dst = out + (size_t)t * ldo + (size_t)h * Dv + d;
  if (sizeof(TO) == 2) {
    union { uint2 u; bf16_t e[4]; } e;
#pragma unroll
    for (int i = 0; i < 4; ++i) e.e[i] = float_to_bf16(v[i]);
    *reinterpret_cast<uint2*>(dst) = e.u;
  } else {
    *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
  }
}

template <typename TO>
static bool head_norm_gate_vec(void* out, long ldo, const float* a, const float* w, int w_stride, float mult,
                               const float* gate, long ldg, int g_off, int act, float eps, long items, int H, int Dv,
                               hipStream_t st) {
  if (Dv % 4 || Dv > 256 || ldo % 4 || (((uintptr_t)a | (uintptr_t)out) & 15) ||
      (gate && (ldg % 4 || g_off % 4 || ((uintptr_t)gate & 15))))
    return false;
  const int lanes = Dv / 4;
#define GO(LPH)                                                                                                    \
  if (lanes <= LPH) {                                                                                              \
    head_norm_gate_vec_kernel<LPH, TO><<<(int)((items * LPH + 255) / 256), 256, 0, st>>>(                          \
        (TO*)out, ldo, a, w, w_stride, mult, gate, ldg, g_off, act, eps, items, H, Dv);                            \
    return true;                                                                                                   \
  }
  GO(4) GO(8) GO(16) GO(32) GO(64)
#undef GO
  return false;
}

// a float32 [T, H * maps, Dv] dense; out [T, ldo] (H * Dv columns used); gate float32 [T, ldg] read
// at columns g_off .. g_off + H * Dv, or null; w float32 (w_stride 0: [Dv] for all heads, Dv: [H, Dv]),
// or null.
extern "C" int ptl_head_norm_gate(void* out, long ldo, const float* a, int maps, float lam, const float* w,
                                  int w_stride, float mult, const float* gate, long ldg, int g_off, int act,
                                  float eps, int T_, int H, int Dv, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (H <= 0 || Dv <= 0 || maps < 1 || maps > 2 || act < 0 || act > 2 || (gate && act == ACT_NONE))
    return PTL_ERR_ARG;
  const long items = (long)T_ * H;
  const long blocks = (items + 3) / 4;
  if (items > 0x7fffffff / 16) return PTL_ERR_ARG;
  if (maps == 1 && dtype == PTL_DTYPE_F32 &&
      head_norm_gate_vec<float>(out, ldo, a, w, w_stride, mult, gate, ldg, g_off, act, eps, items, H, Dv, st))
    return ptl_launch_status();
  if (maps == 1 && dtype == PTL_DTYPE_BF16 &&
      head_norm_gate_vec<bf16_t>(out, ldo, a, w, w_stride, mult, gate, ldg, g_off, act, eps, items, H, Dv, st))
    return ptl_launch_status();
#define GO(TO)                                                                                         \
  {                                                                                                    \
    head_norm_gate_kernel<TO><<<(int)blocks, 256, 0, st>>>((TO*)out, ldo, a, maps, lam, w, w_stride,   \
                                                           mult, gate, ldg, g_off, act, eps, T_, H, Dv); \
    return ptl_launch_status();                                                                        \
  }
  if (dtype == PTL_DTYPE_F32) GO(float)
  if (dtype == PTL_DTYPE_BF16) GO(bf16_t)
#undef GO
  return PTL_ERR_ARG;
}

// The kept inputs of a short convolution of the first n_rows rows, each a sequence of one token:
// tail [taps - 1, C] at tail_off of the sequence's slot; x[t * ldx + c] the token's input.
struct TailArgs {
  float* state; long slot_stride; long tail_off;
  const float* x; long ldx;
  const int32_t* state_slots;
  int n_rows, C, taps;
};

// Channels part * per .. of row t's kept inputs, the lanes of ``width`` threads side by side.
__device__ __forceinline__ void advance_tail(const TailArgs& a, int t, int part, int parts, int lane, int width) {
  float* kept = a.state + (size_t)a.state_slots[t] * a.slot_stride + a.tail_off;
  const int per = (a.C + parts - 1) / parts;
  for (int c = part * per + lane; c < min(a.C, (part + 1) * per); c += width) {
    float v[4];                              // the first inputs read before any is written
    const float x = a.x[(size_t)t * a.ldx + c];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = i + 2 < a.taps ? kept[(size_t)(i + 1) * a.C + c] : x;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i + 2 <= a.taps) kept[(size_t)i * a.C + c] = v[i];
    for (int i = 4; i + 2 <= a.taps; ++i) kept[(size_t)i * a.C + c] = i + 2 < a.taps ? kept[(size_t)(i + 1) * a.C + c] : x;
  }
}

template <typename TO>
__global__ void __launch_bounds__(256)
gate_group_norm_kernel(TO* __restrict__ out, const float* __restrict__ y, const float* __restrict__ z, long ldz,
                       const float* __restrict__ w, int n, int groups, float eps, TailArgs tail) {
  extern __shared__ float us[];
  __shared__ float scratch[16];
  const int t = blockIdx.x, part = blockIdx.y, tid = threadIdx.x, nt = blockDim.x;
  const int size = n / groups, c0 = part * size;
  const float* yr = y + (size_t)t * n + c0;
  const float* zr = z + (size_t)t * ldz + c0;
  float ss = 0.f;
  for (int c = tid; c < size; c += nt) {
    const float g = zr[c];
    const float u = yr[c] * (g / (1.0f + expf(-g)));
    us[c] = u;
    ss = fmaf(u, u, ss);
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)size + eps);
  TO* dst = out + (size_t)t * n + c0;
  for (int c = tid; c < size; c += nt) dst[c] = from_float<TO>(us[c] * r * w[c0 + c]);
  if (t < tail.n_rows) advance_tail(tail, t, part, groups, tid, nt);
}

// A wave a (token, group): the group's columns as NV float4 a lane, nothing through LDS.
template <int NV, typename TO>
__global__ void __launch_bounds__(256)
gate_group_norm_wave_kernel(TO* __restrict__ out, const float* __restrict__ y, const float* __restrict__ z, long ldz,
                            const float* __restrict__ w, int n, int groups, float eps, long items, TailArgs tail) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int lane = threadIdx.x & 63;
  const long t = item / groups;
  const int part = (int)(item - t * groups);
  const int size = n / groups, c0 = part * size;
  const float* yr = y + (size_t)t * n + c0;
  const float* zr = z + (size_t)t * ldz + c0;
  float4 a[NV], b[NV];
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = 4 * (lane + 64 * k);
    a[k] = b[k] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c < size) {
      a[k] = *reinterpret_cast<const float4*>(yr + c);
      b[k] = *reinterpret_cast<const float4*>(zr + c);
    }
  }
  auto gated = [](float v, float g) { return v * (g / (1.0f + expf(-g))); };
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    a[k] = make_float4(gated(a[k].x, b[k].x), gated(a[k].y, b[k].y), gated(a[k].z, b[k].z), gated(a[k].w, b[k].w));
    ss = fmaf(a[k].x, a[k].x, fmaf(a[k].y, a[k].y, fmaf(a[k].z, a[k].z, fmaf(a[k].w, a[k].w, ss))));
  }
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)size + eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = 4 * (lane + 64 * k);
    if (c >= size) continue;
    const float4 ww = *reinterpret_cast<const float4*>(w + c0 + c);
    const float v[4] = {a[k].x * r * ww.x, a[k].y * r * ww.y, a[k].z * r * ww.z, a[k].w * r * ww.w};
    TO* dst = out + (size_t)t * n + c0 + c;
    if (sizeof(TO) == 2) {
      union { uint2 u; bf16_t e[4]; } o;
#pragma unroll
      for (int j = 0; j < 4; ++j) o.e[j] = float_to_bf16(v[j]);
      *reinterpret_cast<uint2*>(dst) = o.u;
    } else {
      *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
    }
  }
  if (t < tail.n_rows) advance_tail(tail, (int)t, part, groups, lane, 64);
}

template <typename TO>
static bool gate_group_norm_waves(void* out, const float* y, const float* z, long ldz, const float* w, int groups,
                                  float eps, int T_, int n, const TailArgs& tail, hipStream_t st) {
  const int size = n / groups;
  const long items = (long)T_ * groups;
  if (size % 4 || ldz % 4 || size > 2048 || (((uintptr_t)y | (uintptr_t)z | (uintptr_t)w | (uintptr_t)out) & 15) ||
      items > 4L * 0x7fffffff)
    return false;
  const int blocks = (int)((items + 3) / 4);
#define GO(NV)                                                                                                       \
  if (size <= 256 * NV) {                                                                                            \
    gate_group_norm_wave_kernel<NV, TO><<<blocks, 256, 0, st>>>((TO*)out, y, z, ldz, w, n, groups, eps, items, tail); \
    return true;                                                                                                     \
  }
  GO(1) GO(2) GO(4) GO(8)
#undef GO
  return false;
}

// y float32 [T, n] dense, z float32 [T, ldz] (its first n columns), w float32 [n], out [T, n] dense.
// tail_rows > 0 and taps > 1: rows 0 .. tail_rows - 1 also advance the kept inputs of their slots.
extern "C" int ptl_gate_group_norm(void* out, const float* y, const float* z, long ldz, const float* w, int groups,
                                   float eps, int T_, int n, float* state, long slot_stride, long tail_off,
                                   const float* x, long ldx, const int32_t* state_slots, int tail_rows, int C,
                                   int taps, int dtype, hipStream_t st) {
  if (T_ <= 0) return PTL_OK;
  if (n <= 0 || groups <= 0 || n % groups || groups > 65535 || (size_t)(n / groups) * sizeof(float) > 60 * 1024 ||
      tail_rows > T_ || (tail_rows > 0 && taps > 1 && (!state || !x || !state_slots || C <= 0)))
    return PTL_ERR_ARG;
  const TailArgs tail{state, slot_stride, tail_off, x, ldx, state_slots, taps > 1 ? tail_rows : 0, C, taps};
  // enough of them: a wave a (token, group)
  if ((long)T_ * groups >= 1024) {
    bool done = false;
    if (dtype == PTL_DTYPE_F32) done = gate_group_norm_waves<float>(out, y, z, ldz, w, groups, eps, T_, n, tail, st);
    else if (dtype == PTL_DTYPE_BF16) done = gate_group_norm_waves<bf16_t>(out, y, z, ldz, w, groups, eps, T_, n, tail, st);
    if (done) return ptl_launch_status();
  }
  const int size = n / groups;
  const int threads = size >= 256 ? 256 : (size + 63) / 64 * 64;
  const size_t lds = (size_t)size * sizeof(float);
  if (dtype == PTL_DTYPE_F32)
    gate_group_norm_kernel<float><<<dim3(T_, groups), threads, lds, st>>>((float*)out, y, z, ldz, w, n, groups, eps, tail);
  else if (dtype == PTL_DTYPE_BF16)
    gate_group_norm_kernel<bf16_t><<<dim3(T_, groups), threads, lds, st>>>((bf16_t*)out, y, z, ldz, w, n, groups, eps,
                                                                           tail);
  else
    return PTL_ERR_ARG;
  return ptl_launch_status();
}
