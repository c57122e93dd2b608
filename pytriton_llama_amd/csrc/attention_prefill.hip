// Attention of prompt portions over the paged cache on the matrix cores (bfloat16).
// The cache layout, the meaning of the arguments and the reference formulas are those of
// attention.hip; this kernel has a source file of its own because it is compiled with one more
// option (see max2 below).
#include "attention.h"
#include "common.h"
#include "mfma.h"
#include <math.h>
#include <type_traits>

// ===========================================================================
// ptl_attention_prefill_mfma: bfloat16 prompt portions on the matrix cores.
//
// A workgroup of four waves takes 64 or 128 query rows of one head (16 or 32 per
// wave) and walks the sequence's keys in tiles of 64. Key and value tiles go
// through LDS as they lie in the cache (rows of D), in two buffers: while tile t
// is used, tile t+1 is on its way from global memory straight into the other
// buffer (global_load_lds_dwordx4, no register in between; its page numbers were
// read one tile earlier still), so a tile costs one barrier. Both products are
// computed transposed so that the scores leave the first MFMA in the register
// layout the second one wants, without a shuffle:
//   S^T[key, query] = K[key, :] . Q[query, :]      (A = K tile, B = Q^T)
//   O^T[d, query]  += V^T[d, key] . P^T[key, query] (A = V^T tile, B = P^T)
// with v_mfma_f32_16x16x32_bf16: a lane holds 8 consecutive k-values of row
// (lane % 16), k-group (lane / 16); the result tile holds rows 4*(lane/16)+i,
// column lane % 16. The V^T fragments come from the row-major value tile through
// ds_read_b64_tr_b16: in a group of 16 lanes, lane s gives the address of four
// consecutive elements E[s][0..3], and lane l receives E[4i + l/4][l%4], i = 0..3;
// with lane s pointing at V[key0 + s/4][d0 + 4*(s%4)], lane l gets
// V[key0 + 0..3][d0 + l]. Softmax is the online one of
// lite_llama/kernels/flashattentionv2.py:10-61 in base 2 (scale * log2 e folded
// into the scores, exp2), float32 max / denominator / accumulator; P is rounded
// to bfloat16 for the second product as there (:55). The running maximum is a
// stabiliser, not a result: it follows the scores only when they pass it by more
// than 8 (in the exponent's units), so that what is kept is rescaled rarely.
// Needs D % 32 == 0, D <= 128, a page size that is a power of two.
//
// Keys of size DK and values of size DV need not be alike (both multiples of 32 up to 128), and
// a head may come in several score maps over one set of values, as in the general form of the
// vector kernel (attention.hip): query head j is map j % maps of head j / maps and reads key
// head (kv head) * maps + j % maps and the values of its kv head. The result is bfloat16, or
// float32 for one that is combined further before it is rounded.
// ===========================================================================

#define PF_BN 64


// (This file is compiled with -fno-honor-nans: fmaxf then is one v_max, or half a v_max3,
// without a quieting v_max(x, x) in front of every score that comes out of an MFMA. No inline
// assembly for it: the compiler inserts the wait states between an MFMA and the first read of
// its result only for instructions it knows.)
__device__ __forceinline__ float max2(float a, float b) { return fmaxf(a, b); }
__device__ __forceinline__ s16x4_t lds_read_tr16(const bf16_t* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_t*)p);
}

template <typename TO> __device__ __forceinline__ void store4(TO* p, const float* v);
template <> __device__ __forceinline__ void store4<bf16_t>(bf16_t* p, const float* v) {
  union { uint2 u; bf16_t e[4]; } rr;
#pragma unroll
  for (int i = 0; i < 4; ++i) rr.e[i] = float_to_bf16(v[i]);
  *reinterpret_cast<uint2*>(p) = rr.u;
}
template <> __device__ __forceinline__ void store4<float>(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

// NDK, NDV: key and value sizes in units of 32. RT: 16-row query tiles per wave; the workgroup
// takes 64 * RT query rows. KEPT: a window that keeps the sequence's first keys (keep_first > 0):
// the key tiles then walk a list of two stretches of positions instead of one. CAP: scores are capped:
// tanh_exp2(raw score * cap_in) takes the place of the raw score and scale_log2 is softcap * log2 e.
template <int NDK, int NDV, int RT, typename TO, bool KEPT, bool CAP>
__global__ void __launch_bounds__(256, (NDK + NDV) <= 4 ? 3 : 2)
attn_prefill_mfma_kernel(TO* __restrict__ out, long out_stride, const bf16_t* __restrict__ q,
                         long q_stride, const bf16_t* __restrict__ k_cache,
                         const bf16_t* __restrict__ v_cache, const int32_t* __restrict__ q_start,
                         const int32_t* __restrict__ ctx_len, const int32_t* __restrict__ block_table,
                         int bt_stride, const int32_t* __restrict__ work_seq,
                         const int32_t* __restrict__ work_qoff, int n_work, int Hq, int Hkv, int maps,
                         int page_size, int page_shift, AttnExtras ex, float scale_log2, float cap_in) {
  constexpr int DK = 32 * NDK, DV = 32 * NDV;
  constexpr int PBM = 64 * RT;
  constexpr int CPRK = DK / 8, CPRV = DV / 8;      // 16-byte chunks per row
  constexpr int NCHK = PF_BN * CPRK / 256, NCHV = PF_BN * CPRV / 256;   // chunks of a tile per thread
  // Tiles lie in LDS as rows of D elements without padding; the 16-byte chunks of a row are
  // permuted (chunk c of row r lies at c ^ swz(r)) so that neither the row-wise reads of the
  // first product nor the transposing reads of the second meet in a bank. Two buffers each,
  // as separate arrays: the compiler then knows that a load into one does not touch the other.
  constexpr bool SW8K = CPRK % 8 == 0, SW8V = CPRV % 8 == 0;
  __shared__ __attribute__((aligned(1024))) bf16_t Ks0[PF_BN * DK];
  __shared__ __attribute__((aligned(1024))) bf16_t Ks1[PF_BN * DK];
  __shared__ __attribute__((aligned(1024))) bf16_t Vs0[PF_BN * DV];
  __shared__ __attribute__((aligned(1024))) bf16_t Vs1[PF_BN * DV];
  auto swzk = [](int row) { return SW8K ? (row & 7) : ((row >> 1) & 3); };
  auto swzv = [](int row) { return SW8V ? (row & 7) : ((row >> 1) & 3); };

  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int ln = lane & 15, lg = lane >> 4;
  // Heads run along x, the fast index of the launch, so that workgroups started one after the
  // other land on the eight XCDs in turn; the heads are dealt out so that XCD c gets heads
  // c * Hq/8 .. (c+1) * Hq/8 - 1: the query heads of a kv head meet in one L2, which then holds
  // an eighth of the keys and values instead of all of them.
  const int head = (Hq % 8 == 0) ? (blockIdx.x % 8) * (Hq / 8) + blockIdx.x / 8 : blockIdx.x;
  const int group_at = blockIdx.y, n_groups = gridDim.y;
  // The work list is sorted, the blocks with the most keys first. The n_groups workgroups of a
  // head walk it as a snake: forwards in even rounds, backwards in odd ones, so that the
  // workgroup with the longest block of one round takes the shortest of the next.
  for (int round = 0;; ++round) {
  const int item = round * n_groups + ((round & 1) ? n_groups - 1 - group_at : group_at);
  if (item >= n_work) break;       // (and so is every later item of this workgroup)
  const int seq = work_seq[item];
  const int qoff = work_qoff[item];
  const int qs = q_start[seq];
  const int qlen = q_start[seq + 1] - qs;
  const int ctx = ctx_len[seq];
  const int cached = ctx - qlen;
  const int rows = min(PBM, qlen - qoff);
  if (rows <= 0) continue;
  const int vh = (head / maps) / ((Hq / maps) / Hkv);      // value head
  const int kh = vh * maps + head % maps;                   // key head (of Hkv * maps)
  const int32_t* bt = block_table + (size_t)seq * bt_stride;
  const int first_q = cached + qoff;

  // query rows of this lane: tile r covers rows 16*(RT*wave + r) .. +15 of the block
  int qpos[RT];
  bool row_ok[RT];
  Frag8 qf[RT][NDK];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    const int my_row = 16 * (RT * wave + r) + ln;
    row_ok[r] = my_row < rows;
    const int qrow = row_ok[r] ? my_row : 0;       // rows past the end repeat row 0; never stored
    qpos[r] = first_q + qrow;
    const bf16_t* qp = q + (size_t)(qs + qoff + qrow) * q_stride + (size_t)head * DK + 8 * lg;
#pragma unroll
    for (int kk = 0; kk < NDK; ++kk) qf[r][kk].u = *reinterpret_cast<const uint4*>(qp + 32 * kk);
  }
  const int wave_first_row = 16 * RT * wave;
  const bool wave_has_rows = wave_first_row < rows;
  const int wave_min_q = first_q + (wave_has_rows ? wave_first_row : 0);
  const int wave_max_q = first_q + min(rows, wave_first_row + 16 * RT) - 1;

  // The softmax denominator: o[r][2 NDV] is one more tile of the second product, whose
  // "values" are all one; it sums the probabilities as the product sees them (rounded to
  // bfloat16; float32 sums) and is rescaled with the numerators.
  f32x4_t o[RT][2 * NDV + 1];
  float m_run[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    m_run[r] = -INFINITY;
#pragma unroll
    for (int t = 0; t <= 2 * NDV; ++t) o[r][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  Frag8 ones;
#pragma unroll
  for (int j = 0; j < 8; ++j) ones.v[j] = (__bf16)1.0f;
  // the running maximum follows the scores only when they pass it by more than this (raw
  // units): until then exp2 of a score minus the maximum stays below 2^8, which float32 sums
  // and bfloat16 probabilities hold as well as values below 1, and nothing is rescaled
  const float lazy = 8.0f / scale_log2;

  // The keys this block walks in tiles of 64, from index k_begin (a multiple of 64) on; indices
  // below k_lo and from k_end on are no keys. Without kept keys an index is a position. KEPT: the
  // list is the kept first keys left of the window (positions 0 .. n_kept - 1) and then the
  // positions from the window's start on, index 0 is its first entry, and key_at gives the
  // position of an index.
  const int win_lo = first_seen(ex, first_q);
  const int n_kept = KEPT ? min(max(ex.keep_first, 0), win_lo) : 0;
  const int shift = KEPT ? win_lo - n_kept : 0;
  const int k_lo = KEPT ? 0 : win_lo;
  const int k_end = min(ctx, first_q + rows) - shift;
  const int k_begin = (k_lo / PF_BN) * PF_BN;
  const int n_tiles = (k_end - k_begin + PF_BN - 1) / PF_BN;
  auto key_at = [&](int kw) { return KEPT ? (kw < n_kept ? kw : kw + shift) : kw; };
  // What a row sees, in indices: its own key is index qw; with kept keys, an index from n_kept on
  // is a key of the window (position index + shift, which is no kept position when shift > 0),
  // an index below is a kept key (a position below keep_first), so key_at is not needed there:
  //   seen = kw <= qw && kw < k_end && (kw >= lo || kw < keep_lim),  lo the row's first key
  int qw[RT], lo[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    qw[r] = qpos[r] - shift;
    lo[r] = first_seen(ex, qpos[r]) - shift;
  }
  const int keep_lim = shift == 0 ? ex.keep_first : n_kept;
  // the first keys of the wave's first and last row: left of the one nothing of a tile is seen (no
  // kept keys), from the other on all rows see it
  const int wave_lo_first = first_seen(ex, wave_min_q) - shift, wave_lo_last = first_seen(ex, wave_max_q) - shift;

  // This thread's chunks of a tile. A wave's load instruction fills 64 consecutive 16-byte
  // slots of LDS, lane l the l-th; slot s holds row s / CPR, chunk (s % CPR) ^ swz(row).
  const int wave_u = __builtin_amdgcn_readfirstlane(wave);
  int crowk[NCHK], ccolk[NCHK], crowv[NCHV], ccolv[NCHV];
#pragma unroll
  for (int i = 0; i < NCHK; ++i) {
    const int slot = 64 * (wave_u * NCHK + i) + lane;
    crowk[i] = slot / CPRK;
    ccolk[i] = ((slot - crowk[i] * CPRK) ^ swzk(crowk[i])) * 8;
  }
#pragma unroll
  for (int i = 0; i < NCHV; ++i) {
    const int slot = 64 * (wave_u * NCHV + i) + lane;
    crowv[i] = slot / CPRV;
    ccolv[i] = ((slot - crowv[i] * CPRV) ^ swzv(crowv[i])) * 8;
  }
  const bf16_t* k_head = k_cache + (size_t)kh * page_size * DK;
  const bf16_t* v_head = v_cache + (size_t)vh * page_size * DV;

  int pgk[NCHK], pgv[NCHV];     // pages of the chunks' rows, read one tile ahead of the rows
  const uint32_t page_bytes_k = (uint32_t)Hkv * maps * page_size * DK * 2;     // < 4 GiB, checked by the host
  const uint32_t page_bytes_v = (uint32_t)Hkv * page_size * DV * 2;
  const int page_mask = page_size - 1;                                // page sizes are powers of two
  // a tile that lies wholly inside the keys this block sees needs no tests (uniform)
  auto whole = [&](int t) {
    const int k0 = k_begin + t * PF_BN;
    return t < n_tiles && k0 >= k_lo && k0 + PF_BN <= k_end;
  };
  auto load_pages = [&](int t) {
    const int k0 = k_begin + t * PF_BN;
    if (whole(t)) {
#pragma unroll
      for (int i = 0; i < NCHK; ++i) pgk[i] = bt[key_at(k0 + crowk[i]) >> page_shift];
#pragma unroll
      for (int i = 0; i < NCHV; ++i) pgv[i] = bt[key_at(k0 + crowv[i]) >> page_shift];
    } else {
#pragma unroll
      for (int i = 0; i < NCHK; ++i) {
        const int kp = k0 + crowk[i];
        pgk[i] = -1;
        if (t < n_tiles && kp >= k_lo && kp < k_end) pgk[i] = bt[key_at(kp) >> page_shift];
      }
#pragma unroll
      for (int i = 0; i < NCHV; ++i) {
        const int kp = k0 + crowv[i];
        pgv[i] = -1;
        if (t < n_tiles && kp >= k_lo && kp < k_end) pgv[i] = bt[key_at(kp) >> page_shift];
      }
    }
  };
  // global memory -> LDS without a register in between (global_load_lds_dwordx4): every lane
  // names its own 16 bytes of global memory, the wave's 64 chunks land side by side in LDS
  auto to_lds = [&](const bf16_t* base, uint64_t at, bf16_t* tile_lds, int chunk) {
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) void*)(reinterpret_cast<const char*>(base) + at),
        (__attribute__((address_space(3))) void*)(tile_lds + 512 * chunk), 16, 0, 0);
  };
  auto fetch = [&](int t, bf16_t* Kb, bf16_t* Vb) {
    const int k0 = k_begin + t * PF_BN;
    const bool all = whole(t);
#pragma unroll
    for (int i = 0; i < NCHK; ++i) {
      if (all || pgk[i] >= 0) {
        const uint32_t in_page = (uint32_t)((key_at(k0 + crowk[i]) & page_mask) * DK + ccolk[i]) * 2;
        to_lds(k_head, (uint64_t)(uint32_t)pgk[i] * page_bytes_k + in_page, Kb, wave_u * NCHK + i);
      } else {                                    // rows outside the keys read as zeros
        *reinterpret_cast<uint4*>(Kb + 8 * (64 * (wave_u * NCHK + i) + lane)) = make_uint4(0, 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < NCHV; ++i) {
      if (all || pgv[i] >= 0) {
        const uint32_t in_page = (uint32_t)((key_at(k0 + crowv[i]) & page_mask) * DV + ccolv[i]) * 2;
        to_lds(v_head, (uint64_t)(uint32_t)pgv[i] * page_bytes_v + in_page, Vb, wave_u * NCHV + i);
      } else {
        *reinterpret_cast<uint4*>(Vb + 8 * (64 * (wave_u * NCHV + i) + lane)) = make_uint4(0, 0, 0, 0);
      }
    }
  };
  // where this lane reads: the first product takes row 16 kt + ln, chunk 4 kk + lg; the second
  // points at row 32 half + 16 j + 4 lg + ln / 4, elements 16 dt + 4 (ln % 4) .. +3
  int k_at[NDK], v_at[2 * NDV];
  {
    const int sw = swzk(ln);
#pragma unroll
    for (int kk = 0; kk < NDK; ++kk) k_at[kk] = ln * DK + 8 * ((4 * kk + lg) ^ sw);
    const int vrow = 4 * lg + (ln >> 2);
    const int vsw = swzv(vrow);
#pragma unroll
    for (int dt = 0; dt < 2 * NDV; ++dt)
      v_at[dt] = vrow * DV + 8 * ((2 * dt + ((ln & 3) >> 1)) ^ vsw) + 4 * (ln & 1);
  }

  // one key tile for this wave's rows; MASKED: the tile touches the diagonal, the end of the
  // keys or a window's edge
  auto tile = [&](int k0, const bf16_t* Kb, const bf16_t* Vb, auto masked_tag) {
    constexpr bool MASKED = decltype(masked_tag)::value;
    f32x4_t st[RT][4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
      for (int r = 0; r < RT; ++r) st[r][kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NDK; ++kk) {
        Frag8 a;
        a.u = *reinterpret_cast<const uint4*>(Kb + 16 * kt * DK + k_at[kk]);
#pragma unroll
        for (int r = 0; r < RT; ++r)
          st[r][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, qf[r][kk].v, st[r][kt], 0, 0, 0);
      }
    }
    Frag8 pb[RT][2];
#pragma unroll
    for (int r = 0; r < RT; ++r) {
      if (CAP) {
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int i = 0; i < 4; ++i) st[r][kt][i] = tanh_exp2(st[r][kt][i] * cap_in);
      }
      if (MASKED) {
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int kw = k0 + 16 * kt + 4 * lg + i;
            const bool vis = kw <= qw[r] && kw < k_end &&
                             (kw >= lo[r] || (KEPT && kw < keep_lim));
            st[r][kt][i] = vis ? st[r][kt][i] : -INFINITY;
          }
      }
      // the running max is kept in units of the raw scores; scale * log2(e) enters in the
      // exponent's multiply-add
      float tm[4];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
        tm[kt] = max2(max2(st[r][kt][0], st[r][kt][1]), max2(st[r][kt][2], st[r][kt][3]));
      float tmax = max2(max2(tm[0], tm[1]), max2(tm[2], tm[3]));
      tmax = max_with_lane_xor16(tmax);
      tmax = max_with_lane_xor32(tmax);
      // the maximum moved far enough for this lane's row: rescale what is kept. (A branch per
      // lane, not per wave: the lanes that skip it keep their registers, so nothing is copied
      // where it joins.)
      if (tmax > m_run[r] + lazy) {
        const float alpha = __builtin_amdgcn_exp2f((m_run[r] - tmax) * scale_log2);
        m_run[r] = tmax;
#pragma unroll
        for (int t = 0; t <= 2 * NDV; ++t) {
          o[r][t][0] *= alpha; o[r][t][1] *= alpha; o[r][t][2] *= alpha; o[r][t][3] *= alpha;
        }
      }
      // (a row that has seen no key yet and sees none in this tile: all its scores are -inf)
      const float mc = (MASKED && m_run[r] == -INFINITY) ? 0.f : -m_run[r] * scale_log2;
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float p = __builtin_amdgcn_exp2f(fmaf(st[r][2 * half + t][i], scale_log2, mc));
            pb[r][half].v[4 * t + i] = (__bf16)p;
          }
    }
    // V^T fragments: lane (ln, lg) points at V[key0 + ln/4][16 dt + 4 (ln%4)] and receives
    // V[key0 + 0..3][16 dt + ln], key0 = 32 half + 16 t + 4 lg: the keys of P^T's element 4 t + i
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int dt = 0; dt < 2 * NDV; ++dt) {
        Frag8 a;
        a.s[0] = lds_read_tr16(Vb + (32 * half) * DV + v_at[dt]);
        a.s[1] = lds_read_tr16(Vb + (32 * half + 16) * DV + v_at[dt]);
#pragma unroll
        for (int r = 0; r < RT; ++r)
          o[r][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, pb[r][half].v, o[r][dt], 0, 0, 0);
      }
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int r = 0; r < RT; ++r)
        o[r][2 * NDV] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones.v, pb[r][half].v, o[r][2 * NDV], 0, 0, 0);
  };

  // one turn: tile t + 1 sets out for the other buffer (everyone left it before the last
  // barrier), tile t is used, and what was loaded is waited for before the barrier
  auto turn = [&](int t, bf16_t* Kb, bf16_t* Vb, bf16_t* Kn, bf16_t* Vn) {
    const int k0 = k_begin + t * PF_BN;
    if (t + 1 < n_tiles) {
      fetch(t + 1, Kn, Vn);
      load_pages(t + 2);
    }
    // a wave whose rows all lie before this tile has nothing to do in it
    if (wave_has_rows && k0 <= wave_max_q - shift && (KEPT || k0 + PF_BN > wave_lo_first)) {
      const bool need_mask = (k0 + PF_BN - 1 > wave_min_q - shift) || (k0 + PF_BN > k_end) || k0 < wave_lo_last;
      if (need_mask)
        tile(k0, Kb, Vb, std::true_type{});
      else
        tile(k0, Kb, Vb, std::false_type{});
    }
    __builtin_amdgcn_s_waitcnt(0x0F70);      // vmcnt(0): this wave's loads into LDS have landed
    __syncthreads();
  };
  load_pages(0);
  fetch(0, Ks0, Vs0);
  load_pages(1);
  __builtin_amdgcn_s_waitcnt(0x0F70);
  __syncthreads();
  for (int t = 0; t < n_tiles; t += 2) {
    turn(t, Ks0, Vs0, Ks1, Vs1);
    if (t + 1 < n_tiles) turn(t + 1, Ks1, Vs1, Ks0, Vs0);
  }

#pragma unroll
  for (int r = 0; r < RT; ++r) {
    float l = o[r][2 * NDV][0];                // every row of that tile holds the column's sum
    // one more term of the denominator: exp(sink), in the units of what was summed
    if (ex.sink) l += __builtin_amdgcn_exp2f(ex.sink[head] * 1.4426950408889634f - m_run[r] * scale_log2);
    if (row_ok[r]) {
      const int my_row = 16 * (RT * wave + r) + ln;
      const float inv = l > 0.f ? head_gate(ex, qs + qoff + my_row, head) / l : 0.f;
      TO* op = out + (size_t)(qs + qoff + my_row) * out_stride + (size_t)head * DV + 4 * lg;
#pragma unroll
      for (int dt = 0; dt < 2 * NDV; ++dt) {
        float rr[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) rr[i] = o[r][dt][i] * inv;
        store4<TO>(op + 16 * dt, rr);
      }
    }
  }
  }   // work items
}

template <int NDK, int NDV, int RT, typename TO>
static int launch_prefill_mfma(void* out, long out_stride, const void* q, long q_stride,
                               const void* k_cache, const void* v_cache, const int32_t* q_start,
                               const int32_t* ctx_len, const int32_t* block_table, int bt_stride,
                               const int32_t* work_seq, const int32_t* work_qoff, int n_work,
                               int n_groups, int Hq, int Hkv, int maps, int page_size, const AttnExtras& ex,
                               float scale, hipStream_t stream) {
  dim3 grid(Hq, n_groups < 65535 ? n_groups : 65535);
  int page_shift = -1;
  for (int sh = 0; sh < 31; ++sh)
    if ((1 << sh) == page_size) page_shift = sh;
  const bool kept = ex.window > 0 && ex.keep_first > 0, cap = ex.softcap > 0.f;
  if (kept && cap) return PTL_ERR_ARG;
  const float log2e = 1.4426950408889634f;
  const float scale_log2 = (cap ? ex.softcap : scale) * log2e, cap_in = cap ? 2.0f * log2e * scale / ex.softcap : 0.f;
#define GO(KEPT, CAP)                                                                                       \
  attn_prefill_mfma_kernel<NDK, NDV, RT, TO, KEPT, CAP><<<grid, 256, 0, stream>>>(                          \
      (TO*)out, out_stride, (const bf16_t*)q, q_stride, (const bf16_t*)k_cache, (const bf16_t*)v_cache,     \
      q_start, ctx_len, block_table, bt_stride, work_seq, work_qoff, n_work, Hq, Hkv, maps, page_size,      \
      page_shift, ex, scale_log2, cap_in)
  if (kept) GO(true, false);
  else if (cap) GO(false, true);
  else GO(false, false);
#undef GO
  return ptl_launch_status();
}

// Keys and values of one size, one score map a head, bfloat16 result: the sizes every model
// with ordinary heads brings.
template <int RT>
static int prefill_same_size(int nd, void* out, long out_stride, const void* q, long q_stride,
                             const void* k_cache, const void* v_cache, const int32_t* q_start,
                             const int32_t* ctx_len, const int32_t* block_table, int bt_stride,
                             const int32_t* work_seq, const int32_t* work_qoff, int n_work, int n_groups,
                             int Hq, int Hkv, int page_size, const AttnExtras& ex, float scale,
                             hipStream_t stream) {
#define GO(N) launch_prefill_mfma<N, N, RT, bf16_t>(out, out_stride, q, q_stride, k_cache, v_cache, q_start, \
                                                    ctx_len, block_table, bt_stride, work_seq, work_qoff,  \
                                                    n_work, n_groups, Hq, Hkv, 1, page_size, ex, scale,  \
                                                    stream)
  switch (nd) {
    case 1: return GO(1);
    case 2: return GO(2);
    case 3: return GO(3);
    default: return GO(4);
  }
#undef GO
}

// work_seq / work_qoff list query blocks of ``block_rows`` rows (64 or 128), the longest first;
// n_groups workgroups a head share them (1 <= n_groups <= n_work). bfloat16 only;
// q rows must be 16-byte aligned and output rows 8-byte (q_stride % 8, out_stride % 4); the
// page size is a power of two and a page of all kv heads is smaller than 4 GiB.
extern "C" int ptl_attention_prefill_mfma(void* out, long out_stride, const void* q, long q_stride,
                                          const void* k_cache, const void* v_cache,
                                          const int32_t* q_start, const int32_t* ctx_len,
                                          const int32_t* block_table, int bt_stride,
                                          const int32_t* work_seq, const int32_t* work_qoff,
                                          int n_work, int n_groups, int block_rows, int Hq,
                                          int Hkv, int D,
                                          int page_size, int window, int keep_first, int chunk,
                                          const float* sink, const float* gate, long gate_stride,
                                          float softcap, float scale, hipStream_t stream) {
  if (n_work <= 0) return PTL_OK;
  const AttnExtras ex{window, keep_first, chunk, sink, gate, gate_stride, softcap};
  if (Hq <= 0 || Hkv <= 0 || Hq % Hkv || D % 32 || D <= 0 || D > 128 || page_size <= 0 ||
      (page_size & (page_size - 1)) || (long)Hkv * page_size * D * 2 >= (1L << 32) ||
      Hq > 65535 || n_groups < 1 || n_groups > n_work || q_stride % 8 || out_stride % 4 ||
      (block_rows != 64 && block_rows != 128) || !extras_ok(ex))
    return PTL_ERR_ARG;
  if (block_rows == 64)
    return prefill_same_size<1>(D / 32, out, out_stride, q, q_stride, k_cache, v_cache, q_start, ctx_len,
                                block_table, bt_stride, work_seq, work_qoff, n_work, n_groups, Hq, Hkv,
                                page_size, ex, scale, stream);
  return prefill_same_size<2>(D / 32, out, out_stride, q, q_stride, k_cache, v_cache, q_start, ctx_len,
                              block_table, bt_stride, work_seq, work_qoff, n_work, n_groups, Hq, Hkv,
                              page_size, ex, scale, stream);
}

// The general form: q [T, Hq, Dk] with Hq = heads * maps, k_cache [pages, Hkv * maps, page_size,
// Dk], v_cache [pages, Hkv, page_size, Dv], out [T, Hq, Dv] bfloat16 or (out_f32) float32; Dk and
// Dv multiples of 32 up to 128. 64-row blocks.
extern "C" int ptl_attention_prefill_mfma_kv(void* out, long out_stride, int out_f32, const void* q,
                                             long q_stride, const void* k_cache, const void* v_cache,
                                             const int32_t* q_start, const int32_t* ctx_len,
                                             const int32_t* block_table, int bt_stride,
                                             const int32_t* work_seq, const int32_t* work_qoff,
                                             int n_work, int n_groups, int Hq, int Hkv, int maps, int Dk,
                                             int Dv, int page_size, int window, int keep_first, int chunk,
                                             const float* sink, const float* gate, long gate_stride,
                                             float softcap, float scale, hipStream_t stream) {
  if (n_work <= 0) return PTL_OK;
  const AttnExtras ex{window, keep_first, chunk, sink, gate, gate_stride, softcap};
  if (Hq <= 0 || Hkv <= 0 || maps <= 0 || Hq % maps || (Hq / maps) % Hkv || Dk % 32 || Dk <= 0 ||
      Dk > 128 || Dv % 32 || Dv <= 0 || Dv > 128 || page_size <= 0 || (page_size & (page_size - 1)) ||
      (long)Hkv * maps * page_size * Dk * 2 >= (1L << 32) || (long)Hkv * page_size * Dv * 2 >= (1L << 32) ||
      Hq > 65535 || n_groups < 1 || n_groups > n_work || q_stride % 8 || out_stride % 4 || !extras_ok(ex))
    return PTL_ERR_ARG;
#define GO(NK, NV, TO)                                                                                  \
  launch_prefill_mfma<NK, NV, 1, TO>(out, out_stride, q, q_stride, k_cache, v_cache, q_start, ctx_len, \
                                     block_table, bt_stride, work_seq, work_qoff, n_work, n_groups, Hq, \
                                     Hkv, maps, page_size, ex, scale, stream)
#define BY_V(NK, TO)                   \
  switch (Dv / 32) {                   \
    case 1: return GO(NK, 1, TO);      \
    case 2: return GO(NK, 2, TO);      \
    case 3: return GO(NK, 3, TO);      \
    default: return GO(NK, 4, TO);     \
  }
#define BY_K(TO)                       \
  switch (Dk / 32) {                   \
    case 1: BY_V(1, TO)                \
    case 2: BY_V(2, TO)                \
    case 3: BY_V(3, TO)                \
    default: BY_V(4, TO)               \
  }
  if (out_f32) { BY_K(float) }
  BY_K(bf16_t)
#undef BY_K
#undef BY_V
#undef GO
}
