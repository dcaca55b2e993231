// Kernels of mixers that carry a fixed-size state from token to token instead of a paged cache:
// token shift (fused with the RMSNorm in front of it), the linear recurrence with a matrix state per
// head (gated linear attention with a decay per key channel, and the mLSTM with scalar gates, a
// normaliser and a running maximum), the per-head RMS norm with an output gate behind it, and the
// gated unit of a feed-forward with a choice of activation.
//
// Everything here is 32-bit arithmetic whatever the mode: the state, the gates, their logarithms and
// exponentials, the norms.  The mode only decides the dtype of what is handed to the next matrix product.
//
// A step's rows of one request are consecutive and in position order; ``seq_rows`` holds for every
// request of the step (first row, number of rows) and ``slots`` its state slot.  A request with no rows,
// a negative slot or a negative first position is padding and is skipped: its state is not touched.
#include "common.h"
#include "api.h"

#include <math.h>

#include <type_traits>

namespace {

__device__ __forceinline__ float log_sigmoid(float z) {
  // log(1 / (1 + e^-z)) = min(z, 0) - log1p(e^-|z|)
  return fminf(z, 0.0f) - log1pf(bw_expf(-fabsf(z)));
}

__device__ __forceinline__ float softplus(float z) {
  // log(1 + e^z) = max(z, 0) + log1p(e^-|z|)
  return fmaxf(z, 0.0f) + log1pf(bw_expf(-fabsf(z)));
}

__device__ __forceinline__ float silu(float z) { return z * (1.0f / (1.0f + bw_expf(-z))); }

template <typename OT>
__device__ __forceinline__ void store_act(OT* p, float v) {
  if constexpr (sizeof(OT) == 2) *p = f32_to_bf16(v);
  else *p = v;
}

// Sum of squares of a row: lane l runs one fused multiply-add chain over elements l, l+64, ... in ascending order,
// the lanes are joined by the butterflies of wave_sum.  The order depends on the width alone.
__device__ __forceinline__ float row_sumsq(const float* __restrict__ xr, int dim, int lane) {
  float acc = 0.0f;
  for (int i = lane; i < dim; i += 64) acc = fmaf(xr[i], xr[i], acc);
  return wave_sum(acc);
}

// ------------------------------------------------------------------------- RMSNorm + token shift

// out[r][m] = h[r] + (h'[r] - h[r]) * mix[m] for each of nmix mixing vectors (out rows hold nmix blocks of dim elements), with
// h = (x * inv_rms) * w and h' the h of the request's previous token: the
// row above, or for the first row of a request in this step what the state slot holds (zeros for a new request).
// The wave of a request's first row also leaves the h of the request's last row in the slot, after it has read it:
// nothing else reads or writes that slot in this launch.  A wave a row.
template <typename OT>
__global__ __launch_bounds__(256) void norm_shift_kernel(const float* __restrict__ x, int ldx, const float* __restrict__ w,
                                                         const float* __restrict__ mix, float* __restrict__ state,
                                                         long long state_ld, const int32_t* __restrict__ positions,
                                                         const int32_t* __restrict__ row_seq,
                                                         const int32_t* __restrict__ seq_rows,
                                                         const int32_t* __restrict__ slots, OT* __restrict__ out, int ldo,
                                                         int rows, int dim, float eps, int nmix) {
  const int lane = threadIdx.x & 63;
  const int row = blockIdx.x * (blockDim.x >> 6) + wave_index();
  if (row >= rows) return;
  if (positions[row] < 0) return;
  const int seq = row_seq[row];
  const int first = seq_rows[2 * seq], count = seq_rows[2 * seq + 1];
  const int slot = slots[seq];
  if (slot < 0 || count <= 0) return;
  const float* xr = x + (size_t)row * ldx;
  float* st = state + (size_t)slot * state_ld;
  OT* o = out + (size_t)row * ldo;
  if ((dim & 3) == 0 && (ldx & 3) == 0 && (ldo & 3) == 0 && (state_ld & 3) == 0) {
    // rows of whole 16-byte vectors: lane l owns vectors l, l+64, ...; four of them (and of everything that goes with them) are
    // asked for before the first is used
    const int nvec = dim >> 2;
    const bool is_first = row == first;
    const int last = first + count - 1;
    const f32x4* xv = reinterpret_cast<const f32x4*>(xr);
    const f32x4* pv = is_first ? reinterpret_cast<const f32x4*>(st) : reinterpret_cast<const f32x4*>(xr - ldx);
    const f32x4* lv = reinterpret_cast<const f32x4*>(x + (size_t)last * ldx);
    const f32x4* wv = reinterpret_cast<const f32x4*>(w);
    const f32x4* mv = reinterpret_cast<const f32x4*>(mix);
    const float inv = 1.0f / sqrtf(row_sumsq_vec(xv, nvec, lane) / (float)dim + eps);
    const float invp = is_first ? 1.0f : 1.0f / sqrtf(row_sumsq_vec(pv, nvec, lane) / (float)dim + eps);
    const float invl = !is_first || last == row ? inv : 1.0f / sqrtf(row_sumsq_vec(lv, nvec, lane) / (float)dim + eps);
    constexpr int UN = 4;
    for (int c0 = 0; c0 < nvec; c0 += 64 * UN) {
      f32x4 xq[UN], pq[UN], lq[UN], wq[UN], mq[UN];
#pragma unroll
      for (int jj = 0; jj < UN; ++jj) {
        const int c = min(c0 + 64 * jj + lane, nvec - 1);
        xq[jj] = xv[c];
        pq[jj] = pv[c];
        wq[jj] = wv[c];
        mq[jj] = mv[c];
        lq[jj] = is_first ? lv[c] : xq[jj];
      }
#pragma unroll
      for (int jj = 0; jj < UN; ++jj) {
        const int c = c0 + 64 * jj + lane;
        if (c >= nvec) continue;
        f32x4 hq, dq, keep;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          hq[e] = (xq[jj][e] * inv) * wq[jj][e];
          const float hp = is_first ? pq[jj][e] : (pq[jj][e] * invp) * wq[jj][e];
          dq[e] = hp - hq[e];
          keep[e] = (lq[jj][e] * invl) * wq[jj][e];
        }
        // (the further mixing vectors four at a time: their loads are all asked for before the first is used)
        for (int m0 = 0; m0 < nmix; m0 += 4) {
          f32x4 mm[4];
#pragma unroll
          for (int k = 0; k < 4; ++k) mm[k] = m0 + k == 0 ? mq[jj] : mv[(size_t)min(m0 + k, nmix - 1) * nvec + c];
#pragma unroll
          for (int k = 0; k < 4; ++k) {
            if (m0 + k >= nmix) continue;
            f32x4 r;
#pragma unroll
            for (int e = 0; e < 4; ++e) r[e] = fmaf(dq[e], mm[k][e], hq[e]);
            OT* om = o + (size_t)(m0 + k) * dim;
            if constexpr (sizeof(OT) == 2) {
              *reinterpret_cast<u32x2*>(om + 4 * c) = (u32x2){pack_bf16x2(r[0], r[1]), pack_bf16x2(r[2], r[3])};
            } else {
              *reinterpret_cast<f32x4*>(om + 4 * c) = r;
            }
          }
        }
        if (is_first) reinterpret_cast<f32x4*>(st)[c] = keep;
      }
    }
    return;
  }
  const float inv = 1.0f / sqrtf(row_sumsq(xr, dim, lane) / (float)dim + eps);
  if (row != first) {
    const float* xp = xr - ldx;
    const float invp = 1.0f / sqrtf(row_sumsq(xp, dim, lane) / (float)dim + eps);
    for (int i = lane; i < dim; i += 64) {
      const float h = (xr[i] * inv) * w[i];
      const float hp = (xp[i] * invp) * w[i];
      for (int m = 0; m < nmix; ++m) store_act(o + (size_t)m * dim + i, fmaf(hp - h, mix[(size_t)m * dim + i], h));
    }
    return;
  }
  const int last = first + count - 1;
  const float* xl = x + (size_t)last * ldx;
  const float invl = last == row ? inv : 1.0f / sqrtf(row_sumsq(xl, dim, lane) / (float)dim + eps);
  for (int i = lane; i < dim; i += 64) {
    const float h = (xr[i] * inv) * w[i];
    const float hp = st[i];
    for (int m = 0; m < nmix; ++m) store_act(o + (size_t)m * dim + i, fmaf(hp - h, mix[(size_t)m * dim + i], h));
    st[i] = (xl[i] * invl) * w[i];
  }
}

// The same for steps of few rows, a workgroup a row: all of a row's operands (the row, the row before or the slot's, the
// request's last row, the weight and up to eight mixing vectors) are asked for at once, the rows pass through LDS, and a
// wave each runs row_sumsq_vec over them from there: the chains, and so the bits, of the kernel above.  Rows of whole
// 16-byte vectors, up to 4,096 elements.
#define SHIFT_ROW_MAXV 4
#define SHIFT_ROW_MAXMIX 8
template <typename OT>
__global__ __launch_bounds__(256) void norm_shift_row_kernel(const float* __restrict__ x, int ldx, const float* __restrict__ w,
                                                             const float* __restrict__ mix, float* __restrict__ state,
                                                             long long state_ld, const int32_t* __restrict__ positions,
                                                             const int32_t* __restrict__ row_seq,
                                                             const int32_t* __restrict__ seq_rows,
                                                             const int32_t* __restrict__ slots, OT* __restrict__ out, int ldo,
                                                             int rows, int dim, float eps, int nmix) {
  extern __shared__ float shift_lds[];            // three rows of dim elements, then three numbers
  const int row = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  if (positions[row] < 0) return;
  const int seq = row_seq[row];
  const int first = seq_rows[2 * seq], count = seq_rows[2 * seq + 1];
  const int slot = slots[seq];
  if (slot < 0 || count <= 0) return;
  const float* xr = x + (size_t)row * ldx;
  float* st = state + (size_t)slot * state_ld;
  OT* o = out + (size_t)row * ldo;
  const int nvec = dim >> 2;
  const bool is_first = row == first;
  const int last = first + count - 1;
  const bool need_p = !is_first, need_l = is_first && last != row;
  const f32x4* xv = reinterpret_cast<const f32x4*>(xr);
  const f32x4* pv = is_first ? reinterpret_cast<const f32x4*>(st) : reinterpret_cast<const f32x4*>(xr - ldx);
  const f32x4* lv = reinterpret_cast<const f32x4*>(x + (size_t)last * ldx);
  const f32x4* wvp = reinterpret_cast<const f32x4*>(w);
  const f32x4* mv = reinterpret_cast<const f32x4*>(mix);
  f32x4* sx = reinterpret_cast<f32x4*>(shift_lds);
  f32x4* sp = sx + nvec;
  f32x4* sl = sp + nvec;
  float* invs = reinterpret_cast<float*>(sl + nvec);
  f32x4 xq[SHIFT_ROW_MAXV], pq[SHIFT_ROW_MAXV], lq[SHIFT_ROW_MAXV], wq[SHIFT_ROW_MAXV], mm[SHIFT_ROW_MAXV][SHIFT_ROW_MAXMIX];
#pragma unroll
  for (int j = 0; j < SHIFT_ROW_MAXV; ++j) {
    const int c = min(tid + 256 * j, nvec - 1);
    xq[j] = xv[c];
    pq[j] = pv[c];
    wq[j] = wvp[c];
    lq[j] = need_l ? lv[c] : xq[j];
#pragma unroll
    for (int m = 0; m < SHIFT_ROW_MAXMIX; ++m) mm[j][m] = mv[(size_t)min(m, nmix - 1) * nvec + c];
  }
#pragma unroll
  for (int j = 0; j < SHIFT_ROW_MAXV; ++j) {
    const int c = tid + 256 * j;
    if (c < nvec) {
      sx[c] = xq[j];
      if (need_p) sp[c] = pq[j];
      if (need_l) sl[c] = lq[j];
    }
  }
  __syncthreads();
  if (wv == 0 || (wv == 1 && need_p) || (wv == 2 && need_l)) {
    const float ss = row_sumsq_vec(wv == 0 ? sx : (wv == 1 ? sp : sl), nvec, lane);
    if (lane == 0) invs[wv] = 1.0f / sqrtf(ss / (float)dim + eps);
  }
  __syncthreads();
  const float inv = invs[0];
  const float invp = need_p ? invs[1] : 1.0f;
  const float invl = need_l ? invs[2] : inv;
#pragma unroll
  for (int j = 0; j < SHIFT_ROW_MAXV; ++j) {
    const int c = tid + 256 * j;
    if (c >= nvec) continue;
    f32x4 hq, dq, keep;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      hq[e] = (xq[j][e] * inv) * wq[j][e];
      const float hp = is_first ? pq[j][e] : (pq[j][e] * invp) * wq[j][e];
      dq[e] = hp - hq[e];
      keep[e] = (lq[j][e] * invl) * wq[j][e];
    }
#pragma unroll
    for (int m = 0; m < SHIFT_ROW_MAXMIX; ++m) {
      if (m >= nmix) continue;
      f32x4 r;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = fmaf(dq[e], mm[j][m][e], hq[e]);
      OT* om = o + (size_t)m * dim;
      if constexpr (sizeof(OT) == 2) {
        *reinterpret_cast<u32x2*>(om + 4 * c) = (u32x2){pack_bf16x2(r[0], r[1]), pack_bf16x2(r[2], r[3])};
      } else {
        *reinterpret_cast<f32x4*>(om + 4 * c) = r;
      }
    }
    if (is_first) reinterpret_cast<f32x4*>(st)[c] = keep;
  }
}

// ------------------------------------------------------------------------- the linear recurrence

enum { RECUR_DECAY_PER_CHANNEL = 0, RECUR_SCALAR_GATES = 1, RECUR_BONUS_DECAY = 2, RECUR_FIXED_DECAY = 3, RECUR_STEP_DECAY = 4, RECUR_DELTA = 5 };

// The sum over the SPLIT neighbouring lanes that hold the parts of one column (every one of them gets it): an addition a
// stage whose second operand comes through a data-parallel move within a row of 16 lanes.  Behind the first two stages the
// lanes of a quad hold the same value, so the mirror images of 8 and of 16 lanes fetch the other half's.
template <int SPLIT>
__device__ __forceinline__ float join_parts(float v) {
  static_assert(SPLIT <= 16, "a column's parts lie within a row of 16 lanes");
  if constexpr (SPLIT >= 2) v += lane_xor<1>(v);
  if constexpr (SPLIT >= 4) v += lane_xor<2>(v);
  if constexpr (SPLIT >= 8) v += __uint_as_float((unsigned)__builtin_amdgcn_mov_dpp((int)__float_as_uint(v), 0x141, 0xf, 0xf, true));      // row_half_mirror
  if constexpr (SPLIT >= 16) v += __uint_as_float((unsigned)__builtin_amdgcn_mov_dpp((int)__float_as_uint(v), 0x140, 0xf, 0xf, true));     // row_mirror
  return v;
}

struct RecurArgs {
  const float* proj;       // [rows, ldp]: the rows' stacked projections
  int ldp, q_off, k_off, v_off;
  const float* gate;       // per channel: decay logits [rows, ldg] at gate_off + head*dim + d;
  int ldg, gate_off, gate2_off;   // scalar gates: input gate at gate_off + head, forget gate at gate2_off + head
  const float* bias;       // per channel: [heads*dim]; scalar gates: input-gate bias [heads]; step: bias of the step size [heads]
  const float* bias2;      // scalar gates: forget-gate bias [heads]; step: the decay's rate [heads]
  const float* skip;       // step: [heads], the weight of the token's own v in the read-out (null: none)
  int heads_per_key;       // neighbouring heads that share one q and one k (1: every head has its own)
  float param;             // per channel: 1 / tau; scalar gates: the cap
  float qscale, kscale;
  int silu;                // fixed decay: q, k and v pass SiLU on their way into LDS
  float* state;            // [slots, state_ld]: S [heads][vdim][dim]; scalar gates then, per
                           // workgroup of a head, n [heads][dim] and m [heads]
  long long state_ld;
  float* out;              // [rows, ldo]: head h at columns h*vdim ..
  int ldo;
  const int32_t* seq_rows;
  const int32_t* slots;
  const int32_t* positions;
  int heads, dim, vdim;
  // long prompt portions in three passes (PHASE 1 to 3): chunks [n][4] = (first row, rows, request of the step, 1 if it is
  // the request's last chunk); heads records of recur_record floats per chunk
  const int32_t* chunks;
  float* local;            // per chunk, from zero state: S [vdim][dim], and the decay over the chunk (per channel: the product of the
                           // decays; scalar gates: n, the maximum from -inf, the sum of the log forget gates)
  float* start;            // per chunk: the state it starts from (S; scalar gates: n, m)
};

// A wave holds the state of 64 / SPLIT value columns of one head in registers: SPLIT lanes a column, each with DH
// key channels, so that a head has many short waves; the parts' read-outs are added by lane exchanges in one order whatever
// runs the head (a single token, a portion, a chunk): the split depends on the head's size alone.  The tokens' q, k, decays
// and v come through LDS in chunks of a few tokens, shared by the workgroup's waves (neighbouring column blocks of one head);
// the next chunk is on its way from memory while one is worked on.  In memory a column's channels lie side by side,
// [column][channel], so a lane's part is a run of whole vectors.
//
// RECUR_DECAY_PER_CHANNEL:  S[d][j] <- alpha[d] S[d][j] + k[d] v[j],  alpha = exp(logsigmoid(z + bias) / tau);  o[j] = sum_d S[d][j] q[d].
// RECUR_SCALAR_GATES:  i = cap tanh((gi + bi) / cap), f = logsigmoid(cap tanh((gf + bf) / cap)), m' = max(f + m, i),
//   S <- e^(f + m - m') S + e^(i - m') k v^T, n likewise with k alone, o[j] = (S^T q)[j] / (max(|n.q|, e^-m') + 1e-6).
//   n is spread over the lanes (lane l holds n[l], n[l+64], ...); every wave of a head computes it, the wave of
//   column block 0 stores it.
//
// RECUR_BONUS_DECAY:  alpha[d] = exp(-exp(z[d] + bias[d]));  o[j] = sum_d (S[d][j] + u[d] k[d] v[j]) q[d] with the S of the token
//   before (the token's own k v^T is read through the bonus u = bias2 [heads*dim]), then S[d][j] <- alpha[d] S[d][j] + k[d] v[j].
// RECUR_FIXED_DECAY:  as per channel with one constant decay a head, alpha[d] = bias[head]; no logits are read.
// RECUR_STEP_DECAY:  a step size per head and token, delta = softplus(z + bias[head]) with z at gate_off + head;
//   S[d][j] <- e^(-bias2[head] delta) S[d][j] + k[d] (delta v[j]),  o[j] = (S^T q)[j] + skip[head] v[j].
// RECUR_DELTA:  a step size beta (at gate_off + head) and a decay a (at gate2_off + head) per head and token;
//   u[j] = beta (v[j] - a (S^T k)[j]),  S[d][j] <- a S[d][j] + k[d] u[j],  o[j] = (S^T q)[j]: what k reads is replaced towards v.
//   The read-out is formed from the memory before the write, o = a (S^T q) + (k.q) u, so that only S^T k stands between a token
//   and the next; k.q comes with the gates (at gate2_off + heads + key group).
//   (The step of a chunk as a whole is a full matrix and not a decay, so there are no passes over chunks.)
// (a head's q and k are those of key group head / heads_per_key.)
// (q is multiplied by qscale and k by kscale on their way into LDS.)
//
// A request's long portion can also run in three passes over chunks of its rows, which gives every chunk waves of its
// own: PHASE 1 runs every chunk from a zero state (no read-out) and leaves the chunk's own contribution and its decay;
// recurrence_scan_kernel walks a request's chunks in order and leaves the state each one starts from; PHASE 3 runs every
// chunk from there with the read-out, and the request's last chunk leaves the state in the slot.  PHASE 0 walks
// the whole portion; PHASE 4 does so for steps of a few tokens a request (decoding), where what counts is how many waves are
// on the chip with their states' loads under way: no groups of tokens, no second buffer, few registers, the same arithmetic.  The passes differ from PHASE 0 by the rounding of the scan's sums only.
#define RW 4             // waves of a workgroup
// floats of a chunk's record for one head: S, a vector, two scalars, in whole vectors of four
__host__ __device__ __forceinline__ size_t recur_record(int dim, int vdim) { return ((size_t)dim * vdim + dim + 2 + 3) & ~(size_t)3; }

// Lanes a column.  A portion walked whole (and a single token) gets many short waves; the passes over chunks have waves
// enough and keep more of a column in a lane, which reads less through LDS for every multiply-add.
__host__ __device__ constexpr int recur_split(int dpad) { return dpad >= 128 ? 16 : dpad / 8; }
__host__ __device__ constexpr int recur_chunk_split(int dpad) { return dpad >= 64 ? 4 : (dpad >= 32 ? 2 : 1); }
// value columns of a workgroup, and how many workgroups share a head
__host__ __device__ constexpr int recur_columns(int dim, bool chunks) {
  const int dpad = dim <= 16 ? 16 : (dim <= 32 ? 32 : (dim <= 64 ? 64 : 128));
  return RW * 64 / (chunks ? recur_chunk_split(dpad) : recur_split(dpad));
}
__host__ __device__ constexpr int recur_blocks(int dim, int vdim, bool chunks = false) {
  return (vdim + recur_columns(dim, chunks) - 1) / recur_columns(dim, chunks);
}

// What a lane needs of N tokens.
template <int TOKENS, int DH, bool CHANNELS>
struct RecurOps {
  static constexpr int N = TOKENS;
  float k[N][DH], q[N][DH], a[CHANNELS ? N : 1][CHANNELS ? DH : 1], v[N], g1[N], g2[N], kq[N];
};

template <int MODE, int DPAD, int PHASE>
__global__ __launch_bounds__(64 * RW) void linear_recurrence_kernel(RecurArgs a) {
  constexpr bool GATES = MODE == RECUR_SCALAR_GATES;
  constexpr bool BONUS = MODE == RECUR_BONUS_DECAY, FIXED = MODE == RECUR_FIXED_DECAY, STEP = MODE == RECUR_STEP_DECAY;
  constexpr bool DELTA = MODE == RECUR_DELTA;
  constexpr bool CHANNELS = !GATES && !STEP && !DELTA && !FIXED;   // a decay per channel comes through LDS
  constexpr int NN = (DPAD + 63) / 64;
  constexpr bool READ_OUT = PHASE != 1;
  constexpr bool WALK = PHASE == 0 || PHASE == 4;
  constexpr int SPLIT = WALK ? recur_split(DPAD) : recur_chunk_split(DPAD);
  constexpr int DH = DPAD / SPLIT, COLS = 64 / SPLIT, WCOLS = RW * COLS;
  constexpr int TU = PHASE != 0 ? 1 : (SPLIT >= 4 && DPAD <= 64 ? 4 : 2);      // tokens of a group (two groups' operands fit the registers, with room for a second wave)
  constexpr int BUFS = PHASE != 0 ? 1 : 2;               // (the passes over chunks hide the loads behind other waves)
  constexpr int RC = PHASE == 4 && DPAD >= 64 ? 4 : (PHASE == 0 && DPAD <= 128 ? 32 : 16);     // tokens staged together
  constexpr int NQ = RC * DPAD / (64 * RW), NV = (RC * WCOLS + 64 * RW - 1) / (64 * RW);
  static_assert(NQ * 64 * RW == RC * DPAD && RC % TU == 0, "a chunk is whole loads and whole groups of tokens");
  __shared__ __attribute__((aligned(16))) float qs[BUFS][RC][DPAD];
  __shared__ __attribute__((aligned(16))) float ks[BUFS][RC][DPAD];
  __shared__ __attribute__((aligned(16))) float as[CHANNELS ? BUFS : 1][CHANNELS ? RC : 1][CHANNELS ? DPAD : 4];
  __shared__ float gi[BUFS][RC], gf[BUFS][RC], gd[DELTA ? BUFS : 1][DELTA ? RC : 1];
  __shared__ float vs[BUFS][RC][WCOLS];
  const int lane = threadIdx.x & 63, wv = wave_index();
  const int h = blockIdx.y;
  const int dim = a.dim, vdim = a.vdim;
  const size_t rec = recur_record(dim, vdim);
  int first, count, slot;
  bool leaves_state = true;
  if constexpr (WALK) {
    const int s = blockIdx.z;
    first = a.seq_rows[2 * s];
    count = a.seq_rows[2 * s + 1];
    slot = a.slots[s];
  } else {
    const int c = blockIdx.z;
    first = a.chunks[4 * c];
    count = a.chunks[4 * c + 1];
    slot = a.slots[a.chunks[4 * c + 2]];
    leaves_state = a.chunks[4 * c + 3] != 0;
  }
  if (count <= 0 || slot < 0) return;
  if (a.positions[first] < 0) return;
  const int col = lane / SPLIT, part = lane % SPLIT;
  // a lane's channels: runs of four, the column's lanes side by side (what they read together lies side by side, too)
  auto channel = [&](int d) { return (d >> 2) * 4 * SPLIT + 4 * part + (d & 3); };
  const int j_wg = blockIdx.x * WCOLS, j_in = wv * COLS + col, j = j_wg + j_in;
  const bool live = j < vdim;
  float* st = a.state + (size_t)slot * a.state_ld;
  float* S = st + (size_t)h * dim * vdim;
  // (every workgroup of a head carries the normaliser and the maximum, so each keeps a copy of its own in the slot: one that
  // starts late must not find what another has already written)
  const size_t copy = (size_t)a.heads * dim + a.heads;
  const size_t own = GATES && WALK ? blockIdx.x * copy : 0;
  float* nv = st + (size_t)a.heads * dim * vdim + own + (size_t)h * dim;
  float* mv = st + (size_t)a.heads * dim * vdim + own + (size_t)a.heads * dim + h;
  // where this wave's state comes from: the slot, nothing, or the chunk's start record
  const float* S_in = S;
  const float* nv_in = nv;
  const float* mv_in = mv;
  if constexpr (PHASE == 3) {
    S_in = a.start + ((size_t)blockIdx.z * a.heads + h) * rec;
    nv_in = S_in + (size_t)dim * vdim;
    mv_in = nv_in + dim;
  }

  float Sreg[DH];
  const bool in_vectors = (dim & 3) == 0 && (reinterpret_cast<uintptr_t>(S_in) & 15) == 0;     // (scalar)
  if (PHASE != 1 && in_vectors) {
    const f32x4* src = reinterpret_cast<const f32x4*>(S_in + (size_t)min(j, vdim - 1) * dim);
#pragma unroll
    for (int d = 0; d < DH; d += 4) {
      const f32x4 v = src[min(channel(d), dim - 4) >> 2];
#pragma unroll
      for (int e = 0; e < 4; ++e) Sreg[d + e] = live && channel(d) < dim ? v[e] : 0.0f;
    }
  } else {
#pragma unroll
    for (int d = 0; d < DH; ++d) Sreg[d] = (PHASE != 1 && live && channel(d) < dim) ? S_in[(size_t)j * dim + channel(d)] : 0.0f;
  }
  float nreg[NN];          // scalar gates: the normaliser; otherwise in PHASE 1: the product of the chunk's decays
  float m = 0.0f, fsum = 0.0f;
  if constexpr (GATES) {
#pragma unroll
    for (int i = 0; i < NN; ++i) nreg[i] = (PHASE != 1 && lane + 64 * i < dim) ? nv_in[lane + 64 * i] : 0.0f;
    m = PHASE == 1 ? -INFINITY : *mv_in;
  } else {
#pragma unroll
    for (int i = 0; i < NN; ++i) nreg[i] = 1.0f;
  }
  float ureg[BONUS ? DH : 1];
  if constexpr (BONUS) {
#pragma unroll
    for (int d = 0; d < DH; ++d) ureg[d] = channel(d) < dim ? a.bias2[h * dim + channel(d)] : 0.0f;
  }
  const float fixed_decay = FIXED ? a.bias[h] : 0.0f;
  const float skip = STEP && a.skip != nullptr ? a.skip[h] : 0.0f;
  const int hk = h / a.heads_per_key;

  // a chunk's operands on their way from memory (every load clamped into its row; what lies outside is zeroed on the way to LDS);
  // q, k and decay logits as 16-byte vectors where the rows allow it: vector u of a thread is elements 4u .. 4u + 3 of its rq
  constexpr bool WIDE = NQ % 4 == 0;
  const bool vectors = WIDE && (dim & 3) == 0 && ((a.q_off | a.k_off | a.ldp) & 3) == 0 && (reinterpret_cast<uintptr_t>(a.proj) & 15) == 0 &&
                       (!CHANNELS || (((a.ldg | a.gate_off) & 3) == 0 && ((reinterpret_cast<uintptr_t>(a.gate) | reinterpret_cast<uintptr_t>(a.bias)) & 15) == 0));   // (scalar)
  float rq[NQ], rk[NQ], rz[CHANNELS ? NQ : 1], rv[NV], rg[3];
  auto fetch = [&](int t0) {
    if (t0 >= count) return;                             // (scalar)
    const int tc = min(RC, count - t0);
    if (vectors) {
#pragma unroll
      for (int u = 0; u < NQ / 4; ++u) {
        if (256 * RW * u < tc * DPAD) {                  // (scalar)
          const int e = 64 * RW * u + (int)threadIdx.x;
          const size_t row = (size_t)(first + t0 + min(e / (DPAD / 4), tc - 1));
          const int d = min(4 * (e % (DPAD / 4)), dim - 4);
          const float* pr = a.proj + row * a.ldp + hk * dim + d;
          const f32x4 q4 = *reinterpret_cast<const f32x4*>(pr + a.q_off), k4 = *reinterpret_cast<const f32x4*>(pr + a.k_off);
          f32x4 z4 = {0.f, 0.f, 0.f, 0.f};
          if constexpr (CHANNELS)
            z4 = *reinterpret_cast<const f32x4*>(a.gate + row * a.ldg + a.gate_off + h * dim + d) + *reinterpret_cast<const f32x4*>(a.bias + h * dim + d);
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            rq[4 * u + x] = q4[x];
            rk[4 * u + x] = k4[x];
            if constexpr (CHANNELS) rz[4 * u + x] = z4[x];
          }
        }
      }
    } else {
#pragma unroll
      for (int u = 0; u < NQ; ++u) {
        if (64 * RW * u < tc * DPAD) {                   // (scalar)
          const int e = 64 * RW * u + (int)threadIdx.x;
          const size_t row = (size_t)(first + t0 + min(e / DPAD, tc - 1));
          const int d = min(e % DPAD, dim - 1);
          const float* pr = a.proj + row * a.ldp;
          rq[u] = pr[a.q_off + hk * dim + d];
          rk[u] = pr[a.k_off + hk * dim + d];
          if constexpr (CHANNELS) rz[u] = a.gate[row * a.ldg + a.gate_off + h * dim + d] + a.bias[h * dim + d];
        }
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      if (64 * RW * u < tc * WCOLS) {
        const int e = 64 * RW * u + (int)threadIdx.x;
        const size_t row = (size_t)(first + t0 + min(e / WCOLS, tc - 1));
        rv[u] = a.proj[row * a.ldp + a.v_off + h * vdim + min(j_wg + e % WCOLS, vdim - 1)];
      }
    }
    if constexpr (GATES || STEP || DELTA) {
      const float* gr = a.gate + (size_t)(first + t0 + min((int)threadIdx.x, tc - 1)) * a.ldg;
      rg[0] = gr[a.gate_off + h];
      rg[1] = GATES || DELTA ? gr[a.gate2_off + h] : 0.0f;
      rg[2] = DELTA ? gr[a.gate2_off + a.heads + hk] : 0.0f;
    }
  };
  auto decay_of = [&](float z) { return BONUS ? bw_expf(-bw_expf(z)) : bw_expf(log_sigmoid(z) * a.param); };
  auto stash = [&](int t0, int buf) {
    if (t0 >= count) return;
    const int tc = min(RC, count - t0);
    if constexpr (FIXED) {
      if (a.silu) {                                      // (scalar)
#pragma unroll
        for (int u = 0; u < NQ; ++u) {
          rq[u] = silu(rq[u]);
          rk[u] = silu(rk[u]);
        }
#pragma unroll
        for (int u = 0; u < NV; ++u) rv[u] = silu(rv[u]);
      }
    }
    if (vectors) {
#pragma unroll
      for (int u = 0; u < NQ / 4; ++u) {
        if (256 * RW * u < tc * DPAD) {
          const int e = 64 * RW * u + (int)threadIdx.x;
          const int t = e / (DPAD / 4), d = 4 * (e % (DPAD / 4));
          const bool in = d < dim;
          f32x4 q4, k4, a4;
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            q4[x] = in ? rq[4 * u + x] * a.qscale : 0.0f;
            k4[x] = in ? rk[4 * u + x] * a.kscale : 0.0f;
            if constexpr (CHANNELS) a4[x] = in ? decay_of(rz[4 * u + x]) : 0.0f;
          }
          *reinterpret_cast<f32x4*>(&qs[buf][t][d]) = q4;
          *reinterpret_cast<f32x4*>(&ks[buf][t][d]) = k4;
          if constexpr (CHANNELS) *reinterpret_cast<f32x4*>(&as[buf][t][d]) = a4;
        }
      }
    } else {
#pragma unroll
      for (int u = 0; u < NQ; ++u) {
        if (64 * RW * u < tc * DPAD) {
          const int e = 64 * RW * u + (int)threadIdx.x;
          const int t = e / DPAD, d = e % DPAD;
          const bool in = d < dim;
          qs[buf][t][d] = in ? rq[u] * a.qscale : 0.0f;
          ks[buf][t][d] = in ? rk[u] * a.kscale : 0.0f;
          if constexpr (CHANNELS) as[buf][t][d] = in ? decay_of(rz[u]) : 0.0f;
        }
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int e = 64 * RW * u + (int)threadIdx.x;
      if (64 * RW * u < tc * WCOLS && e < RC * WCOLS) vs[buf][e / WCOLS][e % WCOLS] = j_wg + e % WCOLS < vdim ? rv[u] : 0.0f;
    }
    if constexpr (GATES) {
      if ((int)threadIdx.x < tc) {
        const float cap = a.param;
        gi[buf][threadIdx.x] = cap * tanhf((rg[0] + a.bias[h]) / cap);
        gf[buf][threadIdx.x] = log_sigmoid(cap * tanhf((rg[1] + a.bias2[h]) / cap));
      }
    }
    if constexpr (DELTA) {
      if ((int)threadIdx.x < tc) {
        gi[buf][threadIdx.x] = rg[0];
        gf[buf][threadIdx.x] = rg[1];
        gd[buf][threadIdx.x] = rg[2];
      }
    }
    if constexpr (STEP) {
      if ((int)threadIdx.x < tc) {
        const float delta = softplus(rg[0] + a.bias[h]);
        gi[buf][threadIdx.x] = delta;
        gf[buf][threadIdx.x] = bw_expf(-(a.bias2[h] * delta));
      }
    }
  };

  // N tokens' operands out of LDS, from token t of the chunk on
  auto load_tokens = [&](auto& O, int buf, int t) {
    constexpr int N = std::remove_reference_t<decltype(O)>::N;
#pragma unroll
    for (int n = 0; n < N; ++n) {
#pragma unroll
      for (int d = 0; d < DH; d += 4) {
        const f32x4 kv = *reinterpret_cast<const f32x4*>(&ks[buf][t + n][channel(d)]);
        const f32x4 qv = *reinterpret_cast<const f32x4*>(&qs[buf][t + n][channel(d)]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          O.k[n][d + e] = kv[e];
          O.q[n][d + e] = qv[e];
        }
        if constexpr (CHANNELS) {
          const f32x4 av = *reinterpret_cast<const f32x4*>(&as[buf][t + n][channel(d)]);
#pragma unroll
          for (int e = 0; e < 4; ++e) O.a[n][d + e] = av[e];
        }
      }
      O.v[n] = vs[buf][t + n][j_in];
      if constexpr (GATES || STEP || DELTA) {
        O.g1[n] = gi[buf][t + n];
        O.g2[n] = gf[buf][t + n];
      }
      if constexpr (DELTA) O.kq[n] = gd[buf][t + n];
    }
  };

  // those tokens one after the other
  auto run_tokens = [&](auto& O, int t0, int buf, int t) {
    constexpr int N = std::remove_reference_t<decltype(O)>::N;
    float o[N], w[DELTA ? N : 1];
#pragma unroll
    for (int n = 0; n < N; ++n) {
      o[n] = 0.0f;
      if constexpr (STEP) {
        const float fa = O.g2[n], bv = O.g1[n] * O.v[n];
#pragma unroll
        for (int d = 0; d < DH; ++d) {
          Sreg[d] = fmaf(fa, Sreg[d], O.k[n][d] * bv);
          if constexpr (READ_OUT) o[n] = fmaf(Sreg[d], O.q[n][d], o[n]);
        }
        if constexpr (PHASE == 1) {
#pragma unroll
          for (int i = 0; i < NN; ++i) nreg[i] *= fa;
        }
      } else if constexpr (DELTA) {
        // (what the next token waits for: two chains over a lane's channels, the column's lanes, and then one fused
        // multiply-add for u and one for each channel)
        const float fa = O.g2[n], step_v = O.g1[n] * O.v[n], step_a = -(O.g1[n] * fa);
        float r0 = 0.0f, r1 = 0.0f, o1 = 0.0f;
#pragma unroll
        for (int d = 0; d < DH; d += 2) {
          r0 = fmaf(Sreg[d], O.k[n][d], r0);
          r1 = fmaf(Sreg[d + 1], O.k[n][d + 1], r1);
        }
        const float u = fmaf(step_a, join_parts<SPLIT>(r0 + r1), step_v);
#pragma unroll
        for (int d = 0; d < DH; d += 2) {
          o[n] = fmaf(Sreg[d], O.q[n][d], o[n]);
          o1 = fmaf(Sreg[d + 1], O.q[n][d + 1], o1);
        }
        o[n] += o1;
        w[n] = O.kq[n] * u;
#pragma unroll
        for (int d = 0; d < DH; ++d) Sreg[d] = fmaf(O.k[n][d], u, fa * Sreg[d]);
      } else if constexpr (!GATES) {
#pragma unroll
        for (int d = 0; d < DH; ++d) {
          const float kv = O.k[n][d] * O.v[n];
          if constexpr (BONUS) {
            if constexpr (READ_OUT) o[n] = fmaf(fmaf(ureg[d], kv, Sreg[d]), O.q[n][d], o[n]);
            Sreg[d] = fmaf(O.a[n][d], Sreg[d], kv);
          } else {
            Sreg[d] = fmaf(FIXED ? fixed_decay : O.a[CHANNELS ? n : 0][CHANNELS ? d : 0], Sreg[d], kv);
            if constexpr (READ_OUT) o[n] = fmaf(Sreg[d], O.q[n][d], o[n]);
          }
        }
        if constexpr (PHASE == 1) {
#pragma unroll
          for (int i = 0; i < NN; ++i)
            if (lane + 64 * i < DPAD) nreg[i] *= FIXED ? fixed_decay : as[CHANNELS ? buf : 0][CHANNELS ? t + n : 0][CHANNELS ? lane + 64 * i : 0];
        }
      } else {
        const float ig = O.g1[n], fg = O.g2[n];
        const float mn = fmaxf(fg + m, ig);
        const float fa = bw_expf(fg + m - mn);
        const float ib = bw_expf(ig - mn);
        m = mn;
        fsum += fg;
        const float bv = ib * O.v[n];
#pragma unroll
        for (int d = 0; d < DH; ++d) {
          Sreg[d] = fmaf(fa, Sreg[d], O.k[n][d] * bv);
          if constexpr (READ_OUT) o[n] = fmaf(Sreg[d], O.q[n][d], o[n]);
        }
        float sum = 0.0f;
#pragma unroll
        for (int i = 0; i < NN; ++i) {
          const int d = lane + 64 * i;
          if (d < DPAD) {
            nreg[i] = fmaf(fa, nreg[i], ib * ks[buf][t + n][d]);
            sum = fmaf(nreg[i], qs[buf][t + n][d], sum);
          }
        }
        if constexpr (READ_OUT) {
          o[n] = join_parts<SPLIT>(o[n]);
          const float nq = wave_sum(sum);
          o[n] = o[n] / (fmaxf(fabsf(nq), bw_expf(-mn)) + 1e-6f);
        }
      }
    }
    if constexpr (READ_OUT) {
      float* orow = a.out + (size_t)(first + t0 + t) * a.ldo + h * vdim + j;
      // (part n of a column stores token t + n)
      float mine = 0.0f;
#pragma unroll
      for (int n = 0; n < N; ++n) {
        float v = o[n];
        if constexpr (!GATES) v = join_parts<SPLIT>(v);
        if constexpr (STEP) v = fmaf(skip, O.v[n], v);
        if constexpr (DELTA) v = fmaf(O.g2[n], v, w[n]);
        mine = part == n ? v : mine;
      }
      if (live && part < N) orow[(size_t)part * a.ldo] = mine;
    }
  };
  using Group = RecurOps<TU, DH, CHANNELS>;
  using Single = RecurOps<1, DH, CHANNELS>;

  if constexpr (BUFS == 2) {
    fetch(0);
    stash(0, 0);
    __syncthreads();
  }
  int buf = 0;
  for (int t0 = 0; t0 < count; t0 += RC) {
    const int tc = min(RC, count - t0);
    if constexpr (BUFS == 2) {
      fetch(t0 + RC);
    } else {
      fetch(t0);
      __syncthreads();
      stash(t0, 0);
      __syncthreads();
    }
    int t = 0;
    if (BUFS == 2 && tc == RC) {
      // a whole chunk: a group's operands are on their way while the group before it is worked on
      Group even, odd;
      load_tokens(even, buf, 0);
#pragma unroll
      for (int g = 0; g < RC / TU; g += 2) {
        load_tokens(odd, buf, (g + 1) * TU);
        __builtin_amdgcn_sched_barrier(0);
        run_tokens(even, t0, buf, g * TU);
        if (g + 2 < RC / TU) load_tokens(even, buf, (g + 2) * TU);
        __builtin_amdgcn_sched_barrier(0);
        run_tokens(odd, t0, buf, (g + 1) * TU);
      }
      t = RC;
    }
    for (; t + TU <= tc; t += TU) {
      Group group;
      load_tokens(group, buf, t);
      run_tokens(group, t0, buf, t);
    }
    for (; t < tc; ++t) {
      Single single;
      load_tokens(single, buf, t);
      run_tokens(single, t0, buf, t);
    }
    if constexpr (BUFS == 2) {
      stash(t0 + RC, buf ^ 1);
      __syncthreads();
      buf ^= 1;
    }
  }
  // where the state goes: the slot (PHASE 3: from the request's last chunk only), or the chunk's own record
  float* S_out = S;
  float* nv_out = nv;
  float* mv_out = mv;
  if constexpr (PHASE == 1) {
    S_out = a.local + ((size_t)blockIdx.z * a.heads + h) * rec;
    nv_out = S_out + (size_t)dim * vdim;
    mv_out = nv_out + dim;
  }
  if (PHASE == 3 && !leaves_state) return;
  if (live) {
    if ((dim & 3) == 0 && (reinterpret_cast<uintptr_t>(S_out) & 15) == 0) {
      f32x4* dst = reinterpret_cast<f32x4*>(S_out + (size_t)j * dim);
#pragma unroll
      for (int d = 0; d < DH; d += 4)
        if (channel(d) < dim) dst[channel(d) >> 2] = (f32x4){Sreg[d], Sreg[d + 1], Sreg[d + 2], Sreg[d + 3]};
    } else {
#pragma unroll
      for (int d = 0; d < DH; ++d)
        if (channel(d) < dim) S_out[(size_t)j * dim + channel(d)] = Sreg[d];
    }
  }
  if (wv == 0 && (WALK ? GATES : blockIdx.x == 0 && (GATES || PHASE == 1))) {
    // (the last of the passes leaves every workgroup's copy)
    const int copies = PHASE == 3 ? recur_blocks(dim, vdim) : 1;
    for (int k = 0; k < copies; ++k) {
#pragma unroll
      for (int i = 0; i < NN; ++i)
        if (lane + 64 * i < dim) nv_out[k * copy + lane + 64 * i] = nreg[i];
      if (GATES && lane == 0) {
        mv_out[k * copy] = m;
        if (PHASE == 1) mv_out[1] = fsum;
      }
    }
  }
}

// A request's chunks in order: the state each one starts from, out of the slot's state and the chunks' own contributions
// and decays.  A thread per element of a head's record; every thread of a head walks the same scalars.
//   per channel:   S' = decay[d] * S + S_local
//   scalar gates:  m' = max(F + m, b), S' = e^(F + m - m') S + e^(b - m') S_local, n likewise (F: the chunk's sum of log
//                  forget gates, b: its maximum from -inf)
template <int MODE>
__global__ __launch_bounds__(256) void recurrence_scan_kernel(RecurArgs a, const int32_t* __restrict__ spans) {
  constexpr bool GATES = MODE == RECUR_SCALAR_GATES;
  const int dim = a.dim, vdim = a.vdim, h = blockIdx.y;
  const int seq = spans[3 * blockIdx.z], c0 = spans[3 * blockIdx.z + 1], nc = spans[3 * blockIdx.z + 2];
  const int slot = a.slots[seq];
  if (slot < 0 || nc <= 0) return;
  const size_t rec = recur_record(dim, vdim);
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int sd = dim * vdim;
  const int mine = GATES ? sd + dim + 1 : sd;          // elements a head has to carry: S, and with scalar gates n and m
  if (e >= mine) return;
  const float* st = a.state + (size_t)slot * a.state_ld;
  float val, m = 0.0f;
  if (e < sd) val = st[(size_t)h * sd + e];
  else if (e < sd + dim) val = st[(size_t)a.heads * sd + (size_t)h * dim + (e - sd)];
  else val = 0.0f;
  if constexpr (GATES) m = st[(size_t)a.heads * sd + (size_t)a.heads * dim + h];
  for (int c = c0; c < c0 + nc; ++c) {
    const float* loc = a.local + ((size_t)c * a.heads + h) * rec;
    float* out = a.start + ((size_t)c * a.heads + h) * rec;
    if constexpr (GATES) {
      out[e] = e == sd + dim ? m : val;
      const float b = loc[sd + dim], F = loc[sd + dim + 1];
      const float mn = fmaxf(F + m, b);
      const float ca = bw_expf(F + m - mn), cl = bw_expf(b - mn);
      if (e < sd + dim) val = fmaf(ca, val, cl * loc[e]);
      m = mn;
    } else {
      out[e] = val;
      val = fmaf(loc[sd + e % dim], val, loc[e]);
    }
  }
}

template <int MODE, int PHASE>
int launch_recurrence(const RecurArgs& a, int units, hipStream_t s) {
  const dim3 grid(recur_blocks(a.dim, a.vdim, PHASE == 1 || PHASE == 3), a.heads, units), block(64 * RW);
  if (a.dim <= 16) hipLaunchKernelGGL((linear_recurrence_kernel<MODE, 16, PHASE>), grid, block, 0, s, a);
  else if (a.dim <= 32) hipLaunchKernelGGL((linear_recurrence_kernel<MODE, 32, PHASE>), grid, block, 0, s, a);
  else if (a.dim <= 64) hipLaunchKernelGGL((linear_recurrence_kernel<MODE, 64, PHASE>), grid, block, 0, s, a);
  else if (a.dim <= 128) hipLaunchKernelGGL((linear_recurrence_kernel<MODE, 128, PHASE>), grid, block, 0, s, a);
  else if (a.dim <= 256) hipLaunchKernelGGL((linear_recurrence_kernel<MODE, 256, PHASE>), grid, block, 0, s, a);
  else return -4;
  return BW_LAUNCH_CHECK();
}

template <int MODE>
int launch_recurrence_passes(const RecurArgs& a, int nseq, bool few, int nchunks, const int32_t* spans, int nspans, hipStream_t s) {
  int rc = 0;
  if (nseq > 0) rc = few ? launch_recurrence<MODE, 4>(a, nseq, s) : launch_recurrence<MODE, 0>(a, nseq, s);
  if (rc != 0 || nchunks <= 0) return rc;
  if constexpr (MODE == RECUR_DELTA) {
    return -2;
  } else {
    rc = launch_recurrence<MODE, 1>(a, nchunks, s);
    if (rc != 0) return rc;
    const int mine = a.dim * a.vdim + (MODE == RECUR_SCALAR_GATES ? a.dim + 1 : 0);
    hipLaunchKernelGGL(recurrence_scan_kernel<MODE>, dim3((mine + 255) / 256, a.heads, nspans), dim3(256), 0, s, a, spans);
    rc = BW_LAUNCH_CHECK();
    if (rc != 0) return rc;
    return launch_recurrence<MODE, 3>(a, nchunks, s);
  }
}

// ------------------------------------------------------------------------- per-head RMS norm and output gate

enum { GATE_SIGMOID = 0, GATE_SILU = 1 };

// out[r][h*vdim + j] = o[r][h][j] / sqrt(mean_j o^2 + eps) * weight[h*wstride + j] * gate(g[r][h*vdim + j]); a wave per (row, head).
template <typename OT>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float* __restrict__ o, int ldi, const float* __restrict__ weight,
                                                             int wstride, const float* __restrict__ g, int ldg, int gate,
                                                             OT* __restrict__ out, int ldo, const int32_t* __restrict__ positions,
                                                             int rows, int heads, int vdim, float eps) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.x * (blockDim.x >> 6) + wave_index();
  if (item >= rows * heads) return;
  const int row = item / heads, h = item % heads;
  if (positions[row] < 0) return;
  const float* orow = o + (size_t)row * ldi + h * vdim;
  const float inv = 1.0f / sqrtf(row_sumsq(orow, vdim, lane) / (float)vdim + eps);
  const float* grow = g + (size_t)row * ldg + h * vdim;
  const float* wr = weight + (size_t)h * wstride;
  OT* dst = out + (size_t)row * ldo + h * vdim;
  for (int jj = lane; jj < vdim; jj += 64) {
    const float z = grow[jj];
    const float sg = 1.0f / (1.0f + bw_expf(-z));
    const float gv = gate == GATE_SILU ? z * sg : sg;
    store_act(dst + jj, ((orow[jj] * inv) * wr[jj]) * gv);
  }
}

// ------------------------------------------------------------------------- output gate and an RMS norm in equal parts

// A row's parts are equal stretches of ``size`` elements.  BEHIND false: v = o[r][e] * act(z[r][e]), out = v / sqrt(mean of v^2
// over the part + eps) * weight[e].  BEHIND true: v = o[r][e], and the norm's result is multiplied by act(z[r][e]).  act: SiLU
// or sigmoid.  A workgroup per (row, part): thread t owns elements t, t + 256, ... (one chain over its squares), the waves'
// sums are joined by wave_sum and added in wave order.  Parts of up to 256 GP_MAXV elements keep their values in registers;
// the same chain either way.
template <typename OT, bool BEHIND, int GP_MAXV>
__global__ __launch_bounds__(256) void gated_part_norm_kernel(const float* __restrict__ o, int ldi, const float* __restrict__ z, int ldz,
                                                              const float* __restrict__ weight, OT* __restrict__ out, int ldo,
                                                              const int32_t* __restrict__ positions, int size, float eps, int gate) {
  __shared__ float part[4];
  const int row = blockIdx.x, base = blockIdx.y * size, tid = threadIdx.x;
  if (positions[row] < 0) return;
  const float* orow = o + (size_t)row * ldi + base;
  const float* zrow = z + (size_t)row * ldz + base;
  const float* wr = weight + base;
  OT* dst = out + (size_t)row * ldo + base;
  auto act = [&](float zv) {
    const float sg = 1.0f / (1.0f + bw_expf(-zv));
    return gate == GATE_SILU ? zv * sg : sg;
  };
  auto before = [&](float ov, float zv) { return BEHIND ? ov : ov * act(zv); };
  auto after = [&](float v, float inv, float we, float zv) {
    const float y = (v * inv) * we;
    return BEHIND ? y * act(zv) : y;
  };
  const bool small = size <= 256 * GP_MAXV;
  float v[GP_MAXV], zv[GP_MAXV], wv[GP_MAXV];
  float acc = 0.0f;
  if (small) {
    float ov[GP_MAXV];
#pragma unroll
    for (int j = 0; j < GP_MAXV; ++j) {
      const int e = min(tid + 256 * j, size - 1);
      ov[j] = orow[e];
      zv[j] = zrow[e];
      wv[j] = wr[e];
    }
#pragma unroll
    for (int j = 0; j < GP_MAXV; ++j) {
      v[j] = tid + 256 * j < size ? before(ov[j], zv[j]) : 0.0f;
      acc = fmaf(v[j], v[j], acc);
    }
  } else {
    for (int e = tid; e < size; e += 256) {
      const float ve = before(orow[e], zrow[e]);
      acc = fmaf(ve, ve, acc);
    }
  }
  acc = wave_sum(acc);
  if ((tid & 63) == 0) part[tid >> 6] = acc;
  __syncthreads();
  const float inv = 1.0f / sqrtf((((part[0] + part[1]) + part[2]) + part[3]) / (float)size + eps);
  if (small) {
#pragma unroll
    for (int j = 0; j < GP_MAXV; ++j) {
      const int e = tid + 256 * j;
      if (e < size) store_act(dst + e, after(v[j], inv, wv[j], zv[j]));
    }
  } else {
    for (int e = tid; e < size; e += 256) store_act(dst + e, after(before(orow[e], zrow[e]), inv, wr[e], zrow[e]));
  }
}

// ------------------------------------------------------------------------- gated unit

enum { ACT_SILU = 0, ACT_GELU_TANH = 1, ACT_CLAMPED_SWISH = 2 };

template <typename OT>
__global__ void glu_kernel(const float* __restrict__ gu, int ldg, OT* __restrict__ hout, long long n, int inter, int act, float limit,
                           float alpha, const float* __restrict__ row_gate, int ld_row_gate) {
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= n) return;
  const long long row = idx / inter;
  const int c = (int)(idx % inter);
  float g = gu[row * ldg + c], u = gu[row * ldg + inter + c];
  float h;
  if (act == ACT_GELU_TANH) {
    const float inner = 0.7978845608028654f * (g + 0.044715f * ((g * g) * g));
    h = ((0.5f * g) * (1.0f + tanhf(inner))) * u;
  } else if (act == ACT_CLAMPED_SWISH) {
    h = clamped_swish_times<sizeof(OT) == 2>(g, u, limit, alpha);
  } else {
    h = (g * (1.0f / (1.0f + bw_expf(-g)))) * u;
  }
  if (row_gate != nullptr) h *= 1.0f / (1.0f + bw_expf(-row_gate[row * ld_row_gate]));
  store_act(hout + idx, h);
}


// ------------------------------------------------------------------------- activation without a gate

// h = act(z) of a 32-bit product.  PLAIN_RELU2: max(z, 0)^2.  PLAIN_XIELU (p0 and p1 positive): z > 0: p0 z^2 + z/2;
// z <= 0: (1/2 + p1) (e^z - 1 - z) + z/2.  PLAIN_GELU_ERF: z/2 (1 + erf(z / sqrt 2)).
enum { PLAIN_RELU2 = 0, PLAIN_XIELU = 1, PLAIN_GELU_ERF = 2 };

template <typename OT>
__global__ __launch_bounds__(256) void activate_kernel(const float* __restrict__ x, int ldx, OT* __restrict__ out, int ldo, int rows,
                                                       int cols, int act, float p0, float p1) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= cols) return;
  for (int r = blockIdx.y; r < rows; r += gridDim.y) {
    const float z = x[(size_t)r * ldx + c];
    float h;
    if (act == PLAIN_XIELU) {
      h = z > 0.0f ? fmaf(p0 * z, z, 0.5f * z) : fmaf(0.5f + p1, expm1f(z) - z, 0.5f * z);
    } else if (act == PLAIN_GELU_ERF) {
      h = gelu_erf(z);
    } else {
      const float m = fmaxf(z, 0.0f);
      h = m * m;
    }
    store_act(out + (size_t)r * ldo + c, h);
  }
}

// ------------------------------------------------------------------------- rotation of 32-bit projections in place

// Sections of a row of 32-bit projections ([heads][dim] each, at columns off[s]) turned in place by the row's position:
// of every head's first rot elements, element i < rot/2 is paired with element i + rot/2, (u, v) -> (u c - v s, v c + u s)
// with c, s from the tables' row of the position.  A thread a pair.
struct RotateRowsArgs {
  float* x;
  int ldx, rows, heads, dim, rot, sections;
  int off[2];
  const float* cos_table;     // [positions, rot / 2]
  const float* sin_table;
  const int32_t* positions;
};

__global__ __launch_bounds__(256) void rotate_halves_rows_kernel(RotateRowsArgs a) {
  const int half = a.rot / 2;
  const int per_row = a.sections * a.heads * half;
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)a.rows * per_row) return;
  const int row = (int)(idx / per_row);
  int r = (int)(idx % per_row);
  const int sec = r / (a.heads * half);
  r %= a.heads * half;
  const int h = r / half, i = r % half;
  const int pos = a.positions[row];
  if (pos < 0) return;
  float* p = a.x + (size_t)row * a.ldx + a.off[sec] + (size_t)h * a.dim;
  const float c = a.cos_table[(size_t)pos * half + i], s = a.sin_table[(size_t)pos * half + i];
  const float u = p[i], v = p[i + half];
  p[i] = u * c - v * s;
  p[i + half] = v * c + u * s;
}

// x <- tanh(x) over [rows, cols] of 32-bit values
__global__ __launch_bounds__(256) void tanh_rows_kernel(float* __restrict__ x, int ld, int rows, int cols) {
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)rows * cols) return;
  float* p = x + (idx / cols) * ld + (idx % cols);
  *p = tanhf(*p);
}

// x <- silu(x) likewise
__global__ __launch_bounds__(256) void silu_rows_kernel(float* __restrict__ x, int ld, int rows, int cols) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= cols) return;
  for (int r = blockIdx.y; r < rows; r += gridDim.y) {
    float* p = x + (size_t)r * ld + c;
    *p = silu(*p);
  }
}

}  // namespace

extern "C" int bw_norm_shift(const float* x, int ldx, const float* w, const float* mix, float* state, long long state_ld,
                             const int32_t* positions, const int32_t* row_seq, const int32_t* seq_rows,
                             const int32_t* slots, void* out, int out_is_bf16, int ldo, int rows, int dim, float eps,
                             int nmix, void* stream) {
  if (rows <= 0) return 0;
  if (dim <= 0 || nmix < 1 || ldx < dim || (long long)ldo < (long long)nmix * dim || state_ld < dim) return -2;
  hipStream_t s = (hipStream_t)stream;
  if (rows <= 64 && (dim & 3) == 0 && (ldx & 3) == 0 && (ldo & 3) == 0 && (state_ld & 3) == 0 && dim <= 1024 * SHIFT_ROW_MAXV &&
      nmix <= SHIFT_ROW_MAXMIX) {
    const size_t bytes = (size_t)(3 * dim + 4) * sizeof(float);
    if (out_is_bf16)
      hipLaunchKernelGGL(norm_shift_row_kernel<bf16_t>, dim3(rows), dim3(256), bytes, s, x, ldx, w, mix, state, state_ld, positions,
                         row_seq, seq_rows, slots, (bf16_t*)out, ldo, rows, dim, eps, nmix);
    else
      hipLaunchKernelGGL(norm_shift_row_kernel<float>, dim3(rows), dim3(256), bytes, s, x, ldx, w, mix, state, state_ld, positions,
                         row_seq, seq_rows, slots, (float*)out, ldo, rows, dim, eps, nmix);
    return BW_LAUNCH_CHECK();
  }
  const dim3 grid((rows + 3) / 4), block(256);
  if (out_is_bf16)
    hipLaunchKernelGGL(norm_shift_kernel<bf16_t>, grid, block, 0, s, x, ldx, w, mix, state, state_ld, positions, row_seq,
                       seq_rows, slots, (bf16_t*)out, ldo, rows, dim, eps, nmix);
  else
    hipLaunchKernelGGL(norm_shift_kernel<float>, grid, block, 0, s, x, ldx, w, mix, state, state_ld, positions, row_seq,
                       seq_rows, slots, (float*)out, ldo, rows, dim, eps, nmix);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_linear_recurrence(int mode, const float* proj, int ldp, int q_off, int k_off, int v_off, const float* gate,
                                    int ldg, int gate_off, int gate2_off, const float* bias, const float* bias2, float param,
                                    float qscale, float kscale, const float* skip, int heads_per_key, int silu, int few, float* state, long long state_ld, float* out, int ldo,
                                    const int32_t* seq_rows, const int32_t* slots, const int32_t* positions, int nseq,
                                    int heads, int dim, int vdim, const int32_t* chunks, int nchunks, const int32_t* spans,
                                    int nspans, float* scan_local, float* scan_start, long long scan_floats, void* stream) {
  if (nseq <= 0 && nchunks <= 0) return 0;
  if (nchunks > 0) {
    if (chunks == nullptr || spans == nullptr || nspans <= 0 || scan_local == nullptr || scan_start == nullptr) return -2;
    if (scan_floats < (long long)nchunks * heads * (long long)recur_record(dim, vdim)) return -6;
  }
  if (heads <= 0 || dim <= 0 || vdim <= 0 || ldo < heads * vdim || heads_per_key < 1 || heads % heads_per_key) return -2;
  const long long need = (long long)heads * dim * vdim + (mode == RECUR_SCALAR_GATES ? (long long)recur_blocks(dim, vdim) * ((long long)heads * dim + heads) : 0);
  if (state_ld < need) return -2;
  if (silu && mode != RECUR_FIXED_DECAY) return -2;
  if ((bias == nullptr && mode != RECUR_DELTA) || (mode != RECUR_FIXED_DECAY && gate == nullptr) || ((mode == RECUR_SCALAR_GATES || mode == RECUR_BONUS_DECAY || mode == RECUR_STEP_DECAY) && bias2 == nullptr))
    return -2;
  RecurArgs a{proj, ldp, q_off, k_off, v_off, gate, ldg, gate_off, gate2_off, bias, bias2, skip, heads_per_key, param, qscale, kscale, silu, state, state_ld,
              out, ldo, seq_rows, slots, positions, heads, dim, vdim, chunks, scan_local, scan_start};
  hipStream_t s = (hipStream_t)stream;
  if (mode == RECUR_SCALAR_GATES) return launch_recurrence_passes<RECUR_SCALAR_GATES>(a, nseq, few != 0, nchunks, spans, nspans, s);
  if (mode == RECUR_DECAY_PER_CHANNEL) return launch_recurrence_passes<RECUR_DECAY_PER_CHANNEL>(a, nseq, few != 0, nchunks, spans, nspans, s);
  if (mode == RECUR_BONUS_DECAY) return launch_recurrence_passes<RECUR_BONUS_DECAY>(a, nseq, few != 0, nchunks, spans, nspans, s);
  if (mode == RECUR_FIXED_DECAY) return launch_recurrence_passes<RECUR_FIXED_DECAY>(a, nseq, few != 0, nchunks, spans, nspans, s);
  if (mode == RECUR_STEP_DECAY) return launch_recurrence_passes<RECUR_STEP_DECAY>(a, nseq, few != 0, nchunks, spans, nspans, s);
  if (mode == RECUR_DELTA) return launch_recurrence_passes<RECUR_DELTA>(a, nseq, few != 0, nchunks, spans, nspans, s);
  return -2;
}

extern "C" long long bw_recurrence_record(int dim, int vdim) { return (long long)recur_record(dim, vdim); }

extern "C" int bw_head_norm_gate(const float* o, int ldi, const float* weight, int wstride, const float* g, int ldg, int gate,
                                 void* out, int out_is_bf16, int ldo, const int32_t* positions, int rows, int heads, int vdim,
                                 float eps, void* stream) {
  if (rows <= 0) return 0;
  if (heads <= 0 || vdim <= 0 || ldi < heads * vdim || ldo < heads * vdim) return -2;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((rows * heads + 3) / 4), block(256);
  if (out_is_bf16)
    hipLaunchKernelGGL(head_norm_gate_kernel<bf16_t>, grid, block, 0, s, o, ldi, weight, wstride, g, ldg, gate, (bf16_t*)out,
                       ldo, positions, rows, heads, vdim, eps);
  else
    hipLaunchKernelGGL(head_norm_gate_kernel<float>, grid, block, 0, s, o, ldi, weight, wstride, g, ldg, gate, (float*)out,
                       ldo, positions, rows, heads, vdim, eps);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_gated_part_norm(const float* o, int ldi, const float* z, int ldz, const float* weight, void* out, int out_is_bf16,
                                  int ldo, const int32_t* positions, int rows, int parts, int size, float eps, int gate, int behind,
                                  void* stream) {
  if (rows <= 0) return 0;
  if (parts <= 0 || parts > 65535 || size <= 0 || ldi < parts * size || ldz < parts * size || ldo < parts * size) return -2;
  if (gate != GATE_SIGMOID && gate != GATE_SILU) return -2;
  const dim3 grid(rows, parts), block(256);
  hipStream_t s = (hipStream_t)stream;
  auto launch = [&](auto kernel, auto op) {
    hipLaunchKernelGGL(kernel, grid, block, 0, s, o, ldi, z, ldz, weight, op, ldo, positions, size, eps, gate);
  };
  const bool wide = size > 2048;
  if (out_is_bf16 && behind) wide ? launch(gated_part_norm_kernel<bf16_t, true, 16>, (bf16_t*)out) : launch(gated_part_norm_kernel<bf16_t, true, 8>, (bf16_t*)out);
  else if (out_is_bf16) wide ? launch(gated_part_norm_kernel<bf16_t, false, 16>, (bf16_t*)out) : launch(gated_part_norm_kernel<bf16_t, false, 8>, (bf16_t*)out);
  else if (behind) wide ? launch(gated_part_norm_kernel<float, true, 16>, (float*)out) : launch(gated_part_norm_kernel<float, true, 8>, (float*)out);
  else wide ? launch(gated_part_norm_kernel<float, false, 16>, (float*)out) : launch(gated_part_norm_kernel<float, false, 8>, (float*)out);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_glu(const float* gate_up, int ldg, void* h, int out_is_bf16, int rows, int inter, int act, float limit, float alpha,
                      const float* row_gate, int ld_row_gate, void* stream) {
  if (rows <= 0 || inter <= 0) return 0;
  if (act != ACT_SILU && act != ACT_GELU_TANH && act != ACT_CLAMPED_SWISH) return -2;
  if (ldg < 2 * inter || (act == ACT_CLAMPED_SWISH && !(limit > 0.0f))) return -2;
  const long long n = (long long)rows * inter;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((unsigned)((n + 255) / 256)), block(256);
  if (out_is_bf16) hipLaunchKernelGGL(glu_kernel<bf16_t>, grid, block, 0, s, gate_up, ldg, (bf16_t*)h, n, inter, act, limit, alpha, row_gate, ld_row_gate);
  else hipLaunchKernelGGL(glu_kernel<float>, grid, block, 0, s, gate_up, ldg, (float*)h, n, inter, act, limit, alpha, row_gate, ld_row_gate);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_activate(const float* x, int ldx, void* out, int out_is_bf16, int ldo, int rows, int cols, int act, float p0,
                           float p1, void* stream) {
  if (rows <= 0 || cols <= 0) return 0;
  if (ldx < cols || ldo < cols || (act != PLAIN_RELU2 && act != PLAIN_XIELU && act != PLAIN_GELU_ERF)) return -2;
  const dim3 grid((cols + 255) / 256, rows < 65535 ? rows : 65535), block(256);
  if (out_is_bf16) hipLaunchKernelGGL(activate_kernel<bf16_t>, grid, block, 0, (hipStream_t)stream, x, ldx, (bf16_t*)out, ldo, rows, cols, act, p0, p1);
  else hipLaunchKernelGGL(activate_kernel<float>, grid, block, 0, (hipStream_t)stream, x, ldx, (float*)out, ldo, rows, cols, act, p0, p1);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_rotate_halves_rows(float* x, int ldx, int rows, int heads, int dim, int rot, int sections, int off0, int off1,
                                     const float* cos_table, const float* sin_table, const int32_t* positions, void* stream) {
  if (rows <= 0 || rot == 0) return 0;
  if (heads <= 0 || dim <= 0 || rot < 0 || rot % 2 || rot > dim || sections < 1 || sections > 2) return -2;
  if (off0 < 0 || off0 + heads * dim > ldx || (sections == 2 && (off1 < 0 || off1 + heads * dim > ldx))) return -2;
  RotateRowsArgs a{x, ldx, rows, heads, dim, rot, sections, {off0, off1}, cos_table, sin_table, positions};
  const long long n = (long long)rows * sections * heads * (rot / 2);
  hipLaunchKernelGGL(rotate_halves_rows_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, (hipStream_t)stream, a);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_tanh_rows(float* x, int ld, int rows, int cols, void* stream) {
  if (rows <= 0 || cols <= 0) return 0;
  if (ld < cols) return -2;
  const long long n = (long long)rows * cols;
  hipLaunchKernelGGL(tanh_rows_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, (hipStream_t)stream, x, ld, rows, cols);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_silu_rows(float* x, int ld, int rows, int cols, void* stream) {
  if (rows <= 0 || cols <= 0) return 0;
  if (ld < cols) return -2;
  hipLaunchKernelGGL(silu_rows_kernel, dim3((cols + 255) / 256, rows < 65535 ? rows : 65535), dim3(256), 0, (hipStream_t)stream, x, ld, rows, cols);
  return BW_LAUNCH_CHECK();
}
