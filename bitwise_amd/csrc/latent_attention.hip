// Attention over a compressed cache: every token leaves one vector [latent | rotated key part] in its
// page slot, shared by all heads.  A head's query is brought into that space first (its unrotated part
// through the transposed key up-projection, its rotated part as it is), so that a score is one dot
// product with the cached vector and the weighted sum of cached latents is projected up to the head's
// values afterwards: the cache is read once for all heads of a row tile.
//
//   latent_prep:         RMSNorm of the latent, rotation of the shared key part and of the queries' rotated
//                        parts, cache write; where the queries go through a latent of their own, its RMSNorm
//                        instead of the queries' rotation.
//   headwise_linear:     out[r][h] = W[h] x[r][h], a product per head with weights of its own, optionally times a
//                        sigmoid gate per head, optionally with the rotation of a query part beside it.
//   shared_key_attention: causal softmax attention of all heads over the shared keys, values a prefix of
//                        the key vector, with an optional sink per head in the denominator and an optional window.
//
// Scores, softmax weights, norms and rotations are 32-bit whatever the cache's dtype.
#include "common.h"
#include "api.h"

#include <math.h>

namespace {

template <typename T>
__device__ __forceinline__ float load_f(const T* p) {
  if constexpr (sizeof(T) == 2) return bf16_to_f32(*p);
  else return *p;
}

template <typename T>
__device__ __forceinline__ void store_f(T* p, float v) {
  if constexpr (sizeof(T) == 2) *p = f32_to_bf16(v);
  else *p = v;
}

// ------------------------------------------------------------------------- prep

// A rotated part's element i: of its first ``rotary`` elements, i and i + rotary/2 are a pair (pairs 0), or 2k and 2k + 1
// (pairs 1), turned by column (i mod rotary/2, or k) of the position's row of the tables; the rest pass unchanged.
__device__ __forceinline__ float rotated_element(const float* __restrict__ x, int i, int rotary, int pairs, const float* __restrict__ ct,
                                                 const float* __restrict__ st) {
  const int half = rotary / 2;
  if (i >= rotary) return x[i];
  if (pairs) {
    const int k = i >> 1;
    return (i & 1) ? x[i] * ct[k] + x[i - 1] * st[k] : x[i] * ct[k] - x[i + 1] * st[k];
  }
  if (i < half) return x[i] * ct[i] - x[i + half] * st[i];
  return x[i] * ct[i - half] + x[i - half] * st[i - half];
}

struct PrepArgs {
  const float* proj;     // [rows, ldp]: q at q_off (heads x (dim + rot)), the down projection at dkv_off (rank + rot)
  int ldp, q_off, dkv_off;
  const float* norm_w;   // [rank]
  float eps;
  const float* cos_table;   // [positions, rotary / 2]
  const float* sin_table;
  const int32_t* positions;
  const int32_t* row_seq;
  const int32_t* block_table;
  int table_stride;
  void* qa;              // [rows, ldqa] (32-bit, or bfloat16 for the matrix-core attention): head h at h * (rank + rot); the
  int ldqa, qa_is_bf16;  // rotated part goes to its last rot elements
  int heads, dim, rot, rotary, rank, page_size, write_cache, pairs;
  // queries that go through a latent of their own (q_rank > 0; qa is not written then): the latent at q_off, normed into cq
  int q_rank;
  const float* q_norm_w;    // [q_rank]
  void* cq;                 // [rows, ldcq]
  int ldcq, cq_is_bf16;
};

// A workgroup a row.
template <typename CT>
__global__ __launch_bounds__(256) void latent_prep_kernel(PrepArgs a, CT* __restrict__ cache, CT* __restrict__ latent_t) {
  const int row = blockIdx.x;
  const int pos = a.positions[row];
  if (pos < 0) return;
  const int lane = threadIdx.x & 63;
  const float* pr = a.proj + (size_t)row * a.ldp;
  const float* dkv = pr + a.dkv_off;
  const int half = a.rotary / 2;
  const float* ct = a.cos_table + (size_t)pos * half;
  const float* st = a.sin_table + (size_t)pos * half;
  const int width = a.rank + a.rot;
  if (a.write_cache) {
    // every wave sums the latent's squares in the same order; the lanes are joined by the butterflies of wave_sum
    float acc = 0.0f;
#pragma unroll 8
    for (int i = lane; i < a.rank; i += 64) acc = fmaf(dkv[i], dkv[i], acc);
    const float inv = 1.0f / sqrtf(wave_sum(acc) / (float)a.rank + a.eps);
    const int page = a.block_table[(size_t)a.row_seq[row] * a.table_stride + pos / a.page_size];
    CT* dst = cache + ((size_t)page * a.page_size + pos % a.page_size) * width;
    for (int i = threadIdx.x; i < a.rank; i += blockDim.x) store_f(dst + i, (dkv[i] * inv) * a.norm_w[i]);
    if (latent_t != nullptr) {      // the latent once more, transposed within its page: [page][element][slot]
      CT* tp = latent_t + (size_t)page * a.rank * a.page_size + pos % a.page_size;
      for (int i = threadIdx.x; i < a.rank; i += blockDim.x) store_f(tp + (size_t)i * a.page_size, (dkv[i] * inv) * a.norm_w[i]);
    }
    const float* kr = dkv + a.rank;
    for (int i = threadIdx.x; i < a.rot; i += blockDim.x) store_f(dst + a.rank + i, rotated_element(kr, i, a.rotary, a.pairs, ct, st));
  }
  if (a.q_rank > 0) {
    const float* ql = pr + a.q_off;
    float acc = 0.0f;
#pragma unroll 8
    for (int i = lane; i < a.q_rank; i += 64) acc = fmaf(ql[i], ql[i], acc);
    const float inv = 1.0f / sqrtf(wave_sum(acc) / (float)a.q_rank + a.eps);
    for (int i = threadIdx.x; i < a.q_rank; i += blockDim.x) {
      const float v = (ql[i] * inv) * a.q_norm_w[i];
      const size_t at = (size_t)row * a.ldcq + i;
      if (a.cq_is_bf16) reinterpret_cast<bf16_t*>(a.cq)[at] = f32_to_bf16(v);
      else reinterpret_cast<float*>(a.cq)[at] = v;
    }
    return;
  }
  const int per = a.dim + a.rot;
  for (int e = threadIdx.x; e < a.heads * a.rot; e += blockDim.x) {
    const int h = e / a.rot, i = e % a.rot;
    const float v = rotated_element(pr + a.q_off + h * per + a.dim, i, a.rotary, a.pairs, ct, st);
    const size_t at = (size_t)row * a.ldqa + h * width + a.rank + i;
    if (a.qa_is_bf16) reinterpret_cast<bf16_t*>(a.qa)[at] = f32_to_bf16(v);
    else reinterpret_cast<float*>(a.qa)[at] = v;
  }
}

// ------------------------------------------------------------------------- a product per head

// out[r][h*ohs + o] = sum_i wt[h][i][o] * x[r][h*xhs + i]: the weights lie input-major, so that neighbouring threads
// (outputs) read neighbouring weights; HL_ROWS rows share every weight that is loaded.  One fused multiply-add chain
// per output, i ascending.
// A workgroup is 64 outputs by four quarters of the inner size (a wave a quarter, eight weights asked for at a time); the
// quarters' sums meet in LDS and are added in quarter order.
// gate (optional): the outputs of head h are multiplied by sigmoid(gate[r][h]).  rot (optional): the workgroups of an extra
// block of outputs write, for their rows and head, the rotated ``n`` elements at x[.. + src] to out[.. + dst].
struct HeadExtras {
  const float* gate;
  int ldg;
  int rot_n, rotary, pairs, src, dst;
  const float* cos_table;
  const float* sin_table;
  const int32_t* positions;
};

#define HL_ROWS 8
template <typename WT, typename OT>
__global__ __launch_bounds__(256) void headwise_linear_kernel(const float* __restrict__ x, int ldx, int xhs,
                                                              const WT* __restrict__ wt, int in, int outn,
                                                              OT* __restrict__ out, int ldo, int ohs, int rows, HeadExtras ex) {
  extern __shared__ float hl_x[];      // [HL_ROWS][in], then [4][HL_ROWS][64] partial sums
  float* hl_part = hl_x + HL_ROWS * in;
  const int r0 = blockIdx.x * HL_ROWS, h = blockIdx.y;
  if ((int)blockIdx.z * 64 >= outn) {      // the extra block
    const int half = ex.rotary / 2;
    for (int e = threadIdx.x; e < HL_ROWS * ex.rot_n; e += 256) {
      const int r = r0 + e / ex.rot_n, i = e % ex.rot_n;
      const int pos = r < rows ? ex.positions[r] : -1;
      if (pos < 0) continue;
      store_f(out + (size_t)r * ldo + h * ohs + ex.dst + i,
              rotated_element(x + (size_t)r * ldx + h * xhs + ex.src, i, ex.rotary, ex.pairs, ex.cos_table + (size_t)pos * half,
                              ex.sin_table + (size_t)pos * half));
    }
    return;
  }
  const int lane = threadIdx.x & 63, quarter = wave_index();
  const int o = blockIdx.z * 64 + lane;
  for (int e = threadIdx.x; e < HL_ROWS * in; e += 256) {
    const int r = e / in, i = e % in;
    hl_x[e] = (r0 + r < rows) ? x[(size_t)(r0 + r) * ldx + h * xhs + i] : 0.0f;
  }
  __syncthreads();
  float acc[HL_ROWS];
#pragma unroll
  for (int r = 0; r < HL_ROWS; ++r) acc[r] = 0.0f;
  const int per = (in + 3) / 4;
  const int i0 = quarter * per, i1 = min(in, i0 + per);
  const WT* wp = wt + (size_t)h * in * outn + min(o, outn - 1);
  for (int i = i0; i < i1; i += 8) {
    float w[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) w[u] = load_f(wp + (size_t)min(i + u, i1 - 1) * outn);
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (i + u < i1) {
#pragma unroll
        for (int r = 0; r < HL_ROWS; ++r) acc[r] = fmaf(hl_x[r * in + i + u], w[u], acc[r]);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < HL_ROWS; ++r) hl_part[(quarter * HL_ROWS + r) * 64 + lane] = acc[r];
  __syncthreads();
  if (quarter != 0 || o >= outn) return;
#pragma unroll
  for (int r = 0; r < HL_ROWS; ++r) {
    const float sum = ((hl_part[r * 64 + lane] + hl_part[(HL_ROWS + r) * 64 + lane]) + hl_part[(2 * HL_ROWS + r) * 64 + lane]) +
                      hl_part[(3 * HL_ROWS + r) * 64 + lane];
    if (r0 + r >= rows) continue;
    const float gate = ex.gate != nullptr ? 1.0f / (1.0f + bw_expf(-ex.gate[(size_t)(r0 + r) * ex.ldg + h])) : 1.0f;
    store_f(out + (size_t)(r0 + r) * ldo + h * ohs + o, sum * gate);
  }
}

// The same product on the matrix cores, for bfloat16 weights that lie output-major, [head][outn][in] with in a multiple of 8:
// x is rounded to bfloat16 where it enters (if it is not bfloat16 already), the sums are 32-bit, one chain of
// v_mfma_f32_16x16x32_bf16 over the inner size ascending from zero for every block of 16 outputs x 16 rows, so a row's
// bits depend neither on the rows beside it nor on the shape of the launch.  A wave owns 16 rows and 16 OB outputs; ROW_WAVES:
// a workgroup's four waves are 64 rows (prompt portions), else 64 outputs of 16 rows.
struct HeadGemmArgs {
  const void* x;
  int ldx, xhs;
  const bf16_t* w;
  int in, outn;
  void* out;
  int ldo, ohs, rows;
  int heads, oz;           // oz: blocks of 64 outputs (and one more for the rotated part)
  int aligned;             // 1: rows and heads of out start at whole groups of four elements, outn is a multiple of 4; 2: of eight
};

template <typename XT, typename OT, int OB, bool ROW_WAVES>
__global__ __launch_bounds__(256) void headwise_mfma_kernel(HeadGemmArgs a, HeadExtras ex) {
  const int lane = threadIdx.x & 63, n = lane & 15, g = lane >> 4, wv = wave_index();
  // Workgroups are dealt to the eight dies in turn.  Of those of one die, the blocks of outputs of one (rows, head) follow each
  // other: they read the same rows of x, from the die's own L2 after the first.
  const int die = blockIdx.x & 7, nth = blockIdx.x >> 3;
  const int zb = nth % a.oz, unit = (nth / a.oz) * 8 + die;
  const int h = unit % a.heads, row_block = unit / a.heads;
  const int r_wg = row_block * (ROW_WAVES ? 64 : 16);
  if (r_wg >= a.rows) return;
  const XT* xh = reinterpret_cast<const XT*>(a.x) + (size_t)h * a.xhs;
  OT* oh = reinterpret_cast<OT*>(a.out) + (size_t)h * a.ohs;
  if (zb * 64 >= a.outn) {      // the extra block: the rotated part beside the product
    if constexpr (sizeof(XT) == 4) {
      const int half = ex.rotary / 2;
      for (int e = threadIdx.x; e < (ROW_WAVES ? 64 : 16) * ex.rot_n; e += 256) {
        const int r = r_wg + e / ex.rot_n, i = e % ex.rot_n;
        const int pos = r < a.rows ? ex.positions[r] : -1;
        if (pos < 0) continue;
        store_f(oh + (size_t)r * a.ldo + ex.dst + i,
                rotated_element(xh + (size_t)r * a.ldx + ex.src, i, ex.rotary, ex.pairs, ex.cos_table + (size_t)pos * half,
                                ex.sin_table + (size_t)pos * half));
      }
    }
    return;
  }
  const int r0 = r_wg + (ROW_WAVES ? 16 * wv : 0);
  const int o0 = zb * 64 + (ROW_WAVES ? 0 : 16 * wv);
  if (r0 >= a.rows || o0 >= a.outn) return;
  const XT* xr = xh + (size_t)min(r0 + n, a.rows - 1) * a.ldx;
  // block b's row k of the product is output o0 + 4 OB (k / 4) + 4 b + k % 4: a lane's results are 4 OB neighbours
  auto output_of = [](int b, int k) { return 4 * OB * (k >> 2) + 4 * b + (k & 3); };
  const bf16_t* wr[OB];
#pragma unroll
  for (int b = 0; b < OB; ++b) wr[b] = a.w + ((size_t)h * a.outn + min(o0 + output_of(b, n), a.outn - 1)) * a.in;
  f32x4 acc[OB];
#pragma unroll
  for (int b = 0; b < OB; ++b) acc[b] = (f32x4){0.f, 0.f, 0.f, 0.f};
  constexpr int U = 4;                       // steps of 32 elements whose loads are in flight together
  for (int k0 = 0; k0 < a.in; k0 += 32 * U) {
    u32x4 xf[U], wf[U][OB];
#pragma unroll
    for (int s = 0; s < U; ++s) {
      const int k = k0 + 32 * s + 8 * g, kc = min(k, a.in - 8);
#pragma unroll
      for (int b = 0; b < OB; ++b) wf[s][b] = *reinterpret_cast<const u32x4*>(wr[b] + kc);
      if constexpr (sizeof(XT) == 2) {
        xf[s] = *reinterpret_cast<const u32x4*>(xr + kc);
      } else {
        const f32x4 lo = *reinterpret_cast<const f32x4*>(xr + kc), hi = *reinterpret_cast<const f32x4*>(xr + kc + 4);
        xf[s] = (u32x4){pack_bf16x2(lo[0], lo[1]), pack_bf16x2(lo[2], lo[3]), pack_bf16x2(hi[0], hi[1]), pack_bf16x2(hi[2], hi[3])};
      }
      if (k >= a.in) xf[s] = (u32x4){0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int s = 0; s < U; ++s)
      if (k0 + 32 * s < a.in) {              // (scalar)
#pragma unroll
        for (int b = 0; b < OB; ++b)
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(wf[s][b]), as_bf16x8(xf[s]), acc[b], 0, 0, 0);
      }
  }
  const int r = r0 + n;
  if (r >= a.rows) return;
  const float gate = ex.gate != nullptr ? 1.0f / (1.0f + bw_expf(-ex.gate[(size_t)r * ex.ldg + h])) : 1.0f;
  if constexpr (OB == 4 && sizeof(OT) == 2) {
    if (a.aligned == 2 && o0 + 16 * g + 15 < a.outn) {
      OT* dst = oh + (size_t)r * a.ldo + o0 + 16 * g;
#pragma unroll
      for (int b = 0; b < OB; b += 2)
        *reinterpret_cast<u32x4*>(dst + 4 * b) = (u32x4){pack_bf16x2(acc[b][0] * gate, acc[b][1] * gate), pack_bf16x2(acc[b][2] * gate, acc[b][3] * gate),
                                                         pack_bf16x2(acc[b + 1][0] * gate, acc[b + 1][1] * gate),
                                                         pack_bf16x2(acc[b + 1][2] * gate, acc[b + 1][3] * gate)};
      return;
    }
  }
#pragma unroll
  for (int b = 0; b < OB; ++b) {
    const int o = o0 + output_of(b, 4 * g);  // outputs o .. o + 3 of this lane's row
    OT* dst = oh + (size_t)r * a.ldo + o;
    if (a.aligned) {
      if (o >= a.outn) continue;
      if constexpr (sizeof(OT) == 2)
        *reinterpret_cast<u32x2*>(dst) = (u32x2){pack_bf16x2(acc[b][0] * gate, acc[b][1] * gate), pack_bf16x2(acc[b][2] * gate, acc[b][3] * gate)};
      else
        *reinterpret_cast<f32x4*>(dst) = acc[b] * gate;
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (o + i < a.outn) store_f(dst + i, acc[b][i] * gate);
    }
  }
}

template <typename XT, typename OT>
int launch_headwise_mfma(const HeadGemmArgs& a, const HeadExtras& ex, hipStream_t s) {
  const int row_blocks = a.rows > 64 ? (a.rows + 63) / 64 : (a.rows + 15) / 16;
  const dim3 grid((unsigned)((row_blocks * a.heads + 7) / 8 * 8 * a.oz));
  if (a.rows > 64)
    hipLaunchKernelGGL((headwise_mfma_kernel<XT, OT, 4, true>), grid, dim3(256), 0, s, a, ex);
  else
    hipLaunchKernelGGL((headwise_mfma_kernel<XT, OT, 1, false>), grid, dim3(256), 0, s, a, ex);
  return BW_LAUNCH_CHECK();
}

// ------------------------------------------------------------------------- attention over shared keys

struct SharedKeyArgs {
  const float* q;          // [rows, ldq]: head h at h * dk
  int ldq;
  const int32_t* positions;
  const int32_t* block_table;
  int table_stride;
  const int32_t* tiles;    // [num_tiles, 4] = (first row, rows, request, 0); null: tile t is row t of request t
  const float* sink;       // [heads] or null
  float* out;              // [rows, ldo]: head h at h * dv
  int ldo;
  int heads, dk, dv, page_size, window, hg, num_pages;
  float scale;
};

// A workgroup of four waves per (tile of rows, group of ``hg`` heads): 16 query vectors, four a wave (16 / hg rows a
// tile: hg = 4 for prompt portions, 16 for single tokens).  Keys come through LDS in blocks of KB as 32-bit rows;
// for the scores a lane is a key (each key element it reads serves the wave's four queries), for the weighted sum a
// lane is NVC value columns.  The running maximum starts at the sink and the denominator at 1 = e^(sink - sink): the sink is
// one more score that has no value.
template <typename CT, int KB, int NVC>
__global__ __launch_bounds__(256) void shared_key_attention_kernel(SharedKeyArgs a, const CT* __restrict__ cache) {
  extern __shared__ float lds[];
  const int dkp = (a.dk + 3) & ~3;
  const int kstride = dkp + 4;
  float* Ks = lds;                         // [KB][kstride]
  float* Qs = Ks + KB * kstride;           // [16][dkp]
  float* Ps = Qs + 16 * dkp;               // [16][KB]
  const int lane = threadIdx.x & 63, w = wave_index();
  const int t = blockIdx.x;
  int r0, nr, seq;
  if (a.tiles != nullptr) {
    r0 = a.tiles[4 * t];
    nr = a.tiles[4 * t + 1];
    seq = a.tiles[4 * t + 2];
  } else {
    r0 = t;
    nr = 1;
    seq = t;
  }
  if (nr <= 0) return;
  const int pos0 = a.positions[r0];
  if (pos0 < 0) return;
  const int pmax = pos0 + nr - 1;
  const int h0 = blockIdx.y * a.hg;

  // this wave's four query vectors
  int qrow[4], qh[4], qpos[4];
  bool qok[4];
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    const int qv = 4 * w + g;
    const int rl = qv / a.hg;
    qh[g] = h0 + qv % a.hg;
    qok[g] = rl < nr && qh[g] < a.heads;
    qrow[g] = r0 + (rl < nr ? rl : 0);
    qpos[g] = qok[g] ? pos0 + rl : -1;
  }
  for (int e = threadIdx.x; e < 16 * dkp; e += 256) {
    const int qv = e / dkp, d = e % dkp;
    const int rl = qv / a.hg, h = h0 + qv % a.hg;
    Qs[e] = (rl < nr && h < a.heads && d < a.dk) ? a.q[(size_t)(r0 + rl) * a.ldq + h * a.dk + d] : 0.0f;
  }
  float m[4], l[4], acc[4][NVC];
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    const bool has = a.sink != nullptr && qok[g];
    m[g] = has ? a.sink[qh[g]] : -INFINITY;
    l[g] = has ? 1.0f : 0.0f;
#pragma unroll
    for (int c = 0; c < NVC; ++c) acc[g][c] = 0.0f;
  }
  const int lo_first = a.window > 0 ? max(0, pos0 - a.window + 1) : 0;
  const int32_t* table = a.block_table + (size_t)seq * a.table_stride;

  for (int kb0 = lo_first / KB * KB; kb0 <= pmax; kb0 += KB) {
    __syncthreads();
    // the block's keys, widened to 32-bit; keys beyond the tile's last position and the padding are zero
    for (int e = threadIdx.x; e < KB * dkp; e += 256) {
      const int jj = e / dkp, d = e % dkp;
      const int kj = kb0 + jj;
      float v = 0.0f;
      if (kj <= pmax && kj >= lo_first && d < a.dk) {
        int page = table[kj / a.page_size];
        page = min(max(page, 0), a.num_pages - 1);
        v = load_f(cache + ((size_t)page * a.page_size + kj % a.page_size) * a.dk + d);
      }
      Ks[jj * kstride + d] = v;
    }
    __syncthreads();
    float sc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (lane < KB) {
      const float* kr = Ks + lane * kstride;
      for (int d = 0; d < dkp; d += 4) {
        const f32x4 kv = *reinterpret_cast<const f32x4*>(kr + d);
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const f32x4 qv = *reinterpret_cast<const f32x4*>(Qs + (4 * w + g) * dkp + d);
          sc[g] = fmaf(kv[0], qv[0], sc[g]);
          sc[g] = fmaf(kv[1], qv[1], sc[g]);
          sc[g] = fmaf(kv[2], qv[2], sc[g]);
          sc[g] = fmaf(kv[3], qv[3], sc[g]);
        }
      }
    }
    const int kj = kb0 + lane;
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int lo = a.window > 0 ? max(0, qpos[g] - a.window + 1) : 0;
      const bool valid = lane < KB && kj <= qpos[g] && kj >= lo;
      const float s = valid ? sc[g] * a.scale : -INFINITY;
      const float mn = fmaxf(m[g], wave_max(s));
      const float base = mn == -INFINITY ? 0.0f : mn;
      float p, corr;
      if constexpr (sizeof(CT) == 2) {
        p = valid ? fast_exp(s - base) : 0.0f;
        corr = m[g] == -INFINITY ? 0.0f : fast_exp(m[g] - base);
      } else {
        p = valid ? bw_expf(s - base) : 0.0f;
        corr = m[g] == -INFINITY ? 0.0f : bw_expf(m[g] - base);
      }
      l[g] = l[g] * corr + wave_sum(p);
      m[g] = mn;
#pragma unroll
      for (int c = 0; c < NVC; ++c) acc[g][c] *= corr;
      if (lane < KB) Ps[(4 * w + g) * KB + lane] = p;
    }
    __syncthreads();
    for (int jj = 0; jj < KB; jj += 4) {
      f32x4 p4[4];
#pragma unroll
      for (int g = 0; g < 4; ++g) p4[g] = *reinterpret_cast<const f32x4*>(Ps + (4 * w + g) * KB + jj);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
#pragma unroll
        for (int c = 0; c < NVC; ++c) {
          const int col = lane + 64 * c;
          const float v = col < a.dv ? Ks[(jj + u) * kstride + col] : 0.0f;
#pragma unroll
          for (int g = 0; g < 4; ++g) acc[g][c] = fmaf(p4[g][u], v, acc[g][c]);
        }
      }
    }
  }
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    if (!qok[g]) continue;
    const float inv = l[g] > 0.0f ? 1.0f / l[g] : 0.0f;
#pragma unroll
    for (int c = 0; c < NVC; ++c) {
      const int col = lane + 64 * c;
      if (col < a.dv) a.out[(size_t)qrow[g] * a.ldo + qh[g] * a.dv + col] = acc[g][c] * inv;
    }
  }
}

template <typename CT, int KB>
int launch_shared_key_kb(const SharedKeyArgs& a, const CT* cache, int num_tiles, hipStream_t s) {
  const int dkp = (a.dk + 3) & ~3;
  const size_t bytes = ((size_t)KB * (dkp + 4) + 16 * dkp + 16 * KB) * sizeof(float);
  const dim3 grid(num_tiles, (a.heads + a.hg - 1) / a.hg), block(256);
  const int nvc = (a.dv + 63) / 64;
#define BW_SK_LAUNCH(N)                                                                                                  \
  do {                                                                                                                   \
    static bool attr_set = false;                                                                                        \
    if (!attr_set) {                                                                                                     \
      (void)hipFuncSetAttribute((const void*)shared_key_attention_kernel<CT, KB, N>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                          150 * 1024);                                                                                   \
      attr_set = true;                                                                                                   \
    }                                                                                                                    \
    hipLaunchKernelGGL((shared_key_attention_kernel<CT, KB, N>), grid, block, bytes, s, a, cache);                        \
  } while (0)
  if (nvc <= 1) BW_SK_LAUNCH(1);
  else if (nvc <= 2) BW_SK_LAUNCH(2);
  else if (nvc <= 4) BW_SK_LAUNCH(4);
  else if (nvc <= 8) BW_SK_LAUNCH(8);
  else return -4;
#undef BW_SK_LAUNCH
  return BW_LAUNCH_CHECK();
}

template <typename CT>
int launch_shared_key(const SharedKeyArgs& a, const CT* cache, int num_tiles, hipStream_t s) {
  const int dkp = (a.dk + 3) & ~3;
  const size_t budget = 144 * 1024;
  auto bytes = [&](int kb) { return ((size_t)kb * (dkp + 4) + 16 * dkp + 16 * kb) * sizeof(float); };
  // (blocks of 64 keys while two workgroups still fit a compute unit's LDS, else what fits)
  if (bytes(64) <= 72 * 1024) return launch_shared_key_kb<CT, 64>(a, cache, num_tiles, s);
  if (bytes(32) <= budget) return launch_shared_key_kb<CT, 32>(a, cache, num_tiles, s);
  if (bytes(16) <= budget) return launch_shared_key_kb<CT, 16>(a, cache, num_tiles, s);
  return -8;
}


// ------------------------------------------------------------------------- the same attention on the matrix cores

// bfloat16 caches whose key vectors are whole 16-byte groups.  A workgroup of NW waves per (tile of rows, group of ``hg``
// heads): 16 QT query vectors (16 QT / hg rows x hg heads).  The keys are cut into pieces of SK_PIECE keys at absolute
// positions, and a piece is one unit of arithmetic: its scores, the largest of them that a query sees, the weights relative to
// that maximum (32-bit, rounded to bfloat16 where they enter the product with the values), their sum, and the weighted sum of
// the values as one chain over the piece's keys.  Pieces are then folded in order, (m, l, o) <- fold((m, l, o), piece) by
// ``fold_piece``.  A prompt's tile walks the pieces of its window and folds as it goes; a single token's pieces get a workgroup
// each, leave (maximum, sum, values) in memory, and shared_key_combine_kernel folds them by the same operations in the same
// order: a position's bits do not depend on whether it came alone or inside a portion.
//
// Within a piece: scores by v_mfma_f32_16x16x32_bf16 with the keys as rows (operand A, straight from the cache: a wave takes
// its share of the piece's keys in tiles of 16, a lane reads 8 consecutive elements of its key) and the queries as columns (operand B, from LDS).  The
// weights go through LDS; a wave then owns every NW-th block of 16 value elements, read from the second copy of the latent that
// the cache write leaves transposed, [page][element][slot]: a lane's 8 keys are 16 consecutive bytes of its element's row.
#define SK_PIECE 128
#define SK_TILE_QUERIES 32          // query vectors of a prompt tile's workgroup: two of them fit a compute unit's registers
#define SK_PSTRIDE (SK_PIECE + 8)

struct MfmaAttnArgs {
  const bf16_t* q;         // [rows, ldq] bfloat16: head h at h * dk
  int ldq;
  const int32_t* positions;
  const int32_t* block_table;
  int table_stride;
  const int32_t* tiles;
  const float* sink;
  void* out;               // [rows, ldo], bfloat16 or 32-bit
  int ldo, out_is_bf16;
  float* partial;          // [tiles][heads][max_pieces][dv], then as many (maximum, sum)
  float* partial_ml;
  int heads, dk, dv, page_size, window, hg, num_pages, max_pieces;
  float scale;
};

__device__ __forceinline__ float across_groups_max(float v) {
  float a, b;
  lane_halves<32>(v, a, b);
  v = fmaxf(a, b);
  lane_halves<16>(v, a, b);
  return fmaxf(a, b);
}

__device__ __forceinline__ float across_groups_sum(float v) {
  float a, b;
  lane_halves<32>(v, a, b);
  v = a + b;
  lane_halves<16>(v, a, b);
  return a + b;
}

// A piece with maximum mp and sum lp joins what was folded so far: the factors for the old sums (c1) and the piece's (c2).
__device__ __forceinline__ void fold_piece(float& m, float& l, float mp, float lp, float& c1, float& c2) {
  const float mn = fmaxf(m, mp);
  c1 = m == -INFINITY ? 0.0f : fast_exp(m - mn);
  c2 = mp == -INFINITY ? 0.0f : fast_exp(mp - mn);
  l = fmaf(lp, c2, l * c1);
  m = mn;
}

// The factor on a query's folded sums: 1 / (denominator with the sink), scaled to the sink if that is larger.
__device__ __forceinline__ float finish_softmax(float m, float l, float sk) {
  const float mf = fmaxf(m, sk);
  const float cm = m == -INFINITY ? 0.0f : fast_exp(m - mf);
  const float lt = l * cm + (sk == -INFINITY ? 0.0f : fast_exp(sk - mf));
  return lt > 0.0f ? cm / lt : 0.0f;
}

__device__ __forceinline__ void store_out(const MfmaAttnArgs& a, size_t at, float v) {
  if (a.out_is_bf16) reinterpret_cast<bf16_t*>(a.out)[at] = f32_to_bf16(v);
  else reinterpret_cast<float*>(a.out)[at] = v;
}

// NDT: blocks of 16 value elements a wave owns (wave w: blocks w, w + NW, ...).  QT 1: a workgroup a piece (single tokens).
// The sums of the weights are kept by tiles of 16 keys and added in tile order, whatever the number of waves.
template <int QT, int NW, int NDT>
__global__ __launch_bounds__(64 * NW, QT == 1 ? 1 : 2) void shared_key_attention_mfma_kernel(MfmaAttnArgs a, const bf16_t* __restrict__ kc,
                                                                        const bf16_t* __restrict__ vt) {
  constexpr bool PIECES = QT == 1;
  constexpr int NQ = 16 * QT;
  constexpr int KT = SK_PIECE / 16, U = KT / NW;           // tiles of 16 keys: of a piece, of a wave
  extern __shared__ bf16_t sk_lds[];       // queries [NQ][qstride], weights [NQ][SK_PSTRIDE]
  __shared__ float red_max[NW][NQ], red_sum[KT][NQ];
  const int lane = threadIdx.x & 63, n = lane & 15, g = lane >> 4, wv = wave_index();
  const int t = blockIdx.x, h0 = blockIdx.y * a.hg;
  int r0, nr, seq;
  if (a.tiles != nullptr) {
    r0 = __builtin_amdgcn_readfirstlane(a.tiles[4 * t]);
    nr = __builtin_amdgcn_readfirstlane(a.tiles[4 * t + 1]);
    seq = __builtin_amdgcn_readfirstlane(a.tiles[4 * t + 2]);
  } else {
    r0 = t;
    nr = 1;
    seq = t;
  }
  if (nr <= 0) return;
  const int pos0 = __builtin_amdgcn_readfirstlane(a.positions[r0]);
  if (pos0 < 0) return;
  const int pmax = pos0 + nr - 1;
  const int lo_first = a.window > 0 ? max(0, pos0 - a.window + 1) : 0;
  int piece = lo_first / SK_PIECE;
  const int last = pmax / SK_PIECE;
  if constexpr (PIECES) {
    piece += blockIdx.z;
    if (piece > last) return;
  }
  const int dk = a.dk, dv = a.dv, ps = a.page_size;
  const int dkp = (dk + 31) & ~31, qstride = dkp + 8;
  bf16_t* qs = sk_lds;
  bf16_t* pw = sk_lds + NQ * qstride;
  {
    const int groups = dkp >> 3;             // 16-byte groups of a query vector (dk is a multiple of 8)
    for (int e = threadIdx.x; e < NQ * groups; e += 64 * NW) {
      const int qn = e / groups, d = (e % groups) * 8;
      const int r2 = qn / a.hg, h2 = h0 + qn % a.hg;
      u32x4 v = {0u, 0u, 0u, 0u};
      if (r2 < nr && h2 < a.heads && d < dk) v = *reinterpret_cast<const u32x4*>(a.q + (size_t)(r0 + r2) * a.ldq + h2 * dk + d);
      *reinterpret_cast<u32x4*>(qs + qn * qstride + d) = v;
    }
  }
  int qpos[QT], qlo[QT];
#pragma unroll
  for (int c = 0; c < QT; ++c) {
    const int qn = 16 * c + n, rl = qn / a.hg;
    const bool ok = rl < nr && h0 + qn % a.hg < a.heads;
    qpos[c] = ok ? pos0 + rl : -1;
    qlo[c] = a.window > 0 ? max(0, qpos[c] - a.window + 1) : 0;
  }
  const int32_t* table = a.block_table + (size_t)seq * a.table_stride;
  float m[QT], l[QT];
  f32x4 acc[NDT][QT];
#pragma unroll
  for (int c = 0; c < QT; ++c) {
    m[c] = -INFINITY;
    l[c] = 0.0f;
#pragma unroll
    for (int j = 0; j < NDT; ++j) acc[j][c] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  __syncthreads();

  for (; piece <= last; ++piece) {
    const int k0 = piece * SK_PIECE, kw = k0 + 16 * U * wv;
    // where this lane's keys and runs of values lie
    const bf16_t* krow[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kj = min(kw + 16 * u + n, pmax);
      krow[u] = kc + ((size_t)min(max(table[kj / ps], 0), a.num_pages - 1) * ps + kj % ps) * dk;
    }
    const bf16_t* vrun[4];
#pragma unroll
    for (int sg = 0; sg < 4; ++sg) {
      const int c = min(k0 + 32 * sg + 8 * g, pmax & ~7);
      vrun[sg] = vt + (size_t)min(max(table[c / ps], 0), a.num_pages - 1) * dv * ps + c % ps;
    }
    auto load_values = [&](int sg, int j) -> u32x4 {
      // (rows past the values are computed and never stored)
      const uint32_t d = (uint32_t)min(16 * (NW * j + wv) + n, dv - 1);
      return *reinterpret_cast<const u32x4*>(vrun[sg] + d * (uint32_t)ps);
    };

    // ---- scores of this wave's keys: lane (n, g) gets keys kw + 16u + 4g + i of query n of every tile
    f32x4 st[U][QT];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int c = 0; c < QT; ++c) st[u][c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (kw <= pmax && kw + 16 * U - 1 >= lo_first) {                 // (scalar: some query of the tile may see one of them)
      constexpr int KST = QT == 1 ? 18 : 6;                                // steps of 32 elements whose loads are in flight together
      for (int d1 = 0; d1 < dkp; d1 += 32 * KST) {
        u32x4 kf[KST][U];
#pragma unroll
        for (int s4 = 0; s4 < KST; ++s4) {
          // (elements past the key vector meet zeros in the query)
          const int d0 = min(d1 + 32 * s4 + 8 * g, dk - 8);
          if (d1 + 32 * s4 < dkp) {                          // (scalar)
#pragma unroll
            for (int u = 0; u < U; ++u) kf[s4][u] = *reinterpret_cast<const u32x4*>(krow[u] + d0);
          }
        }
#pragma unroll
        for (int s4 = 0; s4 < KST; ++s4) {
          if (d1 + 32 * s4 < dkp) {
#pragma unroll
            for (int c = 0; c < QT; ++c) {
              {
                const u32x4 qf = *reinterpret_cast<const u32x4*>(qs + (16 * c + n) * qstride + d1 + 32 * s4 + 8 * g);
#pragma unroll
                for (int u = 0; u < U; ++u)
                  st[u][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(kf[s4][u]), as_bf16x8(qf), st[u][c], 0, 0, 0);
              }
            }
          }
        }
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    // the first blocks of values are asked for before the weights are formed (what is asked for when is as written: left to
    // itself the scheduler asks for everything at once and runs out of registers)
    __builtin_amdgcn_sched_barrier(0);
    constexpr int MOST = QT == 1 ? 4 : 2;
    constexpr int AHEAD = NDT < MOST ? NDT : MOST;
    u32x4 vf[AHEAD][4];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
#pragma unroll
      for (int sg = 0; sg < 4; ++sg) vf[j][sg] = load_values(sg, j);

    // ---- the piece's softmax, relative to its own maximum
#pragma unroll
    for (int c = 0; c < QT; ++c) {
      float mx = -INFINITY;
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kw + 16 * u + 4 * g + i;
          const float sv = key <= qpos[c] && key >= qlo[c] ? st[u][c][i] * a.scale : -INFINITY;
          st[u][c][i] = sv;
          mx = fmaxf(mx, sv);
        }
      mx = across_groups_max(mx);
      if (g == 0) red_max[wv][16 * c + n] = mx;
    }
    __syncthreads();
    float mp[QT];
#pragma unroll
    for (int c = 0; c < QT; ++c) {
      mp[c] = red_max[0][16 * c + n];
#pragma unroll
      for (int k = 1; k < NW; ++k) mp[c] = fmaxf(mp[c], red_max[k][16 * c + n]);
      const float base = mp[c] == -INFINITY ? 0.0f : mp[c];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        float p[4], psum = 0.0f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          p[i] = st[u][c][i] == -INFINITY ? 0.0f : fast_exp(st[u][c][i] - base);
          psum += p[i];
        }
        *reinterpret_cast<u32x2*>(pw + (16 * c + n) * SK_PSTRIDE + 16 * (U * wv + u) + 4 * g) = (u32x2){pack_bf16x2(p[0], p[1]), pack_bf16x2(p[2], p[3])};
        psum = across_groups_sum(psum);
        if (g == 0) red_sum[U * wv + u][16 * c + n] = psum;
      }
    }
    __syncthreads();
    float c1[QT], c2[QT], lp = 0.0f;
    u32x4 pf[4][QT];
#pragma unroll
    for (int c = 0; c < QT; ++c) {
      lp = red_sum[0][16 * c + n];
#pragma unroll
      for (int k = 1; k < KT; ++k) lp += red_sum[k][16 * c + n];
      fold_piece(m[c], l[c], mp[c], lp, c1[c], c2[c]);
#pragma unroll
      for (int sg = 0; sg < 4; ++sg) pf[sg][c] = *reinterpret_cast<const u32x4*>(pw + (16 * c + n) * SK_PSTRIDE + 32 * sg + 8 * g);
    }

    // ---- the weighted sum of the values: a chain over the piece's keys for every block of 16 elements, then the fold
    const bool ragged = k0 + SK_PIECE - 1 > pmax || k0 < lo_first;       // slots outside may hold anything
#pragma unroll
    for (int j = 0; j < NDT; ++j) {
      u32x4 v[4];
#pragma unroll
      for (int sg = 0; sg < 4; ++sg) {
        v[sg] = vf[j % AHEAD][sg];
        if (j + AHEAD < NDT) vf[j % AHEAD][sg] = load_values(sg, j + AHEAD);
      }
      if (ragged) {                                          // (scalar)
#pragma unroll
        for (int sg = 0; sg < 4; ++sg)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int key = k0 + 32 * sg + 8 * g + 2 * e;
            v[sg][e] &= (key <= pmax && key >= lo_first ? 0xffffu : 0u) | (key + 1 <= pmax && key + 1 >= lo_first ? 0xffff0000u : 0u);
          }
      }
#pragma unroll
      for (int c = 0; c < QT; ++c) {
        {
          f32x4 pv = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int sg = 0; sg < 4; ++sg) pv = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(v[sg]), as_bf16x8(pf[sg][c]), pv, 0, 0, 0);
          if constexpr (PIECES) {
            acc[j][c] = pv;
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[j][c][i] = fmaf(pv[i], c2[c], acc[j][c][i] * c1[c]);
            // (the fold happens here: put off to the end of the piece, every block's sums would be held twice)
            asm volatile("" : "+v"(acc[j][c]));
          }
        }
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    if constexpr (PIECES) {
      if (qpos[0] < 0) return;
      const size_t at = ((size_t)t * a.heads + h0 + n % a.hg) * a.max_pieces + blockIdx.z;
      if (wv == 0 && g == 0) {
        a.partial_ml[2 * at] = mp[0];
        a.partial_ml[2 * at + 1] = lp;
      }
      float* part = a.partial + at * dv;
#pragma unroll
      for (int j = 0; j < NDT; ++j) {
        const int d = 16 * (NW * j + wv) + 4 * g;
        if ((dv & 3) == 0) {
          if (d < dv) *reinterpret_cast<f32x4*>(part + d) = acc[j][0];
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (d + i < dv) part[d + i] = acc[j][0][i];
        }
      }
      return;
    }
  }
  if constexpr (!PIECES) {
#pragma unroll
    for (int c = 0; c < QT; ++c) {
      if (qpos[c] < 0) continue;
      const int qn = 16 * c + n, rl = qn / a.hg, h = h0 + qn % a.hg;
      const float w = finish_softmax(m[c], l[c], a.sink != nullptr ? a.sink[h] : -INFINITY);
      const size_t at = (size_t)(r0 + rl) * a.ldo + h * dv;
#pragma unroll
      for (int j = 0; j < NDT; ++j) {
        const int d = 16 * (NW * j + wv) + 4 * g;
        if (a.out_is_bf16 && (dv & 3) == 0 && (a.ldo & 3) == 0) {
          if (d < dv)
            *reinterpret_cast<u32x2*>(reinterpret_cast<bf16_t*>(a.out) + at + d) =
                (u32x2){pack_bf16x2(acc[j][c][0] * w, acc[j][c][1] * w), pack_bf16x2(acc[j][c][2] * w, acc[j][c][3] * w)};
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (d + i < dv) store_out(a, at + d + i, acc[j][c][i] * w);
        }
      }
    }
  }
}

// The pieces of one (single-row tile, head) folded in order, a thread a value element.
__global__ __launch_bounds__(256) void shared_key_combine_kernel(MfmaAttnArgs a) {
  const int t = blockIdx.x, h = blockIdx.y;
  const int r0 = a.tiles != nullptr ? a.tiles[4 * t] : t;
  if (a.tiles != nullptr && a.tiles[4 * t + 1] <= 0) return;
  const int pos = a.positions[r0];
  if (pos < 0) return;
  const int d = blockIdx.z * 256 + threadIdx.x;
  if (d >= a.dv) return;
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int np = pos / SK_PIECE - lo / SK_PIECE + 1;
  const size_t at = ((size_t)t * a.heads + h) * a.max_pieces;
  const float* ml = a.partial_ml + 2 * at;
  const float* part = a.partial + at * a.dv + d;
  float m = -INFINITY, l = 0.0f, o = 0.0f;
  constexpr int UN = 8;
  for (int p0 = 0; p0 < np; p0 += UN) {
    float pv[UN], pm[UN], pl[UN];
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int p = min(p0 + u, np - 1);
      pv[u] = part[(size_t)p * a.dv];
      pm[u] = ml[2 * p];
      pl[u] = ml[2 * p + 1];
    }
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      if (p0 + u < np) {
        float c1, c2;
        fold_piece(m, l, pm[u], pl[u], c1, c2);
        o = fmaf(pv[u], c2, o * c1);
      }
    }
  }
  store_out(a, (size_t)r0 * a.ldo + h * a.dv + d, o * finish_softmax(m, l, a.sink != nullptr ? a.sink[h] : -INFINITY));
}

template <int QT, int NW, int NDT>
int launch_shared_key_mfma_shape(const MfmaAttnArgs& a, const bf16_t* kc, const bf16_t* vt, int num_tiles, hipStream_t s) {
  const int dkp = (a.dk + 31) & ~31;
  const size_t bytes = (size_t)16 * QT * (dkp + 8 + SK_PSTRIDE) * sizeof(bf16_t);
  static bool allowed = false;
  if (!allowed) {
    if (hipFuncSetAttribute((const void*)shared_key_attention_mfma_kernel<QT, NW, NDT>, hipFuncAttributeMaxDynamicSharedMemorySize,
                            150 * 1024) != hipSuccess)
      return -8;
    allowed = true;
  }
  if (bytes > 150 * 1024) return -8;
  const dim3 grid(num_tiles, (a.heads + a.hg - 1) / a.hg, QT == 1 ? a.max_pieces : 1);
  hipLaunchKernelGGL((shared_key_attention_mfma_kernel<QT, NW, NDT>), grid, dim3(64 * NW), bytes, s, a, kc, vt);
  return BW_LAUNCH_CHECK();
}

template <int QT>
int launch_shared_key_mfma(const MfmaAttnArgs& a, const bf16_t* kc, const bf16_t* vt, int num_tiles, hipStream_t s) {
  constexpr int NW = 4;
  const int per_wave = (a.dv + 16 * NW - 1) / (16 * NW);     // blocks of 16 value elements a wave
  if (per_wave <= 1) return launch_shared_key_mfma_shape<QT, NW, 1>(a, kc, vt, num_tiles, s);
  if (per_wave <= 2) return launch_shared_key_mfma_shape<QT, NW, 2>(a, kc, vt, num_tiles, s);
  if (per_wave <= 4) return launch_shared_key_mfma_shape<QT, NW, 4>(a, kc, vt, num_tiles, s);
  if (per_wave <= 8) return launch_shared_key_mfma_shape<QT, NW, 8>(a, kc, vt, num_tiles, s);
  return -4;
}

}  // namespace

extern "C" int bw_latent_prep(const float* proj, int ldp, int q_off, int dkv_off, const float* norm_w, float eps,
                              const float* cos_table, const float* sin_table, const int32_t* positions,
                              const int32_t* row_seq, const int32_t* block_table, int table_stride, void* cache,
                              void* latent_t, int cache_is_bf16, void* qa, int qa_is_bf16, int ldqa, int rows, int heads, int dim, int rot, int rotary,
                              int rank, int page_size, int write_cache, int pairs, int q_rank,
                              const float* q_norm_w, void* cq, int cq_is_bf16, int ldcq, void* stream) {
  if (rows <= 0) return 0;
  if (heads <= 0 || dim < 0 || rot < 0 || rotary < 0 || rotary > rot || (rotary & 1) || rank <= 0 || page_size <= 0) return -2;
  if (q_rank < 0 || (q_rank > 0 ? (cq == nullptr || q_norm_w == nullptr || ldcq < q_rank) : ldqa < heads * (rank + rot))) return -2;
  PrepArgs a{proj, ldp, q_off, dkv_off, norm_w, eps, cos_table, sin_table, positions, row_seq, block_table, table_stride,
             qa, ldqa, qa_is_bf16, heads, dim, rot, rotary, rank, page_size, write_cache, pairs, q_rank, q_norm_w, cq, ldcq, cq_is_bf16};
  hipStream_t s = (hipStream_t)stream;
  if (cache_is_bf16) hipLaunchKernelGGL(latent_prep_kernel<bf16_t>, dim3(rows), dim3(256), 0, s, a, (bf16_t*)cache, (bf16_t*)latent_t);
  else hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(rows), dim3(256), 0, s, a, (float*)cache, (float*)latent_t);
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_headwise_linear(const float* x, int ldx, int xhs, const void* wt, int w_is_bf16, int in, int outn,
                                  void* out, int out_is_bf16, int ldo, int ohs, int rows, int heads, const float* gate, int ldg,
                                  int rot_n, int rotary, int pairs, int rot_src, int rot_dst, const float* cos_table,
                                  const float* sin_table, const int32_t* positions, void* stream) {
  if (rows <= 0 || heads <= 0 || outn <= 0) return 0;
  if (in <= 0 || (size_t)HL_ROWS * in * sizeof(float) > 48 * 1024) return -2;
  if (gate != nullptr && ldg < heads) return -2;
  if (rot_n < 0 || (rot_n > 0 && (rotary < 0 || rotary > rot_n || (rotary & 1) || positions == nullptr ||
                                  (rotary > 0 && (cos_table == nullptr || sin_table == nullptr)))))
    return -2;
  const HeadExtras ex{gate, ldg, rot_n, rotary, pairs, rot_src, rot_dst, cos_table, sin_table, positions};
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((rows + HL_ROWS - 1) / HL_ROWS, heads, (outn + 63) / 64 + (rot_n > 0 ? 1 : 0)), block(256);
  const size_t bytes = (size_t)HL_ROWS * (in + 4 * 64) * sizeof(float);
#define BW_HL_LAUNCH(WT, OT) \
  hipLaunchKernelGGL((headwise_linear_kernel<WT, OT>), grid, block, bytes, s, x, ldx, xhs, (const WT*)wt, in, outn, (OT*)out, ldo, ohs, rows, ex)
  if (w_is_bf16) {
    if (out_is_bf16) BW_HL_LAUNCH(bf16_t, bf16_t);
    else BW_HL_LAUNCH(bf16_t, float);
  } else {
    if (out_is_bf16) BW_HL_LAUNCH(float, bf16_t);
    else BW_HL_LAUNCH(float, float);
  }
#undef BW_HL_LAUNCH
  return BW_LAUNCH_CHECK();
}

extern "C" int bw_shared_key_attention(const float* q, int ldq, const int32_t* positions, const int32_t* block_table,
                                       int table_stride, const int32_t* tiles, int num_tiles, const void* cache,
                                       int cache_is_bf16, int num_pages, const float* sink, float* out, int ldo, int heads,
                                       int dk, int dv, int page_size, int window, float scale, int heads_per_group,
                                       void* stream) {
  if (num_tiles <= 0) return 0;
  if (heads <= 0 || dk <= 0 || dv <= 0 || dv > dk || page_size <= 0 || num_pages <= 0) return -2;
  if (heads_per_group != 4 && heads_per_group != 16) return -2;
  if (ldq < heads * dk || ldo < heads * dv) return -2;
  SharedKeyArgs a{q, ldq, positions, block_table, table_stride, tiles, sink, out, ldo, heads, dk, dv, page_size, window,
                  heads_per_group, num_pages, scale};
  hipStream_t s = (hipStream_t)stream;
  if (cache_is_bf16) return launch_shared_key<bf16_t>(a, (const bf16_t*)cache, num_tiles, s);
  return launch_shared_key<float>(a, (const float*)cache, num_tiles, s);
}

// The product per head on the matrix cores: weights [heads][outn][in] bfloat16, in a multiple of 8; x 32-bit (16-byte aligned
// rows and heads) or bfloat16 (likewise).
extern "C" int bw_headwise_linear_mfma(const void* x, int x_is_bf16, int ldx, int xhs, const void* w, int in, int outn, void* out,
                                       int out_is_bf16, int ldo, int ohs, int rows, int heads, const float* gate, int ldg, int rot_n,
                                       int rotary, int pairs, int rot_src, int rot_dst, const float* cos_table, const float* sin_table,
                                       const int32_t* positions, void* stream) {
  if (rows <= 0 || heads <= 0 || outn <= 0) return 0;
  if (in < 8 || in % 8 || ((long long)rows / 16 + 1) * heads * ((outn + 63) / 64 + 1) > 0x3fffffffLL) return -2;
  const int unit = x_is_bf16 ? 8 : 4;
  if (ldx % unit || xhs % unit || (reinterpret_cast<uintptr_t>(x) & 15) || (reinterpret_cast<uintptr_t>(w) & 15)) return -3;
  if (gate != nullptr && ldg < heads) return -2;
  if (rot_n < 0 || (rot_n > 0 && (x_is_bf16 || rotary < 0 || rotary > rot_n || (rotary & 1) || positions == nullptr ||
                                  (rotary > 0 && (cos_table == nullptr || sin_table == nullptr)))))
    return -2;
  const uintptr_t mask = out_is_bf16 ? 7 : 15;
  int aligned = outn % 4 == 0 && ldo % 4 == 0 && ohs % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & mask) == 0;
  if (aligned && outn % 8 == 0 && ldo % 8 == 0 && ohs % 8 == 0 && (reinterpret_cast<uintptr_t>(out) & 15) == 0) aligned = 2;
  const HeadGemmArgs a{x, ldx, xhs, (const bf16_t*)w, in, outn, out, ldo, ohs, rows, heads, (outn + 63) / 64 + (rot_n > 0 ? 1 : 0), aligned};
  const HeadExtras ex{gate, ldg, rot_n, rotary, pairs, rot_src, rot_dst, cos_table, sin_table, positions};
  hipStream_t s = (hipStream_t)stream;
  if (x_is_bf16) return out_is_bf16 ? launch_headwise_mfma<bf16_t, bf16_t>(a, ex, s) : launch_headwise_mfma<bf16_t, float>(a, ex, s);
  return out_is_bf16 ? launch_headwise_mfma<float, bf16_t>(a, ex, s) : launch_headwise_mfma<float, float>(a, ex, s);
}

extern "C" int bw_shared_key_piece() { return SK_PIECE; }

// The matrix-core route: bfloat16 cache with key vectors of a multiple of 8 elements, pages of 8 slots or a larger power of two, and the
// transposed latents beside it.  Prompt tiles (max_pieces 0): up to SK_TILE_QUERIES / heads_per_group rows.  Single tokens (max_pieces > 0:
// tiles of one row, 16 heads a group): ``partial`` holds tiles * heads * max_pieces * (dv + 2) floats, max_pieces covers the
// pieces of SK_PIECE keys that a token's window, or its whole context, can touch.
extern "C" int bw_shared_key_attention_mfma(const void* q, int ldq, const int32_t* positions, const int32_t* block_table,
                                            int table_stride, const int32_t* tiles, int num_tiles, const void* cache,
                                            const void* latent_t, int num_pages, const float* sink, void* out, int out_is_bf16,
                                            int ldo, int heads, int dk, int dv, int page_size, int window, float scale,
                                            int heads_per_group, int max_pieces, float* partial, long long partial_floats,
                                            void* stream) {
  if (num_tiles <= 0) return 0;
  if (heads <= 0 || dk <= 0 || (dk % 8) || dv <= 0 || dv > dk || dv > 512 || page_size < 8 || (page_size & (page_size - 1)) || num_pages <= 0) return -2;
  if (heads_per_group < 1 || heads_per_group > 16 || (16 % heads_per_group)) return -2;
  if (ldq < heads * dk || (ldq % 8) || ldo < heads * dv || max_pieces < 0 || max_pieces > 65535) return -2;
  if (reinterpret_cast<uintptr_t>(q) & 15) return -3;
  if ((reinterpret_cast<uintptr_t>(cache) & 15) || (reinterpret_cast<uintptr_t>(latent_t) & 15)) return -3;
  const long long pieces = (long long)num_tiles * heads * max_pieces;
  if (max_pieces > 0) {
    if (heads_per_group != 16 || partial == nullptr || (reinterpret_cast<uintptr_t>(partial) & 15)) return -2;
    // (what a block table can name; a window touches at most one piece more than it fills)
    const long long span = ((long long)table_stride * page_size + SK_PIECE - 1) / SK_PIECE;
    const long long in_window = window > 0 ? ((long long)window + SK_PIECE - 2) / SK_PIECE + 1 : span;
    if (max_pieces < (span < in_window ? span : in_window)) return -2;
    if (partial_floats < pieces * (dv + 2)) return -6;
  }
  MfmaAttnArgs a{(const bf16_t*)q, ldq, positions, block_table, table_stride, tiles, sink, out, ldo, out_is_bf16, partial,
                 partial == nullptr ? nullptr : partial + pieces * dv, heads, dk, dv, page_size, window, heads_per_group, num_pages,
                 max_pieces, scale};
  hipStream_t s = (hipStream_t)stream;
  if (max_pieces == 0) return launch_shared_key_mfma<SK_TILE_QUERIES / 16>(a, (const bf16_t*)cache, (const bf16_t*)latent_t, num_tiles, s);
  const int rc = launch_shared_key_mfma<1>(a, (const bf16_t*)cache, (const bf16_t*)latent_t, num_tiles, s);
  if (rc != 0) return rc;
  hipLaunchKernelGGL(shared_key_combine_kernel, dim3(num_tiles, heads, (dv + 255) / 256), dim3(256), 0, s, a);
  return BW_LAUNCH_CHECK();
}
