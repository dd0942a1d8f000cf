// Linear recurrence with one decay per head and token, on an fp32 state S [dim, vdim] per head:
//   S <- e^g S + w k v^T;   o = S^T q + skip v
// g and w come from a step size (w = softplus(dt + dt_bias), g = -exp(a_log) w: a state-space layer whose
// heads share queries and keys by group), are constant (g = log_decay[head], w = 1) or are given per row
// (a matrix memory with exponential gates: matrix_memory_gates forms them).  q, k and v may pass an
// activation on their way in; q may be scaled.
//
// Normalizer (a matrix memory): beside S a vector n [dim] runs through the same recurrence with the value
// 1 -- its product with the query is the row sum of P plus the part of the block's start, so it costs no
// product -- and the scan leaves 1 / (max(|n . q|, floor) + eps) per (token, head) for whoever reads o.
// A head's state is then S followed by n.
//
// matrix_memory_gates: log input gate i = cap tanh((zi + bi) / cap), log forget gate
// f = -softplus(-cap tanh((zf + bf) / cap)), running maximum m_t = max(f + m_(t-1), i) from 0 on; what
// the scan needs is g = f + m_(t-1) - m_t <= 0, w = e^(i - m_t) <= 1 and the floor e^(-m_t).  S and n are
// scaled by e^(-m_t), so any rounding of m cancels as long as g, w and the floor come from the same
// numbers.  m -> max(a + m, b) composes, so a workgroup scans its rows in log steps.
//
// Blocks of 64 rows (runs of more than a few rows).  With c_i the sum of g over a block's rows 0 .. i,
//   o_i = e^(c_i) S^T q_i + sum_(j <= i) e^(c_i - c_j) w_j (q_i . k_j) v_j + skip v_i
//   S  <- e^(c_last) S + sum_j e^(c_last - c_j) w_j k_j v_j^T
// are three matrix products per block around the products P = Q K^T; every exponent is a sum of
// g <= 0, so nothing overflows; c is summed in fp64 and kept as two fp32 numbers, so that differences of
// large sums stay exact to fp32.  All of it runs on fp32 matrix cores (16x16x4): nothing is rounded
// below fp32 after it has been read.  Layout, lane = (g, c) = (lane >> 4, lane & 15):
//   A operand  lane: row c, contraction index g       B operand  lane: column c, contraction index g
//   result     lane: column c, rows 4 g .. 4 g + 3
// The contraction index is a free relabelling, so element i of a 16-byte read at 16 kb + 4 g serves as
// step i of block kb, and what a lane holds of a result with rows 16 db + 4 g + i is the B operand of
// that step: a wave keeps S of its value columns in registers as a result and uses it as an operand
// where it lies.  A workgroup walks one run (or piece of a run) of one head for 64 or 128 value
// columns, 16 per wave; rows come one block ahead through registers into LDS.  bfloat16 queries and
// keys without an activation stay bfloat16 there (half the LDS: two workgroups per CU) and P comes from
// the bfloat16 products, which are exact in fp32 as well; everything else sees them as fp32.
//
// Long runs are cut into pieces of VLA_DECAY_SCAN_PIECE rows: (1) every piece but the last forms the
// state its own rows leave from a zero state; (2) a chain over a sequence's pieces turns these
// into the state every piece starts from; (3) all pieces walk at once from their start states.
//
// Steps of a few rows (decoding) go token by token: a workgroup per (head, sequence) reads and
// writes the state once per token, coalesced along vdim.
//
// gated_group_rms_norm: what follows such a recurrence, per token: gate and RMS norm over equal
// parts of the concatenated heads.
#include <atomic>
#include <type_traits>

#include "seq_common.h"

namespace vla {
namespace seq {
namespace {

constexpr int kBlock = 64;
constexpr int kStepRows = 4;
constexpr int kMaxBlockDim = 128;   // largest dim the block kernels take
std::atomic<int> g_decay_kernel{0};

__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
// for values that were read as 16-bit numbers: hardware exponential and reciprocal, a few 1e-7 off
__device__ __forceinline__ float silu_fast(float z) {
  return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

struct DecayScan {
  float* o;
  const void* q;
  int64_t q_stride;
  const void* k;
  int64_t k_stride;
  const void* v;
  int64_t v_stride;
  const void* dt;
  int64_t dt_stride;
  const float* dt_bias;
  const float* a_log;
  const float* log_decay;
  const float* skip;
  const float* row_log;       // [T][heads]: g per row
  const float* row_weight;    // [T][heads]: w per row
  const float* row_floor;     // [T][heads]
  float* norm_scale;          // [T][heads]; null: no normalizer
  float norm_eps, q_scale;
  int64_t head_size;          // state numbers per head: dim * vdim, plus dim with a normalizer
  float* state;
  float* piece_state;     // [piece slots][heads][head_size]
  float* piece_decay;     // [piece slots][heads]
  const int* query_start_loc;
  const int* context_lens;
  const int* state_slots;
  int num_seqs, heads, groups, dim, vdim, act, dtype, mode;
  int piece_rows;         // 0: runs are not cut
  bool vec_q, vec_k, vec_v;
};

__device__ __forceinline__ float load_one(const void* p, int64_t i, int dtype) {
  if (dtype == VLA_BF16) return BF16::to_f32(((const __bf16*)p)[i]);
  if (dtype == VLA_F16) return F16::to_f32(((const _Float16*)p)[i]);
  return ((const float*)p)[i];
}

// what a row's decay comes from: its step size's projection, or its log decay and weight
struct RowDecay {
  float dt = 0.f, weight = 0.f;
};
__device__ __forceinline__ RowDecay load_decay(const DecayScan& a, int64_t t, int h) {
  RowDecay r;
  if (a.row_log != nullptr) {
    r.dt = a.row_log[t * a.heads + h];
    r.weight = a.row_weight[t * a.heads + h];
  } else if (a.dt != nullptr) {
    r.dt = load_one(a.dt, t * a.dt_stride + h, a.dtype);
  }
  return r;
}

// the log decay and the input's factor of a row
__device__ __forceinline__ void row_decay(const DecayScan& a, const RowDecay& r, int h, float& g, float& w) {
  if (a.row_log != nullptr) {
    w = r.weight;
    g = fminf(r.dt, 0.f);
  } else if (a.dt != nullptr) {
    w = softplus_f(r.dt + a.dt_bias[h]);
    g = -expf(a.a_log[h]) * w;
  } else {
    w = 1.f;
    g = a.log_decay[h];
  }
}

// eight consecutive values as they lie in memory
template <bool W16>
struct Piece;
template <>
struct Piece<true> {
  u32x4 x;
};
template <>
struct Piece<false> {
  f32x4 x, y;
};

// values first .. first + 7 of a row; with vec, width is a multiple of eight and a piece behind the row's
// end reads its first piece instead (the reader of the pieces masks it), so that no load waits for
// another's branch; otherwise columns from `width` on are zeros
template <bool W16>
__device__ __forceinline__ Piece<W16> read_piece(const void* base, int64_t at, int first, int width, bool vec) {
  Piece<W16> p;
  if (vec) first = first < width ? first : 0;
  if constexpr (W16) {
    const uint16_t* src = (const uint16_t*)base + at + first;
    if (vec) {
      p.x = *reinterpret_cast<const u32x4*>(src);
    } else {
      p.x = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (first + e < width) p.x[e >> 1] |= (uint32_t)src[e] << (16 * (e & 1));
    }
  } else {
    const float* src = (const float*)base + at + first;
    if (vec) {
      p.x = *reinterpret_cast<const f32x4*>(src);
      p.y = *reinterpret_cast<const f32x4*>(src + 4);
    } else {
      p.x = p.y = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (first + e < width) p.x[e] = src[e];
        if (first + 4 + e < width) p.y[e] = src[4 + e];
      }
    }
  }
  return p;
}

template <bool W16>
__device__ __forceinline__ void mask_piece(Piece<W16>& p, bool live) {
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    if constexpr (W16) {
      p.x[e] = live ? p.x[e] : 0u;
    } else {
      p.x[e] = live ? p.x[e] : 0.f;
      p.y[e] = live ? p.y[e] : 0.f;
    }
  }
}

// a piece's values in fp32 after the activation, to LDS (16-byte aligned)
template <bool W16>
__device__ __forceinline__ void land_piece(float* dst, const Piece<W16>& p, int act, int dtype) {
  f32x4 lo, hi;
  if constexpr (W16) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float a, b;
      if (dtype == VLA_BF16) {
        a = __builtin_bit_cast(float, p.x[e] << 16);
        b = __builtin_bit_cast(float, p.x[e] & 0xffff0000u);
      } else {
        a = lo16<F16>(p.x[e]);
        b = hi16<F16>(p.x[e]);
      }
      if (act == VLA_ACT_SILU) {
        a = silu_fast(a);
        b = silu_fast(b);
      }
      (e < 2 ? lo : hi)[2 * (e & 1)] = a;
      (e < 2 ? lo : hi)[2 * (e & 1) + 1] = b;
    }
  } else {
    lo = p.x;
    hi = p.y;
    if (act == VLA_ACT_SILU) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        lo[e] = silu_f(lo[e]);
        hi[e] = silu_f(hi[e]);
      }
    }
  }
  *reinterpret_cast<f32x4*>(dst) = lo;
  *reinterpret_cast<f32x4*>(dst + 4) = hi;
}

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// Which sequence and piece a piece slot is: sequence b's pieces are slots start_b / R + b + 0, 1, ...
// (enough for ceil(n / R) of them; slots behind a sequence's last piece stay empty).
__device__ __forceinline__ bool find_piece(const DecayScan& a, int z, int& b, int& piece) {
  if (a.piece_rows == 0) {
    b = z;
    piece = 0;
    return z < a.num_seqs;
  }
  int lo = 0, hi = a.num_seqs - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (a.query_start_loc[mid] / a.piece_rows + mid <= z)
      lo = mid;
    else
      hi = mid - 1;
  }
  b = lo;
  piece = z - (a.query_start_loc[b] / a.piece_rows + b);
  return piece >= 0 && (int64_t)piece * a.piece_rows < a.query_start_loc[b + 1] - a.query_start_loc[b];
}

// How a block kernel reads and keeps its rows
enum RowKind {
  kRowsF32,      // fp32 in memory and in LDS
  kRows16,       // 16-bit in memory, fp32 in LDS (after the activation)
  kRowsBf16      // queries and keys bfloat16 in LDS too (no activation)
};

template <int DB, int WAVES, RowKind KIND, bool STATE_ONLY>
constexpr size_t block_lds_floats() {
  constexpr int DP = 16 * DB, QK = KIND == kRowsBf16 ? (DP + 8) / 2 : DP + 4;     // floats per query / key row
  return (size_t)kBlock * ((STATE_ONLY ? 1 : 2) * QK + (16 * WAVES + 4) + (STATE_ONLY ? 0 : kBlock + 4)) + 5 * kBlock +
         2 * DP;
}

template <int DB, int WAVES, RowKind KIND, bool STATE_ONLY>
__global__ __launch_bounds__(64 * WAVES) void decay_block_kernel(DecayScan a) {
  constexpr bool W16 = KIND != kRowsF32, QK16 = KIND == kRowsBf16;
  constexpr int THREADS = 64 * WAVES;
  constexpr int DP = 16 * DB, KR = QK16 ? DP + 8 : DP + 4;      // elements of a query / key row
  constexpr int QK_FLOATS = QK16 ? KR / 2 : KR;
  constexpr int VB = 16 * WAVES, VR = VB + 4, PR = kBlock + 4;
  constexpr int NQ = (DP * kBlock / 8 + THREADS - 1) / THREADS;         // pieces of eight values per thread
  constexpr int NVP = VB * kBlock / 8 / THREADS;
  using E = typename std::conditional<QK16, uint16_t, float>::type;
  extern __shared__ __align__(16) float lds[];
  E* k_lds = reinterpret_cast<E*>(lds);                 // [64][KR]
  float* v_lds = lds + kBlock * QK_FLOATS;              // [64][VR]
  float* num = v_lds + kBlock * VR;                     // c | w | e^c | e^(c_last - c) w | c's low part
  float* n_lds = num + 5 * kBlock;                      // [2][DP] the normalizer, before / after a block
  E* q_lds = reinterpret_cast<E*>(n_lds + 2 * DP);      // [64][KR]
  float* p_lds = n_lds + 2 * DP + kBlock * QK_FLOATS;   // [64][PR]
  const int h = blockIdx.x, v0 = blockIdx.y * VB, z = blockIdx.z;
  int b, piece;
  if (!find_piece(a, z, b, piece)) return;
  const int run = a.query_start_loc[b + 1] - a.query_start_loc[b];
  if (a.mode == 0 && run <= kStepRows) return;          // the step kernel's
  const bool cut = a.piece_rows > 0 && run > a.piece_rows;
  const int first = piece * a.piece_rows;               // 0 when runs are not cut
  const bool last = !cut || first + a.piece_rows >= run;
  if (STATE_ONLY && last) return;
  const int t_begin = a.query_start_loc[b] + first, t_end = last ? a.query_start_loc[b + 1] : t_begin + a.piece_rows;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15;
  const int D = a.dim, V = a.vdim, hg = h / (a.heads / a.groups);
  const int v_mine = v0 + 16 * w + c;                   // this lane's value column
  const int64_t state_size = a.head_size;
  const bool normed = a.norm_scale != nullptr && blockIdx.y == 0;   // one workgroup of a head keeps n
  const float* from = nullptr;
  if (!STATE_ONLY) {
    if (cut)
      from = a.piece_state + ((int64_t)z * a.heads + h) * state_size;
    else if (a.context_lens[b] > 0)
      from = a.state + ((int64_t)a.state_slots[b] * a.heads + h) * state_size;
  }
  f32x4 s[DB];
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * db + 4 * g + r;
      s[db][r] = from != nullptr && d < D && v_mine < V ? from[(int64_t)d * V + v_mine] : 0.f;
    }
  if (normed)
    for (int d = tid; d < DP; d += THREADS) n_lds[d] = from != nullptr && d < D ? from[(int64_t)D * V + d] : 0.f;
  int n_at = 0;
  const float skip = a.skip != nullptr && !STATE_ONLY ? a.skip[h] : 0.f, q_scale = a.q_scale;
  double log_total = 0.0;

  Piece<W16> pq[NQ], pk[NQ], pv[NVP];
  RowDecay row_next;
  auto fetch = [&](int t0) {
    const int n = min(kBlock, t_end - t0);
#pragma unroll
    for (int u = 0; u < NQ; ++u) {
      const int i = tid + THREADS * u, r = i / (DP / 8), d = 8 * (i % (DP / 8));
      const int64_t t = t0 + min(r, n - 1);
      pk[u] = read_piece<W16>(a.k, t * a.k_stride + (int64_t)hg * D, d, D, a.vec_k);
      if (!STATE_ONLY) pq[u] = read_piece<W16>(a.q, t * a.q_stride + (int64_t)hg * D, d, D, a.vec_q);
    }
#pragma unroll
    for (int u = 0; u < NVP; ++u) {
      const int i = tid + THREADS * u, r = i / (VB / 8), d = v0 + 8 * (i % (VB / 8));
      pv[u] = read_piece<W16>(a.v, (int64_t)(t0 + min(r, n - 1)) * a.v_stride + (int64_t)h * V, d, V, a.vec_v);
    }
    if (tid < kBlock) row_next = load_decay(a, t0 + min(tid, n - 1), h);
  };
  auto land_qk = [&](E* dst, Piece<W16>& p, bool live) {
    mask_piece<W16>(p, live);
    if constexpr (QK16)
      *reinterpret_cast<u32x4*>(dst) = p.x;
    else
      land_piece<W16>(dst, p, a.act, a.dtype);
  };
  auto land = [&](int n) {
    if (w == 0) {
      float row_g = 0.f, row_w = 0.f;
      if (lane < n) row_decay(a, row_next, h, row_g, row_w);
      double cs = row_g;                                // inclusive sum over the 64 rows
#pragma unroll
      for (int m = 1; m < 64; m <<= 1) {
        const double other = __shfl_up(cs, m, 64);
        cs += lane >= m ? other : 0.0;
      }
      const double end = __shfl(cs, 63, 64);
      num[lane] = (float)cs;
      num[kBlock + lane] = row_w;
      num[2 * kBlock + lane] = expf((float)cs);
      num[3 * kBlock + lane] = expf(fminf((float)(end - cs), 0.f)) * row_w;
      num[4 * kBlock + lane] = (float)(cs - (double)(float)cs);
    }
#pragma unroll
    for (int u = 0; u < NQ; ++u) {
      const int i = tid + THREADS * u, r = i / (DP / 8), d = 8 * (i % (DP / 8));
      if (DP * kBlock / 8 % THREADS != 0 && r >= kBlock) continue;
      land_qk(k_lds + r * KR + d, pk[u], r < n && d < D);
      if (!STATE_ONLY) land_qk(q_lds + r * KR + d, pq[u], r < n && d < D);
    }
#pragma unroll
    for (int u = 0; u < NVP; ++u) {
      const int i = tid + THREADS * u, r = i / (VB / 8), d = 8 * (i % (VB / 8));
      mask_piece<W16>(pv[u], r < n && v0 + d < V);
      land_piece<W16>(v_lds + r * VR + d, pv[u], a.act, a.dtype);
    }
  };
  // four consecutive values of a query / key row, and one, as fp32
  auto four = [&](const E* src) {
    if constexpr (QK16) {
      const u32x2 x = *reinterpret_cast<const u32x2*>(src);
      return f32x4{__builtin_bit_cast(float, x[0] << 16), __builtin_bit_cast(float, x[0] & 0xffff0000u),
                   __builtin_bit_cast(float, x[1] << 16), __builtin_bit_cast(float, x[1] & 0xffff0000u)};
    } else {
      return *reinterpret_cast<const f32x4*>(src);
    }
  };
  auto one = [&](const E* src) {
    if constexpr (QK16)
      return __builtin_bit_cast(float, (uint32_t)*src << 16);
    else
      return *src;
  };

  fetch(t_begin);
  for (int t0 = t_begin; t0 < t_end; t0 += kBlock) {
    const int n = min(kBlock, t_end - t0);
    land(n);
    __syncthreads();
    if (t0 + kBlock < t_end) fetch(t0 + kBlock);
    if constexpr (!STATE_ONLY) {
      // P_ij = (q_i . k_j) e^(c_i - c_j) w_j for j <= i: ten 16 x 16 tiles, dealt to the waves
      for (int ti = w; ti < 10; ti += WAVES) {
        const int ib = ti < 1 ? 0 : ti < 3 ? 1 : ti < 6 ? 2 : 3, jb = ti - ib * (ib + 1) / 2;
        if (16 * ib >= n) break;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if constexpr (QK16) {
#pragma unroll
          for (int kb = 0; kb < DP / 32; ++kb) {
            const u32x4 qa = *reinterpret_cast<const u32x4*>(q_lds + (16 * ib + c) * KR + 32 * kb + 8 * g);
            const u32x4 ka = *reinterpret_cast<const u32x4*>(k_lds + (16 * jb + c) * KR + 32 * kb + 8 * g);
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, qa), __builtin_bit_cast(bf16x8, ka),
                                                          acc, 0, 0, 0);
          }
        } else {
#pragma unroll
          for (int kb = 0; kb < DB; ++kb) {
            const f32x4 qa = four(q_lds + (16 * ib + c) * KR + 16 * kb + 4 * g);
            const f32x4 ka = four(k_lds + (16 * jb + c) * KR + 16 * kb + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = mfma4(qa[i], ka[i], acc);
          }
        }
        const int j = 16 * jb + c;
        const float cj = num[j], lj = num[4 * kBlock + j], wj = num[kBlock + j];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * ib + 4 * g + r;
          const float diff = fminf((num[i] - cj) + (num[4 * kBlock + i] - lj), 0.f);
          p_lds[i * PR + j] = j <= i ? acc[r] * (expf(diff) * wj * q_scale) : 0.f;
        }
      }
      __syncthreads();
      if (normed) {
        // n . q of every row: PARTS neighbouring threads share one
        constexpr int PARTS = THREADS / kBlock;
        const int i = tid / PARTS, part = tid % PARTS;
        float dot = 0.f, sum = 0.f;
        for (int d = 4 * part; d < DP; d += 4 * PARTS) {
          const f32x4 qv = four(q_lds + i * KR + d), nv = *reinterpret_cast<const f32x4*>(n_lds + n_at * DP + d);
#pragma unroll
          for (int e = 0; e < 4; ++e) dot += qv[e] * nv[e];
        }
        for (int j = part; j <= i; j += PARTS) sum += p_lds[i * PR + j];
        sum += dot * (num[2 * kBlock + i] * q_scale);
#pragma unroll
        for (int m = 1; m < PARTS; m <<= 1) sum += __shfl_xor(sum, m, 64);
        if (part == 0 && i < n) {
          const int64_t at = (int64_t)(t0 + i) * a.heads + h;
          a.norm_scale[at] = 1.f / (fmaxf(fabsf(sum), a.row_floor[at]) + a.norm_eps);
        }
      }
    }
    // this wave's value columns as B operands: rows 16 kb + 4 g + i
    float vf[4][4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int i = 0; i < 4; ++i) vf[kb][i] = v_lds[(16 * kb + 4 * g + i) * VR + 16 * w + c];
    if constexpr (!STATE_ONLY) {
#pragma unroll
      for (int rb = 0; rb < 4; ++rb) {
        if (16 * rb < n) {
          f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int db = 0; db < DB; ++db) {
            const f32x4 qa = four(q_lds + (16 * rb + c) * KR + 16 * db + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = mfma4(qa[i], s[db][i], acc);
          }
          const f32x4 ec = *reinterpret_cast<const f32x4*>(num + 2 * kBlock + 16 * rb + 4 * g);
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[r] = acc[r] * (ec[r] * q_scale) + skip * vf[rb][r];
#pragma unroll
          for (int kb = 0; kb <= rb; ++kb) {
            const f32x4 pa = *reinterpret_cast<const f32x4*>(p_lds + (16 * rb + c) * PR + 16 * kb + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = mfma4(pa[i], vf[kb][i], acc);
          }
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int i = 16 * rb + 4 * g + r;
            if (i < n && v_mine < V) a.o[((int64_t)(t0 + i) * a.heads + h) * V + v_mine] = acc[r];
          }
        }
      }
    }
    const float e_last = num[2 * kBlock + kBlock - 1];
    if (normed) {                                        // readers of the other half are behind the last barrier
      for (int d = tid; d < DP; d += THREADS) {
        float nv = e_last * n_lds[n_at * DP + d];
#pragma unroll 8
        for (int j = 0; j < kBlock; ++j) nv += num[3 * kBlock + j] * one(k_lds + j * KR + d);
        n_lds[(1 - n_at) * DP + d] = nv;
      }
      n_at = 1 - n_at;
    }
    log_total += (double)num[kBlock - 1] + (double)num[5 * kBlock - 1];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      const f32x4 tw = *reinterpret_cast<const f32x4*>(num + 3 * kBlock + 16 * kb + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) vf[kb][i] *= tw[i];
    }
#pragma unroll
    for (int db = 0; db < DB; ++db) {
#pragma unroll
      for (int r = 0; r < 4; ++r) s[db][r] *= e_last;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb) {
        if (16 * kb < n) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            s[db] = mfma4(one(k_lds + (16 * kb + 4 * g + i) * KR + 16 * db + c), vf[kb][i], s[db]);
        }
      }
    }
    __syncthreads();                                     // the block's rows are done with
  }
  float* to;
  if (STATE_ONLY) {
    to = a.piece_state + ((int64_t)z * a.heads + h) * state_size;
    if (tid == 0 && blockIdx.y == 0) a.piece_decay[(int64_t)z * a.heads + h] = expf((float)log_total);
  } else {
    if (!last) return;
    to = a.state + ((int64_t)a.state_slots[b] * a.heads + h) * state_size;
  }
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * db + 4 * g + r;
      if (d < D && v_mine < V) to[(int64_t)d * V + v_mine] = s[db][r];
    }
  if (normed)                                            // written before the last barrier
    for (int d = tid; d < D; d += THREADS) to[(int64_t)D * V + d] = n_lds[n_at * DP + d];
}

// Over one sequence's pieces: what piece i leaves from zero (in its slot) becomes what it starts from.
constexpr int kChainAhead = 8;
__global__ __launch_bounds__(256) void decay_chain_kernel(DecayScan a) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int run = a.query_start_loc[b + 1] - a.query_start_loc[b];
  if (run <= a.piece_rows) return;
  const int count = (run + a.piece_rows - 1) / a.piece_rows;
  const int z0 = a.query_start_loc[b] / a.piece_rows + b;
  const int64_t size = a.head_size;
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= size) return;
  float s = a.context_lens[b] > 0 ? a.state[((int64_t)a.state_slots[b] * a.heads + h) * size + e] : 0.f;
  const int64_t step = (int64_t)a.heads * size;
  float* at = a.piece_state + ((int64_t)z0 * a.heads + h) * size + e;
  const float* dec = a.piece_decay + (int64_t)z0 * a.heads + h;
  for (int i0 = 0; i0 < count; i0 += kChainAhead) {
    float left[kChainAhead], fac[kChainAhead];
#pragma unroll
    for (int i = 0; i < kChainAhead; ++i) {
      const bool has = i0 + i + 1 < count;               // the last piece leaves nothing here
      left[i] = has ? at[(int64_t)(i0 + i) * step] : 0.f;
      fac[i] = has ? dec[(int64_t)(i0 + i) * a.heads] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < kChainAhead; ++i) {
      if (i0 + i < count) {
        at[(int64_t)(i0 + i) * step] = s;
        s = fac[i] * s + left[i];
      }
    }
  }
}

// Token by token.  Thread (rg, cg) owns rows rg, rg + groups, ... of the VW columns from VW cg on.
template <int VW>
__global__ __launch_bounds__(256) void decay_step_kernel(DecayScan a) {
  extern __shared__ __align__(16) float lds[];
  const int h = blockIdx.x, b = blockIdx.y;
  const int t_begin = a.query_start_loc[b], t_end = a.query_start_loc[b + 1];
  if (a.mode == 0 && t_end - t_begin > kStepRows) return;
  const int D = a.dim, V = a.vdim, hg = h / (a.heads / a.groups);
  const int cols = (V + VW - 1) / VW, groups = 256 / cols;
  const int tid = threadIdx.x, cg = tid % cols, rg = tid / cols;
  const bool mine = rg < groups;
  float* q_lds = lds;                    // [D]
  float* k_lds = q_lds + D;              // [D]
  float* v_lds = k_lds + D;              // [V]
  float* part = v_lds + V;               // [groups][V]
  float* red = part + groups * V;        // [4]
  float* head = a.state + ((int64_t)a.state_slots[b] * a.heads + h) * a.head_size;
  float* st = head + VW * cg;
  float* n_st = head + (int64_t)D * V;
  const bool resume = a.context_lens[b] > 0;
  const float skip = a.skip != nullptr ? a.skip[h] : 0.f;
  auto load = [&](const void* p, int64_t i) {
    const float x = load_one(p, i, a.dtype);
    return a.act == VLA_ACT_SILU ? silu_f(x) : x;
  };
  for (int t = t_begin; t < t_end; ++t) {
    float g, wt;
    row_decay(a, load_decay(a, t, h), h, g, wt);
    const float e = expf(g);
    for (int d = tid; d < D; d += 256) {
      q_lds[d] = load(a.q, (int64_t)t * a.q_stride + (int64_t)hg * D + d) * a.q_scale;
      k_lds[d] = load(a.k, (int64_t)t * a.k_stride + (int64_t)hg * D + d);
    }
    for (int d = tid; d < V; d += 256) v_lds[d] = load(a.v, (int64_t)t * a.v_stride + (int64_t)h * V + d);
    __syncthreads();
    const bool zero = !resume && t == t_begin;
    if (a.norm_scale != nullptr) {
      float dot = 0.f;
      for (int d = tid; d < D; d += 256) {
        const float nv = (zero ? 0.f : e * n_st[d]) + wt * k_lds[d];
        n_st[d] = nv;
        dot += q_lds[d] * nv;
      }
      dot = wave_sum(dot);
      if ((tid & 63) == 0) red[tid >> 6] = dot;
    }
    float o[VW], wv[VW];
#pragma unroll
    for (int x = 0; x < VW; ++x) {
      o[x] = 0.f;
      wv[x] = mine ? wt * v_lds[VW * cg + x] : 0.f;
    }
    if (mine) {
      constexpr int U = 4;               // rows in flight
      for (int d0 = rg; d0 < D; d0 += U * groups) {
        float s[U][VW];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int d = d0 + u * groups;
          if constexpr (VW == 4) {
            f32x4 got = {0.f, 0.f, 0.f, 0.f};
            if (d < D && !zero) got = *reinterpret_cast<const f32x4*>(st + (int64_t)d * V);
#pragma unroll
            for (int x = 0; x < 4; ++x) s[u][x] = got[x];
          } else {
            s[u][0] = d < D && !zero ? st[(int64_t)d * V] : 0.f;
          }
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int d = d0 + u * groups;
          if (d < D) {
            const float kd = k_lds[d], qd = q_lds[d];
#pragma unroll
            for (int x = 0; x < VW; ++x) {
              s[u][x] = e * s[u][x] + kd * wv[x];
              o[x] += qd * s[u][x];
            }
            if constexpr (VW == 4)
              *reinterpret_cast<f32x4*>(st + (int64_t)d * V) = f32x4{s[u][0], s[u][1], s[u][2], s[u][3]};
            else
              st[(int64_t)d * V] = s[u][0];
          }
        }
      }
#pragma unroll
      for (int x = 0; x < VW; ++x) part[rg * V + VW * cg + x] = o[x];
    }
    __syncthreads();
    for (int v = tid; v < V; v += 256) {
      float sum = skip * v_lds[v];
      for (int r = 0; r < groups; ++r) sum += part[r * V + v];
      a.o[((int64_t)t * a.heads + h) * V + v] = sum;
    }
    if (a.norm_scale != nullptr && tid == 0) {
      const int64_t at = (int64_t)t * a.heads + h;
      a.norm_scale[at] = 1.f / (fmaxf(fabsf(red[0] + red[1] + red[2] + red[3]), a.row_floor[at]) + a.norm_eps);
    }
    __syncthreads();
  }
}

__device__ __forceinline__ float capped(float z, float cap) { return cap * tanhf(z / cap); }

// One workgroup per (head, sequence): each thread one row of a stretch of blockDim.x.
template <class S>
__global__ __launch_bounds__(1024) void matrix_memory_gates_kernel(
    float* __restrict__ row_log, float* __restrict__ row_weight, float* __restrict__ row_floor,
    const typename S::T* __restrict__ zi, int64_t zi_stride, const typename S::T* __restrict__ zf,
    int64_t zf_stride, const float* __restrict__ bias_i, const float* __restrict__ bias_f, float cap,
    float* __restrict__ maximum, const int* __restrict__ query_start_loc,
    const int* __restrict__ context_lens, const int* __restrict__ state_slots, int heads) {
  __shared__ double wave_a[16];
  __shared__ float wave_b[16];
  __shared__ float m_lds[1025];
  const int h = blockIdx.x, b = blockIdx.y;
  const int t_begin = query_start_loc[b], t_end = query_start_loc[b + 1];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  float* m_state = maximum + (int64_t)state_slots[b] * heads + h;
  float m0 = context_lens[b] > 0 ? *m_state : 0.f;      // every thread holds the maximum before the stretch
  for (int t0 = t_begin; t0 < t_end; t0 += blockDim.x) {
    const int t = t0 + tid, n = min((int)blockDim.x, t_end - t0);
    const bool live = tid < n;
    float i = -INFINITY, f = 0.f;                       // a row behind the end changes nothing
    if (live) {
      i = capped(S::to_f32(zi[(int64_t)t * zi_stride + h]) + bias_i[h], cap);
      const float c = capped(S::to_f32(zf[(int64_t)t * zf_stride + h]) + bias_f[h], cap);
      f = -(fmaxf(-c, 0.f) + log1pf(expf(-fabsf(c))));
    }
    double a = f;                                       // m -> max(a + m, best) over the rows so far
    float best = i;
#pragma unroll
    for (int s = 1; s < 64; s <<= 1) {
      const double oa = __shfl_up(a, s, 64);
      const float ob = __shfl_up(best, s, 64);
      if (lane >= s) {
        best = fmaxf((float)(a + (double)ob), best);
        a += oa;
      }
    }
    if (lane == 63) {
      wave_a[w] = a;
      wave_b[w] = best;
    }
    __syncthreads();
    float m_in = m0;
    for (int o = 0; o < w; ++o) m_in = fmaxf((float)(wave_a[o] + (double)m_in), wave_b[o]);
    const float m = fmaxf((float)(a + (double)m_in), best);
    m_lds[tid + 1] = m;
    if (tid == 0) m_lds[0] = m0;
    __syncthreads();
    if (live) {
      const int64_t at = (int64_t)t * heads + h;
      row_log[at] = (float)((double)f + (double)m_lds[tid] - (double)m);
      row_weight[at] = expf(i - m);
      row_floor[at] = expf(-m);
    }
    m0 = m_lds[n];
    __syncthreads();
  }
  if (tid == 0) *m_state = m0;
}

// Parts of up to 256 numbers, 16-byte aligned: LANES lanes share a part, four numbers each, and norm it
// with lane sums; 256 / LANES parts per workgroup.
template <class S, int LANES>
__global__ __launch_bounds__(256) void gated_small_part_norm_kernel(
    typename S::T* __restrict__ out, int64_t out_stride, const float* __restrict__ o,
    const float* __restrict__ weight, const typename S::T* __restrict__ gate, int64_t gate_stride,
    int gate_act, int gate_first, float eps, int groups, int part, int64_t parts,
    const float* __restrict__ part_scale) {
  const int64_t p = (int64_t)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  const int c = 4 * (threadIdx.x % LANES);
  if (p >= parts) return;                               // whole groups of lanes
  const int64_t t = p / groups;
  const int first = (int)(p - t * groups) * part;
  const bool mine = c < part;
  f32x4 x = {0.f, 0.f, 0.f, 0.f}, z = x, wv = x;
  if (mine) {
    x = *reinterpret_cast<const f32x4*>(o + p * part + c);
    wv = *reinterpret_cast<const f32x4*>(weight + first + c);
    const typename S::T* gr = gate + t * gate_stride + first + c;
    if constexpr (sizeof(typename S::T) == 2) {
      const u32x2 zz = *reinterpret_cast<const u32x2*>(gr);
      z = f32x4{lo16<S>(zz[0]), hi16<S>(zz[0]), lo16<S>(zz[1]), hi16<S>(zz[1])};
    } else {
      z = *reinterpret_cast<const f32x4*>(gr);
    }
  }
  const float ps = part_scale != nullptr ? part_scale[p] : 1.f;
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    z[e] = gate_act == VLA_GATE_SILU ? silu_f(z[e]) : 1.f / (1.f + expf(-z[e]));
    x[e] *= ps;
    if (gate_first) x[e] *= z[e];
    ss += x[e] * x[e];
  }
#pragma unroll
  for (int m = 1; m < LANES; m <<= 1) ss += __shfl_xor(ss, m, 64);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
  if (!mine) return;
  float r[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) r[e] = x[e] * inv * wv[e] * (gate_first ? 1.f : z[e]);
  typename S::T* dst = out + t * out_stride + first + c;
  if constexpr (sizeof(typename S::T) == 2)
    *reinterpret_cast<u32x2*>(dst) = u32x2{pack16<S>(r[0], r[1]), pack16<S>(r[2], r[3])};
  else
    *reinterpret_cast<f32x4*>(dst) = f32x4{r[0], r[1], r[2], r[3]};
}

// One workgroup per (token, part).  A thread keeps up to four vectors of its part in registers.
template <class S, int VW>
__global__ __launch_bounds__(256) void gated_group_rms_norm_kernel(
    typename S::T* __restrict__ out, int64_t out_stride, const float* __restrict__ o,
    const float* __restrict__ weight, const typename S::T* __restrict__ gate, int64_t gate_stride,
    int gate_act, int gate_first, float eps, int n, int part, const float* __restrict__ part_scale) {
  __shared__ float red[16];
  constexpr int KEEP = 16 / VW;
  const int64_t t = blockIdx.x;
  const int first = blockIdx.y * part;
  const float* orow = o + t * n + first;
  const typename S::T* grow = gate + t * gate_stride + first;
  typename S::T* out_row = out + t * out_stride + first;
  const float* wrow = weight + first;
  const int step = blockDim.x * VW;
  const float ps = part_scale != nullptr ? part_scale[t * gridDim.y + blockIdx.y] : 1.f;
  auto gated = [&](float z) { return gate_act == VLA_GATE_SILU ? silu_f(z) : 1.f / (1.f + expf(-z)); };
  auto read = [&](int c, float (&u)[VW], float (&f)[VW]) {     // the value to norm, and the factor after it
    float x[VW], z[VW];
    if constexpr (VW == 4) {
      const f32x4 got = *reinterpret_cast<const f32x4*>(orow + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = got[e];
      if constexpr (sizeof(typename S::T) == 2) {
        const u32x2 zz = *reinterpret_cast<const u32x2*>(grow + c);
        z[0] = lo16<S>(zz[0]);
        z[1] = hi16<S>(zz[0]);
        z[2] = lo16<S>(zz[1]);
        z[3] = hi16<S>(zz[1]);
      } else {
        const f32x4 zz = *reinterpret_cast<const f32x4*>(grow + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) z[e] = zz[e];
      }
    } else {
      x[0] = orow[c];
      z[0] = S::to_f32(grow[c]);
    }
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      const float gv = gated(z[e]);
      u[e] = x[e] * ps * (gate_first ? gv : 1.f);
      f[e] = gate_first ? 1.f : gv;
    }
  };
  auto write = [&](int c, const float (&u)[VW], const float (&f)[VW], float inv) {
    float r[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) r[e] = u[e] * inv * wrow[c + e] * f[e];
    if constexpr (VW == 4 && sizeof(typename S::T) == 2) {
      *reinterpret_cast<u32x2*>(out_row + c) = u32x2{pack16<S>(r[0], r[1]), pack16<S>(r[2], r[3])};
    } else {
#pragma unroll
      for (int e = 0; e < VW; ++e) out_row[c + e] = S::from_f32(r[e]);
    }
  };
  float u[KEEP][VW], f[KEEP][VW];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = threadIdx.x * VW + i * step;
    if (c < part) {
      read(c, u[i], f[i]);
#pragma unroll
      for (int e = 0; e < VW; ++e) ss += u[i][e] * u[i][e];
    }
  }
  for (int c = threadIdx.x * VW + KEEP * step; c < part; c += step) {
    float uu[VW], ff[VW];
    read(c, uu, ff);
#pragma unroll
    for (int e = 0; e < VW; ++e) ss += uu[e] * uu[e];
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = threadIdx.x * VW + i * step;
    if (c < part) write(c, u[i], f[i], inv);
  }
  for (int c = threadIdx.x * VW + KEEP * step; c < part; c += step) {
    float uu[VW], ff[VW];
    read(c, uu, ff);
    write(c, uu, ff, inv);
  }
}

template <int DB, int WAVES, RowKind KIND, bool STATE_ONLY>
int launch_block(const DecayScan& a, int pieces, hipStream_t stream) {
  constexpr size_t lds = block_lds_floats<DB, WAVES, KIND, STATE_ONLY>() * sizeof(float);
  static std::atomic<bool> allowed{false};              // raised once per kernel, not per launch
  if (lds > 64 * 1024 && !allowed.load(std::memory_order_relaxed)) {
    VLA_SEQ_HIP_CHECK(hipFuncSetAttribute(
        reinterpret_cast<const void*>(&decay_block_kernel<DB, WAVES, KIND, STATE_ONLY>),
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    allowed.store(true, std::memory_order_relaxed);
  }
  const dim3 grid(a.heads, (a.vdim + 16 * WAVES - 1) / (16 * WAVES), pieces);
  decay_block_kernel<DB, WAVES, KIND, STATE_ONLY><<<grid, 64 * WAVES, lds, stream>>>(a);
  VLA_SEQ_HIP_CHECK(hipGetLastError());
  return VLA_OK;
}

template <int DB, int WAVES, RowKind KIND>
int launch_blocks(const DecayScan& a, int pieces, hipStream_t stream) {
  if (a.piece_rows > 0) {
    const int rc = launch_block<DB, WAVES, KIND, true>(a, pieces, stream);
    if (rc != VLA_OK) return rc;
    decay_chain_kernel<<<dim3((unsigned)((a.head_size + 255) / 256), a.heads, a.num_seqs), 256, 0, stream>>>(a);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
  }
  return launch_block<DB, WAVES, KIND, false>(a, pieces, stream);
}

template <RowKind KIND>
int launch_by_size(const DecayScan& a, int pieces, hipStream_t stream) {
  const bool wide = a.vdim > 64;
  switch ((a.dim + 31) / 32) {
    case 1: return wide ? launch_blocks<2, 8, KIND>(a, pieces, stream) : launch_blocks<2, 4, KIND>(a, pieces, stream);
    case 2: return wide ? launch_blocks<4, 8, KIND>(a, pieces, stream) : launch_blocks<4, 4, KIND>(a, pieces, stream);
    case 3: return wide ? launch_blocks<6, 8, KIND>(a, pieces, stream) : launch_blocks<6, 4, KIND>(a, pieces, stream);
    case 4: return wide ? launch_blocks<8, 8, KIND>(a, pieces, stream) : launch_blocks<8, 4, KIND>(a, pieces, stream);
    default: return VLA_ERR_HEAD_SIZE;
  }
}

bool cuts_runs(int max_query_len, int dim) {
  return max_query_len > VLA_DECAY_SCAN_PIECE && dim <= kMaxBlockDim &&
         g_decay_kernel.load(std::memory_order_relaxed) != 1;
}
int64_t piece_slots(int num_tokens, int num_seqs) {
  return (int64_t)num_tokens / VLA_DECAY_SCAN_PIECE + num_seqs;
}

}  // namespace
}  // namespace seq
}  // namespace vla

using namespace vla;
using namespace vla::seq;

extern "C" int64_t vla_seq_decay_scan_scratch_floats(int num_tokens, int num_seqs, int max_query_len,
                                                     int heads, int dim, int vdim, int normalizer) {
  if (!cuts_runs(max_query_len, dim)) return 0;
  return piece_slots(num_tokens, num_seqs) * heads * ((int64_t)dim * (vdim + (normalizer ? 1 : 0)) + 1);
}

extern "C" int vla_seq_set_decay_scan_kernel(int mode) {
  if (mode < 0 || mode > 2) return VLA_ERR_ARG;
  g_decay_kernel.store(mode, std::memory_order_relaxed);
  return VLA_OK;
}

extern "C" int vla_seq_decay_scan(float* o, const void* q, int64_t q_stride, const void* k,
                                  int64_t k_stride, const void* v, int64_t v_stride, const void* dt,
                                  int64_t dt_stride, const float* dt_bias, const float* a_log,
                                  const float* log_decay, const float* skip, const float* row_log,
                                  const float* row_weight, const float* row_floor,
                                  float* norm_scale, float norm_eps, float q_scale, float* state,
                                  const int* query_start_loc, const int* context_lens,
                                  const int* state_slots, int num_tokens, int num_seqs,
                                  int num_slots, int max_query_len, int heads, int groups, int dim,
                                  int vdim, int act, float* scratch, int64_t scratch_floats,
                                  int dtype, void* stream) {
  if (num_tokens == 0 || num_seqs == 0) return VLA_OK;
  if (!o || !q || !k || !v || !state || !query_start_loc || !context_lens || !state_slots ||
      num_tokens < 0 || num_seqs < 0 || num_seqs > 65535 || num_slots <= 0 || max_query_len <= 0 ||
      heads <= 0 || groups <= 0 || heads % groups != 0 || dim <= 0 || vdim <= 0 ||
      q_stride < (int64_t)groups * dim || k_stride < (int64_t)groups * dim ||
      v_stride < (int64_t)heads * vdim || (act != VLA_ACT_NONE && act != VLA_ACT_SILU) ||
      (row_log ? !row_weight : dt ? (!dt_bias || !a_log || dt_stride < heads) : !log_decay) ||
      (norm_scale && !row_floor))
    return VLA_ERR_ARG;
  if (dim > 1024 || vdim > (vdim % 4 == 0 ? 1024 : 256)) return VLA_ERR_HEAD_SIZE;
  if (dtype != VLA_F16 && dtype != VLA_BF16 && dtype != VLA_F32) return VLA_ERR_DTYPE;
  hipStream_t st = (hipStream_t)stream;
  const int elem = dtype == VLA_F32 ? 4 : 2;
  auto aligned = [&](const void* p, int64_t stride, int size) {
    return size % 8 == 0 && ((uintptr_t)p % 16) == 0 && (stride * elem) % 16 == 0;
  };
  DecayScan a;
  a.o = o;
  a.q = q;
  a.q_stride = q_stride;
  a.k = k;
  a.k_stride = k_stride;
  a.v = v;
  a.v_stride = v_stride;
  a.dt = dt;
  a.dt_stride = dt_stride;
  a.dt_bias = dt_bias;
  a.a_log = a_log;
  a.log_decay = log_decay;
  a.skip = skip;
  a.row_log = row_log;
  a.row_weight = row_weight;
  a.row_floor = row_floor;
  a.norm_scale = norm_scale;
  a.norm_eps = norm_eps;
  a.q_scale = q_scale;
  a.head_size = (int64_t)dim * (vdim + (norm_scale ? 1 : 0));
  a.state = state;
  a.query_start_loc = query_start_loc;
  a.context_lens = context_lens;
  a.state_slots = state_slots;
  a.num_seqs = num_seqs;
  a.heads = heads;
  a.groups = groups;
  a.dim = dim;
  a.vdim = vdim;
  a.act = act;
  a.dtype = dtype;
  a.mode = g_decay_kernel.load(std::memory_order_relaxed);
  if (dim > kMaxBlockDim) a.mode = 1;
  a.vec_q = aligned(q, q_stride, dim);
  a.vec_k = aligned(k, k_stride, dim);
  a.vec_v = aligned(v, v_stride, vdim);
  a.piece_rows = 0;
  a.piece_state = a.piece_decay = nullptr;
  int pieces = num_seqs;
  if (a.mode != 1 && cuts_runs(max_query_len, dim)) {
    const int64_t slots = piece_slots(num_tokens, num_seqs);
    const int64_t need = slots * heads * (a.head_size + 1);
    if (!scratch || scratch_floats < need || slots > 65535) return VLA_ERR_ARG;
    a.piece_rows = VLA_DECAY_SCAN_PIECE;
    a.piece_state = scratch;
    a.piece_decay = scratch + slots * heads * a.head_size;
    pieces = (int)slots;
  }
  // a step of several sequences may hold runs of both kinds: each launch skips the other's sequences
  const bool steps = a.mode == 1 || (a.mode == 0 && (max_query_len <= kStepRows || num_seqs > 1));
  const bool blocks = a.mode == 2 || (a.mode == 0 && max_query_len > kStepRows);
  if (steps) {
    const int vw = vdim % 4 == 0 && a.head_size % 4 == 0 && ((uintptr_t)state % 16) == 0 ? 4 : 1;
    const int cols = (vdim + vw - 1) / vw, groups_of_rows = 256 / cols;
    if (groups_of_rows < 1) return VLA_ERR_HEAD_SIZE;
    const size_t lds = sizeof(float) * (2 * (size_t)dim + vdim + (size_t)groups_of_rows * vdim + 4);
    const dim3 grid(heads, num_seqs);
    if (vw == 4)
      decay_step_kernel<4><<<grid, 256, lds, st>>>(a);
    else
      decay_step_kernel<1><<<grid, 256, lds, st>>>(a);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
  }
  if (!blocks) return VLA_OK;
  if (dtype == VLA_F32) return launch_by_size<kRowsF32>(a, pieces, st);
  if (dtype == VLA_BF16 && act == VLA_ACT_NONE) return launch_by_size<kRowsBf16>(a, pieces, st);
  return launch_by_size<kRows16>(a, pieces, st);
}

extern "C" int vla_seq_gated_group_rms_norm(void* out, int64_t out_stride, const float* o,
                                            const float* weight, const void* gate,
                                            int64_t gate_stride, int gate_act, int gate_first,
                                            int groups, float eps, int num_tokens, int n, int dtype,
                                            const float* part_scale, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!out || !o || !weight || !gate || num_tokens < 0 || n <= 0 || groups <= 0 || n % groups != 0 ||
      groups > 65535 || out_stride < n || gate_stride < n ||
      (gate_act != VLA_GATE_SILU && gate_act != VLA_GATE_SIGMOID))
    return VLA_ERR_ARG;
  const int part = n / groups;
  return with_dtype(dtype, [&](auto s) {
    using S = decltype(s);
    using T = typename S::T;
    const int threads = part <= 256 ? 64 : part <= 512 ? 128 : 256;
    const dim3 grid(num_tokens, groups);
    const int64_t bytes = 4 * sizeof(T);
    const bool vec = part % 4 == 0 && ((uintptr_t)o % 16) == 0 && (uintptr_t)gate % bytes == 0 &&
                     (uintptr_t)out % bytes == 0 && gate_stride % 4 == 0 && out_stride % 4 == 0;
    if (vec && groups > 1 && part <= 256 && ((uintptr_t)weight % 16) == 0) {
      const int64_t parts = (int64_t)num_tokens * groups;
      auto small = [&](auto kernel, int lanes) {
        const int per = 256 / lanes;
        kernel<<<(unsigned)((parts + per - 1) / per), 256, 0, (hipStream_t)stream>>>(
            (T*)out, out_stride, o, weight, (const T*)gate, gate_stride, gate_act, gate_first, eps, groups, part,
            parts, part_scale);
      };
      if (part <= 64)
        small(gated_small_part_norm_kernel<S, 16>, 16);
      else if (part <= 128)
        small(gated_small_part_norm_kernel<S, 32>, 32);
      else
        small(gated_small_part_norm_kernel<S, 64>, 64);
      VLA_SEQ_HIP_CHECK(hipGetLastError());
      return (int)VLA_OK;
    }
    if (vec)
      gated_group_rms_norm_kernel<S, 4><<<grid, threads, 0, (hipStream_t)stream>>>(
          (T*)out, out_stride, o, weight, (const T*)gate, gate_stride, gate_act, gate_first, eps, n, part,
          part_scale);
    else
      gated_group_rms_norm_kernel<S, 1><<<grid, threads, 0, (hipStream_t)stream>>>(
          (T*)out, out_stride, o, weight, (const T*)gate, gate_stride, gate_act, gate_first, eps, n, part,
          part_scale);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    return (int)VLA_OK;
  });
}

extern "C" int vla_seq_matrix_memory_gates(float* row_log, float* row_weight, float* row_floor,
                                           const void* zi, int64_t zi_stride, const void* zf,
                                           int64_t zf_stride, const float* bias_i,
                                           const float* bias_f, float cap, float* maximum,
                                           const int* query_start_loc, const int* context_lens,
                                           const int* state_slots, int num_seqs, int num_slots,
                                           int max_query_len, int heads, int dtype, void* stream) {
  if (num_seqs == 0) return VLA_OK;
  if (!row_log || !row_weight || !row_floor || !zi || !zf || !bias_i || !bias_f || !maximum ||
      !query_start_loc || !context_lens || !state_slots || num_seqs < 0 || num_seqs > 65535 ||
      num_slots <= 0 || max_query_len <= 0 || heads <= 0 || zi_stride < heads || zf_stride < heads ||
      !(cap > 0.f))
    return VLA_ERR_ARG;
  const int threads = max_query_len <= 64 ? 64 : max_query_len <= 256 ? 256 : 1024;
  return with_dtype(dtype, [&](auto s) {
    using S = decltype(s);
    using T = typename S::T;
    matrix_memory_gates_kernel<S><<<dim3(heads, num_seqs), threads, 0, (hipStream_t)stream>>>(
        row_log, row_weight, row_floor, (const T*)zi, zi_stride, (const T*)zf, zf_stride, bias_i, bias_f, cap,
        maximum, query_start_loc, context_lens, state_slots, heads);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    return VLA_OK;
  });
}
