// Delta rule with a decay per key channel: per head a state S [dim, vdim] in fp32,
//   S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// with k and q unit vectors per key head (q also times dim^-1/2), beta = sigmoid(b) and
// g = exp(-exp(A_log) softplus(z + dt_bias)) per head and channel.  Several value heads may share one
// query / key head.  o leaves in fp32, before whatever norms and gates it.  State: [slot, head, vdim,
// dim].
//
// Blocks of 16 rows (runs of more than a few rows).  With G_i the product of g over a block's rows
// 0 .. i (per channel), and G_i / G_j formed as the product over j + 1 .. i (nothing is divided and no
// sum of logarithms is subtracted, so any decay between 0 and 1 is exact to fp32):
//   B_ij = beta_i k_i . (G_i / G_j) k_j  (j < i),   A_ij = q_i . (G_i / G_j) k_j  (j <= i)
//   T = (I + B)^-1 diag(beta),   M = A T                                 (16 x 16, lower triangular)
//   U = T V - (T K~) S,   O = M V + (Q~ - M K~) S                        K~_i = G_i k_i, Q~_i = G_i q_i
//   S <- diag(G_last) S + K^^T U                                         K^_j = (G_last / G_j) k_j
// Everything but the last two lines' products with S depends on the block alone.  delta_prepare_kernel
// forms it for all blocks at once (one workgroup per block and head) and leaves W = T K~, Q~ - M K~,
// K^, G_last and T V in scratch and M V in o; delta_walk_kernel then goes over a run's blocks in order
// with two products of 16 rows and one update of S per block.  A column of S never meets another, so
// workgroups take 16 value columns each; four waves split the rows of S, add their partial products
// through LDS (one barrier per block), and keep S in registers as a matrix-core result that is the
// next product's operand where it lies (the contraction index of a product may be relabelled freely).
// All products run on 16x16x4 fp32 matrix cores.  Layout, lane = (g, c) = (lane >> 4, lane & 15):
//   A operand  lane: row c, contraction index g       B operand  lane: column c, contraction index g
//   result     lane: column c, rows 4 g .. 4 g + 3
// and a block's scratch is stored in the order in which the walking waves read it, 16 bytes per lane.
//
// Runs of at most four rows (decode steps) go token by token: thread (column, r) keeps R rows of a
// column in registers, the `split` threads of a column add their dot products with lane exchanges, and
// the channels' decays of a token are formed once per workgroup.
#include <algorithm>
#include <atomic>

#include "seq_common.h"

namespace vla {
namespace seq {
namespace {

constexpr int kRows = 16;
constexpr int kStepRows = 4;
constexpr int kMaxBlockDim = 256;
constexpr int kMaxSplit = 16;
constexpr int kTri = 20;            // floats per row of a 16 x 16 matrix in LDS
std::atomic<int> g_channel_delta_kernel{0};

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

struct ChannelDelta {
  float* o;                   // [T][heads * vdim]
  const void* q;
  int64_t q_stride;
  const void* k;
  int64_t k_stride;
  const void* v;
  int64_t v_stride;
  const void* beta;
  int64_t beta_stride;
  const float* z;
  int64_t z_stride;
  const float* dt_bias;       // [heads * dim]
  const float* a_log;         // [heads]
  float* state;
  float* scratch;
  const int* query_start_loc;
  const int* context_lens;
  const int* state_slots;
  int num_seqs, heads, kv_heads, dim, vdim, mode;
  bool vec_qk, vec_z, vec_state;
};

// four values d .. d + 3 of a row of `dim`, zeros behind its end
template <class S>
__device__ __forceinline__ f32x4 load4(const typename S::T* row, int d, int dim, bool vec) {
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (vec) {
    if (d < dim) {
      if constexpr (sizeof(typename S::T) == 2) {
        const u32x2 x = *reinterpret_cast<const u32x2*>(row + d);
        r = f32x4{lo16<S>(x[0]), hi16<S>(x[0]), lo16<S>(x[1]), hi16<S>(x[1])};
      } else {
        r = *reinterpret_cast<const f32x4*>(row + d);
      }
    }
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (d + e < dim) r[e] = S::to_f32(row[d + e]);
  }
  return r;
}

__device__ __forceinline__ float channel_decay(float rate, float z) { return expf(-rate * softplusf(z)); }

// floats of a block's scratch: W | Q~ - M K~ | K^ (each 16 x DP) | G_last (DP) | T V (16 x VP)
__host__ __device__ __forceinline__ int64_t block_floats(int dp, int vp) { return (int64_t)(3 * kRows + 1) * dp + kRows * vp; }

// Which sequence and block a block slot is: sequence b's blocks are slots start_b / 16 + b + 0, 1, ...
__device__ __forceinline__ bool find_block(const ChannelDelta& a, int slot, int& b, int& block) {
  int lo = 0, hi = a.num_seqs - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (a.query_start_loc[mid] / kRows + mid <= slot)
      lo = mid;
    else
      hi = mid - 1;
  }
  b = lo;
  block = slot - (a.query_start_loc[b] / kRows + b);
  return block >= 0 && block * kRows < a.query_start_loc[b + 1] - a.query_start_loc[b];
}

template <class S, int DX>
__global__ __launch_bounds__(256) void delta_prepare_kernel(ChannelDelta a) {
  constexpr int DP = 64 * DX, RS = DP + 4;
  __shared__ __align__(16) float k_lds[kRows * RS];
  __shared__ __align__(16) float q_lds[kRows * RS];
  __shared__ __align__(16) float g_lds[kRows * RS];
  __shared__ __align__(16) float b_lds[kRows * kTri];      // B, strictly lower
  __shared__ __align__(16) float a_lds[kRows * kTri];      // A, lower
  __shared__ __align__(16) float t_lds[kRows * kTri];      // T
  __shared__ __align__(16) float m_lds[kRows * kTri];      // M
  __shared__ float beta_lds[kRows];
  const int slot = blockIdx.x, h = blockIdx.y;
  int b, block;
  if (!find_block(a, slot, b, block)) return;
  const int run = a.query_start_loc[b + 1] - a.query_start_loc[b];
  if (a.mode == 0 && run <= kStepRows) return;             // the step kernel's
  const int t0 = a.query_start_loc[b] + block * kRows, n = min(kRows, run - block * kRows);
  const int D = a.dim, V = a.vdim, hg = h / (a.heads / a.kv_heads);
  const int vb = (V + 15) / 16;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15;
  const int row = tid >> 4, part = tid & 15;               // 16 neighbouring lanes share a row
  float* out = a.scratch + ((int64_t)slot * a.heads + h) * block_floats(DP, 16 * vb);
  float* w_out = out;                                      // [DP / 16][row][16]
  float* q_out = w_out + kRows * DP;                       // the same
  float* k_out = q_out + kRows * DP;                       // [DP][row]
  float* g_out = k_out + kRows * DP;                       // [DP]
  float* u_out = g_out + DP;                               // [vb][16 columns][row]
  using T = typename S::T;

  // rows, unit norms, decays
  {
    const bool live = row < n;
    const int64_t t = t0 + (live ? row : 0);
    const T* qr = (const T*)a.q + t * a.q_stride + (int64_t)hg * D;
    const T* kr = (const T*)a.k + t * a.k_stride + (int64_t)hg * D;
    const float* zr = a.z + t * a.z_stride + (int64_t)h * D;
    const float* br = a.dt_bias + (int64_t)h * D;
    const float rate = expf(a.a_log[h]);
    f32x4 qv[DX], kv[DX], gv[DX];
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int x = 0; x < DX; ++x) {
      const int d = 4 * part + 64 * x;
      qv[x] = load4<S>(qr, d, D, a.vec_qk);
      kv[x] = load4<S>(kr, d, D, a.vec_qk);
      const f32x4 zv = load4<F32>(zr, d, D, a.vec_z), bv = load4<F32>(br, d, D, a.vec_z);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        qq += qv[x][e] * qv[x][e];
        kk += kv[x][e] * kv[x][e];
        gv[x][e] = live && d + e < D ? channel_decay(rate, zv[e] + bv[e]) : 1.f;
      }
    }
    group_sums(qq, kk, 16);
    const float qs = live ? 1.f / (sqrtf(qq + 1e-6f) * sqrtf((float)D)) : 0.f, ks = live ? 1.f / sqrtf(kk + 1e-6f) : 0.f;
#pragma unroll
    for (int x = 0; x < DX; ++x) {
      const int d = 4 * part + 64 * x;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        qv[x][e] *= qs;
        kv[x][e] *= ks;
      }
      *reinterpret_cast<f32x4*>(q_lds + row * RS + d) = qv[x];
      *reinterpret_cast<f32x4*>(k_lds + row * RS + d) = kv[x];
      *reinterpret_cast<f32x4*>(g_lds + row * RS + d) = gv[x];
    }
    if (part == 0)
      beta_lds[row] = live ? 1.f / (1.f + expf(-S::to_f32(((const T*)a.beta)[t * a.beta_stride + h]))) : 0.f;
  }
  __syncthreads();

  // column j = row of B and A: r = (G_i / G_j) k_j, decayed row by row
  f32x4 r[DX];
  {
    const int j = row;
    float qk = 0.f, none = 0.f;
#pragma unroll
    for (int x = 0; x < DX; ++x) {
      const int d = 4 * part + 64 * x;
      r[x] = *reinterpret_cast<const f32x4*>(k_lds + j * RS + d);
      const f32x4 qv = *reinterpret_cast<const f32x4*>(q_lds + j * RS + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) qk += qv[e] * r[x][e];
    }
    group_sums(qk, none, 16);
    if (part == 0) a_lds[j * kTri + j] = qk;
    for (int i = 4 * w + 1; i < kRows; ++i) {              // uniform over the wave: its columns start at 4 w
      float ik = 0.f, iq = 0.f;
      const bool below = i > j;
#pragma unroll
      for (int x = 0; x < DX; ++x) {
        const int d = 4 * part + 64 * x;
        const f32x4 gv = *reinterpret_cast<const f32x4*>(g_lds + i * RS + d);
        const f32x4 kv = *reinterpret_cast<const f32x4*>(k_lds + i * RS + d);
        const f32x4 qv = *reinterpret_cast<const f32x4*>(q_lds + i * RS + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          r[x][e] *= below ? gv[e] : 1.f;
          ik += kv[e] * r[x][e];
          iq += qv[e] * r[x][e];
        }
      }
      group_sums(ik, iq, 16);
      if (part == 0 && below) {
        b_lds[i * kTri + j] = beta_lds[i] * ik;
        a_lds[i * kTri + j] = iq;
      }
    }
  }
  __syncthreads();

  // wave 0: T column by column; the other waves: K~, Q~ in place and G_last
  if (w == 0) {
    if (lane < kRows) {
      float x[kRows];
#pragma unroll
      for (int i = 0; i < kRows; ++i) {
        float acc = i == lane ? beta_lds[i] : 0.f;
#pragma unroll
        for (int j = 0; j < i; ++j) acc -= b_lds[i * kTri + j] * x[j];
        x[i] = i < lane ? 0.f : acc;
      }
#pragma unroll
      for (int i = 0; i < kRows; ++i) t_lds[i * kTri + lane] = x[i];
    }
  } else {
    for (int d = tid - 64; d < DP; d += 192) {
      float p = 1.f;
#pragma unroll
      for (int i = 0; i < kRows; ++i) {
        p *= g_lds[i * RS + d];
        k_lds[i * RS + d] *= p;
        q_lds[i * RS + d] *= p;
      }
      g_out[d] = p;
    }
  }
  __syncthreads();

  // M = A T; K^ takes the decays' place
  {
    float acc = 0.f;
    for (int j = part; j <= row; ++j) acc += a_lds[row * kTri + j] * t_lds[j * kTri + part];
    m_lds[row * kTri + part] = acc;
#pragma unroll
    for (int x = 0; x < DX; ++x) *reinterpret_cast<f32x4*>(g_lds + row * RS + 4 * part + 64 * x) = r[x];
  }
  __syncthreads();
  for (int i = tid; i < kRows * DP; i += 256) k_out[i] = g_lds[(i & 15) * RS + (i >> 4)];

  const f32x4 tv = *reinterpret_cast<const f32x4*>(t_lds + c * kTri + 4 * g);
  const f32x4 mv = *reinterpret_cast<const f32x4*>(m_lds + c * kTri + 4 * g);
  for (int tile = w; tile < 4 * DX + vb; tile += 4) {
    f32x4 xt = {0.f, 0.f, 0.f, 0.f}, ym = xt;
    if (tile < 4 * DX) {
      // the products transposed (K~^T T^T), so that a lane ends with four channels of a row of W
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float kv = k_lds[(4 * g + i) * RS + 16 * tile + c];
        xt = mfma4(kv, tv[i], xt);
        ym = mfma4(kv, mv[i], ym);
      }
      const f32x4 qv = *reinterpret_cast<const f32x4*>(q_lds + c * RS + 16 * tile + 4 * g);
      *reinterpret_cast<f32x4*>(w_out + (tile * 16 + c) * 16 + 4 * g) = xt;
      *reinterpret_cast<f32x4*>(q_out + (tile * 16 + c) * 16 + 4 * g) = f32x4{qv[0] - ym[0], qv[1] - ym[1], qv[2] - ym[2], qv[3] - ym[3]};
    } else {
      const int v0 = 16 * (tile - 4 * DX), col = v0 + c;
      const T* vr = (const T*)a.v + (int64_t)h * V + (col < V ? col : 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = 4 * g + i;
        const float got = S::to_f32(vr[(int64_t)(t0 + min(j, n - 1)) * a.v_stride]);
        const float vv = j < n && col < V ? got : 0.f;
        xt = mfma4(tv[i], vv, xt);
        ym = mfma4(mv[i], vv, ym);
      }
      *reinterpret_cast<f32x4*>(u_out + (v0 + c) * 16 + 4 * g) = xt;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (4 * g + e < n && col < V) a.o[((int64_t)(t0 + 4 * g + e) * a.heads + h) * V + col] = ym[e];
    }
  }
}

template <int DX>
__global__ __launch_bounds__(256) void delta_walk_kernel(ChannelDelta a) {
  constexpr int DP = 64 * DX;
  __shared__ __align__(16) float u_part[2][4][64][4];      // a wave's part of W S
  __shared__ __align__(16) float o_part[2][4][4][64];      // of (Q~ - M K~) S, by component
  const int h = blockIdx.x, v0 = 16 * blockIdx.y, b = blockIdx.z;
  const int t_begin = a.query_start_loc[b], run = a.query_start_loc[b + 1] - t_begin;
  if (run <= 0 || (a.mode == 0 && run <= kStepRows)) return;
  const int D = a.dim, V = a.vdim, vp = (V + 15) / 16 * 16;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, g = lane >> 4, c = lane & 15;
  const int col = v0 + c;
  const int64_t per = block_floats(DP, vp);
  const float* base = a.scratch + ((int64_t)(t_begin / kRows + b) * a.heads + h) * per;
  const int64_t step = (int64_t)a.heads * per;
  float* st = a.state + (((int64_t)a.state_slots[b] * a.heads + h) * V + (col < V ? col : 0)) * D;
  const bool resume = a.context_lens[b] > 0;
  f32x4 s[DX];
#pragma unroll
  for (int x = 0; x < DX; ++x) {
    const int d = 16 * (w * DX + x) + 4 * g;
    s[x] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (resume && col < V) s[x] = load4<F32>(st, d, D, a.vec_state);
  }
  const int blocks = (run + kRows - 1) / kRows;
  struct Block {
    f32x4 wv[DX], qv[DX], kv[DX], gv[DX], u;
    float o;
  };
  auto fetch = [&](Block& f, int i) {
    const float* p = base + (int64_t)i * step;
#pragma unroll
    for (int x = 0; x < DX; ++x) {
      const int db = w * DX + x, at = (16 * db + c) * 16 + 4 * g;
      f.wv[x] = *reinterpret_cast<const f32x4*>(p + at);
      f.qv[x] = *reinterpret_cast<const f32x4*>(p + kRows * DP + at);
      f.kv[x] = *reinterpret_cast<const f32x4*>(p + 2 * kRows * DP + at);
      f.gv[x] = *reinterpret_cast<const f32x4*>(p + 3 * kRows * DP + 16 * db + 4 * g);
    }
    f.u = *reinterpret_cast<const f32x4*>(p + (3 * kRows + 1) * DP + col * 16 + 4 * g);
    // wave w finishes rows 4 g + w of the block's outputs
    const int row = min(i * kRows + 4 * g + w, run - 1);
    f.o = a.o[((int64_t)(t_begin + row) * a.heads + h) * V + (col < V ? col : 0)];
  };
  auto advance = [&](const Block& f, int i) {
    const int buf = i & 1;
    f32x4 xu = {0.f, 0.f, 0.f, 0.f}, xo = xu;
#pragma unroll
    for (int x = 0; x < DX; ++x)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        xu = mfma4(f.wv[x][e], s[x][e], xu);
        xo = mfma4(f.qv[x][e], s[x][e], xo);
      }
    *reinterpret_cast<f32x4*>(&u_part[buf][w][lane][0]) = xu;
#pragma unroll
    for (int e = 0; e < 4; ++e) o_part[buf][w][e][lane] = xo[e];
    __syncthreads();
    f32x4 u = f.u;
#pragma unroll
    for (int o = 0; o < 4; ++o) {
      const f32x4 p = *reinterpret_cast<const f32x4*>(&u_part[buf][o][lane][0]);
#pragma unroll
      for (int e = 0; e < 4; ++e) u[e] -= p[e];
    }
#pragma unroll
    for (int x = 0; x < DX; ++x) {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[x][e] *= f.gv[x][e];
#pragma unroll
      for (int e = 0; e < 4; ++e) s[x] = mfma4(f.kv[x][e], u[e], s[x]);
    }
    const float o = f.o + ((o_part[buf][0][w][lane] + o_part[buf][1][w][lane]) +
                           (o_part[buf][2][w][lane] + o_part[buf][3][w][lane]));
    const int row = i * kRows + 4 * g + w;
    if (row < run && col < V) a.o[((int64_t)(t_begin + row) * a.heads + h) * V + col] = o;
  };
  // two blocks in turn, so that one is asked for while the other is worked on
  Block f0, f1;
  fetch(f0, 0);
  for (int i = 0; i < blocks; i += 2) {
    fetch(f1, min(i + 1, blocks - 1));
    advance(f0, i);
    if (i + 1 >= blocks) break;
    fetch(f0, min(i + 2, blocks - 1));
    advance(f1, i + 1);
  }
  if (col < V) {
#pragma unroll
    for (int x = 0; x < DX; ++x) {
      const int d = 16 * (w * DX + x) + 4 * g;
      if (a.vec_state) {
        if (d < D) *reinterpret_cast<f32x4*>(st + d) = s[x];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < D) st[d + e] = s[x][e];
      }
    }
  }
}

// Token by token.  The `split` lanes of a column hold all rows of it between them, so a token's unit
// norms are lane sums of what they read for the dot products anyway.
template <class S, int R>
__global__ __launch_bounds__(256) void channel_delta_step_kernel(ChannelDelta a, int split, int cols) {
  extern __shared__ __align__(16) float g_lds[];           // [2][split * R]
  using T = typename S::T;
  const int h = blockIdx.y, b = blockIdx.z, j0 = blockIdx.x * cols;
  const int start = a.query_start_loc[b], end = a.query_start_loc[b + 1];
  if (a.mode == 0 && end - start > kStepRows) return;      // the block kernels'
  const int D = a.dim, V = a.vdim, dp = split * R, hg = h / (a.heads / a.kv_heads);
  const int tid = threadIdx.x;
  const int jl = tid / split, r = tid - jl * split;
  const int j = j0 + jl;
  const bool col = jl < cols && j < V;
  float* st = a.state + (((int64_t)a.state_slots[b] * a.heads + h) * V + (col ? j : 0)) * D;
  const bool resume = a.context_lens[b] > 0;
  const float rate = expf(a.a_log[h]), q_unit = 1.f / sqrtf((float)D);
  float s[R];
#pragma unroll
  for (int ii = 0; ii < R / 4; ++ii) {
    f32x4 got = {0.f, 0.f, 0.f, 0.f};
    if (col && resume) got = load4<F32>(st, 4 * (ii * split + r), D, a.vec_state);
#pragma unroll
    for (int e = 0; e < 4; ++e) s[4 * ii + e] = got[e];
  }
  for (int t = start; t < end; ++t) {
    float* g_row = g_lds + ((t - start) & 1) * dp;         // the other half may still be read
    for (int d = tid; d < dp; d += blockDim.x)
      g_row[d] = d < D ? channel_decay(rate, a.z[(int64_t)t * a.z_stride + (int64_t)h * D + d] + a.dt_bias[(int64_t)h * D + d]) : 1.f;
    const T* qr = (const T*)a.q + (int64_t)t * a.q_stride + (int64_t)hg * D;
    const T* kr = (const T*)a.k + (int64_t)t * a.k_stride + (int64_t)hg * D;
    float kv[R], qv[R];
#pragma unroll
    for (int ii = 0; ii < R / 4; ++ii) {
      const int d = 4 * (ii * split + r);
      const f32x4 q4 = load4<S>(qr, d, D, a.vec_qk), k4 = load4<S>(kr, d, D, a.vec_qk);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        qv[4 * ii + e] = q4[e];
        kv[4 * ii + e] = k4[e];
      }
    }
    const float vj = S::to_f32(((const T*)a.v)[(int64_t)t * a.v_stride + (int64_t)h * V + (col ? j : 0)]);
    const float be = 1.f / (1.f + expf(-S::to_f32(((const T*)a.beta)[(int64_t)t * a.beta_stride + h])));
    __syncthreads();
    float qq = 0.f, kk = 0.f, kq = 0.f, dk = 0.f, dq = 0.f, none = 0.f;
#pragma unroll
    for (int ii = 0; ii < R / 4; ++ii) {
      const f32x4 g4 = *reinterpret_cast<const f32x4*>(g_row + 4 * (ii * split + r));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 4 * ii + e;
        s[i] *= g4[e];
        qq += qv[i] * qv[i];
        kk += kv[i] * kv[i];
        kq += kv[i] * qv[i];
        dk += s[i] * kv[i];
        dq += s[i] * qv[i];
      }
    }
    group_sums(qq, kk, split);
    group_sums(kq, none, split);
    group_sums(dk, dq, split);
    const float ks = 1.f / sqrtf(kk + 1e-6f), qs = q_unit / sqrtf(qq + 1e-6f);
    const float u = be * (vj - ks * dk);
    const float ku = ks * u;
#pragma unroll
    for (int i = 0; i < R; ++i) s[i] += kv[i] * ku;
    if (col && r == 0) a.o[((int64_t)t * a.heads + h) * V + j] = qs * dq + kq * ks * qs * u;
  }
  if (col && end > start) {
#pragma unroll
    for (int ii = 0; ii < R / 4; ++ii) {
      const int d = 4 * (ii * split + r);
      if (a.vec_state) {
        if (d < D) *reinterpret_cast<f32x4*>(st + d) = f32x4{s[4 * ii], s[4 * ii + 1], s[4 * ii + 2], s[4 * ii + 3]};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < D) st[d + e] = s[4 * ii + e];
      }
    }
  }
}

int pow2_at_least(int n) {
  int p = 1;
  while (p < n) p <<= 1;
  return p;
}

// what a step needs: token by token, in blocks, or both (each skips the other's sequences)
bool wants_steps(int mode, int max_query_len, int num_seqs, int dim) {
  return mode == 1 || dim > kMaxBlockDim || (mode == 0 && (max_query_len <= kStepRows || num_seqs > 1));
}
bool wants_blocks(int mode, int max_query_len, int dim) {
  return dim <= kMaxBlockDim && (mode == 2 || (mode == 0 && max_query_len > kStepRows));
}
int64_t block_slots(int num_tokens, int num_seqs) { return (int64_t)num_tokens / kRows + num_seqs; }

template <class S, int DX>
int launch_blocks(const ChannelDelta& a, int64_t slots, hipStream_t stream) {
  delta_prepare_kernel<S, DX><<<dim3((unsigned)slots, a.heads), 256, 0, stream>>>(a);
  VLA_SEQ_HIP_CHECK(hipGetLastError());
  delta_walk_kernel<DX><<<dim3(a.heads, (a.vdim + 15) / 16, a.num_seqs), 256, 0, stream>>>(a);
  VLA_SEQ_HIP_CHECK(hipGetLastError());
  return VLA_OK;
}

}  // namespace
}  // namespace seq
}  // namespace vla

using namespace vla;
using namespace vla::seq;

extern "C" int64_t vla_seq_channel_delta_scratch_floats(int num_tokens, int num_seqs, int max_query_len,
                                                        int heads, int dim, int vdim) {
  if (!wants_blocks(g_channel_delta_kernel.load(std::memory_order_relaxed), max_query_len, dim)) return 0;
  return block_slots(num_tokens, num_seqs) * heads * block_floats((dim + 63) / 64 * 64, (vdim + 15) / 16 * 16);
}

extern "C" int vla_seq_set_channel_delta_kernel(int mode) {
  if (mode < 0 || mode > 2) return VLA_ERR_ARG;
  g_channel_delta_kernel.store(mode, std::memory_order_relaxed);
  return VLA_OK;
}

extern "C" int vla_seq_channel_delta_scan(
    float* o, const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v,
    int64_t v_stride, const void* beta, int64_t beta_stride, const float* z, int64_t z_stride,
    const float* dt_bias, const float* a_log, float* state, const int* query_start_loc,
    const int* context_lens, const int* state_slots, int num_tokens, int num_seqs, int num_slots,
    int max_query_len, int heads, int kv_heads, int dim, int vdim, float* scratch,
    int64_t scratch_floats, int dtype, void* stream) {
  if (num_seqs == 0 || num_tokens == 0) return VLA_OK;
  if (!o || !q || !k || !v || !beta || !z || !dt_bias || !a_log || !state || !query_start_loc ||
      !context_lens || !state_slots || num_seqs < 0 || num_seqs > 65535 || num_tokens < 0 ||
      num_slots <= 0 || max_query_len <= 0 || heads <= 0 || heads > 65535 || kv_heads <= 0 ||
      heads % kv_heads != 0 || dim <= 0 || vdim <= 0 || q_stride < (int64_t)kv_heads * dim ||
      k_stride < (int64_t)kv_heads * dim || v_stride < (int64_t)heads * vdim || beta_stride < heads ||
      z_stride < (int64_t)heads * dim)
    return VLA_ERR_ARG;
  hipStream_t st = (hipStream_t)stream;
  const int elem = dtype == VLA_F32 ? 4 : 2;
  ChannelDelta a;
  a.o = o;
  a.q = q;
  a.q_stride = q_stride;
  a.k = k;
  a.k_stride = k_stride;
  a.v = v;
  a.v_stride = v_stride;
  a.beta = beta;
  a.beta_stride = beta_stride;
  a.z = z;
  a.z_stride = z_stride;
  a.dt_bias = dt_bias;
  a.a_log = a_log;
  a.state = state;
  a.scratch = scratch;
  a.query_start_loc = query_start_loc;
  a.context_lens = context_lens;
  a.state_slots = state_slots;
  a.num_seqs = num_seqs;
  a.heads = heads;
  a.kv_heads = kv_heads;
  a.dim = dim;
  a.vdim = vdim;
  const int mode = g_channel_delta_kernel.load(std::memory_order_relaxed);
  a.mode = dim > kMaxBlockDim ? 1 : mode;
  auto fours = [&](const void* p, int64_t stride, int size) {      // four values per access
    return dim % 4 == 0 && stride % 4 == 0 && (uintptr_t)p % (4 * size) == 0;
  };
  a.vec_qk = fours(q, q_stride, elem) && fours(k, k_stride, elem);
  a.vec_z = fours(z, z_stride, 4) && fours(dt_bias, 0, 4);
  a.vec_state = fours(state, 0, 4);
  const bool steps = wants_steps(mode, max_query_len, num_seqs, dim), blocks = wants_blocks(mode, max_query_len, dim);
  const int64_t slots = block_slots(num_tokens, num_seqs);
  const int dx = (dim + 63) / 64;
  if (blocks && (!scratch || (uintptr_t)scratch % 16 || (vdim + 15) / 16 > 65535 ||
                 scratch_floats < slots * heads * block_floats(64 * dx, (vdim + 15) / 16 * 16)))
    return VLA_ERR_ARG;
  int rows = 0, split = 0;         // the fewest rows per thread whose columns are at most kMaxSplit lanes
  for (int r = 8; r <= 64 && rows == 0; r *= 2) {
    const int sp = pow2_at_least((dim + r - 1) / r);
    if (sp <= kMaxSplit) {
      rows = r;
      split = sp;
    }
  }
  if (rows == 0) return VLA_ERR_HEAD_SIZE;
  return with_dtype(dtype, [&](auto s) -> int {
    using S = decltype(s);
    if (steps) {
      const int cols = std::min(256 / split, vdim);
      const int threads = (cols * split + 63) / 64 * 64;
      const dim3 grid((vdim + cols - 1) / cols, heads, num_seqs);
      const size_t lds = 2 * (size_t)split * rows * sizeof(float);
      switch (rows) {
        case 8: channel_delta_step_kernel<S, 8><<<grid, threads, lds, st>>>(a, split, cols); break;
        case 16: channel_delta_step_kernel<S, 16><<<grid, threads, lds, st>>>(a, split, cols); break;
        case 32: channel_delta_step_kernel<S, 32><<<grid, threads, lds, st>>>(a, split, cols); break;
        default: channel_delta_step_kernel<S, 64><<<grid, threads, lds, st>>>(a, split, cols); break;
      }
      VLA_SEQ_HIP_CHECK(hipGetLastError());
    }
    if (!blocks) return VLA_OK;
    switch (dx) {
      case 1: return launch_blocks<S, 1>(a, slots, st);
      case 2: return launch_blocks<S, 2>(a, slots, st);
      case 3: return launch_blocks<S, 3>(a, slots, st);
      default: return launch_blocks<S, 4>(a, slots, st);
    }
  });
}
