// Row-wise steps of decoder layers that norm the stream itself after every sublayer (the norm
// follows the sum, so the fp32 stream is what the next sublayer reads):
//   post_norm         x <- N(alpha x + y) * w, and a copy of the new x in the activation dtype
//   rms_norm_rows     plain RMS norm of projected rows (a latent before its up-projection)
//   short_conv        causal convolution over time per channel with bias and activation, the last
//                     taps - 1 inputs of every sequence in state slots
//   gated_act_lookup  act(gate) * table[id, columns]: a per-token embedding gates a projection
//   embed_scaled      table[id] * scale as the fp32 stream
//   softcap           z <- cap * tanh(z / cap)
// One workgroup per row, fp32 arithmetic throughout; rows are read / written in the types named.
#include <atomic>
#include <type_traits>

#include "seq_common.h"

namespace vla {
namespace seq {
namespace {

std::atomic<int> g_conv_kernel{0};
constexpr int kThreads = 256;
constexpr int kKeep = 8;          // row elements a thread keeps in registers (rows up to 2048)
constexpr int kMaxTaps = 32;

__device__ __forceinline__ float activate(float z, int act) {
  switch (act) {
    case VLA_ACT_NONE: return z;
    case VLA_ACT_RELU: return fmaxf(z, 0.f);
    case VLA_ACT_RELU2: {
      const float r = fmaxf(z, 0.f);
      return r * r;
    }
    case VLA_ACT_SILU: return z / (1.f + expf(-z));
    default: return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  }
}

template <class SY, class SO>
__global__ __launch_bounds__(kThreads) void post_norm_kernel(
    float* __restrict__ x, float alpha, const typename SY::T* __restrict__ y, int64_t y_stride,
    const float* __restrict__ weight, float eps, typename SO::T* __restrict__ out, int width) {
  __shared__ float red[16];
  const int64_t base = (int64_t)blockIdx.x * width;
  const typename SY::T* yr = y + (int64_t)blockIdx.x * y_stride;
  float keep[kKeep];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int c = threadIdx.x + i * kThreads;
    keep[i] = 0.f;
    if (c < width) {
      keep[i] = alpha * x[base + c] + SY::to_f32(yr[c]);
      ss += keep[i] * keep[i];
    }
  }
  for (int c = threadIdx.x + kKeep * kThreads; c < width; c += kThreads) {
    const float v = alpha * x[base + c] + SY::to_f32(yr[c]);
    x[base + c] = v;                // parked in the stream until the scale is known
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int c = threadIdx.x + i * kThreads;
    if (c < width) {
      const float v = keep[i] * inv * weight[c];
      x[base + c] = v;
      if (out != nullptr) out[base + c] = SO::from_f32(v);
    }
  }
  for (int c = threadIdx.x + kKeep * kThreads; c < width; c += kThreads) {
    const float v = x[base + c] * inv * weight[c];
    x[base + c] = v;
    if (out != nullptr) out[base + c] = SO::from_f32(v);
  }
}

template <class SI, class SO>
__global__ __launch_bounds__(kThreads) void rms_norm_rows_kernel(
    typename SO::T* __restrict__ out, int64_t out_stride, const typename SI::T* __restrict__ in,
    int64_t in_stride, const float* __restrict__ weight, float eps, int n) {
  __shared__ float red[16];
  const typename SI::T* r = in + (int64_t)blockIdx.x * in_stride;
  float ss = 0.f;
  for (int c = threadIdx.x; c < n; c += kThreads) {
    const float v = SI::to_f32(r[c]);
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
  for (int c = threadIdx.x; c < n; c += kThreads)
    out[(int64_t)blockIdx.x * out_stride + c] = SO::from_f32(SI::to_f32(r[c]) * inv * weight[c]);
}

// out[t, c] = act(bias[c] + sum_d w[c, taps - 1 - d] * u at position p - d); rows of earlier
// steps come from the state slot, positions before the sequence's start are zeros.
template <class SI, class SO>
__global__ __launch_bounds__(kThreads) void short_conv_kernel(
    typename SO::T* __restrict__ out, int64_t out_stride, const typename SI::T* __restrict__ u,
    int64_t u_stride, const float* __restrict__ w, const float* __restrict__ bias,
    const float* __restrict__ state, const int* __restrict__ query_start_loc,
    const int* __restrict__ context_lens, const int* __restrict__ state_slots,
    const int* __restrict__ token_seq, int channels, int taps, int act) {
  const int t = blockIdx.x;
  const int b = token_seq[t];
  const int start = query_start_loc[b], ctx = context_lens[b];
  const int p = ctx + (t - start);
  const float* st = state + (int64_t)state_slots[b] * (taps - 1) * channels;
  for (int c = threadIdx.x; c < channels; c += kThreads) {
    float acc = bias != nullptr ? bias[c] : 0.f;
    for (int d = 0; d < taps; ++d) {
      const int s = p - d;
      if (s < 0) break;
      const float v = s >= ctx ? SI::to_f32(u[(int64_t)(t - d) * u_stride + c])
                               : st[(int64_t)(s - ctx + taps - 1) * channels + c];
      acc += w[(int64_t)c * taps + (taps - 1 - d)] * v;
    }
    out[(int64_t)t * out_stride + c] = SO::from_f32(activate(acc, act));
  }
}

// Two to four taps, silu or no activation, rows and channels in whole 16-byte pieces: a thread takes 16 bytes of channels
// through kRun consecutive rows of one sequence and keeps the taps - 1 inputs before the current row in
// registers.  Runs are counted from a sequence's first row of the step (sequence b's are slots
// start_b / kRun + b + 0, 1, ...), so only its first run needs the old state, and the thread that has it
// leaves the new one: one launch, no thread reads what another writes.
constexpr int kRun = 8;

template <class S, int VC>
__device__ __forceinline__ void unpack_channels(u32x4 got, float (&x)[VC]) {
  if constexpr (sizeof(typename S::T) == 2) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      x[2 * e] = lo16<S>(got[e]);
      x[2 * e + 1] = hi16<S>(got[e]);
    }
  } else {
    const f32x4 f = __builtin_bit_cast(f32x4, got);
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = f[e];
  }
}
template <class S, int VC>
__device__ __forceinline__ void load_channels(const typename S::T* p, float (&x)[VC]) {
  unpack_channels<S, VC>(*reinterpret_cast<const u32x4*>(p), x);
}

template <class SI, class SO, int TAPS, int ACT>
__global__ __launch_bounds__(kThreads) void short_conv_run_kernel(
    typename SO::T* __restrict__ out, int64_t out_stride, const typename SI::T* __restrict__ u,
    int64_t u_stride, const float* __restrict__ w, const float* __restrict__ bias, float* state,
    const int* __restrict__ query_start_loc, const int* __restrict__ context_lens,
    const int* __restrict__ state_slots, int num_seqs, int channels) {
  constexpr int VC = 16 / sizeof(typename SI::T), B = TAPS - 1;
  const int c = VC * (blockIdx.x * blockDim.x + threadIdx.x);
  if (c >= channels) return;
  int lo = 0, hi = num_seqs - 1;                // the last sequence whose first slot is not behind this one
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (query_start_loc[mid] / kRun + mid <= (int)blockIdx.y)
      lo = mid;
    else
      hi = mid - 1;
  }
  const int start = query_start_loc[lo], end = query_start_loc[lo + 1];
  const int run = blockIdx.y - (start / kRun + lo);
  const int t0 = start + run * kRun, t1 = min(t0 + kRun, end);
  if (t0 >= end) return;                        // a slot behind the sequence's last run
  u32x4 rows[kRun];                             // the whole run is asked for before anything is used
#pragma unroll
  for (int i = 0; i < kRun; ++i)
    rows[i] = *reinterpret_cast<const u32x4*>(u + (int64_t)min(t0 + i, t1 - 1) * u_stride + c);
  float wt[TAPS][VC], bs[VC];
#pragma unroll
  for (int i = 0; i < VC * TAPS; i += 4) {      // the weights of VC channels lie side by side
    const f32x4 got = *reinterpret_cast<const f32x4*>(w + (int64_t)c * TAPS + i);
#pragma unroll
    for (int e = 0; e < 4; ++e) wt[(i + e) % TAPS][(i + e) / TAPS] = got[e];
  }
#pragma unroll
  for (int v = 0; v < VC; v += 4) {
    f32x4 got = {0.f, 0.f, 0.f, 0.f};
    if (bias != nullptr) got = *reinterpret_cast<const f32x4*>(bias + c + v);
#pragma unroll
    for (int e = 0; e < 4; ++e) bs[v + e] = got[e];
  }
  float before[B][VC];                          // the inputs B, ..., 1 rows back
  const int ctx = context_lens[lo];
  float* st = state + (int64_t)state_slots[lo] * B * channels + c;
#pragma unroll
  for (int i = 0; i < B; ++i) {
    if (run > 0) {
      load_channels<SI, VC>(u + (int64_t)(t0 - B + i) * u_stride + c, before[i]);
    } else {
#pragma unroll
      for (int v = 0; v < VC; v += 4) {         // entry i of the old state is position ctx - B + i
        f32x4 got = {0.f, 0.f, 0.f, 0.f};
        if (ctx - B + i >= 0) got = *reinterpret_cast<const f32x4*>(st + (int64_t)i * channels + v);
#pragma unroll
        for (int e = 0; e < 4; ++e) before[i][v + e] = got[e];
      }
    }
  }
#pragma unroll
  for (int k = 0; k < kRun; ++k) {
    const int t = t0 + k;
    if (t >= t1) break;
    float cur[VC], r[VC];
    unpack_channels<SI, VC>(rows[k], cur);
#pragma unroll
    for (int v = 0; v < VC; ++v) {
      float acc = bs[v];
#pragma unroll
      for (int i = 0; i < B; ++i) acc += wt[i][v] * before[i][v];
      acc += wt[B][v] * cur[v];
      if constexpr (ACT == VLA_ACT_SILU && sizeof(typename SO::T) == 2)      // rounded to 16 bits right away
        r[v] = acc * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * acc));
      else
        r[v] = activate(acc, ACT);
    }
    typename SO::T* o = out + (int64_t)t * out_stride + c;
    if constexpr (sizeof(typename SO::T) == 2) {
      uint32_t word[VC / 2];
#pragma unroll
      for (int e = 0; e < VC / 2; ++e) word[e] = pack16<SO>(r[2 * e], r[2 * e + 1]);
      if constexpr (VC == 8)
        *reinterpret_cast<u32x4*>(o) = u32x4{word[0], word[1], word[2], word[3]};
      else
        *reinterpret_cast<u32x2*>(o) = u32x2{word[0], word[1]};
    } else {
#pragma unroll
      for (int v = 0; v < VC; v += 4) *reinterpret_cast<f32x4*>(o + v) = f32x4{r[v], r[v + 1], r[v + 2], r[v + 3]};
    }
#pragma unroll
    for (int v = 0; v < VC; ++v) {
#pragma unroll
      for (int i = 0; i + 1 < B; ++i) before[i][v] = before[i + 1][v];
      before[B - 1][v] = cur[v];
    }
  }
  if (run > 0) return;
  if (t1 < end) {                               // the sequence goes on: its last inputs are other runs' rows
#pragma unroll
    for (int i = 0; i < B; ++i) load_channels<SI, VC>(u + (int64_t)(end - B + i) * u_stride + c, before[i]);
  }
#pragma unroll
  for (int i = 0; i < B; ++i)
#pragma unroll
    for (int v = 0; v < VC; v += 4)
      *reinterpret_cast<f32x4*>(st + (int64_t)i * channels + v) =
          f32x4{before[i][v], before[i][v + 1], before[i][v + 2], before[i][v + 3]};
}

// The last taps - 1 inputs of every sequence of the step, oldest first.  A thread owns a channel:
// it reads what it keeps of the old state before it writes.
template <class SI>
__global__ __launch_bounds__(kThreads) void short_conv_state_kernel(
    float* __restrict__ state, const typename SI::T* __restrict__ u, int64_t u_stride,
    const int* __restrict__ query_start_loc, const int* __restrict__ context_lens,
    const int* __restrict__ state_slots, int channels, int taps) {
  const int b = blockIdx.y;
  const int c = blockIdx.x * kThreads + threadIdx.x;
  if (c >= channels) return;
  const int start = query_start_loc[b], n = query_start_loc[b + 1] - start, ctx = context_lens[b];
  float* st = state + (int64_t)state_slots[b] * (taps - 1) * channels;
  float keep[kMaxTaps];
  for (int i = 0; i < taps - 1; ++i) {
    const int s = ctx + n - (taps - 1) + i;     // position that lands in entry i
    float v = 0.f;
    if (s >= ctx)
      v = SI::to_f32(u[(int64_t)(start + s - ctx) * u_stride + c]);
    else if (s >= 0)
      v = st[(int64_t)(s - ctx + taps - 1) * channels + c];
    keep[i] = v;
  }
  for (int i = 0; i < taps - 1; ++i) st[(int64_t)i * channels + c] = keep[i];
}

template <class SI, class ST, class SO>
__global__ __launch_bounds__(kThreads) void gated_act_lookup_kernel(
    typename SO::T* __restrict__ out, int64_t out_stride, const typename SI::T* __restrict__ gate,
    int64_t gate_stride, const typename ST::T* __restrict__ table, int64_t table_stride,
    const int64_t* __restrict__ ids, int rows, int first_col, int features, int act) {
  const int64_t t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= rows ? rows - 1 : id);
  for (int c = threadIdx.x; c < features; c += kThreads)
    out[t * out_stride + c] = SO::from_f32(activate(SI::to_f32(gate[t * gate_stride + c]), act) *
                                           ST::to_f32(table[id * table_stride + first_col + c]));
}

template <class S>
__global__ __launch_bounds__(kThreads) void embed_scaled_kernel(
    float* __restrict__ out, const typename S::T* __restrict__ table, const int64_t* __restrict__ ids,
    float scale, int width, int vocab) {
  const int t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const typename S::T* row = table + id * (int64_t)width;
  for (int c = threadIdx.x; c < width; c += kThreads)
    out[(int64_t)t * width + c] = S::to_f32(row[c]) * scale;
}

__global__ __launch_bounds__(kThreads) void softcap_kernel(float* __restrict__ z, int64_t n, float cap) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i < n) z[i] = cap * tanhf(z[i] / cap);
}

template <class F>
int with_two(int a, int b, F&& f) {
  return with_dtype(a, [&](auto sa) { return with_dtype(b, [&](auto sb) { return f(sa, sb); }); });
}

}  // namespace
}  // namespace seq
}  // namespace vla

using namespace vla;
using namespace vla::seq;

extern "C" int vla_seq_post_norm(float* x, float alpha, const void* y, int64_t y_stride, int y_dtype,
                                 const float* weight, float eps, void* out, int out_dtype,
                                 int num_tokens, int width, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!x || !y || !weight || num_tokens < 0 || width <= 0 || y_stride < width) return VLA_ERR_ARG;
  return with_two(y_dtype, out ? out_dtype : VLA_F32, [&](auto sy, auto so) {
    using SY = decltype(sy);
    using SO = decltype(so);
    post_norm_kernel<SY, SO><<<num_tokens, kThreads, 0, (hipStream_t)stream>>>(
        x, alpha, (const typename SY::T*)y, y_stride, weight, eps, (typename SO::T*)out, width);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    return VLA_OK;
  });
}

extern "C" int vla_seq_rms_norm_rows(void* out, int64_t out_stride, int out_dtype, const void* in,
                                     int64_t in_stride, int in_dtype, const float* weight, float eps,
                                     int num_tokens, int n, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!out || !in || !weight || num_tokens < 0 || n <= 0 || out_stride < n || in_stride < n)
    return VLA_ERR_ARG;
  return with_two(in_dtype, out_dtype, [&](auto si, auto so) {
    using SI = decltype(si);
    using SO = decltype(so);
    rms_norm_rows_kernel<SI, SO><<<num_tokens, kThreads, 0, (hipStream_t)stream>>>(
        (typename SO::T*)out, out_stride, (const typename SI::T*)in, in_stride, weight, eps, n);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    return VLA_OK;
  });
}

extern "C" int vla_seq_short_conv(void* out, int64_t out_stride, int out_dtype, const void* u,
                                  int64_t u_stride, int u_dtype, const float* weight,
                                  const float* bias, float* state, const int* query_start_loc,
                                  const int* context_lens, const int* state_slots,
                                  const int* token_seq, int num_tokens, int num_seqs, int num_slots,
                                  int channels, int taps, int act, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!out || !u || !weight || !query_start_loc || !context_lens || !state_slots || !token_seq ||
      num_tokens < 0 || num_seqs <= 0 || num_seqs > 65535 || channels <= 0 || taps < 1 ||
      taps > kMaxTaps || out_stride < channels || u_stride < channels || act < VLA_ACT_NONE ||
      act > VLA_ACT_GELU_TANH || (taps > 1 && (!state || num_slots <= 0)))
    return VLA_ERR_ARG;
  return with_two(u_dtype, out_dtype, [&](auto si, auto so) {
    using SI = decltype(si);
    using SO = decltype(so);
    using TI = typename SI::T;
    using TO = typename SO::T;
    constexpr int VC = 16 / sizeof(TI);
    const bool vec = taps >= 2 && taps <= 4 && (act == VLA_ACT_NONE || act == VLA_ACT_SILU) && channels % VC == 0 && ((uintptr_t)u % 16) == 0 &&
                     u_stride % VC == 0 && (uintptr_t)out % (VC * sizeof(TO) < 16 ? VC * sizeof(TO) : 16) == 0 &&
                     out_stride % VC == 0 && ((uintptr_t)state % 16) == 0 &&
                     ((uintptr_t)weight % 16) == 0 && ((uintptr_t)bias % 16) == 0 &&
                     num_tokens / kRun + num_seqs <= 65535 && g_conv_kernel.load(std::memory_order_relaxed) == 0;
    if (vec) {
      const int pieces = channels / VC, blocks = (pieces + kThreads - 1) / kThreads;
      const int threads = ((pieces + blocks - 1) / blocks + kWave - 1) / kWave * kWave;
      const dim3 grid(blocks, num_tokens / kRun + num_seqs);
      auto launch = [&](auto kernel) {
        kernel<<<grid, threads, 0, (hipStream_t)stream>>>((TO*)out, out_stride, (const TI*)u, u_stride, weight, bias,
                                                          state, query_start_loc, context_lens, state_slots,
                                                          num_seqs, channels);
      };
      auto by_act = [&](auto n) {
        if (act == VLA_ACT_SILU)
          launch(short_conv_run_kernel<SI, SO, decltype(n)::value, VLA_ACT_SILU>);
        else
          launch(short_conv_run_kernel<SI, SO, decltype(n)::value, VLA_ACT_NONE>);
      };
      if (taps == 2)
        by_act(std::integral_constant<int, 2>{});
      else if (taps == 3)
        by_act(std::integral_constant<int, 3>{});
      else
        by_act(std::integral_constant<int, 4>{});
    } else {
      short_conv_kernel<SI, SO><<<num_tokens, kThreads, 0, (hipStream_t)stream>>>(
          (TO*)out, out_stride, (const TI*)u, u_stride, weight, bias, state, query_start_loc, context_lens,
          state_slots, token_seq, channels, taps, act);
    }
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    if (taps > 1 && !vec) {
      short_conv_state_kernel<SI><<<dim3((channels + kThreads - 1) / kThreads, num_seqs), kThreads, 0,
                                    (hipStream_t)stream>>>(state, (const typename SI::T*)u, u_stride,
                                                           query_start_loc, context_lens, state_slots,
                                                           channels, taps);
      VLA_SEQ_HIP_CHECK(hipGetLastError());
    }
    return VLA_OK;
  });
}

// 0: short_conv picks its kernel per shape; 1: always the one for any taps and alignment (tests run both)
extern "C" int vla_seq_set_short_conv_kernel(int mode) {
  if (mode < 0 || mode > 1) return VLA_ERR_ARG;
  g_conv_kernel.store(mode, std::memory_order_relaxed);
  return VLA_OK;
}

extern "C" int vla_seq_gated_act_lookup(void* out, int64_t out_stride, int out_dtype,
                                        const void* gate, int64_t gate_stride, int gate_dtype,
                                        const void* table, int64_t table_stride, int table_dtype,
                                        const int64_t* ids, int rows, int first_col, int num_tokens,
                                        int features, int act, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!out || !gate || !table || !ids || num_tokens < 0 || features <= 0 || rows <= 0 ||
      first_col < 0 || out_stride < features || gate_stride < features ||
      table_stride < (int64_t)first_col + features || act < VLA_ACT_NONE || act > VLA_ACT_GELU_TANH)
    return VLA_ERR_ARG;
  return with_two(gate_dtype, out_dtype, [&](auto si, auto so) {
    return with_dtype(table_dtype, [&](auto st) {
      using SI = decltype(si);
      using SO = decltype(so);
      using ST = decltype(st);
      gated_act_lookup_kernel<SI, ST, SO><<<num_tokens, kThreads, 0, (hipStream_t)stream>>>(
          (typename SO::T*)out, out_stride, (const typename SI::T*)gate, gate_stride,
          (const typename ST::T*)table, table_stride, ids, rows, first_col, features, act);
      VLA_SEQ_HIP_CHECK(hipGetLastError());
      return VLA_OK;
    });
  });
}

extern "C" int vla_seq_embed_scaled(float* out, const void* table, const int64_t* ids, float scale,
                                    int num_tokens, int width, int vocab, int dtype, void* stream) {
  if (num_tokens == 0) return VLA_OK;
  if (!out || !table || !ids || num_tokens < 0 || width <= 0 || vocab <= 0) return VLA_ERR_ARG;
  return with_dtype(dtype, [&](auto s) {
    using S = decltype(s);
    embed_scaled_kernel<S><<<num_tokens, kThreads, 0, (hipStream_t)stream>>>(
        out, (const typename S::T*)table, ids, scale, width, vocab);
    VLA_SEQ_HIP_CHECK(hipGetLastError());
    return VLA_OK;
  });
}

extern "C" int vla_seq_softcap(float* z, int64_t n, float cap, void* stream) {
  if (n == 0) return VLA_OK;
  if (!z || n < 0 || !(cap > 0.f)) return VLA_ERR_ARG;
  softcap_kernel<<<(unsigned)((n + kThreads - 1) / kThreads), kThreads, 0, (hipStream_t)stream>>>(z, n, cap);
  VLA_SEQ_HIP_CHECK(hipGetLastError());
  return VLA_OK;
}
