// The residual stream around sub-layers whose output is normalized before it is added, and token tables.
//
//   stream += norm(y) * w,   y = the sub-layer's output, or scale * (norm(a) * wa + norm(b) * wb) for a sub-layer
//   made of two whose outputs are normalized first
// with norm(y) = y / sqrt(mean(y^2) + eps), everything in float; the new stream is also written in the activation type
// (what the next sub-layer reads). An output is one tensor or float slices that are summed first.
//
// The gather with a bigram table: row = table[id] + bigram[(previous id * mul_prev + id * mul_cur) mod buckets], or
// bigram[buckets] for a sequence's first token; the previous token of a step's first token of an item lies in the
// item's state slot (as id + 1, 0: there is none), where the item's last token goes.

#include <algorithm>

#include "api.h"
#include "common.h"

namespace psamd {

struct NormInput {
  const void* y;
  int dtype;
  int slices;
  int64_t stride;                          // elements between slices
  const float* w;                          // null: the output is not normalized on its own
};

// V neighbouring values of row r of an output, its slices summed in ascending order.
template <int V>
__device__ __forceinline__ void sum_slices(const NormInput& in, int64_t at, float (&out)[V]) {
#pragma unroll
  for (int e = 0; e < V; ++e) out[e] = 0.f;
  if constexpr (V == 4) {
    if (in.dtype == kBF16) {
      const uint2 q = *reinterpret_cast<const uint2*>(static_cast<const bf16_t*>(in.y) + at);
      out[0] = __uint_as_float(q.x << 16), out[1] = __uint_as_float(q.x & 0xffff0000u);
      out[2] = __uint_as_float(q.y << 16), out[3] = __uint_as_float(q.y & 0xffff0000u);
      return;
    }
    const float* y = static_cast<const float*>(in.y) + at;
    for (int p = 0; p < in.slices; p += 8) {
      float4 t[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) t[u] = *reinterpret_cast<const float4*>(y + min(p + u, in.slices - 1) * in.stride);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (p + u < in.slices) out[0] += t[u].x, out[1] += t[u].y, out[2] += t[u].z, out[3] += t[u].w;
    }
  } else {
    for (int p = 0; p < in.slices; ++p) out[0] += load_as_float(in.y, in.dtype, at + p * in.stride);
  }
}

// Two sums over the workgroup at once; every thread gets both.
template <int WAVES>
__device__ __forceinline__ float2 block_sum2(float a, float b, float* scratch) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int lane = threadIdx.x & (kWave - 1), w = threadIdx.x / kWave;
  __syncthreads();
  if (lane == 0) {
    scratch[2 * w] = a;
    scratch[2 * w + 1] = b;
  }
  __syncthreads();
  float2 t = make_float2(0.f, 0.f);
#pragma unroll
  for (int i = 0; i < WAVES; ++i) t.x += scratch[2 * i], t.y += scratch[2 * i + 1];
  return t;
}

// One workgroup per row. Every thread owns the same columns in every pass, so rows lie in LDS (or registers) without
// barriers of their own. CACHE > 0: up to CACHE pieces of V columns a thread stay in registers; 0: rows in LDS.
template <typename OT, int V, int CACHE, int THREADS, bool TWO>
__global__ __launch_bounds__(THREADS) void output_norm_kernel(float* __restrict__ residual, NormInput a, NormInput b, float scale,
                                                              float in_eps, const float* __restrict__ w, float eps,
                                                              OT* __restrict__ out, int hidden) {
  extern __shared__ __align__(16) float norm_smem[];    // CACHE 0: the rows of a (and b)
  __shared__ float scratch[2 * (THREADS / kWave)];
  constexpr int WAVES = THREADS / kWave;
  constexpr int N = CACHE > 0 ? CACHE : 1;
  const int64_t r = static_cast<int64_t>(blockIdx.x) * hidden;
  const float inv_n = 1.f / static_cast<float>(hidden);
  float ya[N][V], yb[TWO ? N : 1][V];
  float sa = 0.f, sb = 0.f;
  auto pieces = [&](auto body) {                          // body(piece, first column) for every piece of the thread
    if constexpr (CACHE > 0) {
#pragma unroll
      for (int p = 0; p < CACHE; ++p) {
        const int i = (static_cast<int>(threadIdx.x) + p * THREADS) * V;
        if (i < hidden) body(p, i);
      }
    } else {
      for (int i = threadIdx.x * V; i < hidden; i += THREADS * V) body(0, i);
    }
  };
  auto load_row = [&](int p, int i) {
    if constexpr (CACHE == 0) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        ya[p][e] = norm_smem[i + e];
        if constexpr (TWO) yb[p][e] = norm_smem[hidden + i + e];
      }
    }
  };
  auto keep_row = [&](int p, int i) {
    if constexpr (CACHE == 0) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        norm_smem[i + e] = ya[p][e];
        if constexpr (TWO) norm_smem[hidden + i + e] = yb[p][e];
      }
    }
  };
  pieces([&](int p, int i) {
    sum_slices<V>(a, r + i, ya[p]);
    if constexpr (TWO) sum_slices<V>(b, r + i, yb[p]);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      sa = fmaf(ya[p][e], ya[p][e], sa);
      if constexpr (TWO) sb = fmaf(yb[p][e], yb[p][e], sb);
    }
    keep_row(p, i);
  });
  float2 sums = block_sum2<WAVES>(sa, sb, scratch);
  if constexpr (TWO) {
    const float ia = scale / sqrtf(sums.x * inv_n + in_eps), ib = scale / sqrtf(sums.y * inv_n + in_eps);
    sa = 0.f;
    pieces([&](int p, int i) {
      load_row(p, i);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        ya[p][e] = ya[p][e] * ia * a.w[i + e] + yb[p][e] * ib * b.w[i + e];
        sa = fmaf(ya[p][e], ya[p][e], sa);
      }
      keep_row(p, i);
    });
    sums = block_sum2<WAVES>(sa, 0.f, scratch);
  }
  const float inv = 1.f / sqrtf(sums.x * inv_n + eps);
  pieces([&](int p, int i) {
    load_row(p, i);
    float* x = residual + r + i;
    float y[V];
    if constexpr (V == 4) {
      const float4 old = *reinterpret_cast<const float4*>(x);
      y[0] = old.x, y[1] = old.y, y[2] = old.z, y[3] = old.w;
    } else {
      y[0] = x[0];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] += ya[p][e] * inv * w[i + e];
    if constexpr (V == 4) {
      *reinterpret_cast<float4*>(x) = make_float4(y[0], y[1], y[2], y[3]);
      if (out != nullptr) {
        if constexpr (sizeof(OT) == 2)
          *reinterpret_cast<ushort4*>(out + r + i) = ushort4{float_to_bf16(y[0]), float_to_bf16(y[1]), float_to_bf16(y[2]), float_to_bf16(y[3])};
        else
          *reinterpret_cast<float4*>(out + r + i) = make_float4(y[0], y[1], y[2], y[3]);
      }
    } else {
      x[0] = y[0];
      if (out != nullptr) out[r + i] = from_float<OT>(y[0]);
    }
  });
}

// One workgroup per token (see above). The workgroup of an item's first token reads the saved token and then replaces
// it by the item's last one: nobody else touches the slot.
template <typename W>
__global__ __launch_bounds__(256) void embed_bigram_kernel(
    const int32_t* __restrict__ ids, const W* __restrict__ table, const W* __restrict__ bigram, float* __restrict__ out,
    W* __restrict__ copy, int hidden, int vocab, int64_t buckets, int64_t mul_prev, int64_t mul_cur, int32_t* __restrict__ state,
    int64_t state_row, const int32_t* __restrict__ tok_item, const int32_t* __restrict__ item_start, const int32_t* __restrict__ slots) {
  const int64_t t = blockIdx.x;
  const int item = tok_item[t];
  const int64_t s0 = item_start[item];
  // Ids a previous step sampled are not checked on the host: one outside the table reads its nearest row.
  const int id = min(max(ids[t], 0), vocab - 1);
  int32_t* saved = state + static_cast<int64_t>(slots[item]) * state_row;
  const int before = t > s0 ? min(max(ids[t - 1], 0), vocab - 1) : *saved - 1;
  if (t == s0) {
    __syncthreads();                                     // every thread has read the saved token
    if (threadIdx.x == 0) *saved = min(max(ids[item_start[item + 1] - 1], 0), vocab - 1) + 1;
  }
  int64_t bucket = buckets;
  if (before >= 0) {
    bucket = (before * mul_prev + id * mul_cur) % buckets;
    if (bucket < 0) bucket += buckets;
  }
  const W* row = table + static_cast<int64_t>(id) * hidden;
  const W* more = bigram + bucket * hidden;
  for (int i = threadIdx.x; i < hidden; i += 256) {
    const float x = to_float<W>(row[i]) + to_float<W>(more[i]);
    out[t * hidden + i] = x;
    if (copy != nullptr) copy[t * hidden + i] = from_float<W>(x);
  }
}

template <typename OT, int V, int CACHE, int THREADS>
static int launch_output_norm(hipStream_t s, float* residual, const NormInput& a, const NormInput& b, float scale, float in_eps,
                              const float* w, float eps, void* out, int64_t rows, int hidden) {
  const dim3 grid(static_cast<unsigned>(rows)), block(THREADS);
  const size_t smem = CACHE > 0 ? 0 : sizeof(float) * static_cast<size_t>(hidden) * (b.y != nullptr ? 2 : 1);
  if (b.y != nullptr)
    output_norm_kernel<OT, V, CACHE, THREADS, true><<<grid, block, smem, s>>>(residual, a, b, scale, in_eps, w, eps, static_cast<OT*>(out), hidden);
  else
    output_norm_kernel<OT, V, CACHE, THREADS, false><<<grid, block, smem, s>>>(residual, a, b, scale, in_eps, w, eps, static_cast<OT*>(out), hidden);
  return check_launch("psamd_output_norm");
}

template <typename OT>
static int by_width(hipStream_t s, float* residual, const NormInput& a, const NormInput& b, float scale, float in_eps, const float* w,
                    float eps, void* out, int64_t rows, int hidden) {
  const auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool wide = hidden % 4 == 0 && a.stride % 4 == 0 && b.stride % 4 == 0 && aligned(residual) && aligned(a.y) && aligned(b.y) &&
                    aligned(a.w) && aligned(b.w) && aligned(w) && aligned(out);
  if (wide && hidden <= 1024) return launch_output_norm<OT, 4, 1, 256>(s, residual, a, b, scale, in_eps, w, eps, out, rows, hidden);
  if (wide && hidden <= 2048) return launch_output_norm<OT, 4, 2, 256>(s, residual, a, b, scale, in_eps, w, eps, out, rows, hidden);
  if (wide && hidden <= 4096) return launch_output_norm<OT, 4, 2, 512>(s, residual, a, b, scale, in_eps, w, eps, out, rows, hidden);
  if (wide && hidden <= 8192) return launch_output_norm<OT, 4, 2, 1024>(s, residual, a, b, scale, in_eps, w, eps, out, rows, hidden);
  PSAMD_REQUIRE(sizeof(float) * static_cast<size_t>(hidden) * (b.y != nullptr ? 2 : 1) <= 64 * 1024, "a row does not fit in LDS");
  return launch_output_norm<OT, 1, 0, 256>(s, residual, a, b, scale, in_eps, w, eps, out, rows, hidden);
}

}  // namespace psamd

using namespace psamd;

extern "C" {

int psamd_output_norm(void* stream, float* residual, const void* a, int a_dtype, int a_slices, int64_t a_stride, const float* a_weight,
                      const void* b, int b_dtype, int b_slices, int64_t b_stride, const float* b_weight, float scale, float in_eps,
                      const float* weight, float eps, void* out, int out_dtype, int64_t rows, int hidden) {
  PSAMD_REQUIRE(rows >= 0 && rows <= 2147483647LL && hidden > 0, "bad sizes");
  PSAMD_REQUIRE(a != nullptr && a_slices >= 1 && (a_dtype == kF32 || (a_dtype == kBF16 && a_slices == 1)), "one tensor or float slices");
  PSAMD_REQUIRE(b == nullptr || (b_slices >= 1 && (b_dtype == kF32 || (b_dtype == kBF16 && b_slices == 1))), "one tensor or float slices");
  PSAMD_REQUIRE((b == nullptr) == (b_weight == nullptr) && (b == nullptr) == (a_weight == nullptr),
                "two outputs are normalized on their own, each with a weight");
  PSAMD_REQUIRE(residual != nullptr && weight != nullptr, "missing operands");
  if (rows == 0) return 0;
  const NormInput ia{a, a_dtype, a_slices, a_stride, a_weight}, ib{b, b_dtype, b_slices, b != nullptr ? b_stride : 0, b_weight};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (out != nullptr && out_dtype == kBF16) return by_width<bf16_t>(s, residual, ia, ib, scale, in_eps, weight, eps, out, rows, hidden);
  if (out == nullptr || out_dtype == kF32) return by_width<float>(s, residual, ia, ib, scale, in_eps, weight, eps, out, rows, hidden);
  return fail("psamd_output_norm: the copy is float32 or bfloat16");
}

int psamd_embed_bigram(void* stream, const int32_t* ids, const void* table, const void* bigram, int table_dtype, float* out, void* copy,
                       int64_t tokens, int hidden, int vocab, int64_t buckets, int64_t mul_prev, int64_t mul_cur, int32_t* state,
                       int64_t state_row, const int32_t* tok_item, const int32_t* item_start, const int32_t* slots) {
  PSAMD_REQUIRE(tokens >= 0 && tokens <= 2147483647LL && hidden > 0 && vocab > 0 && buckets >= 1, "bad sizes");
  PSAMD_REQUIRE(state != nullptr && state_row >= 1, "the previous token lies in the state");
  if (tokens == 0) return 0;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid(static_cast<unsigned>(tokens));
  if (table_dtype == kBF16)
    embed_bigram_kernel<bf16_t><<<grid, dim3(256), 0, s>>>(ids, static_cast<const bf16_t*>(table), static_cast<const bf16_t*>(bigram), out,
                                                          static_cast<bf16_t*>(copy), hidden, vocab, buckets, mul_prev, mul_cur, state,
                                                          state_row, tok_item, item_start, slots);
  else if (table_dtype == kF32)
    embed_bigram_kernel<float><<<grid, dim3(256), 0, s>>>(ids, static_cast<const float*>(table), static_cast<const float*>(bigram), out,
                                                         static_cast<float*>(copy), hidden, vocab, buckets, mul_prev, mul_cur, state,
                                                         state_row, tok_item, item_start, slots);
  else
    return fail("psamd_embed_bigram: the tables are float32 or bfloat16");
  return check_launch("psamd_embed_bigram");
}

}  // extern "C"
