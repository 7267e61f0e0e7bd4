// Between the input product of attention with short convolutions and the attention itself, in one launch:
// a causal convolution per channel on q, k and v (continued in front of an item's first token from the inputs
// its state slot saved), an RMS norm per q and k head with an optional weight shared by the heads, the rotation of
// the pairs (i, i + d/2), and the write of keys and values into their pages. Everything between the product's
// output and the stored results is float.
//
// A row of the input holds (hq + 2 hkv) heads of d channels: q heads, k heads, v heads. The results leave the
// input as it is (neighbouring tokens read it): q goes to rows of its own, k and v to the pages.

#include <algorithm>

#include "api.h"
#include "common.h"

namespace psamd {

constexpr int kConvTokens = 4;             // consecutive tokens per workgroup
constexpr int kConvMostTaps = 16;
constexpr int kConvFastTaps = 4;           // up to here the taps' weights and inputs stay in registers

template <typename A>
struct QkvConv {
  const A* in;
  int64_t in_row;
  const float* w;                          // [taps][channels]
  int channels, taps;
  int hq, hkv, d;
  const int32_t* positions;
  const float2* table;                     // [pos][d / 2] or null
  int norm_dim;                            // 0: no norm
  float eps;
  const float* q_weight;                   // [d] or null
  const float* k_weight;
  A* q_out;                                // [tokens][hq * d]
  A* kv;                                   // pages or null
  const int32_t* write_slot;
  float* state;                            // saved inputs of slot s: state + s * state_row, [taps - 1][channels], oldest first
  int64_t state_row;
  const int32_t* tok_item;
  const int32_t* item_start;
  const int32_t* slots;
  int tokens;
};

// What the rest of a token's head needs from memory besides the convolution, asked for before it.
template <int P>
struct TokenRest {
  int first;                               // the item's first token
  int slot;                                // the token's place in the pages
  float2 cs[P];
};

template <typename A, int P>
__device__ __forceinline__ void load_rest(const QkvConv<A>& c, int64_t t, int l, int lanes, TokenRest<P>& r) {
  const int half = c.d >> 1;
  r.first = c.item_start[c.tok_item[t]];
  r.slot = c.kv != nullptr ? c.write_slot[t] : 0;
  const int64_t pos = c.positions[t];
#pragma unroll
  for (int p = 0; p < P; ++p) r.cs[p] = c.table != nullptr ? c.table[pos * half + min(l + p * lanes, half - 1)] : make_float2(1.f, 0.f);
}

// A q or k head's norm weights for the lane (ones where there are none).
template <typename A, int P>
__device__ __forceinline__ void load_norm(const QkvConv<A>& c, int head, int l, int lanes, float (&na)[P], float (&nb)[P]) {
  const int half = c.d >> 1;
  const float* nw = head < c.hq ? c.q_weight : head < c.hq + c.hkv ? c.k_weight : nullptr;
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = min(l + p * lanes, half - 1);
    na[p] = nw != nullptr ? nw[i] : 1.f;
    nb[p] = nw != nullptr ? nw[i + half] : 1.f;
  }
}

// Norm, rotation and write of one token's head; a, b: the convolution's results for the lane's pairs (zeros past the head).
template <typename A, int P>
__device__ __forceinline__ void finish_head(const QkvConv<A>& c, int64_t t, int head, int l, int lanes, const float (&a)[P],
                                            const float (&b)[P], const float (&na)[P], const float (&nb)[P], const TokenRest<P>& r) {
  const int half = c.d >> 1;
  const int64_t page_elems = 2LL * c.hkv * kPage * c.d, page = r.slot / kPage;
  const int off = r.slot % kPage;
  if (head >= c.hq + c.hkv) {                            // a value head: as it is, transposed into its page
    if (c.kv == nullptr) return;
    A* vpage = c.kv + page * page_elems + (static_cast<int64_t>(c.hkv) + (head - c.hq - c.hkv)) * kPage * c.d + off;
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int i = l + p * lanes;
      if (i >= half) continue;
      vpage[static_cast<int64_t>(i) * kPage] = from_float<A>(a[p]);
      vpage[static_cast<int64_t>(i + half) * kPage] = from_float<A>(b[p]);
    }
    return;
  }
  float inv = 1.f;
  if (c.norm_dim > 0) {
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < P; ++p) ss = fmaf(a[p], a[p], fmaf(b[p], b[p], ss));
    for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, kWave);
    inv = 1.f / sqrtf(ss / static_cast<float>(c.norm_dim) + c.eps);
  }
  A* dst = head < c.hq ? c.q_out + t * (static_cast<int64_t>(c.hq) * c.d) + static_cast<int64_t>(head) * c.d
                       : (c.kv != nullptr ? c.kv + page * page_elems + (static_cast<int64_t>(head - c.hq) * kPage + off) * c.d : nullptr);
  if (dst == nullptr) return;
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = l + p * lanes;
    if (i >= half) continue;
    const float u = a[p] * inv * na[p], v = b[p] * inv * nb[p];
    dst[i] = from_float<A>(u * r.cs[p].x - v * r.cs[p].y);
    dst[i + half] = from_float<A>(v * r.cs[p].x + u * r.cs[p].y);
  }
}

// grid (ceil(tokens / kConvTokens) + items, heads / (4 * 64 / lanes)). A token that lies taps - 1 or more behind its
// item's first token needs only the step's own rows: the first kind of workgroup. The first taps - 1 tokens of an
// item read the inputs its slot saved, which are then replaced by the item's last ones: the second kind, where a
// channel belongs to one lane throughout, so that nobody reads a saved input another lane has replaced.
// P: pairs per lane (lanes = 64 and two of them when d > 128). TAPS: their number where the inputs of a workgroup's tokens are
// kept in registers, so that all loads are on their way before the first sum; 0: any number, read tap by tap.
template <typename A, int P, int TAPS>
__global__ __launch_bounds__(256) void qkv_conv_kernel(QkvConv<A> c, int lanes, int chunks) {
  const int lane = threadIdx.x & (kWave - 1), l = lane & (lanes - 1);
  const int head = (static_cast<int>(blockIdx.y) * 4 + static_cast<int>(threadIdx.x >> 6)) * (kWave / lanes) + lane / lanes;
  if (head >= c.hq + 2 * c.hkv) return;
  const int taps = TAPS > 0 ? TAPS : c.taps, keep = taps - 1, half = c.d >> 1;
  constexpr int KEEP = TAPS > 0 ? TAPS - 1 : 0, HELD = TAPS > 0 ? TAPS : 1;
  const A* in = c.in + static_cast<int64_t>(head) * c.d;
  const float* w = c.w + static_cast<int64_t>(head) * c.d;
  int at[P];                                             // the lane's channels at[p], at[p] + half
  bool have[P];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    at[p] = min(l + p * lanes, half - 1);
    have[p] = l + p * lanes < half;
  }
  float wa[HELD][P], wb[HELD][P], na[P], nb[P];
#pragma unroll
  for (int j = 0; j < TAPS; ++j)
#pragma unroll
    for (int p = 0; p < P; ++p) {
      wa[j][p] = have[p] ? w[static_cast<int64_t>(j) * c.channels + at[p]] : 0.f;
      wb[j][p] = have[p] ? w[static_cast<int64_t>(j) * c.channels + at[p] + half] : 0.f;
    }
  load_norm<A, P>(c, head, l, lanes, na, nb);

  if (static_cast<int>(blockIdx.x) < chunks) {
    const int64_t t0 = static_cast<int64_t>(blockIdx.x) * kConvTokens, last = c.tokens - 1;
    TokenRest<P> rest[kConvTokens];
#pragma unroll
    for (int u = 0; u < kConvTokens; ++u) load_rest<A, P>(c, min(t0 + u, last), l, lanes, rest[u]);
    float xa[KEEP + kConvTokens][P], xb[KEEP + kConvTokens][P];
    if (TAPS > 0) {
#pragma unroll
      for (int r = 0; r < KEEP + kConvTokens; ++r)       // rows in front of the step's first are read as row 0, and not used
#pragma unroll
        for (int p = 0; p < P; ++p) {
          const A* x = in + min(max(t0 - KEEP + r, static_cast<int64_t>(0)), last) * c.in_row + at[p];
          xa[r][p] = to_float<A>(x[0]);
          xb[r][p] = to_float<A>(x[half]);
        }
    }
#pragma unroll
    for (int u = 0; u < kConvTokens; ++u) {
      const int64_t t = t0 + u;
      if (t > last) break;
      if (t - rest[u].first < keep) continue;
      float a[P], b[P];
#pragma unroll
      for (int p = 0; p < P; ++p) {
        a[p] = b[p] = 0.f;
        if (TAPS > 0) {
#pragma unroll
          for (int j = 0; j < TAPS; ++j) {
            a[p] = fmaf(wa[j][p], xa[u + j][p], a[p]);
            b[p] = fmaf(wb[j][p], xb[u + j][p], b[p]);
          }
        } else if (have[p]) {
          for (int j = 0; j < taps; ++j) {
            const A* x = in + (t - keep + j) * c.in_row + at[p];
            a[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + at[p]], to_float<A>(x[0]), a[p]);
            b[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + at[p] + half], to_float<A>(x[half]), b[p]);
          }
        }
      }
      finish_head<A, P>(c, t, head, l, lanes, a, b, na, nb, rest[u]);
    }
    return;
  }

  const int item = static_cast<int>(blockIdx.x) - chunks;
  const int64_t s0 = c.item_start[item];
  const int n = static_cast<int>(c.item_start[item + 1] - s0);
  if (n <= 0) return;
  float* saved = c.state + static_cast<int64_t>(c.slots[item]) * c.state_row + static_cast<int64_t>(head) * c.d;
  if (TAPS > 0) {
    TokenRest<P> rest[HELD];
    float xa[2 * HELD][P], xb[2 * HELD][P];              // the saved inputs, then the item's first ones
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
      const int64_t t = s0 + max(min(j, n - 1), 0);
      load_rest<A, P>(c, t, l, lanes, rest[j]);
#pragma unroll
      for (int p = 0; p < P; ++p) {
        xa[j][p] = saved[static_cast<int64_t>(j) * c.channels + at[p]];
        xb[j][p] = saved[static_cast<int64_t>(j) * c.channels + at[p] + half];
        xa[KEEP + j][p] = to_float<A>(in[t * c.in_row + at[p]]);
        xb[KEEP + j][p] = to_float<A>(in[t * c.in_row + at[p] + half]);
      }
    }
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
      if (u >= n) break;
      float a[P], b[P];
#pragma unroll
      for (int p = 0; p < P; ++p) {
        a[p] = b[p] = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
          a[p] = fmaf(wa[j][p], xa[u + j][p], a[p]);
          b[p] = fmaf(wb[j][p], xb[u + j][p], b[p]);
        }
      }
      finish_head<A, P>(c, s0 + u, head, l, lanes, a, b, na, nb, rest[u]);
    }
#pragma unroll
    for (int p = 0; p < P; ++p) {
      if (!have[p]) continue;
#pragma unroll
      for (int j = 0; j < KEEP; ++j) {
        // The item's input n - KEEP + j, which is a saved one where that is negative.
        float u = xa[j][p], v = xb[j][p];
#pragma unroll
        for (int m = 1; m < KEEP; ++m)
          if (n == m) u = xa[m + j][p], v = xb[m + j][p];
        if (n >= KEEP) {
          const A* x = in + (s0 + n - KEEP + j) * c.in_row + at[p];
          u = to_float<A>(x[0]);
          v = to_float<A>(x[half]);
        }
        saved[static_cast<int64_t>(j) * c.channels + at[p]] = u;
        saved[static_cast<int64_t>(j) * c.channels + at[p] + half] = v;
      }
    }
    return;
  }
  auto input = [&](int src, int i) {                     // the item's input src (negative: saved), channel i of the head
    return src >= 0 ? to_float<A>(in[(s0 + src) * c.in_row + i]) : saved[static_cast<int64_t>(keep + src) * c.channels + i];
  };
  for (int u = 0; u < min(n, keep); ++u) {
    TokenRest<P> rest;
    load_rest<A, P>(c, s0 + u, l, lanes, rest);
    float a[P], b[P];
#pragma unroll
    for (int p = 0; p < P; ++p) {
      a[p] = b[p] = 0.f;
      for (int j = 0; have[p] && j < taps; ++j) {
        a[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + at[p]], input(u - keep + j, at[p]), a[p]);
        b[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + at[p] + half], input(u - keep + j, at[p] + half), b[p]);
      }
    }
    finish_head<A, P>(c, s0 + u, head, l, lanes, a, b, na, nb, rest);
  }
  // Ascending j reads saved entries at or behind the one it writes; a channel is the same lane's as above.
#pragma unroll
  for (int p = 0; p < P; ++p)
    for (int j = 0; have[p] && j < keep; ++j) {
      float* to = saved + static_cast<int64_t>(j) * c.channels;
      const float u = input(n - keep + j, at[p]), v = input(n - keep + j, at[p] + half);
      to[at[p]] = u;
      to[at[p] + half] = v;
    }
}

template <typename A, int P>
static void launch_qkv_conv(hipStream_t s, const QkvConv<A>& c, dim3 grid, int lanes, int chunks) {
  static_assert(kConvFastTaps == 4, "the cases below");
  switch (c.taps) {
    case 1: qkv_conv_kernel<A, P, 1><<<grid, dim3(256), 0, s>>>(c, lanes, chunks); break;
    case 2: qkv_conv_kernel<A, P, 2><<<grid, dim3(256), 0, s>>>(c, lanes, chunks); break;
    case 3: qkv_conv_kernel<A, P, 3><<<grid, dim3(256), 0, s>>>(c, lanes, chunks); break;
    case 4: qkv_conv_kernel<A, P, 4><<<grid, dim3(256), 0, s>>>(c, lanes, chunks); break;
    default: qkv_conv_kernel<A, P, 0><<<grid, dim3(256), 0, s>>>(c, lanes, chunks); break;
  }
}

}  // namespace psamd

using namespace psamd;

template <typename A>
static int run_qkv_conv(hipStream_t s, const QkvConv<A>& c, int items) {
  int lanes = 1;
  while (lanes < kWave && lanes < c.d / 2) lanes *= 2;
  const int per_block = 4 * (kWave / lanes);
  const int keep = c.taps - 1;
  const int chunks = static_cast<int>(ceil_div(c.tokens, kConvTokens));
  const dim3 grid(static_cast<unsigned>(chunks + (keep > 0 ? items : 0)), static_cast<unsigned>(ceil_div(c.hq + 2 * c.hkv, per_block)));
  if (c.d > 2 * kWave) launch_qkv_conv<A, 2>(s, c, grid, lanes, chunks);
  else launch_qkv_conv<A, 1>(s, c, grid, lanes, chunks);
  return check_launch("psamd_qkv_conv_append");
}

extern "C" int psamd_qkv_conv_append(void* stream, const void* in, int act_dtype, int64_t in_row, const float* taps_w, int taps, int hq,
                                     int hkv, int d, const int32_t* positions, const float* table, int norm_dim, float eps,
                                     const float* q_weight, const float* k_weight, void* q_out, void* kv, const int32_t* write_slot,
                                     float* state, int64_t state_row, const int32_t* tok_item, const int32_t* item_start,
                                     const int32_t* slots, int64_t tokens, int items) {
  PSAMD_REQUIRE(tokens >= 0 && items >= 0 && hq > 0 && hkv > 0 && d > 0 && d % 2 == 0 && d <= 256, "bad sizes (head size even, at most 256)");
  PSAMD_REQUIRE(taps >= 1 && taps <= kConvMostTaps && norm_dim >= 0 && norm_dim <= d, "at most 16 taps");
  const int64_t channels = (static_cast<int64_t>(hq) + 2 * hkv) * d;
  PSAMD_REQUIRE(in_row >= channels && channels <= 2147483647LL, "rows too short");
  PSAMD_REQUIRE(taps == 1 || (state != nullptr && state_row >= (taps - 1) * channels), "the state's saved inputs");
  PSAMD_REQUIRE(kv == nullptr || write_slot != nullptr, "pages need the tokens' places");
  PSAMD_REQUIRE(tokens + items <= 2147483647LL, "too large for one launch");
  if (tokens == 0) return 0;
  hipStream_t s = static_cast<hipStream_t>(stream);
#define PSAMD_QKV_CONV(A_)                                                                                                        \
  run_qkv_conv<A_>(s, QkvConv<A_>{static_cast<const A_*>(in), in_row, taps_w, static_cast<int>(channels), taps, hq, hkv, d, positions, \
                                  reinterpret_cast<const float2*>(table), norm_dim, eps, q_weight, k_weight, static_cast<A_*>(q_out), \
                                  static_cast<A_*>(kv), write_slot, state, state_row, tok_item, item_start, slots,               \
                                  static_cast<int>(tokens)}, items)
  if (act_dtype == kBF16) return PSAMD_QKV_CONV(bf16_t);
  if (act_dtype == kF32) return PSAMD_QKV_CONV(float);
#undef PSAMD_QKV_CONV
  return fail("psamd_qkv_conv_append: activation dtype must be float32 or bfloat16");
}
