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

// One token of one head by a group of `lanes` lanes; x(j, c) is tap j's input of the head's channel c.
template <typename A, typename Input>
__device__ __forceinline__ void conv_head(const QkvConv<A>& c, int64_t t, int head, int l, int lanes, Input x) {
  const int half = c.d >> 1;
  const float* w = c.w + static_cast<int64_t>(head) * c.d;
  float a[2], b[2], ss = 0.f;
#pragma unroll
  for (int p = 0; p < 2; ++p) {                          // lanes = 64 when d > 128: two pairs per lane
    const int i = l + p * lanes;
    a[p] = b[p] = 0.f;
    if (i < half) {
      for (int j = 0; j < c.taps; ++j) {
        a[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + i], x(j, i), a[p]);
        b[p] = fmaf(w[static_cast<int64_t>(j) * c.channels + i + half], x(j, i + half), b[p]);
      }
      ss = fmaf(a[p], a[p], fmaf(b[p], b[p], ss));
    }
  }
  int64_t page = 0;
  int off = 0;
  if (c.kv != nullptr) {
    const int slot = c.write_slot[t];
    page = slot / kPage;
    off = slot % kPage;
  }
  const int64_t page_elems = 2LL * c.hkv * kPage * c.d;
  if (head >= c.hq + c.hkv) {                            // a value head: as it is, transposed into its page
    if (c.kv == nullptr) return;
    A* vpage = c.kv + page * page_elems + (static_cast<int64_t>(c.hkv) + (head - c.hq - c.hkv)) * kPage * c.d + off;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int i = l + p * lanes;
      if (i >= half) continue;
      vpage[static_cast<int64_t>(i) * kPage] = from_float<A>(a[p]);
      vpage[static_cast<int64_t>(i + half) * kPage] = from_float<A>(b[p]);
    }
    return;
  }
  float inv = 1.f;
  if (c.norm_dim > 0) {
    for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, kWave);
    inv = 1.f / sqrtf(ss / static_cast<float>(c.norm_dim) + c.eps);
  }
  const float* nw = head < c.hq ? c.q_weight : c.k_weight;
  A* dst = head < c.hq ? c.q_out + t * (static_cast<int64_t>(c.hq) * c.d) + static_cast<int64_t>(head) * c.d
                       : (c.kv != nullptr ? c.kv + page * page_elems + (static_cast<int64_t>(head - c.hq) * kPage + off) * c.d : nullptr);
  if (dst == nullptr) return;
  const int pos = c.positions[t];
#pragma unroll
  for (int p = 0; p < 2; ++p) {
    const int i = l + p * lanes;
    if (i >= half) continue;
    float u = a[p] * inv, v = b[p] * inv;
    if (nw != nullptr) {
      u *= nw[i];
      v *= nw[i + half];
    }
    if (c.table != nullptr) {
      const float2 cs = c.table[static_cast<int64_t>(pos) * half + i];
      const float r = u * cs.x - v * cs.y;
      v = v * cs.x + u * cs.y;
      u = r;
    }
    dst[i] = from_float<A>(u);
    dst[i + half] = from_float<A>(v);
  }
}

// grid (ceil(tokens / kConvTokens) + items, heads / (4 * 64 / lanes)). A token that lies taps - 1 or more behind its
// item's first token needs only the step's own rows: the first kind of workgroup. The first taps - 1 tokens of an
// item read the inputs its slot saved, which are then replaced by the item's last ones: the second kind, where a
// channel belongs to one lane throughout, so that nobody reads a saved input another lane has replaced.
template <typename A>
__global__ __launch_bounds__(256) void qkv_conv_kernel(QkvConv<A> c, int lanes, int chunks) {
  const int lane = threadIdx.x & (kWave - 1), l = lane & (lanes - 1);
  const int head = (static_cast<int>(blockIdx.y) * 4 + static_cast<int>(threadIdx.x >> 6)) * (kWave / lanes) + lane / lanes;
  if (head >= c.hq + 2 * c.hkv) return;
  const int keep = c.taps - 1;
  const A* in = c.in + static_cast<int64_t>(head) * c.d;
  if (static_cast<int>(blockIdx.x) < chunks) {
#pragma unroll
    for (int u = 0; u < kConvTokens; ++u) {
      const int64_t t = static_cast<int64_t>(blockIdx.x) * kConvTokens + u;
      if (t >= c.tokens) break;
      if (t - c.item_start[c.tok_item[t]] < keep) continue;
      conv_head(c, t, head, l, lanes, [&](int j, int i) { return to_float<A>(in[(t - keep + j) * c.in_row + i]); });
    }
    return;
  }
  const int item = static_cast<int>(blockIdx.x) - chunks;
  const int64_t s0 = c.item_start[item];
  const int n = static_cast<int>(c.item_start[item + 1] - s0);
  float* saved = c.state + static_cast<int64_t>(c.slots[item]) * c.state_row + static_cast<int64_t>(head) * c.d;
  auto input = [&](int src, int i) {                     // the item's input src (negative: saved), channel i of the head
    return src >= 0 ? to_float<A>(in[(s0 + src) * c.in_row + i]) : saved[static_cast<int64_t>(keep + src) * c.channels + i];
  };
  for (int li = 0; li < min(n, keep); ++li)
    conv_head(c, s0 + li, head, l, lanes, [&](int j, int i) { return input(li - keep + j, i); });
  // Ascending j reads saved entries at or behind the one it writes; a channel is the same lane's as above.
  const int half = c.d >> 1;
  for (int i = l; i < half; i += lanes)
    for (int j = 0; j < keep; ++j) {
      float* to = saved + static_cast<int64_t>(j) * c.channels;
      const float u = input(n - keep + j, i), v = input(n - keep + j, i + half);
      to[i] = u;
      to[i + half] = v;
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
  qkv_conv_kernel<A><<<grid, dim3(256), 0, s>>>(c, lanes, chunks);
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
