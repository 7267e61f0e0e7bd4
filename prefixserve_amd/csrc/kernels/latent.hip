// Latent attention's steps between its products and the attention itself: the token's compressed
// vector is normalized and, with the rotated key part all heads share, written to the token's place
// in the paged cache; where queries have a latent of their own it is normalized for the product that
// makes the heads' queries; every head's query is laid into the form the attention kernels read.
//
// The cache holds one "head" per token, `slots` wide: the key is [compressed (rank) | rotated
// part (rot) | zeros], the value (transposed in the page, as for every attention here) is
// [compressed | zeros]. A head's query is [its un-rotated part folded into the compressed
// space (rank) | its rotated part | zeros], so that query . key is the head's whole score and the
// weighted sum of values is the weighted sum of compressed vectors, which a product per head then
// unfolds.
//
// The rotation pairs neighbours, (2i, 2i + 1), or halves, (i, i + rot/2); statistics, rotation and
// norm are float.

#include "api.h"
#include "common.h"
#include "heads_tile.h"

namespace psamd {

// Entry i of the rotated part v (rot numbers) at an angle table cs [rot/2].
template <typename A>
__device__ __forceinline__ float turned(const A* __restrict__ v, const float2* __restrict__ cs, int i, int rot, int halves) {
  const int half = rot >> 1;
  const int p = halves ? (i < half ? i : i - half) : i >> 1;
  const bool second = halves ? i >= half : (i & 1) != 0;
  const float a = to_float<A>(v[halves ? p : 2 * p]), b = to_float<A>(v[halves ? p + half : 2 * p + 1]);
  const float2 c = cs[p];
  return second ? b * c.x + a * c.y : a * c.x - b * c.y;
}

// One workgroup per token. `low` row: [rank | rot]. c_in (or null): the queries' latent, normalized to
// c_out. q (or null): the heads' queries, whose rotated parts and trailing zeros are laid into q_lat.
template <typename A>
__global__ __launch_bounds__(256) void latent_kv_append_kernel(
    const A* __restrict__ low_rows, int64_t low_row, const A* __restrict__ c_in, int64_t c_row, int c_rank,
    const float* __restrict__ c_norm_w, A* __restrict__ c_out, const A* __restrict__ q_rows, int64_t q_row,
    A* __restrict__ q_lat, int hq, int dim, int rot, int rank, int slots, int halves, const int32_t* __restrict__ positions,
    const float2* __restrict__ table, const float* __restrict__ norm_w, float eps, A* __restrict__ kv,
    const int32_t* __restrict__ write_slot) {
  __shared__ float scratch[4], scratch_c[4];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  const A* low = low_rows + t * low_row;                            // [rank | rot]
  const int pos = positions[t];
  const float2* cs = table + static_cast<int64_t>(pos) * (rot >> 1);

  float ss = 0.f;
  for (int i = tid; i < rank; i += 256) {
    const float v = to_float<A>(low[i]);
    ss += v * v;
  }
  if (c_in != nullptr) {
    const A* c = c_in + t * c_row;
    float cc = 0.f;
    for (int i = tid; i < c_rank; i += 256) {
      const float v = to_float<A>(c[i]);
      cc += v * v;
    }
    cc = block_sum(cc, scratch_c, 4);
    const float cinv = rsqrtf(cc / static_cast<float>(c_rank) + eps);
    for (int i = tid; i < c_rank; i += 256)
      c_out[t * c_rank + i] = from_float<A>(to_float<A>(c[i]) * cinv * c_norm_w[i]);
  }
  ss = block_sum(ss, scratch, 4);
  const float inv = rsqrtf(ss / static_cast<float>(rank) + eps);

  if (kv != nullptr) {
    const int slot = write_slot[t];
    const int64_t page = slot / kPage;
    const int off = slot % kPage;
    A* kpage = kv + page * (2LL * kPage * slots) + static_cast<int64_t>(off) * slots;      // [16][slots]
    A* vpage = kv + page * (2LL * kPage * slots) + static_cast<int64_t>(kPage) * slots + off;   // [slots][16]
    for (int i = tid; i < slots; i += 256) {
      A key = from_float<A>(0.f), val = from_float<A>(0.f);
      if (i < rank) {
        key = val = from_float<A>(to_float<A>(low[i]) * inv * norm_w[i]);
      } else if (i < rank + rot) {
        key = from_float<A>(turned<A>(low + rank, cs, i - rank, rot, halves));
      }
      kpage[i] = key;
      vpage[static_cast<int64_t>(i) * kPage] = val;
    }
  }
  if (q_rows == nullptr) return;

  // Every head's rotated query part and the zeros behind it.
  const A* row = q_rows + t * q_row;
  const int tail = slots - rank;
  A* q_out = q_lat + t * (static_cast<int64_t>(hq) * slots);
  for (int e = tid; e < hq * tail; e += 256) {
    const int h = e / tail, i = e - h * tail;
    float val = 0.f;
    if (i < rot) val = turned<A>(row + static_cast<int64_t>(h) * (dim + rot) + dim, cs, i, rot, halves);
    q_out[static_cast<int64_t>(h) * slots + rank + i] = from_float<A>(val);
  }
}

// The tails alone (see above), for queries that exist only behind the append: tail entry e of token
// blockIdx.y * 256 + ... is a thread.
template <typename A>
__global__ __launch_bounds__(256) void latent_query_tail_kernel(const A* __restrict__ q_rows, int64_t q_row, A* __restrict__ q_lat,
                                                                int64_t tokens, int hq, int dim, int rot, int rank, int slots,
                                                                int halves, const int32_t* __restrict__ positions,
                                                                const float2* __restrict__ table) {
  const int tail = slots - rank;
  const int64_t per = static_cast<int64_t>(hq) * tail, n = tokens * per;
  for (int64_t x = blockIdx.x * 256LL + threadIdx.x; x < n; x += gridDim.x * 256LL) {
    const int64_t t = x / per;
    const int e = static_cast<int>(x - t * per), h = e / tail, i = e - h * tail;
    float val = 0.f;
    if (i < rot)
      val = turned<A>(q_rows + t * q_row + static_cast<int64_t>(h) * (dim + rot) + dim,
                      table + static_cast<int64_t>(positions[t]) * (rot >> 1), i, rot, halves);
    q_lat[(t * hq + h) * slots + rank + i] = from_float<A>(val);
  }
}

// Folding and tails in one kernel on the matrix cores: the grid's last column of workgroups lays the
// tails of its tokens of one head, the others fold (heads_tile.h).
template <int NT, int U, bool FEW>
__global__ __launch_bounds__(256) void latent_query_mfma_kernel(const bf16_t* __restrict__ q_rows, int64_t q_row,
                                                                const bf16_t* __restrict__ w, bf16_t* __restrict__ q_lat, int64_t M,
                                                                int hq, int dim, int rot, int rank, int slots, int halves,
                                                                const int32_t* __restrict__ positions,
                                                                const float2* __restrict__ table) {
  const int h = blockIdx.z;
  const bf16_t* q = q_rows + static_cast<int64_t>(h) * (dim + rot);
  bf16_t* out = q_lat + static_cast<int64_t>(h) * slots;
  const int64_t o_row = static_cast<int64_t>(hq) * slots;
  if (blockIdx.x == gridDim.x - 1) {
    const int tail = slots - rank;
    const int64_t t0 = static_cast<int64_t>(blockIdx.y) * 64;
    const int count = static_cast<int>(min(static_cast<int64_t>(64), M - t0)) * tail;
    for (int e = threadIdx.x; e < count; e += 256) {
      const int64_t t = t0 + e / tail;
      const int i = e % tail;
      float val = 0.f;
      if (i < rot) val = turned<bf16_t>(q + t * q_row + dim, table + static_cast<int64_t>(positions[t]) * (rot >> 1), i, rot, halves);
      out[t * o_row + rank + i] = float_to_bf16(val);
    }
    return;
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int r = lane & 15, g = lane >> 4;
  const HeadPlace<NT, FEW> place(wave);
  const int n0 = place.n0;
  if (place.m0 >= M || n0 >= rank) return;
  const bf16_t* wr[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) wr[nt] = w + (static_cast<int64_t>(h) * rank + min(n0 + nt * 16 + r, rank - 1)) * dim;
  head_f32x4 acc[NT];
  head_tile<NT, U>(q + min(place.m0 + r, M - 1) * q_row, wr, dim, g, acc);
  const int64_t m = place.m0 + r;
  if (m >= M) return;
  bf16_t* o = out + m * o_row;
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    const int n = n0 + nt * 16 + 4 * g;
    if (n + 3 < rank) {                               // slots is a multiple of 4: four results are one 8-byte store
      *reinterpret_cast<ushort4*>(o + n) = ushort4{float_to_bf16(acc[nt][0]), float_to_bf16(acc[nt][1]),
                                                   float_to_bf16(acc[nt][2]), float_to_bf16(acc[nt][3])};
    } else {
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (n + v < rank) o[n + v] = float_to_bf16(acc[nt][v]);
    }
  }
}

template <typename A>
static void launch_append(hipStream_t s, const void* low, int64_t low_row, const void* c_in, int64_t c_row, int c_rank,
                          const float* c_norm_w, void* c_out, const void* q, int64_t q_row, void* q_lat, int64_t tokens,
                          int hq, int dim, int rot, int rank, int slots, int halves, const int32_t* positions,
                          const float* table, const float* norm_w, float eps, void* kv, const int32_t* write_slot) {
  latent_kv_append_kernel<A><<<dim3(static_cast<unsigned>(tokens)), dim3(256), 0, s>>>(
      static_cast<const A*>(low), low_row, static_cast<const A*>(c_in), c_row, c_rank, c_norm_w, static_cast<A*>(c_out),
      static_cast<const A*>(q), q_row, static_cast<A*>(q_lat), hq, dim, rot, rank, slots, halves, positions,
      reinterpret_cast<const float2*>(table), norm_w, eps, static_cast<A*>(kv), write_slot);
}

template <typename A>
static void launch_tail(hipStream_t s, const void* q, int64_t q_row, void* q_lat, int64_t tokens, int hq, int dim, int rot,
                        int rank, int slots, int halves, const int32_t* positions, const float* table) {
  const int64_t n = tokens * hq * (slots - rank);
  const unsigned blocks = static_cast<unsigned>(ceil_div(n, 256) < 65536 ? ceil_div(n, 256) : 65536);
  latent_query_tail_kernel<A><<<dim3(blocks), dim3(256), 0, s>>>(
      static_cast<const A*>(q), q_row, static_cast<A*>(q_lat), tokens, hq, dim, rot, rank, slots, halves, positions,
      reinterpret_cast<const float2*>(table));
}

}  // namespace psamd

using namespace psamd;

extern "C" {

int psamd_latent_kv_append(void* stream, const void* low, int64_t low_row, const void* c_in, int64_t c_row, int c_rank,
                           const float* c_norm_w, void* c_out, const void* q, int64_t q_row, void* q_lat, int act_dtype,
                           int64_t tokens, int hq, int dim, int rot, int rank, int slots, int halves,
                           const int32_t* positions, const float* table, const float* norm_w, float eps, void* kv,
                           const int32_t* write_slot) {
  PSAMD_REQUIRE(tokens >= 0 && hq > 0 && dim >= 0 && rank > 0 && rot >= 0 && rot % 2 == 0, "bad sizes");
  PSAMD_REQUIRE(slots >= rank + rot, "a slot must hold the compressed vector and the rotated part");
  PSAMD_REQUIRE(low != nullptr && low_row >= static_cast<int64_t>(rank) + rot, "input rows too short");
  PSAMD_REQUIRE(q == nullptr || (q_lat != nullptr && q_row >= static_cast<int64_t>(hq) * (dim + rot)), "query rows too short");
  PSAMD_REQUIRE(c_in == nullptr || (c_norm_w != nullptr && c_out != nullptr && c_rank > 0 && c_row >= c_rank), "the queries' latent");
  PSAMD_REQUIRE(rot == 0 || table != nullptr, "a rotated part needs its table");
  PSAMD_REQUIRE(positions != nullptr && norm_w != nullptr, "positions and the norm's weight are needed");
  PSAMD_REQUIRE(kv == nullptr || write_slot != nullptr, "a cache needs write slots");
  PSAMD_REQUIRE(tokens <= 2147483647LL, "too large for one launch");
  PSAMD_REQUIRE(act_dtype == kBF16 || act_dtype == kF32, "activation dtype must be float32 or bfloat16");
  if (tokens == 0) return 0;
  auto launch = act_dtype == kBF16 ? launch_append<bf16_t> : launch_append<float>;
  launch(static_cast<hipStream_t>(stream), low, low_row, c_in, c_row, c_rank, c_norm_w, c_out, q, q_row, q_lat, tokens, hq, dim,
         rot, rank, slots, halves, positions, table, norm_w, eps, kv, write_slot);
  return check_launch("psamd_latent_kv_append");
}

int psamd_latent_query(void* stream, const void* q, int64_t q_row, const void* w_fold, void* q_lat, int act_dtype,
                       int64_t tokens, int hq, int dim, int rot, int rank, int slots, int halves, const int32_t* positions,
                       const float* table) {
  PSAMD_REQUIRE(tokens >= 0 && hq > 0 && dim >= 0 && rank > 0 && rot >= 0 && rot % 2 == 0, "bad sizes");
  PSAMD_REQUIRE(slots >= rank + rot && q_row >= static_cast<int64_t>(hq) * (dim + rot), "rows too short");
  PSAMD_REQUIRE((rot == 0 || table != nullptr) && positions != nullptr && (dim == 0 || w_fold != nullptr), "operands are missing");
  PSAMD_REQUIRE(act_dtype == kBF16 || act_dtype == kF32, "activation dtype must be float32 or bfloat16");
  PSAMD_REQUIRE(hq <= 65535 && ceil_div(tokens, 64) <= 65535, "too large for one launch");
  if (tokens == 0) return 0;
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (act_dtype == kBF16 && dim > 0 && dim % 8 == 0 && rot % 8 == 0 && q_row % 8 == 0 && slots % 4 == 0 &&
      reinterpret_cast<uintptr_t>(q) % 16 == 0 && reinterpret_cast<uintptr_t>(w_fold) % 16 == 0 &&
      reinterpret_cast<uintptr_t>(q_lat) % 8 == 0) {
    const dim3 grid(static_cast<unsigned>(ceil_div(rank, 64)) + 1, static_cast<unsigned>(ceil_div(tokens, 64)),
                    static_cast<unsigned>(hq));
    auto kernel = tokens <= 16 ? latent_query_mfma_kernel<1, 4, true> : latent_query_mfma_kernel<4, 4, false>;
    kernel<<<grid, dim3(256), 0, s>>>(
        static_cast<const bf16_t*>(q), q_row, static_cast<const bf16_t*>(w_fold), static_cast<bf16_t*>(q_lat), tokens, hq, dim, rot,
        rank, slots, halves, positions, reinterpret_cast<const float2*>(table));
    return check_launch("psamd_latent_query");
  }
  if (slots > rank) {
    auto tail = act_dtype == kBF16 ? launch_tail<bf16_t> : launch_tail<float>;
    tail(s, q, q_row, q_lat, tokens, hq, dim, rot, rank, slots, halves, positions, table);
    if (check_launch("psamd_latent_query (tails)")) return 1;
  }
  if (dim == 0) return 0;                             // nothing to fold: the caller has zeroed the front
  return psamd_heads_linear(stream, q, act_dtype, q_row, dim + rot, w_fold, act_dtype, q_lat, act_dtype,
                            static_cast<int64_t>(hq) * slots, slots, tokens, hq, rank, dim, nullptr, 0, 0);
}

}  // extern "C"
