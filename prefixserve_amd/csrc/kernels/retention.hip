// Retention: linear attention with a fixed decay per head. Per head, with S [dim, vdim] in float,
//     S <- g S + k v^T,   o = S^T q,   out = o / rms(o) * silu(gate),
// q and k rotated (pairs (i, i + rot/2) of the first `rot` dimensions) and k times k_scale.
//
// Single tokens: one workgroup per (item, head) rotates, decays, writes, reads, normalizes and gates in
// one pass over the head's state.
//
// Portions: the decay does not depend on the token, so a run of up to 128 tokens needs the state only where
// the run begins. With n tokens in the run, i and j counted inside it and S0 the state in front of it,
//     o_i = g^(i+1) S0^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j
//     S_n = g^n S0 + sum_j g^(n-1-j) k_j v_j^T
// Three launches: the sums of all runs (each on its own), a walk over an item's runs that leaves every run
// the state in front of it, and all runs' outputs side by side. The products run on the matrix cores in
// float (v_mfma_f32_32x32x2_f32): nothing of the recurrence is rounded below 32-bit. Powers of the decays
// come from a table [heads][kRunTokens + 1] made in double.
//
// A row of the step's input holds q, k, v and gate with heads padded to multiples of 16 (zeros), and the
// state of a head is stored [dim_p][vdim_p]: values are neighbours.

#include <algorithm>

#include "api.h"
#include "common.h"

namespace psamd {

typedef __attribute__((ext_vector_type(16))) float f32x16;

constexpr int kTile = 32;                  // tokens per wave: the step's tiles of queries
constexpr int kRunTokens = 128;            // tokens per run: up to four tiles of one item
constexpr int kPowers = kRunTokens + 1;

// What all kernels here take.
struct RetentionCall {
  const void* rows;
  int64_t row;                             // elements per token
  int q_col, k_col, v_col, g_col;
  const int32_t* positions;
  const float2* table;                     // [pos][rot / 2] = (cos, sin)
  int half;                                // rot / 2
  const float* powers;                     // [heads][kPowers]
  float k_scale;
  float* state;
  int64_t state_row;
  const int32_t* item_start;
  const int32_t* slots;
  int heads, dim_p, vdim_p, vdim;
  float eps;
  void* out;                               // [tokens][heads * vdim_p]
};

// Element c of a head's rotated vector (x: the head's first element, cs: the token's row of the table).
template <typename A>
__device__ __forceinline__ float turned(const A* __restrict__ x, const float2* __restrict__ cs, int c, int half) {
  const float a = to_float<A>(x[c]);
  if (c >= 2 * half) return a;
  if (c < half) {
    const float2 t = cs[c];
    return a * t.x - to_float<A>(x[c + half]) * t.y;
  }
  const float2 t = cs[c - half];
  return a * t.x + to_float<A>(x[c - half]) * t.y;
}

// Four neighbouring elements as floats.
template <typename A> __device__ __forceinline__ float4 quad(const A* p);
template <> __device__ __forceinline__ float4 quad<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <> __device__ __forceinline__ float4 quad<bf16_t>(const bf16_t* p) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(raw.x << 16), __uint_as_float(raw.x & 0xFFFF0000u), __uint_as_float(raw.y << 16),
                     __uint_as_float(raw.y & 0xFFFF0000u));
}
template <typename A> __device__ __forceinline__ void put_quad(A* p, float4 v);
template <> __device__ __forceinline__ void put_quad<float>(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
template <> __device__ __forceinline__ void put_quad<bf16_t>(bf16_t* p, float4 v) {
  *reinterpret_cast<ushort4*>(p) = ushort4{float_to_bf16(v.x), float_to_bf16(v.y), float_to_bf16(v.z), float_to_bf16(v.w)};
}

__device__ __forceinline__ float silu(float z) { return z / (1.f + expf(-z)); }

// ------------------------------------------------------------------ single tokens

// grid (single tokens, heads), 256 threads: a thread owns four neighbouring values of the state's rows
// d = group, group + groups, ...
template <typename A>
__global__ __launch_bounds__(256) void retention_step_kernel(RetentionCall c, const int32_t* __restrict__ dec_items) {
  __shared__ float q_s[256], k_s[256];
  __shared__ __align__(16) float part[256 * 4];
  __shared__ float scratch[4];
  const int item = dec_items[blockIdx.x], h = blockIdx.y;
  const int64_t t = c.item_start[item];
  const A* row = static_cast<const A*>(c.rows) + t * c.row;
  const int lanes = c.vdim_p >> 2, groups = 256 / lanes;
  const int l = threadIdx.x % lanes, grp = threadIdx.x / lanes;
  float* st = c.state + static_cast<int64_t>(c.slots[item]) * c.state_row + static_cast<int64_t>(h) * c.dim_p * c.vdim_p + 4 * l;
  const float2* cs = c.table != nullptr ? c.table + static_cast<int64_t>(c.positions[t]) * c.half : nullptr;
  if (static_cast<int>(threadIdx.x) < c.dim_p) {
    q_s[threadIdx.x] = turned<A>(row + c.q_col + static_cast<int64_t>(h) * c.dim_p, cs, threadIdx.x, c.half);
    k_s[threadIdx.x] = turned<A>(row + c.k_col + static_cast<int64_t>(h) * c.dim_p, cs, threadIdx.x, c.half) * c.k_scale;
  }
  const float decay = c.powers[h * kPowers + 1];
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  __syncthreads();
  if (grp < groups) {
    const float4 v = quad<A>(row + c.v_col + static_cast<int64_t>(h) * c.vdim_p + 4 * l);
    constexpr int U = 8;
    for (int d0 = grp; d0 < c.dim_p; d0 += U * groups) {
      float4 s[U];
#pragma unroll
      for (int u = 0; u < U; ++u)
        s[u] = *reinterpret_cast<const float4*>(st + static_cast<int64_t>(min(d0 + u * groups, c.dim_p - 1)) * c.vdim_p);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int d = d0 + u * groups;
        if (d >= c.dim_p) break;
        const float k = k_s[d], q = q_s[d];
        s[u] = make_float4(fmaf(k, v.x, decay * s[u].x), fmaf(k, v.y, decay * s[u].y), fmaf(k, v.z, decay * s[u].z),
                           fmaf(k, v.w, decay * s[u].w));
        *reinterpret_cast<float4*>(st + static_cast<int64_t>(d) * c.vdim_p) = s[u];
        o = make_float4(fmaf(q, s[u].x, o.x), fmaf(q, s[u].y, o.y), fmaf(q, s[u].z, o.z), fmaf(q, s[u].w, o.w));
      }
    }
    *reinterpret_cast<float4*>(part + grp * c.vdim_p + 4 * l) = o;
  }
  __syncthreads();
  const int i = threadIdx.x;
  float y = 0.f;
  if (i < c.vdim_p)
    for (int g = 0; g < groups; ++g) y += part[g * c.vdim_p + i];
  const float ss = block_sum(y * y, scratch, 4);
  if (i < c.vdim_p) {
    const float gate = to_float<A>(row[c.g_col + static_cast<int64_t>(h) * c.vdim_p + i]);
    static_cast<A*>(c.out)[t * (static_cast<int64_t>(c.heads) * c.vdim_p) + static_cast<int64_t>(h) * c.vdim_p + i] =
        from_float<A>(y * (1.f / sqrtf(ss / static_cast<float>(c.vdim) + c.eps)) * silu(gate));
  }
}

// ------------------------------------------------------------------ portions

// The run a workgroup works on.
struct Run {
  int item;
  int q0;                                  // its first token inside the item's portion
  int64_t t0;                              // ... and in the step
  int n;                                   // its tokens
  int rest;                                // the portion's tokens from q0 on
};
__device__ __forceinline__ Run run_of(const int32_t* __restrict__ pf_tiles, const int32_t* __restrict__ pf_blocks,
                                      const int32_t* __restrict__ item_start, int block) {
  const int tile = pf_blocks[block];
  Run r;
  r.item = pf_tiles[2 * tile];
  r.q0 = pf_tiles[2 * tile + 1];
  r.t0 = item_start[r.item] + r.q0;
  r.rest = static_cast<int>(item_start[r.item + 1] - r.t0);
  r.n = min(r.rest, kRunTokens);
  return r;
}

// 32 tokens from token t0 on (count of them real, the others zero) of one head's rotated vectors, times
// `scale`, into LDS rows of `ld` floats; DK columns, of which dim_p exist.
template <typename A, int DK>
__device__ __forceinline__ void stage_turned(const RetentionCall& c, int col, int64_t t0, int count, float scale, float* dst, int ld) {
#pragma unroll 4
  for (int idx = threadIdx.x; idx < kTile * DK; idx += 256) {
    const int r = idx / DK, i = idx % DK;
    float v = 0.f;
    if (r < count && i < c.dim_p) {
      const int64_t t = t0 + r;
      const float2* cs = c.table != nullptr ? c.table + static_cast<int64_t>(c.positions[t]) * c.half : nullptr;
      v = scale * turned<A>(static_cast<const A*>(c.rows) + t * c.row + col, cs, i, c.half);
    }
    dst[r * ld + i] = v;
  }
}

// The same for values (four columns a thread), times weight[r] if given.
template <typename A, int VD>
__device__ __forceinline__ void stage_values(const RetentionCall& c, int col, int64_t t0, int count, const float* weight, int step,
                                             float* dst, int ld) {
#pragma unroll 2
  for (int idx = threadIdx.x; idx < kTile * VD / 4; idx += 256) {
    const int r = idx / (VD / 4), i = 4 * (idx % (VD / 4));
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (r < count && i < c.vdim_p) {
      v = quad<A>(static_cast<const A*>(c.rows) + (t0 + r) * c.row + col + i);
      if (weight != nullptr) {
        const float w = weight[step * r];
        v = make_float4(w * v.x, w * v.y, w * v.z, w * v.w);
      }
    }
    *reinterpret_cast<float4*>(dst + r * ld + i) = v;
  }
}

// grid (heads, runs): sums[run][head] = sum_j g^(n-1-j) k_j v_j^T. The 32 x 32 tiles of the result are dealt out to
// the four waves; keys and values pass through LDS 32 tokens at a time.
template <typename A, int DK, int VD>
__global__ __launch_bounds__(256) void retention_sums_kernel(RetentionCall c, const int32_t* __restrict__ pf_tiles,
                                                             const int32_t* __restrict__ pf_blocks, float* __restrict__ sums) {
  constexpr int MT = DK / 32, NT = VD / 32, TILES = MT * NT;
  constexpr int TPW = (TILES + 3) / 4;
  constexpr int LDK = DK + 4, LDV = VD + 4;
  __shared__ __align__(16) float kbuf[kTile * LDK];
  __shared__ __align__(16) float vbuf[kTile * LDV];
  const int h = blockIdx.x;
  const Run run = run_of(pf_tiles, pf_blocks, c.item_start, blockIdx.y);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 31, g = lane >> 5;
  const float* pw = c.powers + h * kPowers;
  f32x16 acc[TPW];
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[i][v] = 0.f;
  for (int j0 = 0; j0 < run.n; j0 += kTile) {
    const int count = min(kTile, run.n - j0);
    __syncthreads();
    stage_turned<A, DK>(c, c.k_col + h * c.dim_p, run.t0 + j0, count, c.k_scale, kbuf, LDK);
    stage_values<A, VD>(c, c.v_col + h * c.vdim_p, run.t0 + j0, count, pw + (run.n - 1 - j0), -1, vbuf, LDV);
    __syncthreads();
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int key = 2 * v + g;
#pragma unroll
      for (int i = 0; i < TPW; ++i) {
        const int tile = min(wave * TPW + i, TILES - 1), m = tile / NT, n = tile % NT;
        acc[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(kbuf[key * LDK + 32 * m + col], vbuf[key * LDV + 32 * n + col], acc[i], 0, 0, 0);
      }
    }
  }
  float* dst = sums + (static_cast<int64_t>(blockIdx.y) * c.heads + h) * (static_cast<int64_t>(c.dim_p) * c.vdim_p);
#pragma unroll
  for (int i = 0; i < TPW; ++i) {
    const int tile = wave * TPW + i, m = tile / NT, n = tile % NT;
    if (tile >= TILES) break;
    const int j = 32 * n + col;
    if (j >= c.vdim_p) continue;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int d = 32 * m + 8 * (v >> 2) + 4 * g + (v & 3);
      if (d < c.dim_p) dst[static_cast<int64_t>(d) * c.vdim_p + j] = acc[i][v];
    }
  }
}

// grid (pieces of 256 x 4 state entries, heads, runs): the workgroups of a portion's first run walk all of its runs:
// sums[run] is replaced by the state in front of the run, the state behind the last one goes to the slot.
__global__ __launch_bounds__(256) void retention_chain_kernel(RetentionCall c, const int32_t* __restrict__ pf_tiles,
                                                              const int32_t* __restrict__ pf_blocks, float* __restrict__ sums) {
  const Run run = run_of(pf_tiles, pf_blocks, c.item_start, blockIdx.z);
  if (run.q0 != 0) return;
  const int h = blockIdx.y;
  const int64_t size = static_cast<int64_t>(c.dim_p) * c.vdim_p;
  const int64_t e = 4 * (blockIdx.x * 256LL + threadIdx.x);
  if (e >= size) return;
  float4* st = reinterpret_cast<float4*>(c.state + static_cast<int64_t>(c.slots[run.item]) * c.state_row + h * size + e);
  float* first = sums + (static_cast<int64_t>(blockIdx.z) * c.heads + h) * size + e;
  const int64_t stride = c.heads * size;
  const float* pw = c.powers + h * kPowers;
  float4 s = *st;
  const int runs = (run.rest + kRunTokens - 1) / kRunTokens;
  constexpr int U = 4;
  for (int b0 = 0; b0 < runs; b0 += U) {
    float4 add[U];
#pragma unroll
    for (int u = 0; u < U; ++u) add[u] = *reinterpret_cast<const float4*>(first + min(b0 + u, runs - 1) * stride);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (b0 + u >= runs) break;
      const float w = pw[min(run.rest - (b0 + u) * kRunTokens, kRunTokens)];
      *reinterpret_cast<float4*>(first + (b0 + u) * stride) = s;
      s = make_float4(fmaf(w, s.x, add[u].x), fmaf(w, s.y, add[u].y), fmaf(w, s.z, add[u].z), fmaf(w, s.w, add[u].w));
    }
  }
  *st = s;
}

// grid (heads, runs): the outputs of a run. Wave w owns the run's tokens 32 w .. 32 w + 31 and all of the head's values. Scores
// are formed transposed, K Q^T (a lane's column is its query), so that the decayed scores go from the accumulator of
// the first product straight into the second as its B operand: register v of lane (col, g) is key
// 8 (v / 4) + 4 g + v % 4, and the value operand is read in the same order. The output is transposed too (a lane
// holds values of one query), so the norm over a head's values is a sum inside two lanes.
template <typename A, int DK, int VD>
__global__ __launch_bounds__(256) void retention_out_kernel(RetentionCall c, const int32_t* __restrict__ pf_tiles,
                                                            const int32_t* __restrict__ pf_blocks, const float* __restrict__ before) {
  constexpr int NT = VD / 32;
  constexpr int LDK = DK + 4, LDV = VD + 8, LDS = 40;
  constexpr int BUF = kTile * (LDK + LDV) > DK * LDS ? kTile * (LDK + LDV) : DK * LDS;
  __shared__ __align__(16) float buf[BUF];
  __shared__ float pw[kPowers];
  float* kbuf = buf;
  float* vbuf = buf + kTile * LDK;
  const int h = blockIdx.x;
  const Run run = run_of(pf_tiles, pf_blocks, c.item_start, gridDim.y - 1 - blockIdx.y);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 31, g = lane >> 5;
  for (int i = threadIdx.x; i < kPowers; i += 256) pw[i] = c.powers[h * kPowers + i];

  // The wave's queries: lane (col, g) holds the entries 8 j + 4 g + s of query col, s = 0 .. 3.
  float q[DK / 2];
#pragma unroll
  for (int i = 0; i < DK / 2; ++i) q[i] = 0.f;
  for (int w = 0; w * kTile < run.n; ++w) {
    __syncthreads();
    stage_turned<A, DK>(c, c.q_col + h * c.dim_p, run.t0 + w * kTile, min(kTile, run.n - w * kTile), 1.f, kbuf, LDK);
    __syncthreads();
    if (w == wave) {
#pragma unroll
      for (int j = 0; j < DK / 8; ++j) {
        const float4 x = *reinterpret_cast<const float4*>(kbuf + col * LDK + 8 * j + 4 * g);
        q[4 * j] = x.x, q[4 * j + 1] = x.y, q[4 * j + 2] = x.z, q[4 * j + 3] = x.w;
      }
    }
  }

  f32x16 acc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[n][v] = 0.f;

  // What the state in front of the run gives: S0^T q, 32 values at a time.
  const float* s0 = before + (static_cast<int64_t>(gridDim.y - 1 - blockIdx.y) * c.heads + h) * (static_cast<int64_t>(c.dim_p) * c.vdim_p);
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    if (32 * n >= c.vdim_p) break;
    __syncthreads();
    for (int idx = threadIdx.x; idx < DK * 8; idx += 256) {
      const int d = idx >> 3, i = 4 * (idx & 7);
      float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
      if (d < c.dim_p && 32 * n + i < c.vdim_p) x = *reinterpret_cast<const float4*>(s0 + static_cast<int64_t>(d) * c.vdim_p + 32 * n + i);
      *reinterpret_cast<float4*>(buf + d * LDS + i) = x;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < DK / 8; ++j)
#pragma unroll
      for (int s = 0; s < 4; ++s)
        acc[n] = __builtin_amdgcn_mfma_f32_32x32x2f32(buf[(8 * j + 4 * g + s) * LDS + col], q[4 * j + s], acc[n], 0, 0, 0);
  }
  const int i = kTile * wave + col;                      // the lane's query inside the run
  {
    const float w = pw[i + 1];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[n][v] *= w;
  }

  // The run's own tokens up to the query.
  for (int kt = 0; kt * kTile < run.n; ++kt) {
    const int count = min(kTile, run.n - kt * kTile);
    __syncthreads();
    stage_turned<A, DK>(c, c.k_col + h * c.dim_p, run.t0 + kt * kTile, count, c.k_scale, kbuf, LDK);
    stage_values<A, VD>(c, c.v_col + h * c.vdim_p, run.t0 + kt * kTile, count, nullptr, 0, vbuf, LDV);
    __syncthreads();
    if (kt > wave) continue;
    f32x16 s;
#pragma unroll
    for (int v = 0; v < 16; ++v) s[v] = 0.f;
#pragma unroll
    for (int j = 0; j < DK / 8; ++j) {
      const float4 a = *reinterpret_cast<const float4*>(kbuf + col * LDK + 8 * j + 4 * g);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, q[4 * j], s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, q[4 * j + 1], s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, q[4 * j + 2], s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, q[4 * j + 3], s, 0, 0, 0);
    }
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int back = i - (kt * kTile + 8 * (v >> 2) + 4 * g + (v & 3));
      s[v] = back >= 0 ? s[v] * pw[max(back, 0)] : 0.f;
    }
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int v = 0; v < 16; ++v)
        acc[n] = __builtin_amdgcn_mfma_f32_32x32x2f32(vbuf[(8 * (v >> 2) + 4 * g + (v & 3)) * LDV + 32 * n + col], s[v], acc[n], 0, 0, 0);
  }

  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v = 0; v < 16; ++v) ss = fmaf(acc[n][v], acc[n][v], ss);
  ss += __shfl_xor(ss, 32, kWave);
  if (i >= run.n) return;
  const float inv = 1.f / sqrtf(ss / static_cast<float>(c.vdim) + c.eps);
  const A* gate = static_cast<const A*>(c.rows) + (run.t0 + i) * c.row + c.g_col + static_cast<int64_t>(h) * c.vdim_p;
  A* o = static_cast<A*>(c.out) + (run.t0 + i) * (static_cast<int64_t>(c.heads) * c.vdim_p) + static_cast<int64_t>(h) * c.vdim_p;
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v4 = 0; v4 < 4; ++v4) {
      const int d = 32 * n + 8 * v4 + 4 * g;
      if (d >= c.vdim_p) continue;
      const float4 z = quad<A>(gate + d);
      put_quad<A>(o + d, make_float4(acc[n][4 * v4] * inv * silu(z.x), acc[n][4 * v4 + 1] * inv * silu(z.y),
                                     acc[n][4 * v4 + 2] * inv * silu(z.z), acc[n][4 * v4 + 3] * inv * silu(z.w)));
    }
}

template <typename A, int DK, int VD>
static int launch_portions(hipStream_t s, const RetentionCall& c, const int32_t* pf_tiles, const int32_t* pf_blocks, int n_blocks,
                           float* sums) {
  const dim3 grid(static_cast<unsigned>(c.heads), static_cast<unsigned>(n_blocks));
  retention_sums_kernel<A, DK, VD><<<grid, dim3(256), 0, s>>>(c, pf_tiles, pf_blocks, sums);
  if (check_launch("psamd_retention (sums)")) return 1;
  const unsigned pieces = static_cast<unsigned>(ceil_div(static_cast<int64_t>(c.dim_p) * c.vdim_p, 1024));
  retention_chain_kernel<<<dim3(pieces, grid.x, grid.y), dim3(256), 0, s>>>(c, pf_tiles, pf_blocks, sums);
  if (check_launch("psamd_retention (chain)")) return 1;
  retention_out_kernel<A, DK, VD><<<grid, dim3(256), 0, s>>>(c, pf_tiles, pf_blocks, sums);
  return check_launch("psamd_retention (out)");
}

template <typename A, int DK>
static int by_value_size(hipStream_t s, const RetentionCall& c, const int32_t* pf_tiles, const int32_t* pf_blocks, int n_blocks,
                         float* sums) {
  if (c.vdim_p <= 32) return launch_portions<A, DK, 32>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  if (c.vdim_p <= 64) return launch_portions<A, DK, 64>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  if (c.vdim_p <= 128) return launch_portions<A, DK, 128>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  return launch_portions<A, DK, 256>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
}

template <typename A>
static int run_retention(hipStream_t s, const RetentionCall& c, const int32_t* pf_tiles, const int32_t* pf_blocks, int n_blocks,
                         const int32_t* dec_items, int n_dec, float* sums) {
  if (n_dec > 0) {
    retention_step_kernel<A><<<dim3(static_cast<unsigned>(n_dec), static_cast<unsigned>(c.heads)), dim3(256), 0, s>>>(c, dec_items);
    if (check_launch("psamd_retention (step)")) return 1;
  }
  if (n_blocks == 0) return 0;
  if (c.dim_p <= 32) return by_value_size<A, 32>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  if (c.dim_p <= 64) return by_value_size<A, 64>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  if (c.dim_p <= 128) return by_value_size<A, 128>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
  return by_value_size<A, 256>(s, c, pf_tiles, pf_blocks, n_blocks, sums);
}

}  // namespace psamd

using namespace psamd;

extern "C" {

int psamd_retention_powers(void) { return kPowers; }

int psamd_retention(void* stream, const void* rows, int act_dtype, int64_t row, int q_col, int k_col, int v_col, int g_col,
                    const int32_t* positions, const float* table, int rot, const float* powers, float k_scale, float* state,
                    int64_t state_row, const int32_t* item_start, const int32_t* slots, const int32_t* pf_tiles, int n_tiles,
                    int tile_tokens, const int32_t* pf_blocks, int n_blocks, const int32_t* dec_items, int n_dec, float* sums,
                    int heads, int dim_p, int vdim_p, int vdim, float eps, void* out) {
  PSAMD_REQUIRE(heads > 0 && heads <= 65535 && dim_p > 0 && dim_p <= 256 && dim_p % 16 == 0 && vdim_p > 0 && vdim_p <= 256 &&
                    vdim_p % 16 == 0 && vdim > 0 && vdim <= vdim_p, "head sizes are multiples of 16, at most 256");
  PSAMD_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= dim_p && (rot == 0 || table != nullptr), "bad rotation");
  PSAMD_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && g_col >= 0 &&
                    std::max(q_col, k_col) + static_cast<int64_t>(heads) * dim_p <= row &&
                    std::max(v_col, g_col) + static_cast<int64_t>(heads) * vdim_p <= row, "columns outside the rows");
  PSAMD_REQUIRE(row % 4 == 0 && v_col % 4 == 0 && g_col % 4 == 0 && reinterpret_cast<uintptr_t>(rows) % 16 == 0,
                "rows, values and gates start on multiples of four elements");
  PSAMD_REQUIRE(state_row % 4 == 0 && reinterpret_cast<uintptr_t>(state) % 16 == 0 &&
                    state_row >= static_cast<int64_t>(heads) * dim_p * vdim_p, "the state's rows");
  PSAMD_REQUIRE(tile_tokens == kTile && n_tiles >= 0 && n_blocks >= 0 && n_blocks <= n_tiles && 4LL * n_blocks >= n_tiles && n_blocks <= 65535,
                "the portions' runs of up to four tiles of 32 tokens");
  PSAMD_REQUIRE(n_dec >= 0, "bad sizes");
  PSAMD_REQUIRE(n_blocks == 0 || sums != nullptr, "portions need room for their runs' sums");
  const RetentionCall c{rows, row, q_col, k_col, v_col, g_col, positions, rot > 0 ? reinterpret_cast<const float2*>(table) : nullptr,
                        rot / 2, powers, k_scale, state, state_row, item_start, slots, heads, dim_p, vdim_p, vdim, eps, out};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (act_dtype == kBF16) return run_retention<bf16_t>(s, c, pf_tiles, pf_blocks, n_blocks, dec_items, n_dec, sums);
  if (act_dtype == kF32) return run_retention<float>(s, c, pf_tiles, pf_blocks, n_blocks, dec_items, n_dec, sums);
  return fail("psamd_retention: activation dtype must be float32 or bfloat16");
}

}  // extern "C"
