// Retention: linear attention with a fixed decay per head. Per head, with S [dim, vdim] in float,
//     S <- g S + k v^T,   o = S^T q,   out = o / rms(o) * silu(gate),
// q and k rotated and k times k_scale.
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
// A row of the step's input holds q, k, v and gate with heads padded to multiples of 16 (zeros), the rotation's partners
// dim_p / 2 apart (entries that do not rotate meet (1, 0) in the table), and the state of a head is stored
// [dim_p][vdim_p]: values are neighbours.

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
  const float2* table;                     // [pos][dim_p / 2] = (cos, sin)
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
  const float2 t = cs[c < half ? c : c - half];
  return c < half ? to_float<A>(x[c]) * t.x - to_float<A>(x[c + half]) * t.y : to_float<A>(x[c]) * t.x + to_float<A>(x[c - half]) * t.y;
}

// Four neighbouring elements as floats.
template <typename A> __device__ __forceinline__ float4 quad(const A* p);
template <> __device__ __forceinline__ float4 quad<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <> __device__ __forceinline__ float4 quad<bf16_t>(const bf16_t* p) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(raw.x << 16), __uint_as_float(raw.x & 0xFFFF0000u), __uint_as_float(raw.y << 16),
                     __uint_as_float(raw.y & 0xFFFF0000u));
}
// ... and as they lie in memory: a load that is converted later leaves the wait for it to the conversion.
template <typename A> struct RawQuad;
template <> struct RawQuad<float> {
  float4 raw;
  __device__ __forceinline__ float4 value() const { return raw; }
};
template <> struct RawQuad<bf16_t> {
  uint2 raw;
  __device__ __forceinline__ float4 value() const {
    return make_float4(__uint_as_float(raw.x << 16), __uint_as_float(raw.x & 0xFFFF0000u), __uint_as_float(raw.y << 16),
                       __uint_as_float(raw.y & 0xFFFF0000u));
  }
};
template <typename A> __device__ __forceinline__ RawQuad<A> raw_quad(const A* p) { return *reinterpret_cast<const RawQuad<A>*>(p); }
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
  const int half = c.dim_p >> 1;
  const float2* cs = c.table + static_cast<int64_t>(c.positions[t]) * half;
  if (static_cast<int>(threadIdx.x) < c.dim_p) {
    q_s[threadIdx.x] = turned<A>(row + c.q_col + static_cast<int64_t>(h) * c.dim_p, cs, threadIdx.x, half);
    k_s[threadIdx.x] = turned<A>(row + c.k_col + static_cast<int64_t>(h) * c.dim_p, cs, threadIdx.x, half) * c.k_scale;
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

// 32 tokens of one head's rotated vectors on their way into LDS rows of `LD` floats (DK columns, of which dim_p exist), in two
// steps, so that the next tile's loads are in flight while a tile is multiplied: no branch lies around the loads (addresses
// are clamped to the run's tokens), and what they bring is looked at when it is stored. A thread's piece is two groups of four
// neighbouring entries that rotate into each other. T: threads of the workgroup.
template <typename A, int DK, int LD, int T>
struct TurnedTile {
  static constexpr int PER_ROW = DK / 8;
  static constexpr int N = (kTile * PER_ROW + T - 1) / T;
  RawQuad<A> a[N], b[N];
  float4 c[N], d[N];                      // (cos, sin) of the first two pairs, of the last two

  // Tokens from the run's token r0 on; pos: the position of the run's first token.
  __device__ __forceinline__ void load(const RetentionCall& rc, const Run& run, int col, int r0, int pos) {
    const int half = rc.dim_p >> 1;
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, r = min(r0 + idx / PER_ROW, run.n - 1);
      const int u = min(4 * (idx % PER_ROW), half - 4);
      const A* x = static_cast<const A*>(rc.rows) + (run.t0 + r) * rc.row + col + u;
      const float4* cs = reinterpret_cast<const float4*>(rc.table + static_cast<int64_t>(pos + r) * half + u);
      a[p] = raw_quad<A>(x);
      b[p] = raw_quad<A>(x + half);
      c[p] = cs[0];
      d[p] = cs[1];
    }
  }

  // ... of which `count` exist, times scale; zeros behind them.
  __device__ __forceinline__ void store(const RetentionCall& rc, int count, float scale, float* dst) const {
    const int half = rc.dim_p >> 1;
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, r = idx / PER_ROW, u = 4 * (idx % PER_ROW);
      if (kTile * PER_ROW % T != 0 && r >= kTile) break;
      const bool in = u < half;
      const float f = r < count && in ? scale : 0.f;
      const float4 x = a[p].value(), y = b[p].value();
      // A head narrower than DK: the pieces past its halves fill the columns from dim_p on with zeros.
      float* lo = dst + r * LD + (in ? u : 2 * u);
      float* hi = dst + r * LD + (in ? u + half : 2 * u + 4);
      *reinterpret_cast<float4*>(lo) = make_float4(f * (x.x * c[p].x - y.x * c[p].y), f * (x.y * c[p].z - y.y * c[p].w),
                                                   f * (x.z * d[p].x - y.z * d[p].y), f * (x.w * d[p].z - y.w * d[p].w));
      *reinterpret_cast<float4*>(hi) = make_float4(f * (y.x * c[p].x + x.x * c[p].y), f * (y.y * c[p].z + x.y * c[p].w),
                                                   f * (y.z * d[p].x + x.z * d[p].y), f * (y.w * d[p].z + x.w * d[p].w));
    }
  }
};

// The same for 32 tokens' values, of whose VD columns `have` exist.
template <typename A, int VD, int LD, int T>
struct ValueTile {
  static constexpr int PER_ROW = VD / 4;
  static constexpr int N = (kTile * PER_ROW + T - 1) / T;
  RawQuad<A> v[N];

  __device__ __forceinline__ void load(const RetentionCall& rc, const Run& run, int col, int r0, int have) {
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, r = min(r0 + idx / PER_ROW, run.n - 1), i = min(4 * (idx % PER_ROW), have - 4);
      v[p] = raw_quad<A>(static_cast<const A*>(rc.rows) + (run.t0 + r) * rc.row + col + i);
    }
  }

  // The first n rows, row r times weight[-r] (weight is never read past its first entry: n entries lie in front of it); zeros
  // behind them.
  template <bool WEIGHTED>
  __device__ __forceinline__ void store(float* dst, const float* weight, int n, int have) const {
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, r = idx / PER_ROW, i = 4 * (idx % PER_ROW);
      if (kTile * PER_ROW % T != 0 && r >= kTile) break;
      float w = r < n && i < have ? 1.f : 0.f;
      if (WEIGHTED) w *= weight[-min(r, n - 1)];
      const float4 x = v[p].value();
      *reinterpret_cast<float4*>(dst + r * LD + i) = make_float4(w * x.x, w * x.y, w * x.z, w * x.w);
    }
  }
};

// The operands of step i + 1 are read from LDS in front of the matrix instructions of step i, and stay there.
template <int STEPS, typename Operands, typename Read, typename Multiply>
__device__ __forceinline__ void pipelined(Read read, Multiply multiply) {
  Operands op[2];
  read(0, op[0]);
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    if (i + 1 < STEPS) read(i + 1, op[(i + 1) & 1]);
    __builtin_amdgcn_sched_barrier(0);
    multiply(i, op[i & 1]);
  }
}

// grid (heads, runs, pieces of VD values): sums[run][head] = sum_j g^(n-1-j) k_j v_j^T. The 32 x 32 tiles of the result are
// dealt out to the workgroup's waves (eight where there are that many tiles: two waves a SIMD hide each other's waits); keys
// and values pass through LDS 32 tokens at a time.
constexpr int sums_threads(int dk, int vd) { return dk * vd >= 8 * 1024 ? 512 : 256; }
template <typename A, int DK, int VD>
__global__ __launch_bounds__(sums_threads(DK, VD)) void retention_sums_kernel(RetentionCall c, const int32_t* __restrict__ pf_tiles,
                                                                              const int32_t* __restrict__ pf_blocks,
                                                                              float* __restrict__ sums) {
  constexpr int NT = VD / 32, TILES = (DK / 32) * NT;
  constexpr int T = sums_threads(DK, VD);
  constexpr int TPW = (TILES + T / 64 - 1) / (T / 64);
  constexpr int LDK = DK + 4, LDV = VD + 4;
  __shared__ __align__(16) float kbuf[kTile * LDK];
  __shared__ __align__(16) float vbuf[kTile * LDV];
  __shared__ float pw[kPowers];
  const int h = blockIdx.x;
  const Run run = run_of(pf_tiles, pf_blocks, c.item_start, blockIdx.y);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 31, g = lane >> 5;
  const int v0 = VD * static_cast<int>(blockIdx.z), have = c.vdim_p - v0;
  const int pos = c.positions[run.t0], k_col = c.k_col + h * c.dim_p, v_col = c.v_col + h * c.vdim_p + v0;
  TurnedTile<A, DK, LDK, T> keys;
  ValueTile<A, VD, LDV, T> values;
  keys.load(c, run, k_col, 0, pos);
  values.load(c, run, v_col, 0, have);
  for (int i = threadIdx.x; i < kPowers; i += T) pw[i] = c.powers[h * kPowers + i];
  const float* kp[TPW];                                  // the wave's tiles' columns of the first key, for the lane
  const float* vp[TPW];
#pragma unroll
  for (int i = 0; i < TPW; ++i) {
    const int tile = min(wave * TPW + i, TILES - 1);
    kp[i] = kbuf + g * LDK + 32 * (tile / NT) + col;
    vp[i] = vbuf + g * LDV + 32 * (tile % NT) + col;
  }
  f32x16 acc[TPW];
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[i][v] = 0.f;
  for (int j0 = 0; j0 < run.n; j0 += kTile) {
    __syncthreads();
    keys.store(c, run.n - j0, c.k_scale, kbuf);
    values.template store<true>(vbuf, pw + (run.n - 1 - j0), run.n - j0, have);
    __syncthreads();
    keys.load(c, run, k_col, j0 + kTile, pos);           // the next 32, or the run's last token over and over
    values.load(c, run, v_col, j0 + kTile, have);
    struct Pair {
      float k[TPW][2], v[TPW][2];
    };
    pipelined<8, Pair>(                                  // four keys a step, two of them per lane
        [&](int i, Pair& p) {
#pragma unroll
          for (int t = 0; t < TPW; ++t)
#pragma unroll
            for (int e = 0; e < 2; ++e) {
              p.k[t][e] = kp[t][(4 * i + 2 * e) * LDK];
              p.v[t][e] = vp[t][(4 * i + 2 * e) * LDV];
            }
        },
        [&](int, const Pair& p) {
#pragma unroll
          for (int e = 0; e < 2; ++e)
#pragma unroll
            for (int t = 0; t < TPW; ++t) acc[t] = __builtin_amdgcn_mfma_f32_32x32x2f32(p.k[t][e], p.v[t][e], acc[t], 0, 0, 0);
        });
  }
  float* dst = sums + (static_cast<int64_t>(blockIdx.y) * c.heads + h) * (static_cast<int64_t>(c.dim_p) * c.vdim_p);
#pragma unroll
  for (int i = 0; i < TPW; ++i) {
    const int tile = wave * TPW + i, m = tile / NT, n = tile % NT;
    if (tile >= TILES) break;
    const int j = v0 + 32 * n + col;
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

// grid (heads, runs): the outputs of a run. Eight waves: waves w and 7 - w own the run's tokens 32 w .. 32 w + 31, the first the
// lower half of the head's values and the second the upper (both form the scores; a SIMD's two waves then have early tokens
// with few keys and late ones with many, and hide each other's waits). Up to 32 values, four waves with all of them. Scores
// are formed transposed, K Q^T (a lane's column is its query), so that the decayed scores go from the accumulator of
// the first product straight into the second as its B operand: register v of lane (col, g) is key
// 8 (v / 4) + 4 g + v % 4, and the value operand is read in the same order. The output is transposed too (a lane
// holds values of one query), so the norm over a head's values is a sum inside two lanes, and over two waves.
template <typename A, int DK, int VD>
__global__ __launch_bounds__(VD > 32 ? 512 : 256) void retention_out_kernel(RetentionCall c, const int32_t* __restrict__ pf_tiles,
                                                            const int32_t* __restrict__ pf_blocks, const float* __restrict__ before) {
  constexpr int T = VD > 32 ? 512 : 256, HALVES = T / 256;
  constexpr int NT = VD / 32 / HALVES;                   // the wave's tiles of 32 values
  constexpr int SC = VD < 64 ? VD : 64;                  // columns of the state in LDS at a time, of both halves together
  constexpr int SW = SC / HALVES;                        // ... of one
  constexpr int LDK = DK + 4, LDV = VD + 8, LDS = SC + 8;
  constexpr int KV = kTile * (LDK + LDV), QQ = 2 * kTile * LDK, ST = DK * LDS;
  constexpr int BUF = KV > QQ ? (KV > ST ? KV : ST) : (QQ > ST ? QQ : ST);
  __shared__ __align__(16) float buf[BUF];
  __shared__ float pw[kPowers];
  __shared__ float squares[HALVES][kRunTokens];
  float* kbuf = buf;
  float* vbuf = buf + kTile * LDK;
  const int h = blockIdx.x, block = static_cast<int>(gridDim.y - 1 - blockIdx.y);
  const Run run = run_of(pf_tiles, pf_blocks, c.item_start, block);
  const int half = threadIdx.x >> 8, lane = threadIdx.x & 63, col = lane & 31, g = lane >> 5;
  const int wave = half ? 7 - (threadIdx.x >> 6) : threadIdx.x >> 6;        // which 32 tokens
  const int n0 = half * NT;                              // the first of the wave's value tiles
  const int pos = c.positions[run.t0], q_col = c.q_col + h * c.dim_p, k_col = c.k_col + h * c.dim_p, v_col = c.v_col + h * c.vdim_p;
  for (int i = threadIdx.x; i < kPowers; i += T) pw[i] = c.powers[h * kPowers + i];

  // The wave's queries: lane (col, g) holds the entries 8 j + 4 g + s of query col, s = 0 .. 3. The tiles pass through LDS two
  // at a time.
  float q[DK / 2];
#pragma unroll
  for (int i = 0; i < DK / 2; ++i) q[i] = 0.f;
  auto pass_queries = [&](const TurnedTile<A, DK, LDK, T>& one, const TurnedTile<A, DK, LDK, T>& two, int w) {
    one.store(c, run.n - w * kTile, 1.f, buf);
    two.store(c, run.n - (w + 1) * kTile, 1.f, buf + kTile * LDK);
    __syncthreads();
    if ((wave & ~1) == w) {
#pragma unroll
      for (int j = 0; j < DK / 8; ++j) {
        const float4 x = *reinterpret_cast<const float4*>(buf + ((wave & 1) * kTile + col) * LDK + 8 * j + 4 * g);
        q[4 * j] = x.x, q[4 * j + 1] = x.y, q[4 * j + 2] = x.z, q[4 * j + 3] = x.w;
      }
    }
    __syncthreads();
  };
  {
    TurnedTile<A, DK, LDK, T> one, two;
    one.load(c, run, q_col, 0, pos);
    two.load(c, run, q_col, kTile, pos);
    if (run.n > 2 * kTile) {
      TurnedTile<A, DK, LDK, T> three, four;
      three.load(c, run, q_col, 2 * kTile, pos);
      four.load(c, run, q_col, 3 * kTile, pos);
      pass_queries(one, two, 0);
      pass_queries(three, four, 2);
    } else {
      pass_queries(one, two, 0);
    }
  }

  f32x16 acc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[n][v] = 0.f;

  // What the state in front of the run gives: S0^T q, SC values at a time (SW of every half); the next columns are on their
  // way meanwhile.
  const float* s0 = before + (static_cast<int64_t>(block) * c.heads + h) * (static_cast<int64_t>(c.dim_p) * c.vdim_p);
  constexpr int SN = DK * (SC / 4) / T;                  // pieces of four a thread carries
  float4 piece[SN];
  // Column 4 (idx % (SC / 4)) of the round that starts at column j0 of every half.
  auto column = [](int idx, int j0) {
    const int x = 4 * (idx % (SC / 4));
    return HALVES == 1 ? j0 + x : (x / SW) * (VD / 2) + j0 + x % SW;
  };
  auto ask = [&](int j0) {
#pragma unroll
    for (int p = 0; p < SN; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, d = min(idx / (SC / 4), c.dim_p - 1);
      piece[p] = *reinterpret_cast<const float4*>(s0 + static_cast<int64_t>(d) * c.vdim_p + min(column(idx, j0), c.vdim_p - 4));
    }
  };
  ask(0);
  TurnedTile<A, DK, LDK, T> keys;
  ValueTile<A, VD, LDV, T> values;
#pragma unroll
  for (int j0 = 0; j0 < VD / HALVES; j0 += SW) {
    if (j0 > 0) __syncthreads();
#pragma unroll
    for (int p = 0; p < SN; ++p) {
      const int idx = static_cast<int>(threadIdx.x) + T * p, d = idx / (SC / 4);
      const float f = d < c.dim_p && column(idx, j0) < c.vdim_p ? 1.f : 0.f;
      *reinterpret_cast<float4*>(buf + d * LDS + 4 * (idx % (SC / 4))) = make_float4(f * piece[p].x, f * piece[p].y, f * piece[p].z, f * piece[p].w);
    }
    __syncthreads();
    if (j0 + SW < VD / HALVES) {
      ask(j0 + SW);
    } else {
      keys.load(c, run, k_col, 0, pos);
      values.load(c, run, v_col, 0, c.vdim_p);
    }
    struct Four {
      float a[4][SW / 32];
    };
    const float* sb = buf + 4 * g * LDS + half * SW + col;
    pipelined<DK / 8, Four>(
        [&](int j, Four& f) {
#pragma unroll
          for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int n = 0; n < SW / 32; ++n) f.a[s][n] = sb[(8 * j + s) * LDS + 32 * n];
        },
        [&](int j, const Four& f) {
#pragma unroll
          for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int n = 0; n < SW / 32; ++n)
              acc[j0 / 32 + n] = __builtin_amdgcn_mfma_f32_32x32x2f32(f.a[s][n], q[4 * j + s], acc[j0 / 32 + n], 0, 0, 0);
        });
  }
  const int i = kTile * wave + col;                      // the lane's query inside the run
  {
    const float w = pw[i + 1];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[n][v] *= w;
  }
  // The gate's rows are wanted last and asked for now.
  const int64_t t = run.t0 + min(i, run.n - 1);
  const A* gate = static_cast<const A*>(c.rows) + t * c.row + c.g_col + static_cast<int64_t>(h) * c.vdim_p;
  RawQuad<A> z[NT][4];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v4 = 0; v4 < 4; ++v4) z[n][v4] = raw_quad<A>(gate + min(32 * (n0 + n) + 8 * v4 + 4 * g, c.vdim_p - 4));

  // The run's own tokens up to the query.
  for (int kt = 0; kt * kTile < run.n; ++kt) {
    __syncthreads();
    keys.store(c, run.n - kt * kTile, c.k_scale, kbuf);
    values.template store<false>(vbuf, nullptr, run.n - kt * kTile, c.vdim_p);
    __syncthreads();
    keys.load(c, run, k_col, (kt + 1) * kTile, pos);     // the next 32, or the run's last token over and over
    values.load(c, run, v_col, (kt + 1) * kTile, c.vdim_p);
    if (kt > wave) continue;
    f32x16 s;
#pragma unroll
    for (int v = 0; v < 16; ++v) s[v] = 0.f;
    const float* kr = kbuf + col * LDK + 4 * g;
    pipelined<DK / 8, float4>([&](int j, float4& a) { a = *reinterpret_cast<const float4*>(kr + 8 * j); },
                              [&](int j, const float4& a) {
                                s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.x, q[4 * j], s, 0, 0, 0);
                                s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.y, q[4 * j + 1], s, 0, 0, 0);
                                s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.z, q[4 * j + 2], s, 0, 0, 0);
                                s = __builtin_amdgcn_mfma_f32_32x32x2f32(a.w, q[4 * j + 3], s, 0, 0, 0);
                              });
    const int back0 = i - kt * kTile - 4 * g;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int back = back0 - 8 * (v >> 2) - (v & 3);
      s[v] = back >= 0 ? s[v] * pw[max(back, 0)] : 0.f;
    }
    struct Two {
      float a[2][NT];
    };
    const float* vr = vbuf + 4 * g * LDV + 32 * n0 + col;
    pipelined<8, Two>(
        [&](int e, Two& x) {
#pragma unroll
          for (int b = 0; b < 2; ++b) {
            const int v = 2 * e + b;
#pragma unroll
            for (int n = 0; n < NT; ++n) x.a[b][n] = vr[(8 * (v >> 2) + (v & 3)) * LDV + 32 * n];
          }
        },
        [&](int e, const Two& x) {
#pragma unroll
          for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int n = 0; n < NT; ++n) acc[n] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.a[b][n], s[2 * e + b], acc[n], 0, 0, 0);
        });
  }

  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v = 0; v < 16; ++v) ss = fmaf(acc[n][v], acc[n][v], ss);
  ss += __shfl_xor(ss, 32, kWave);
  if (HALVES > 1) {
    if (g == 0) squares[half][i] = ss;
    __syncthreads();
    ss = squares[0][i] + squares[HALVES - 1][i];
  }
  if (i >= run.n) return;
  const float inv = 1.f / sqrtf(ss / static_cast<float>(c.vdim) + c.eps);
  A* o = static_cast<A*>(c.out) + t * (static_cast<int64_t>(c.heads) * c.vdim_p) + static_cast<int64_t>(h) * c.vdim_p;
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int v4 = 0; v4 < 4; ++v4) {
      const int d = 32 * (n0 + n) + 8 * v4 + 4 * g;
      if (d >= c.vdim_p) continue;
      const float4 y = z[n][v4].value();
      put_quad<A>(o + d, make_float4(acc[n][4 * v4] * inv * silu(y.x), acc[n][4 * v4 + 1] * inv * silu(y.y),
                                     acc[n][4 * v4 + 2] * inv * silu(y.z), acc[n][4 * v4 + 3] * inv * silu(y.w)));
    }
}

template <typename A, int DK, int VD>
static int launch_portions(hipStream_t s, const RetentionCall& c, const int32_t* pf_tiles, const int32_t* pf_blocks, int n_blocks,
                           float* sums) {
  const dim3 grid(static_cast<unsigned>(c.heads), static_cast<unsigned>(n_blocks));
  constexpr int VS = VD < 128 ? VD : 128;
  const dim3 sums_grid(grid.x, grid.y, static_cast<unsigned>(ceil_div(c.vdim_p, VS)));
  retention_sums_kernel<A, DK, VS><<<sums_grid, dim3(sums_threads(DK, VS)), 0, s>>>(c, pf_tiles, pf_blocks, sums);
  if (check_launch("psamd_retention (sums)")) return 1;
  const unsigned pieces = static_cast<unsigned>(ceil_div(static_cast<int64_t>(c.dim_p) * c.vdim_p, 1024));
  retention_chain_kernel<<<dim3(pieces, grid.x, grid.y), dim3(256), 0, s>>>(c, pf_tiles, pf_blocks, sums);
  if (check_launch("psamd_retention (chain)")) return 1;
  retention_out_kernel<A, DK, VD><<<grid, dim3(VD > 32 ? 512 : 256), 0, s>>>(c, pf_tiles, pf_blocks, sums);
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
                    const int32_t* positions, const float* table, const float* powers, float k_scale, float* state,
                    int64_t state_row, const int32_t* item_start, const int32_t* slots, const int32_t* pf_tiles, int n_tiles,
                    int tile_tokens, const int32_t* pf_blocks, int n_blocks, const int32_t* dec_items, int n_dec, float* sums,
                    int heads, int dim_p, int vdim_p, int vdim, float eps, void* out) {
  PSAMD_REQUIRE(heads > 0 && heads <= 65535 && dim_p > 0 && dim_p <= 256 && dim_p % 16 == 0 && vdim_p > 0 && vdim_p <= 256 &&
                    vdim_p % 16 == 0 && vdim > 0 && vdim <= vdim_p, "head sizes are multiples of 16, at most 256");
  PSAMD_REQUIRE(table != nullptr && reinterpret_cast<uintptr_t>(table) % 16 == 0, "a rotation table, (1, 0) where nothing turns");
  PSAMD_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && g_col >= 0 &&
                    std::max(q_col, k_col) + static_cast<int64_t>(heads) * dim_p <= row &&
                    std::max(v_col, g_col) + static_cast<int64_t>(heads) * vdim_p <= row, "columns outside the rows");
  PSAMD_REQUIRE(row % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && v_col % 4 == 0 && g_col % 4 == 0 && reinterpret_cast<uintptr_t>(rows) % 16 == 0,
                "rows and columns start on multiples of four elements");
  PSAMD_REQUIRE(state_row % 4 == 0 && reinterpret_cast<uintptr_t>(state) % 16 == 0 &&
                    state_row >= static_cast<int64_t>(heads) * dim_p * vdim_p, "the state's rows");
  PSAMD_REQUIRE(tile_tokens == kTile && n_tiles >= 0 && n_blocks >= 0 && n_blocks <= n_tiles && 4LL * n_blocks >= n_tiles && n_blocks <= 65535,
                "the portions' runs of up to four tiles of 32 tokens");
  PSAMD_REQUIRE(n_dec >= 0, "bad sizes");
  PSAMD_REQUIRE(n_blocks == 0 || sums != nullptr, "portions need room for their runs' sums");
  const RetentionCall c{rows, row, q_col, k_col, v_col, g_col, positions, reinterpret_cast<const float2*>(table),
                        powers, k_scale, state, state_row, item_start, slots, heads, dim_p, vdim_p, vdim, eps, out};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (act_dtype == kBF16) return run_retention<bf16_t>(s, c, pf_tiles, pf_blocks, n_blocks, dec_items, n_dec, sums);
  if (act_dtype == kF32) return run_retention<float>(s, c, pf_tiles, pf_blocks, n_blocks, dec_items, n_dec, sums);
  return fail("psamd_retention: activation dtype must be float32 or bfloat16");
}

}  // extern "C"
