// experts.hip — feed-forward experts: the router, (token, expert) pairs sorted
// by expert, and the experts' products over them.
//
// A pair's inner row is act(weight * up[e] h): the weight scales the expert's
// input, and since the product is linear it is applied to the 32-bit sums.
// Pairs are sorted by expert (stable, so results do not depend on timing) and
// cut into tiles of one expert each; the product kernels take one tile and a
// block of output channels per workgroup:
//   expert_tiles   128 pairs and 256 channels through LDS, for many pairs
//   expert_rows    up to 64 pairs, weights straight into registers, for few:
//                  there the weights' bytes are what counts
//   expert_plain   any size, bf16 or float
#include "elem.h"

#include <type_traits>

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(16))) float f32x16;

// ---- router ----------------------------------------------------------------
// The `top` largest of z[0, E) by one wave: experts and sigmoids of their
// scores, largest first, the lower expert on ties. An expert's place is the
// number of experts ahead of it.
__device__ void take_top(const float* z, int E, int top, int32_t* ids,
                         float* wt) {
  for (int e = threadIdx.x % WAVE; e < E; e += WAVE) {
    const float mine = z[e];
    int place = 0;
#pragma unroll 8
    for (int i = 0; i < E; ++i)
      place += z[i] > mine || (z[i] == mine && i < e);
    if (place < top) {
      ids[place] = e;
      wt[place] = sigmoid_f(mine);
    }
  }
}

// any size; one workgroup per row
template <typename T>
__global__ __launch_bounds__(256) void route_plain_kernel(
    const T* __restrict__ h, const T* __restrict__ w, int32_t* __restrict__ ids,
    float* __restrict__ wt, int K, int E, int top) {
  extern __shared__ float z[];
  const int64_t row = blockIdx.x;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  for (int e = wave; e < E; e += 4) {
    float s = 0.f;
    for (int k = lane; k < K; k += WAVE)
      s += ld(h + row * K + k) * ld(w + (int64_t)e * K + k);
    s = wave_reduce_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (wave == 0) take_top(z, E, top, ids + row * top, wt + row * top);
}

// 16 rows per workgroup, K split among NW waves; ET: 16-expert tiles
template <int ET, int NW>
__global__ __launch_bounds__(NW * WAVE) void route_kernel(
    const short* __restrict__ h, const short* __restrict__ w,
    int32_t* __restrict__ ids, float* __restrict__ wt, int64_t rows, int K,
    int E, int top) {
  extern __shared__ float lds[];       // [NW][16 rows][16 ET]
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane % 16, grp = lane / 16;
  const int64_t row0 = (int64_t)blockIdx.x * 16;
  const int64_t row = row0 + col < rows ? row0 + col : rows - 1;
  const short8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  float4v acc[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = (float4v){0.f, 0.f, 0.f, 0.f};
  // past the end of K the row counts as zero; experts past E are not looked at
  const short* wr[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t)
    wr[t] = w + (int64_t)min(t * 16 + col, E - 1) * K;
  constexpr int AHEAD = ET <= 2 ? 4 : 2;     // steps whose loads go together
  for (int k0 = wave * 64; k0 < K; k0 += AHEAD * NW * 64) {
    short8 a[AHEAD][2], b[AHEAD][2][ET];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int k = k0 + u * NW * 64 + grp * 16 + s * 8, kc = min(k, K - 8);
        a[u][s] = *(const short8*)(h + row * K + kc);
        if (k >= K) a[u][s] = zero;
#pragma unroll
        for (int t = 0; t < ET; ++t)
          b[u][s][t] = *(const short8*)(wr[t] + kc);
      }
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int t = 0; t < ET; ++t)
          acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              __builtin_bit_cast(bf16x8, b[u][s][t]),
              __builtin_bit_cast(bf16x8, a[u][s]), acc[t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < ET; ++t)
    *(float4v*)(lds + (wave * 16 + col) * 16 * ET + t * 16 + grp * 4) = acc[t];
  __syncthreads();
  for (int i = threadIdx.x; i < 256 * ET; i += NW * WAVE) {
    float s = lds[i];
#pragma unroll
    for (int v = 1; v < NW; ++v) s += lds[v * 256 * ET + i];
    lds[i] = s;
  }
  __syncthreads();
  for (int r = wave; r < 16 && row0 + r < rows; r += NW)
    take_top(lds + r * 16 * ET, E, top, ids + (row0 + r) * top,
             wt + (row0 + r) * top);
}

// ---- sorting ---------------------------------------------------------------
constexpr int ST = 1024, SV = 8;   // threads; pairs per thread and sweep

// SV experts from place i on; -1 past the end (i is a multiple of SV)
__device__ __forceinline__ void load_ids(const int32_t* ids, int i, int P,
                                         int* x) {
  if (i + SV <= P) {
    const int4 a = *(const int4*)(ids + i), b = *(const int4*)(ids + i + 4);
    x[0] = a.x; x[1] = a.y; x[2] = a.z; x[3] = a.w;
    x[4] = b.x; x[5] = b.y; x[6] = b.z; x[7] = b.w;
  } else {
#pragma unroll
    for (int j = 0; j < SV; ++j) x[j] = i + j < P ? ids[i + j] : -1;
  }
}

// One workgroup per expert. order [P]: pairs by expert; tiles [1 + max_tiles]
// = (number of tiles, ..), then (expert, first place in order, pairs, 0).
__global__ __launch_bounds__(ST) void sort_pairs_kernel(
    const int32_t* __restrict__ ids, int32_t* __restrict__ order,
    int4* __restrict__ tiles, int P, int E, int tile) {
  extern __shared__ int hist[];        // [E]
  __shared__ int sums[ST / WAVE], at[2];
  const int e = blockIdx.x, tid = threadIdx.x;
  const int wave = tid / WAVE, lane = tid % WAVE;
  for (int i = tid; i < E; i += ST) hist[i] = 0;
  __syncthreads();
  for (int i = tid * SV; i < P; i += ST * SV) {
    int x[SV];
    load_ids(ids, i, P, x);
#pragma unroll
    for (int j = 0; j < SV; ++j)
      if (x[j] >= 0 && x[j] < E) atomicAdd(&hist[x[j]], 1);
  }
  __syncthreads();
  if (wave == 0) {                     // pairs and tiles of lower experts
    int n = 0, t = 0;
    for (int i = lane; i < e; i += WAVE) {
      n += hist[i];
      t += (hist[i] + tile - 1) / tile;
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      n += __shfl_xor(n, o, WAVE);
      t += __shfl_xor(t, o, WAVE);
    }
    if (lane == 0) {
      at[0] = n;
      at[1] = t;
    }
  }
  __syncthreads();
  const int first = at[0], count = hist[e], nt = (count + tile - 1) / tile;
  for (int j = tid; j < nt; j += ST)
    tiles[1 + at[1] + j] =
        make_int4(e, first + j * tile, min(tile, count - j * tile), 0);
  if (e == E - 1 && tid == 0) tiles[0] = make_int4(at[1] + nt, 0, 0, 0);
  int base = first;
  for (int i0 = 0; i0 < P; i0 += ST * SV) {   // workgroup-uniform
    const int i = i0 + tid * SV;
    int mine = 0, x[SV];
    load_ids(ids, i, P, x);
#pragma unroll
    for (int j = 0; j < SV; ++j) mine |= (x[j] == e) << j;
    const int n = __popc(mine);
    int before = n;                    // inclusive sum over the wave
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const int v = __shfl_up(before, o, WAVE);
      if (lane >= o) before += v;
    }
    __syncthreads();
    if (lane == WAVE - 1) sums[wave] = before;
    __syncthreads();
    int total = 0, place = base + before - n;
#pragma unroll
    for (int w = 0; w < ST / WAVE; ++w) {
      if (w < wave) place += sums[w];
      total += sums[w];
    }
#pragma unroll
    for (int j = 0; j < SV; ++j)
      if (mine >> j & 1) order[place++] = i + j;
    base += total;
  }
}

// ---- products --------------------------------------------------------------
struct Pairs {
  const void* a;             // UP: h [T, K]; else inner rows [P, K], sorted
  const void* w;             // [E, N, K]
  void* out;                 // UP: inner rows [P, N], sorted; else [P, N]
  const int32_t* order;      // place -> pair
  const int4* tiles;
  const float* weights;      // [P]
  int N, K, top, act;
};

// input row of a place
template <bool UP>
__device__ __forceinline__ int64_t source(const Pairs& p, int place) {
  return UP ? p.order[place] / p.top : place;
}
template <bool UP>
__device__ __forceinline__ float finish(const Pairs& p, float sum, float wt) {
  return UP ? activate(p.act, sum * wt) : sum;
}

// grid (blocks of channels, tiles)
template <typename T, bool UP>
__global__ __launch_bounds__(256) void expert_plain_kernel(const Pairs p) {
  if ((int)blockIdx.y >= p.tiles[0].x) return;
  const int4 tile = p.tiles[1 + blockIdx.y];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int n1 = min(p.N, (int)(blockIdx.x + 1) * 64);
  for (int i = tile.y; i < tile.y + tile.z; ++i) {
    const int pair = p.order[i];
    const T* a = (const T*)p.a + source<UP>(p, i) * p.K;
    T* o = (T*)p.out + (int64_t)(UP ? i : pair) * p.N;
    for (int n = blockIdx.x * 64 + wave; n < n1; n += 4) {
      const T* w = (const T*)p.w + ((int64_t)tile.x * p.N + n) * p.K;
      float s = 0.f;
      for (int k = lane; k < p.K; k += WAVE) s += ld(a + k) * ld(w + k);
      s = wave_reduce_sum(s);
      if (lane == 0) st(o + n, finish<UP>(p, s, p.weights[pair]));
    }
  }
}

// grid (blocks of 64 channels, tiles of 16 MT pairs). The waves split K; a
// lane reads 32 bytes of a row at a time, 16 rows and 128 bytes of each per
// wave. The order of K inside a step is the same for both operands.
template <int MT, bool UP>
__global__ __launch_bounds__(256) void expert_rows_kernel(const Pairs p) {
  __shared__ float4v red[4][4][MT][WAVE];   // [channel tile][wave]
  if ((int)blockIdx.y >= p.tiles[0].x) return;
  const int4 tile = p.tiles[1 + blockIdx.y];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane % 16, grp = lane / 16, N = p.N, K = p.K;
  const int n0 = blockIdx.x * 64;
  const short *wr[4], *ar[MT];
#pragma unroll
  for (int c = 0; c < 4; ++c)
    wr[c] = (const short*)p.w +
            ((int64_t)tile.x * N + min(n0 + c * 16 + col, N - 1)) * K;
#pragma unroll
  for (int t = 0; t < MT; ++t)
    ar[t] = (const short*)p.a +
            source<UP>(p, tile.y + min(t * 16 + col, tile.z - 1)) * K;
  float4v acc[4][MT];
#pragma unroll
  for (int c = 0; c < 4; ++c)
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[c][t] = (float4v){0.f, 0.f, 0.f, 0.f};
  const short8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  short8 wf[4][2], af[MT][2], wn[4][2], an[MT][2];
  // past the end of K the pairs' rows count as zero
  auto fetch = [&](int k0) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int k = k0 + grp * 16 + s * 8, kc = min(k, K - 8);
#pragma unroll
      for (int c = 0; c < 4; ++c) wn[c][s] = *(const short8*)(wr[c] + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        if constexpr (MT > 2) {      // worth leaving absent pairs out
          an[t][s] = k < K && t * 16 + col < tile.z
                         ? *(const short8*)(ar[t] + k)
                         : zero;
        } else {
          an[t][s] = *(const short8*)(ar[t] + kc);
          if (k >= K) an[t][s] = zero;
        }
      }
    }
  };
  fetch(wave * 64);
  for (int k0 = wave * 64; k0 < K; k0 += 256) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int c = 0; c < 4; ++c) wf[c][s] = wn[c][s];
#pragma unroll
      for (int t = 0; t < MT; ++t) af[t][s] = an[t][s];
    }
    fetch(k0 + 256);
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int t = 0; t < MT; ++t)
          acc[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              __builtin_bit_cast(bf16x8, wf[c][s]),
              __builtin_bit_cast(bf16x8, af[t][s]), acc[c][t], 0, 0, 0);
  }
#pragma unroll
  for (int c = 0; c < 4; ++c)
#pragma unroll
    for (int t = 0; t < MT; ++t) red[c][wave][t][lane] = acc[c][t];
  __syncthreads();
  const int n = n0 + wave * 16 + grp * 4;    // this wave's channels
  if (n >= N) return;
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int i = t * 16 + col;
    if (i >= tile.z) continue;
    const int pair = p.order[tile.y + i];
    const float wt = UP ? p.weights[pair] : 1.f;
    float4v s = red[wave][0][t][lane];
#pragma unroll
    for (int v = 1; v < 4; ++v) s += red[wave][v][t][lane];
    *(short4v*)((short*)p.out + (int64_t)(UP ? tile.y + i : pair) * N + n) =
        (short4v){f32_to_bf16(finish<UP>(p, s[0], wt)),
                  f32_to_bf16(finish<UP>(p, s[1], wt)),
                  f32_to_bf16(finish<UP>(p, s[2], wt)),
                  f32_to_bf16(finish<UP>(p, s[3], wt))};
  }
}

// 256 channels x 128 pairs, K in steps of 64 through three LDS buffers that are
// filled straight from memory, two steps ahead. A row of a step is 128 bytes =
// 8 pieces; piece c of row r lies at place c ^ (r / 2 % 8): the 16 rows a read
// serves at once then meet all 64 banks. 4 waves, 128 x 64 each, CT x PT tiles
// of 32 x 32. Loads and LDS reads are spread between the matrix instructions:
// issued in a row they would hold the wave up.
constexpr int CT = 4, PT = 2, NB = 3, BK = 64;
constexpr int TC = 64 * CT, TILE = 64 * PT;
constexpr int BUF = (TC + TILE) * BK;
constexpr int TILES_LDS = NB * BUF * (int)sizeof(short);
constexpr int TG = 8;                // tiles of pairs that run side by side

template <bool UP>
__global__ __launch_bounds__(256, 1) void expert_tiles_kernel(const Pairs p) {
  extern __shared__ __align__(16) short tile_lds[];  // NB x [weights, pairs]
  const int N = p.N, K = p.K;
  // Workgroups go round the 8 XCDs in turn: each XCD gets a contiguous share
  // of the work, in which TG tiles of pairs walk the channels together.
  const int nx = (N + TC - 1) / TC, total = p.tiles[0].x * nx;
  const int share = (total + 7) / 8;
  const int id = blockIdx.x % 8 * share + blockIdx.x / 8;
  if ((int)blockIdx.x / 8 >= share || id >= total) return;
  const int g = id / (TG * nx), in = id % (TG * nx);
  const int width = min(TG, p.tiles[0].x - g * TG);
  const int4 tile = p.tiles[1 + g * TG + in % width];
  const int n0 = in / width * TC;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane & 31, hi = lane >> 5;
  const int wc = wave & 1, wp = wave >> 1;    // its channels, its pairs

  // A wave fills a quarter of the rows of both, 8 rows per instruction, from
  // byte offsets within the expert's weights and p.a (both under 4 GiB).
  // Rows past the tile repeat its last one: they are computed and dropped.
  constexpr int LW = 2 * CT, LOADS = 2 * CT + 2 * PT;
  const char* wbase = (const char*)p.w + (int64_t)tile.x * N * K * 2;
  const char* abase = (const char*)p.a;
  uint32_t src[LOADS];
  int64_t rows[2 * PT];
#pragma unroll
  for (int j = 0; j < 2 * PT; ++j)
    rows[j] = source<UP>(p, tile.y + min(wave * 16 * PT + j * 8 + lane / 8,
                                         tile.z - 1));
  auto piece = [&](int j) {
    return (lane % 8 ^ (lane / 16 + j % 2 * 4)) * 8;
  };
#pragma unroll
  for (int j = 0; j < LW; ++j)
    src[j] = ((uint32_t)min(n0 + wave * 16 * CT + j * 8 + lane / 8, N - 1) *
                  K + piece(j)) * 2;
  const int steps = K / BK;
  auto column = [&](int s) { return min(s, steps - 1) * BK * 2; };
  auto load = [&](int buf, int k, int j) {
    typedef __attribute__((address_space(1))) const unsigned int gmem;
    typedef __attribute__((address_space(3))) unsigned int smem;
    const int row = j < LW ? wave * 16 * CT + j * 8
                           : TC + wave * 16 * PT + (j - LW) * 8;
    __builtin_amdgcn_global_load_lds(
        (gmem*)((j < LW ? wbase : abase) + k + src[j]),
        (smem*)(tile_lds + buf * BUF + row * BK), 16, 0, 0);
  };
#pragma unroll
  for (int j = 0; j < LW; ++j) load(0, column(0), j);
#pragma unroll
  for (int j = 0; j < 2 * PT; ++j)
    src[LW + j] = ((uint32_t)rows[j] * K + piece(j)) * 2;
#pragma unroll
  for (int j = LW; j < LOADS; ++j) load(0, column(0), j);
#pragma unroll
  for (int j = 0; j < LOADS; ++j) load(1, column(1), j);

  f32x16 acc[CT][PT];
#pragma unroll
  for (int c = 0; c < CT; ++c)
#pragma unroll
    for (int t = 0; t < PT; ++t) acc[c][t] = (f32x16)(0.f);
  int buf = 0, fill = NB - 1;
  for (int s = 0; s < steps; ++s) {
    // this step has landed (the next may be on its way), and the buffer that
    // is filled now is no longer read
    asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"i"(LOADS) : "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    const int k = column(s + NB - 1);          // the last step repeats
    const short* wl = tile_lds + buf * BUF + (wc * 32 * CT + col) * BK;
    const short* al = tile_lds + buf * BUF + (TC + wp * 32 * PT + col) * BK;
    bf16x8 wf[2][CT], af[2][PT];
    auto read = [&](int x, int kk) {
      const int at = ((kk * 2 + hi) ^ (col / 2 & 7)) * 8;
#pragma unroll
      for (int c = 0; c < CT; ++c)
        wf[x][c] = *(const bf16x8*)(wl + c * 32 * BK + at);
#pragma unroll
      for (int t = 0; t < PT; ++t)
        af[x][t] = *(const bf16x8*)(al + t * 32 * BK + at);
    };
    read(0, 0);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int kk = 0; kk < BK / 16; ++kk) {
      const bool more = kk + 1 < BK / 16;
      if (more) read(kk + 1 & 1, kk + 1);
#pragma unroll
      for (int j = 0; j < LOADS / 4; ++j) load(fill, k, kk * LOADS / 4 + j);
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int t = 0; t < PT; ++t)
          acc[c][t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              wf[kk & 1][c], af[kk & 1][t], acc[c][t], 0, 0, 0);
      // the order: matrix, read, (load), ... matrix
#pragma unroll
      for (int i = 0; i < CT + PT; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
        if (more) __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        if (i % 2 == 0) __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
      }
      __builtin_amdgcn_sched_group_barrier(0x008, CT * PT - CT - PT, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
    buf = buf + 1 == NB ? 0 : buf + 1;
    fill = fill + 1 == NB ? 0 : fill + 1;
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // the repeated loads

  auto write = [&](auto act) {
#pragma unroll
    for (int t = 0; t < PT; ++t) {
      const int i = wp * 32 * PT + t * 32 + col;
      if (i >= tile.z) continue;
      const int pair = p.order[tile.y + i];
      const float wt = UP ? p.weights[pair] : 1.f;
      short* o = (short*)p.out + (int64_t)(UP ? tile.y + i : pair) * N;
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int n = n0 + wc * 32 * CT + c * 32 + q * 8 + hi * 4;
          if (n >= N) continue;
          short4v v;
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            const float f = acc[c][t][4 * q + x];
            v[x] = f32_to_bf16(UP ? activate(act, f * wt) : f);
          }
          *(short4v*)(o + n) = v;
        }
    }
  };
  using std::integral_constant;
  if (!UP || p.act == ACT_RELU_SQUARED)
    write(integral_constant<int, ACT_RELU_SQUARED>{});
  else if (p.act == ACT_SILU)
    write(integral_constant<int, ACT_SILU>{});
  else
    write(integral_constant<int, ACT_GELU_TANH>{});
}

template <bool UP>
hipError_t launch_tiles(const Pairs& p, int max_tiles, hipStream_t stream) {
  // every XCD's share is rounded up
  const int64_t n = ((int64_t)max_tiles * ((p.N + TC - 1) / TC) + 7) / 8 * 8;
  if (n > 0x7fffffff || p.N % 8 || p.K % BK || p.K < 2 * BK ||
      (int64_t)p.N * p.K >= 1ll << 31)
    return hipErrorInvalidValue;
  auto fn = expert_tiles_kernel<UP>;
  hipError_t e = hipFuncSetAttribute(
      (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, TILES_LDS);
  if (e != hipSuccess) return e;
  hipLaunchKernelGGL(fn, dim3((uint32_t)n), dim3(256), TILES_LDS, stream, p);
  HIP_CHECK_LAST();
  return hipSuccess;
}

template <bool UP>
hipError_t product(int f32, int plain, int tile, int max_tiles, const Pairs& p,
                   hipStream_t stream) {
  if (tile == TILE) return launch_tiles<UP>(p, max_tiles, stream);
  const dim3 grid((p.N + 63) / 64, max_tiles), block(256);
  if (max_tiles > 65535 || tile > 64) return hipErrorInvalidValue;
#define GO(KERNEL) hipLaunchKernelGGL((KERNEL), grid, block, 0, stream, p)
#define K2(NAME, ARG) NAME<ARG, UP>
  if (f32) GO(K2(expert_plain_kernel, float));
  else if (plain || p.N % 8 || p.K % 8) GO(K2(expert_plain_kernel, short));
  else if (tile <= 16) GO(K2(expert_rows_kernel, 1));
  else if (tile <= 32) GO(K2(expert_rows_kernel, 2));
  else GO(K2(expert_rows_kernel, 4));
#undef K2
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // namespace

extern "C" {

hipError_t lds_route(int f32, const void* h, const void* w, int32_t* ids,
                     float* wt, int64_t rows, int K, int E, int top,
                     hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  if (top < 1 || top > E || E > 8192) return hipErrorInvalidValue;
  if (f32 || K % 8 || E > 256) {
    const size_t lds = E * sizeof(float);
    if (f32)
      hipLaunchKernelGGL(route_plain_kernel<float>, dim3((uint32_t)rows),
                         dim3(256), lds, stream, (const float*)h,
                         (const float*)w, ids, wt, K, E, top);
    else
      hipLaunchKernelGGL(route_plain_kernel<short>, dim3((uint32_t)rows),
                         dim3(256), lds, stream, (const short*)h,
                         (const short*)w, ids, wt, K, E, top);
    HIP_CHECK_LAST();
    return hipSuccess;
  }
#define GO(ET, NW)                                                            \
  hipLaunchKernelGGL((route_kernel<ET, NW>),                                  \
                     dim3((uint32_t)((rows + 15) / 16)), dim3(NW * WAVE),     \
                     NW * 256 * ET * sizeof(float), stream, (const short*)h,  \
                     (const short*)w, ids, wt, rows, K, E, top)
  if (E <= 16) GO(1, 16); else if (E <= 32) GO(2, 16);
  else if (E <= 64) GO(4, 16); else if (E <= 128) GO(8, 8);
  else GO(16, 4);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

// pairs of one expert that a workgroup takes: about as many as an expert has
int lds_expert_tile(int f32, int plain, int P, int T, int E, int N, int K) {
  const int per = (P + E - 1) / E;
  const int64_t limit = 1ll << 31;      // elements: offsets stay under 4 GiB
  if (f32 || plain || per <= 12) return 16;
  if (per <= 24) return 32;
  if (per <= 48 || N % BK || K % BK || N < 2 * BK || K < 2 * BK ||
      (int64_t)N * K >= limit || (int64_t)T * K >= limit ||
      (int64_t)P * N >= limit)
    return 64;
  return TILE;
}

// tiles of P pairs at most
int lds_expert_max_tiles(int P, int E, int tile) {
  const int n = P / tile + E;
  return n < P ? n : P;
}

// order [P], tiles [1 + max_tiles, 4]
hipError_t lds_sort_pairs(const int32_t* ids, int32_t* order, void* tiles,
                          int P, int E, int tile, hipStream_t stream) {
  if (P == 0) return hipSuccess;
  if (E > 8192) return hipErrorInvalidValue;
  hipLaunchKernelGGL(sort_pairs_kernel, dim3(E), dim3(ST), E * sizeof(int),
                     stream, ids, order, (int4*)tiles, P, E, tile);
  HIP_CHECK_LAST();
  return hipSuccess;
}

// One layer of the experts (up: the first). a, out: see Pairs.
hipError_t lds_expert_product(int f32, int plain, int up, const void* a,
                              const void* w, void* out, const int32_t* order,
                              const void* tiles, int max_tiles, int tile,
                              const float* weights, int N, int K, int top,
                              int act, hipStream_t stream) {
  if (max_tiles == 0) return hipSuccess;
  const Pairs p{a, w, out, order, (const int4*)tiles, weights, N, K, top, act};
  return up ? product<true>(f32, plain, tile, max_tiles, p, stream)
            : product<false>(f32, plain, tile, max_tiles, p, stream);
}

}  // extern "C"
