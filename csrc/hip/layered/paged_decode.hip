// paged_decode.hip — attention of single rows over paged keys and values (bf16).
//
// A cached token is one row of W elements per key/value head; its keys are the
// first SW columns, its values R columns from v0 on. Two layouts use it: the
// absorbed form of latent attention (one head for all queries, the latent
// being key part and value at once) and grouped heads (rows [key | value]).
//
// One workgroup per (row, 16 or 32 query heads of one key/value head, part of
// the context), 4 waves per 16 heads. Tiles of 64 tokens pass through LDS
// once, for keys and values; the next tile waits in registers. S' = K Q' (a
// wave owns 16 tokens and 16 heads), softmax across the waves through LDS,
// O' = V' P' for all heads (a wave owns every NW-th 16 value channels; the
// transposing LDS reads give V'). Memory-bound: the matrix work per token is
// small beside its bytes.
#include "elem.h"

namespace {

constexpr int TB = 64;          // tokens per tile
constexpr float NEG = -1e30f;
constexpr int PS = TB + 8;      // row stride of P (shorts)

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

struct Decode {
  // query: columns [0, da) at qa, [da, SW) at qb; strides in elements
  const short *qa, *qb;
  int64_t qa_row, qa_head, qb_row, qb_head;
  int da, SW;
  const short* cache;
  int64_t page, head;      // strides of a page and of a head inside it
  int W, v0, R;
  const int32_t *positions, *row_seq, *block_tables;
  int max_blocks, bs, window;
  short* out;
  int64_t o_row, o_head;
  float* part_o;           // [n, H, parts, R] when parts > 1
  float* part_ml;          // [n, H, parts, 2]
  int H, rep, blocks;      // query heads, per key head, their workgroups
  int parts;
  float scale_log2, sink;  // sink: score (log2) of a key without a value
  int has_sink;
};

// columns of a token's LDS row
__host__ __device__ inline int padded_width(int SW, int W, int v0, int R) {
  const int s = (SW + 31) / 32 * 32, v = v0 + (R + 15) / 16 * 16;
  const int w = s > v ? s : v;
  return ((w > W ? w : W) + 31) / 32 * 32;
}

// RT: value channels / 64, rounded up; NI: 64-column pieces of an LDS row;
// HT: 16-head tiles
template <int RT, int NI, int HT>
__global__ __launch_bounds__(4 * HT * WAVE) void paged_decode_kernel(
    const Decode d_) {
  constexpr int NW = 4 * HT, NT = NW * WAVE;
  constexpr int NTL = (4 * RT + NW - 1) / NW;  // 16-channel tiles per wave
  constexpr int NJ = 8 / NW;           // tokens per thread and tile
  const int W = d_.W, R = d_.R, bs = d_.bs, parts = d_.parts;
  extern __shared__ short lds[];
  const int WP = padded_width(d_.SW, W, d_.v0, R), LS = WP + 8;
  const int SP = (d_.SW + 31) / 32 * 32;
  short* kl = lds;                     // [TB][LS]
  short* ql = kl + TB * LS;            // [16 HT][LS]
  short* pl = ql + 16 * HT * LS;       // [16 HT][PS]
  float* red = (float*)(pl + 16 * HT * PS);   // [2][4][16 HT]
  const int row = blockIdx.x, kvh = blockIdx.y / d_.blocks;
  const int r_lo = blockIdx.y % d_.blocks * 16 * HT;   // in the head's group
  const int h0 = kvh * d_.rep + r_lo, n_h = d_.rep - r_lo;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int col = lane % 16, grp = lane / 16;
  const int tw = wave % 4, hw = wave / 4;   // its 16 tokens, its 16 heads
  const int pos = d_.positions[row];
  const int lo = d_.window > 0 ? max(0, pos + 1 - d_.window) : 0;
  const int span = ((pos + 1 - lo + parts - 1) / parts + TB - 1) / TB * TB;
  const int t_lo = lo + blockIdx.z * span;
  const int t_hi = min(pos + 1, t_lo + span);
  const int32_t* bt =
      d_.block_tables + (int64_t)d_.row_seq[row] * d_.max_blocks;
  const short* cache = d_.cache + kvh * d_.head;
  const bool sink = d_.has_sink && parts == 1;

  float m[HT], l[HT];
  float4v acc[HT][NTL];
#pragma unroll
  for (int a = 0; a < HT; ++a) {
    m[a] = sink ? d_.sink : NEG;
    l[a] = sink ? 1.f : 0.f;
#pragma unroll
    for (int i = 0; i < NTL; ++i) acc[a][i] = (float4v){0.f, 0.f, 0.f, 0.f};
  }

  if (t_lo < t_hi) {                   // workgroup-uniform
    const int pieces = SP / 8;
    for (int i = tid; i < 16 * HT * pieces; i += NT) {
      const int r = i / pieces, d = i % pieces * 8;
      short8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      if (r < n_h && d < d_.SW)
        z = *(const short8*)(d < d_.da
                                 ? d_.qa + row * d_.qa_row +
                                       (h0 + r) * d_.qa_head + d
                                 : d_.qb + row * d_.qb_row +
                                       (h0 + r) * d_.qb_head + (d - d_.da));
      *(short8*)(ql + i / pieces * LS + d) = z;
    }
    // 8 threads share a token (128 bytes at a time), two tokens per thread
    const int r0 = tid / 8, d0 = tid % 8 * 8;
    // and their pages one tile further ahead
    short8 nx[NJ][NI];
    int page[NJ];
    auto find = [&](int t0) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int t = t0 + r0 + 32 * j;
        page[j] = t < t_hi ? bt[t / bs] : 0;
      }
    };
    auto fetch = [&](int t0) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int t = t0 + r0 + 32 * j;
        const short* src = cache + page[j] * d_.page + t % bs * W;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
          const int d = d0 + i * 64;
          nx[j][i] = (short8){0, 0, 0, 0, 0, 0, 0, 0};
          if (t < t_hi && d < W) nx[j][i] = *(const short8*)(src + d);
        }
      }
    };
    find(t_lo);
    fetch(t_lo);
    find(t_lo + TB);
    for (int t0 = t_lo; t0 < t_hi; t0 += TB) {
      lds_barrier();
#pragma unroll
      for (int j = 0; j < NJ; ++j)
#pragma unroll
        for (int i = 0; i < NI; ++i)
          if (d0 + i * 64 < WP)
            *(short8*)(kl + (r0 + 32 * j) * LS + d0 + i * 64) = nx[j][i];
      lds_barrier();
      if (t0 + TB < t_hi) {
        fetch(t0 + TB);
        find(t0 + 2 * TB);
      }

      // scores: rows tokens, columns heads
      float4v sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 6
      for (int kk = 0; kk < SP / 32; ++kk) {
        const bf16x8 kf = *(const bf16x8*)(kl + (tw * 16 + col) * LS +
                                           kk * 32 + grp * 8);
        const bf16x8 qf = *(const bf16x8*)(ql + (hw * 16 + col) * LS +
                                           kk * 32 + grp * 8);
        sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, sc, 0, 0, 0);
      }
      float mx = NEG;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = t0 + tw * 16 + grp * 4 + r;
        sc[r] = t < t_hi ? sc[r] * d_.scale_log2 : NEG;
        mx = fmaxf(mx, sc[r]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      if (grp == 0) red[(tw * HT + hw) * 16 + col] = mx;
      lds_barrier();
      float alpha[HT];
#pragma unroll
      for (int a = 0; a < HT; ++a) {
        float mn = m[a];
#pragma unroll
        for (int w = 0; w < 4; ++w)
          mn = fmaxf(mn, red[(w * HT + a) * 16 + col]);
        alpha[a] = __builtin_amdgcn_exp2f(m[a] - mn);
        m[a] = mn;       // finite: the tile's first token is in range
        if (a == hw) {   // wave-uniform
          float sum = 0.f, e[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            e[r] = __builtin_amdgcn_exp2f(sc[r] - mn);
            sum += e[r];
          }
          *(short4v*)(pl + (a * 16 + col) * PS + tw * 16 + grp * 4) =
              (short4v){f32_to_bf16(e[0]), f32_to_bf16(e[1]),
                        f32_to_bf16(e[2]), f32_to_bf16(e[3])};
          sum += __shfl_xor(sum, 16, WAVE);
          sum += __shfl_xor(sum, 32, WAVE);
          if (grp == 0) red[((4 + tw) * HT + a) * 16 + col] = sum;
        }
      }
      lds_barrier();
      bf16x8 pf[HT][2];
#pragma unroll
      for (int a = 0; a < HT; ++a) {
        float sum = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w)
          sum += red[((4 + w) * HT + a) * 16 + col];
        l[a] = l[a] * alpha[a] + sum;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
          pf[a][ks] = *(const bf16x8*)(pl + (a * 16 + col) * PS + ks * 32 +
                                       grp * 8);
#pragma unroll
        for (int i = 0; i < NTL; ++i) acc[a][i] = acc[a][i] * alpha[a];
      }
#pragma unroll
      for (int i = 0; i < NTL; ++i) {
        const int c0 = (wave + NW * i) * 16;
        if (c0 < R) {                  // wave-uniform
#pragma unroll
          for (int ks = 0; ks < 2; ++ks) {
            const short* v = kl + (ks * 32 + grp * 8 + col / 4) * LS +
                             d_.v0 + c0 + (col % 4) * 4;
            typedef __attribute__((address_space(3))) short4v lds4;
            const short4v a0 =
                __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)v);
            const short4v a1 =
                __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)(v + 4 * LS));
            const short8 vf = {a0[0], a0[1], a0[2], a0[3],
                               a1[0], a1[1], a1[2], a1[3]};
#pragma unroll
            for (int a = 0; a < HT; ++a)
              acc[a][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                  __builtin_bit_cast(bf16x8, vf), pf[a][ks], acc[a][i], 0, 0,
                  0);
          }
        }
      }
    }
  }

#pragma unroll
  for (int a = 0; a < HT; ++a) {
    const int r = a * 16 + col, h = h0 + r;
    if (r >= n_h) continue;
    const int64_t pr = ((int64_t)row * d_.H + h) * parts + blockIdx.z;
    const float inv = parts > 1 ? 1.f : 1.f / l[a];
#pragma unroll
    for (int i = 0; i < NTL; ++i) {
      const int d = (wave + NW * i) * 16 + grp * 4;
      if (d >= R) continue;
      if (parts > 1) {
        *(float4v*)(d_.part_o + pr * R + d) = acc[a][i];
      } else {
        *(short4v*)(d_.out + row * d_.o_row + h * d_.o_head + d) = (short4v){
            f32_to_bf16(acc[a][i][0] * inv), f32_to_bf16(acc[a][i][1] * inv),
            f32_to_bf16(acc[a][i][2] * inv), f32_to_bf16(acc[a][i][3] * inv)};
      }
    }
    if (parts > 1 && wave == 0 && grp == 0) {
      d_.part_ml[pr * 2] = m[a];
      d_.part_ml[pr * 2 + 1] = l[a];
    }
  }
}

// grid (n, H)
__global__ __launch_bounds__(128) void combine_kernel(const Decode d_) {
  const int64_t row = blockIdx.x, h = blockIdx.y;
  const int R = d_.R, parts = d_.parts;
  const int64_t pr = (row * d_.H + h) * parts;
  const float* ml = d_.part_ml + pr * 2;
  float m = d_.has_sink ? d_.sink : NEG;
  for (int p = 0; p < parts; ++p) m = fmaxf(m, ml[p * 2]);
  float l = d_.has_sink ? __builtin_amdgcn_exp2f(d_.sink - m) : 0.f;
  for (int p = 0; p < parts; ++p)
    l += ml[p * 2 + 1] * __builtin_amdgcn_exp2f(ml[p * 2] - m);
  const float inv = 1.f / l;
  for (int d = threadIdx.x; d < R; d += 128) {
    float o = 0.f;
    for (int p = 0; p < parts; ++p)
      o += d_.part_o[(pr + p) * R + d] *
           __builtin_amdgcn_exp2f(ml[p * 2] - m);
    d_.out[row * d_.o_row + h * d_.o_head + d] = f32_to_bf16(o * inv);
  }
}

// query heads per workgroup of a key head with `rep` of them
int head_block(int rep) { return rep > 16 ? 32 : 16; }

// parts of the context that make up about `target` workgroups
int parts_for(int groups, int keys, int target) {
  int parts = target / groups;
  if (parts > (keys + 127) / 128) parts = (keys + 127) / 128;
  return parts < 1 ? 1 : parts > 32 ? 32 : parts;
}

size_t lds_bytes(const Decode& d) {
  const int hb = head_block(d.rep);
  const int LS = padded_width(d.SW, d.W, d.v0, d.R) + 8;
  return (size_t)(TB * LS + hb * LS + hb * PS) * 2 +
         2 * 4 * hb * sizeof(float);
}

hipError_t launch(Decode d, int n, int kv_heads, hipStream_t stream) {
  if (n == 0) return hipSuccess;
  const int hb = head_block(d.rep);
  d.blocks = (d.rep + hb - 1) / hb;
  const size_t lds = lds_bytes(d);
  const dim3 grid(n, kv_heads * d.blocks, d.parts), block(4 * (hb / 16) * WAVE);
#define GO2(N, M, HT)                                                         \
  do {                                                                        \
    auto fn = paged_decode_kernel<N, M, HT>;                                  \
    hipError_t e = hipFuncSetAttribute(                                       \
        (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize,          \
        (int)lds);                                                            \
    if (e != hipSuccess) return e;                                            \
    hipLaunchKernelGGL(fn, grid, block, lds, stream, d);                      \
  } while (0)
#define GO(N, M)                                                              \
  do {                                                                        \
    if (hb == 32) GO2(N, M, 2); else GO2(N, M, 1);                            \
  } while (0)
  const int rt = (d.R + 63) / 64;
  const int ni = (padded_width(d.SW, d.W, d.v0, d.R) + 63) / 64;
  if (rt <= 1 && ni <= 2) GO(1, 2);
  else if (rt <= 2 && ni <= 3) GO(2, 3);
  else if (rt <= 2 && ni <= 4) GO(2, 4);
  else if (rt <= 4 && ni <= 5) GO(4, 5);
  else if (rt <= 4 && ni <= 8) GO(4, 8);
  else if (rt <= 8 && ni <= 9) GO(8, 9);
  else return hipErrorInvalidValue;
#undef GO
#undef GO2
  if (d.parts > 1)
    hipLaunchKernelGGL(combine_kernel, dim3(n, d.H), dim3(128), 0, stream, d);
  HIP_CHECK_LAST();
  return hipSuccess;
}

constexpr float LOG2E = 1.4426950408889634f;

}  // namespace

extern "C" {

// 0 if the sizes have no tiled form
int lds_latent_decode_ok(int R, int rot, int QD) {
  return R % 16 == 0 && rot % 8 == 0 && QD % 8 == 0 && R <= 512 &&
         R + rot <= 576;
}

int lds_latent_decode_parts(int n, int H, int max_ctx, int window) {
  const int keys = window > 0 && window < max_ctx ? window : max_ctx;
  const int hb = head_block(H);
  return parts_for(n * ((H + hb - 1) / hb), keys, 256);
}

hipError_t lds_latent_decode(const void* q_lat, const void* q,
                             const void* cache, const int32_t* positions,
                             const int32_t* row_seq,
                             const int32_t* block_tables, void* out,
                             float* part_o, float* part_ml, int n, int H,
                             int R, int rot, int QD, int max_blocks, int bs,
                             int window, int parts, float scale,
                             hipStream_t stream) {
  if (!lds_latent_decode_ok(R, rot, QD)) return hipErrorInvalidValue;
  Decode d{};
  d.qa = (const short*)q_lat;
  d.qa_row = R;
  d.qa_head = (int64_t)n * R;
  d.da = R;
  d.qb = (const short*)q + QD - rot;
  d.qb_row = (int64_t)H * QD;
  d.qb_head = QD;
  d.SW = d.W = R + rot;
  d.R = R;
  d.cache = (const short*)cache;
  d.page = (int64_t)bs * d.W;
  d.positions = positions;
  d.row_seq = row_seq;
  d.block_tables = block_tables;
  d.max_blocks = max_blocks;
  d.bs = bs;
  d.window = window;
  d.out = (short*)out;
  d.o_row = R;
  d.o_head = (int64_t)n * R;
  d.part_o = part_o;
  d.part_ml = part_ml;
  d.H = d.rep = H;
  d.parts = parts;
  d.scale_log2 = scale * LOG2E;
  return launch(d, n, 1, stream);
}

int lds_grouped_decode_ok(int D, int V, int64_t q_stride) {
  return D % 8 == 0 && V % 8 == 0 && q_stride % 8 == 0 && V <= 256 &&
         padded_width(D, D + V, D, V) <= 512;
}

int lds_grouped_decode_parts(int n, int H, int G, int D, int V, int max_ctx) {
  Decode d{};
  d.rep = H / G;
  d.SW = d.v0 = D;
  d.W = D + V;
  d.R = V;
  const int hb = head_block(d.rep);
  const int per_cu = (int)((160 << 10) / lds_bytes(d));   // workgroups
  return parts_for(n * G * ((d.rep + hb - 1) / hb), max_ctx,
                   256 * (per_cu > 4 ? 4 : per_cu < 1 ? 1 : per_cu));
}

// q: first query of row 0, rows q_stride apart; cache [NB, G, bs, D + V];
// out [rows, H V]
hipError_t lds_grouped_decode(const void* q, int64_t q_stride,
                              const void* cache, const int32_t* positions,
                              const int32_t* row_seq,
                              const int32_t* block_tables, void* out,
                              float* part_o, float* part_ml, int n, int H,
                              int G, int D, int V, int max_blocks, int bs,
                              int parts, float scale, int has_sink, float sink,
                              hipStream_t stream) {
  if (!lds_grouped_decode_ok(D, V, q_stride)) return hipErrorInvalidValue;
  Decode d{};
  d.qa = (const short*)q;
  d.qa_row = q_stride;
  d.qa_head = D;
  d.da = d.SW = d.v0 = D;
  d.W = D + V;
  d.R = V;
  d.cache = (const short*)cache;
  d.head = (int64_t)bs * d.W;
  d.page = G * d.head;
  d.positions = positions;
  d.row_seq = row_seq;
  d.block_tables = block_tables;
  d.max_blocks = max_blocks;
  d.bs = bs;
  d.out = (short*)out;
  d.o_row = (int64_t)H * V;
  d.o_head = V;
  d.part_o = part_o;
  d.part_ml = part_ml;
  d.H = H;
  d.rep = H / G;
  d.parts = parts;
  d.scale_log2 = scale * LOG2E;
  d.has_sink = has_sink;
  d.sink = sink * LOG2E;
  return launch(d, n, G, stream);
}

}  // extern "C"
