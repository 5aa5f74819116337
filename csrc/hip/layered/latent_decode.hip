// latent_decode.hip — absorbed attention of single rows over paged latents
// (bf16): every head of a row reads the same cached token
// [latent (R) | rotated part], the latent being key part and value at once.
//
// One workgroup per (row, 16 or 32 heads, part of the context), 4 waves per 16
// heads. Tiles of 64 tokens pass through LDS once, for keys and values; the
// next tile waits in registers. S' = K Q' (a wave owns 16 tokens and 16 heads),
// softmax across the waves through LDS, O' = V' P' for all heads (a wave owns
// every NW-th 16 latent channels; the transposing LDS reads give V').
// Memory-bound: the matrix work per token is small beside its bytes.
#include "elem.h"

namespace {

constexpr int TB = 64;          // tokens per tile
constexpr float NEG = -1e30f;
constexpr int PS = TB + 8;      // row stride of P (shorts)

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

// RT: latent channels / 64, rounded up; HT: 16-head tiles
template <int RT, int HT>
__global__ __launch_bounds__(4 * HT * WAVE) void latent_decode_kernel(
    const short* __restrict__ q_lat,   // [H, n, R]
    const short* __restrict__ q,       // [rows, H, QD], rotated part last
    const short* __restrict__ cache,   // [NB, BS, W]
    const int32_t* __restrict__ positions, const int32_t* __restrict__ row_seq,
    const int32_t* __restrict__ block_tables, short* __restrict__ out,
    float* __restrict__ part_o,        // [n, H, parts, R] when parts > 1
    float* __restrict__ part_ml,       // [n, H, parts, 2]
    int n, int H, int R, int W, int QD, int max_blocks, int bs, int window,
    int parts, float scale_log2) {
  constexpr int NW = 4 * HT, NT = NW * WAVE;
  constexpr int NTL = (4 * RT + NW - 1) / NW;  // 16-channel tiles per wave
  constexpr int NI = RT + 1;           // 16-byte pieces per thread and token
  constexpr int NJ = 8 / NW;           // tokens per thread and tile
  extern __shared__ short lds[];
  const int WP = (W + 31) / 32 * 32, LS = WP + 8;
  short* kl = lds;                     // [TB][LS]
  short* ql = kl + TB * LS;            // [16 HT][LS]
  short* pl = ql + 16 * HT * LS;       // [16 HT][PS]
  float* red = (float*)(pl + 16 * HT * PS);   // [2][4][16 HT]
  const int row = blockIdx.x, h0 = blockIdx.y * 16 * HT;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int col = lane % 16, grp = lane / 16;
  const int tw = wave % 4, hw = wave / 4;   // its 16 tokens, its 16 heads
  const int pos = positions[row];
  const int lo = window > 0 ? max(0, pos + 1 - window) : 0;
  const int span = ((pos + 1 - lo + parts - 1) / parts + TB - 1) / TB * TB;
  const int t_lo = lo + blockIdx.z * span;
  const int t_hi = min(pos + 1, t_lo + span);
  const int32_t* bt = block_tables + (int64_t)row_seq[row] * max_blocks;
  const int rot = W - R;

  float m[HT], l[HT];
  float4v acc[HT][NTL];
#pragma unroll
  for (int a = 0; a < HT; ++a) {
    m[a] = NEG;
    l[a] = 0.f;
#pragma unroll
    for (int i = 0; i < NTL; ++i) acc[a][i] = (float4v){0.f, 0.f, 0.f, 0.f};
  }

  if (t_lo < t_hi) {                   // workgroup-uniform
    const int pieces = WP / 8;
    for (int i = tid; i < 16 * HT * pieces; i += NT) {
      const int h = h0 + i / pieces, d = i % pieces * 8;
      short8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      if (h < H && d < W)
        z = *(const short8*)(d < R ? q_lat + ((int64_t)h * n + row) * R + d
                                   : q + ((int64_t)row * H + h) * QD + QD -
                                         rot + (d - R));
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
        const short* src = cache + ((int64_t)page[j] * bs + t % bs) * W;
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
      for (int kk = 0; kk < WP / 32; ++kk) {
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
        sc[r] = t < t_hi ? sc[r] * scale_log2 : NEG;
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
            const short* v = kl + (ks * 32 + grp * 8 + col / 4) * LS + c0 +
                             (col % 4) * 4;
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
    const int h = h0 + a * 16 + col;
    if (h >= H) continue;
    const int64_t pr = ((int64_t)row * H + h) * parts + blockIdx.z;
    const float inv = parts > 1 ? 1.f : 1.f / l[a];
#pragma unroll
    for (int i = 0; i < NTL; ++i) {
      const int d = (wave + NW * i) * 16 + grp * 4;
      if (d >= R) continue;
      if (parts > 1) {
        *(float4v*)(part_o + pr * R + d) = acc[a][i];
      } else {
        *(short4v*)(out + ((int64_t)h * n + row) * R + d) = (short4v){
            f32_to_bf16(acc[a][i][0] * inv), f32_to_bf16(acc[a][i][1] * inv),
            f32_to_bf16(acc[a][i][2] * inv), f32_to_bf16(acc[a][i][3] * inv)};
      }
    }
    if (parts > 1 && wave == 0 && grp == 0) {
      part_ml[pr * 2] = m[a];
      part_ml[pr * 2 + 1] = l[a];
    }
  }
}

// grid (n, H)
__global__ __launch_bounds__(128) void latent_combine_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    short* __restrict__ out, int n, int H, int R, int parts) {
  const int row = blockIdx.x, h = blockIdx.y;
  const int64_t pr = ((int64_t)row * H + h) * parts;
  float m = NEG;
  for (int p = 0; p < parts; ++p) m = fmaxf(m, part_ml[(pr + p) * 2]);
  float l = 0.f;
  for (int p = 0; p < parts; ++p)
    l += part_ml[(pr + p) * 2 + 1] *
         __builtin_amdgcn_exp2f(part_ml[(pr + p) * 2] - m);
  const float inv = 1.f / l;
  for (int d = threadIdx.x; d < R; d += 128) {
    float o = 0.f;
    for (int p = 0; p < parts; ++p)
      o += part_o[(pr + p) * R + d] *
           __builtin_amdgcn_exp2f(part_ml[(pr + p) * 2] - m);
    out[((int64_t)h * n + row) * R + d] = f32_to_bf16(o * inv);
  }
}

}  // namespace

extern "C" {

// 0 if the sizes have no tiled form
int lds_latent_decode_ok(int R, int rot, int QD) {
  const int tiles = (R + 63) / 64;
  const int ntl = tiles <= 1 ? 1 : tiles <= 2 ? 2 : tiles <= 4 ? 4 : 8;
  return R % 16 == 0 && rot % 8 == 0 && QD % 8 == 0 && R <= 512 &&
         R + rot <= 64 * (ntl + 1);
}

// parts of the context that fill the chip with n rows
int lds_latent_decode_parts(int n, int H, int max_ctx, int window) {
  const int keys = window > 0 && window < max_ctx ? window : max_ctx;
  const int groups = n * (H > 16 ? (H + 31) / 32 : 1);
  int parts = 256 / groups;         // a workgroup has a CU to itself
  if (parts > (keys + 127) / 128) parts = (keys + 127) / 128;
  return parts < 1 ? 1 : parts > 32 ? 32 : parts;
}

hipError_t lds_latent_decode(const void* q_lat, const void* q,
                             const void* cache, const int32_t* positions,
                             const int32_t* row_seq,
                             const int32_t* block_tables, void* out,
                             float* part_o, float* part_ml, int n, int H,
                             int R, int rot, int QD, int max_blocks, int bs,
                             int window, int parts, float scale,
                             hipStream_t stream) {
  if (n == 0) return hipSuccess;
  if (!lds_latent_decode_ok(R, rot, QD)) return hipErrorInvalidValue;
  const int W = R + rot, LS = (W + 31) / 32 * 32 + 8;
  const int ht = H > 16 ? 2 : 1;
  const size_t lds = (size_t)(TB * LS + 16 * ht * LS + 16 * ht * PS) * 2 +
                     2 * 4 * 16 * ht * sizeof(float);
  const dim3 grid(n, (H + 16 * ht - 1) / (16 * ht), parts), block(4 * ht * WAVE);
  const float s2 = scale * 1.4426950408889634f;
#define GO2(N, HT)                                                            \
  do {                                                                        \
    auto fn = latent_decode_kernel<N, HT>;                                    \
    hipError_t e = hipFuncSetAttribute(                                       \
        (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize,          \
        (int)lds);                                                            \
    if (e != hipSuccess) return e;                                            \
    hipLaunchKernelGGL(fn, grid, block, lds, stream, (const short*)q_lat,     \
                       (const short*)q, (const short*)cache, positions,       \
                       row_seq, block_tables, (short*)out, part_o, part_ml,   \
                       n, H, R, W, QD, max_blocks, bs, window, parts, s2);    \
  } while (0)
#define GO(N)                                                                 \
  do {                                                                        \
    if (ht == 2) GO2(N, 2); else GO2(N, 1);                                   \
  } while (0)
  const int tiles = (R + 63) / 64;
  if (tiles <= 1) GO(1); else if (tiles <= 2) GO(2);
  else if (tiles <= 4) GO(4); else GO(8);
#undef GO
#undef GO2
  if (parts > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(n, H), dim3(128), 0,
                       stream, part_o, part_ml, (short*)out, n, H, R, parts);
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
