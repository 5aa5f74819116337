// latent_prefill.hip — causal windowed prefill attention over expanded keys
// and values (bf16), one key/value head per query head, the rotated key part
// shared by all heads.
//
//   q    [rows, H, D + rot]           rotated
//   kv   [ctx rows, H D + H V]        keys and values expanded from latents
//   lat  [ctx rows, R + rot]          gathered cache rows (rotated part used)
//   a sequence's context row 0 sits at position ctx.pos0
//
// S' = K Q' keeps a query per lane: the online softmax is in-lane work plus
// one exchange between the wave's halves, as in flash_prefill.hip. Rows of
// the LDS tiles are padded instead of swizzled: 16 bytes for K (16-byte row
// reads hit distinct banks), 64 bytes for V (the transposing reads of four
// rows do). The next tile waits in registers while this one is computed.
#include "elem.h"

namespace {

constexpr int NW = 4, NT = NW * WAVE;
constexpr int QW = 32;          // query rows per wave
constexpr int KB = 64;          // keys per tile
constexpr float NEG = -1e30f;

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(4))) unsigned int uint4v;

__device__ __forceinline__ unsigned int pack2(float a, float b) {
  return ((unsigned int)(unsigned short)f32_to_bf16(b) << 16) |
         (unsigned int)(unsigned short)f32_to_bf16(a);
}

// grid (H, tiles); tiles [n, 2] = sequence, first query row of the portion
template <int DK, int DV>
__global__ __launch_bounds__(NT, 2) void latent_prefill_kernel(
    const short* __restrict__ q, const short* __restrict__ kv,
    const short* __restrict__ lat, const int32_t* __restrict__ seq_meta,
    const int32_t* __restrict__ ctx, const int32_t* __restrict__ tiles,
    short* __restrict__ out, int H, int D, int rot, int V, int lat_w,
    int window, float scale_log2) {
  constexpr int KS = DK + 8, VS = DV + 32;      // row strides in LDS (shorts)
  constexpr int NK = DK / 32, NV = DV / 32;     // 16-byte pieces per thread
  __shared__ short k_lds[KB * KS];
  __shared__ short v_lds[KB * VS];
  const int h = blockIdx.x;
  const int seq = tiles[2 * blockIdx.y], p0 = tiles[2 * blockIdx.y + 1];
  const Seq sq = load_seq(seq_meta, seq);
  const int64_t ctx0 = ctx[2 * seq];
  const int off = sq.prior - ctx[2 * seq + 1];  // query p sees keys <= off + p
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int qc = lane & 31, hi = lane >> 5;
  const int p = p0 + wave * QW + qc;
  const bool active = p < sq.n;
  const int QD = D + rot;
  const int64_t kv_w = (int64_t)H * (D + V);

  bf16x8 qf[DK / 16];
  {
    const short* qr =
        q + ((int64_t)(sq.row0 + min(p, sq.n - 1)) * H + h) * QD;
#pragma unroll
    for (int kk = 0; kk < DK / 16; ++kk) {
      const int d = kk * 16 + hi * 8;
      short8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < QD) z = *(const short8*)(qr + d);
      qf[kk] = __builtin_bit_cast(bf16x8, z);
    }
  }
  float m_run = NEG, l_run = 0.f;
  f32x16 acc[DV / 32];
#pragma unroll
  for (int t = 0; t < DV / 32; ++t) acc[t] = (f32x16)(0.f);

  auto first_key = [&](int pp) {
    return window > 0 ? max(0, off + pp - window + 1) : 0;
  };
  const int hi_wg = off + min(p0 + NW * QW, sq.n);     // one past the last key
  const int lo_wg = first_key(p0) / KB * KB;
  const int pw0 = p0 + wave * QW, pw1 = min(pw0 + QW, sq.n);  // [pw0, pw1)
  const int hi_w = pw0 < sq.n ? off + pw1 : 0;
  const int lo_w = first_key(pw0);

  short8 kn[NK], vn[NV];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int ch = tid + i * NT, row = ch / (DK / 8), d = ch % (DK / 8) * 8;
      const int t = t0 + row;
      kn[i] = (short8){0, 0, 0, 0, 0, 0, 0, 0};
      if (t < hi_wg && d < QD)
        kn[i] = *(const short8*)(
            d < D ? kv + (ctx0 + t) * kv_w + (int64_t)h * D + d
                  : lat + (ctx0 + t) * lat_w + (lat_w - rot) + (d - D));
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int ch = tid + i * NT, row = ch / (DV / 8), d = ch % (DV / 8) * 8;
      const int t = t0 + row;
      vn[i] = (short8){0, 0, 0, 0, 0, 0, 0, 0};
      if (t < hi_wg && d < V)
        vn[i] = *(const short8*)(kv + (ctx0 + t) * kv_w + (int64_t)H * D +
                                 (int64_t)h * V + d);
    }
  };
  fetch(lo_wg);

  for (int t0 = lo_wg; t0 < hi_wg; t0 += KB) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int ch = tid + i * NT;
      *(short8*)(k_lds + ch / (DK / 8) * KS + ch % (DK / 8) * 8) = kn[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int ch = tid + i * NT;
      *(short8*)(v_lds + ch / (DV / 8) * VS + ch % (DV / 8) * 8) = vn[i];
    }
    __syncthreads();
    if (t0 + KB < hi_wg) fetch(t0 + KB);

#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const int sub = t0 + 32 * half;
      if (sub >= hi_w || sub + 32 <= lo_w) continue;   // wave-uniform
      f32x16 s = (f32x16)(0.f);
#pragma unroll
      for (int kk = 0; kk < DK / 16; ++kk) {
        const bf16x8 kf = *(const bf16x8*)(k_lds + (32 * half + qc) * KS +
                                           kk * 16 + hi * 8);
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[kk], s, 0, 0, 0);
      }
      // scores in units of log2; keys outside the mask drop out
      float x[16], mx = NEG;
      const bool inside = pw1 - pw0 == QW && sub + 31 <= off + pw0 &&
                          sub >= first_key(pw1 - 1);
      if (inside) {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          x[r] = s[r] * scale_log2;
          mx = fmaxf(mx, x[r]);
        }
      } else {
        const int last = active ? off + p : -1, first = first_key(p);
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int t = sub + (r & 3) + 8 * (r >> 2) + 4 * hi;
          x[r] = t <= last && t >= first ? s[r] * scale_log2 : NEG;
          mx = fmaxf(mx, x[r]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      const float mn = fmaxf(m_run, mx);
      // a query without a key so far keeps m at NEG: its exponents are taken
      // against 0 and underflow to 0
      const float base = mn <= NEG * 0.5f ? 0.f : mn;
      const float alpha = __builtin_amdgcn_exp2f(m_run - base);
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        x[r] = __builtin_amdgcn_exp2f(x[r] - base);
        sum += x[r];
      }
      sum += __shfl_xor(sum, 32, WAVE);
      l_run = l_run * alpha + sum;
      if (__any(mn > m_run)) {
#pragma unroll
        for (int t = 0; t < DV / 32; ++t)
#pragma unroll
          for (int e = 0; e < 16; ++e) acc[t][e] *= alpha;
      }
      m_run = mn;

      // P' as B operands: the halves exchange the rows they lack
      unsigned int w[8], y[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        w[i] = pack2(x[2 * i], x[2 * i + 1]);
        y[i] = __shfl_xor((int)w[i], 32, WAVE);
      }
      const uint4v f0 = hi ? (uint4v){y[2], y[3], w[2], w[3]}
                           : (uint4v){w[0], w[1], y[0], y[1]};
      const uint4v f1 = hi ? (uint4v){y[6], y[7], w[6], w[7]}
                           : (uint4v){w[4], w[5], y[4], y[5]};
      const bf16x8 pf[2] = {__builtin_bit_cast(bf16x8, f0),
                            __builtin_bit_cast(bf16x8, f1)};

      // O' += V' P': transposing reads give V' fragments
      const int i16 = lane % 16;
      const int dcol = 16 * ((lane & 31) >> 4) + (i16 % 4) * 4;
#pragma unroll
      for (int t = 0; t < DV / 32; ++t) {
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          const short* a = v_lds +
                           (32 * half + ks * 16 + hi * 8 + i16 / 4) * VS +
                           t * 32 + dcol;
          typedef __attribute__((address_space(3))) short4v lds4;
          const short4v lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)a);
          const short4v up =
              __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)(a + 4 * VS));
          const short8 vf = {lo[0], lo[1], lo[2], lo[3],
                             up[0], up[1], up[2], up[3]};
          acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              __builtin_bit_cast(bf16x8, vf), pf[ks], acc[t], 0, 0, 0);
        }
      }
    }
  }

  if (active) {
    const float inv = 1.f / l_run;
    short* o = out + ((int64_t)(sq.row0 + p) * H + h) * V;
#pragma unroll
    for (int t = 0; t < DV / 32; ++t)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int d = t * 32 + 8 * g + 4 * hi;
        if (d < V)
          *(uint2*)(o + d) =
              make_uint2(pack2(acc[t][4 * g] * inv, acc[t][4 * g + 1] * inv),
                         pack2(acc[t][4 * g + 2] * inv,
                               acc[t][4 * g + 3] * inv));
      }
  }
}

}  // namespace

extern "C" {

// 0 if the sizes have no tiled form
int lds_latent_prefill_ok(int D, int rot, int V, int R) {
  return D % 8 == 0 && rot % 8 == 0 && V % 8 == 0 && R % 8 == 0 &&
         D + rot <= 192 && V <= 128;
}

hipError_t lds_latent_prefill(const void* q, const void* kv, const void* lat,
                              const int32_t* seq_meta, const int32_t* ctx,
                              const int32_t* tiles, int n_tiles, void* out,
                              int H, int D, int rot, int V, int lat_w,
                              int window, float scale, hipStream_t stream) {
  if (n_tiles == 0) return hipSuccess;
  if (n_tiles > 65535 || !lds_latent_prefill_ok(D, rot, V, lat_w - rot))
    return hipErrorInvalidValue;
  const dim3 grid(H, n_tiles), block(NT);
  const float s2 = scale * 1.4426950408889634f;
#define GO(DK, DV)                                                            \
  hipLaunchKernelGGL((latent_prefill_kernel<DK, DV>), grid, block, 0, stream, \
                     (const short*)q, (const short*)kv, (const short*)lat,    \
                     seq_meta, ctx, tiles, (short*)out, H, D, rot, V, lat_w,  \
                     window, s2)
#define GOV(DK)                                                               \
  do {                                                                        \
    if (V <= 64) GO(DK, 64); else GO(DK, 128);                                \
  } while (0)
  const int qd = D + rot;
  if (qd <= 64) GOV(64); else if (qd <= 96) GOV(96);
  else if (qd <= 128) GOV(128); else GOV(192);
#undef GOV
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
