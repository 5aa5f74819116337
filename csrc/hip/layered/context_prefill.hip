// context_prefill.hip — causal (windowed) prefill attention of long portions
// (bf16). A tile is 128 rows of (query, head): all heads of a key/value head
// share its tiles of keys. Keys and values come from
//   pages        grouped heads: cache rows [key | value], found through the
//                block table a tile ahead
//   context rows latent attention: keys and values expanded from the latents
//                of everything a portion may see, the rotated key part shared
//                by all heads; a sequence's context row 0 sits at ctx.pos0
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

struct Prefill {
  const short* q;
  int64_t q_row;             // rows of q, heads D + rot apart
  // context rows: key columns [0, D) at ka, the rest at kb, values at v
  const short *ka, *kb, *v;
  int64_t ka_tok, ka_head, kb_tok, v_tok, v_head;
  const int32_t* ctx;        // [n_seqs, 2] = first context row, its position
  // pages: rows of D + V elements from ka on
  const int32_t* block_tables;
  int max_blocks, bs;
  int64_t page, head;        // strides of a page and of a head inside it
  const int32_t *seq_meta, *tiles;  // tiles [n, 2] = sequence, first query
  short* out;                // [rows, H V]
  int H, rep, D, rot, V, window;
  float scale_log2, sink;    // sink: score (log2) of a key without a value
  int has_sink;
};

// grid (key/value heads, tiles)
template <int DK, int DV, bool PAGED>
__global__ __launch_bounds__(NT, DK + DV > 320 ? 1 : 2)
void context_prefill_kernel(const Prefill a_) {
  constexpr int KS = DK + 8, VS = DV + 32;      // row strides in LDS (shorts)
  constexpr int NK = DK / 32, NV = DV / 32;     // 16-byte pieces per thread
  extern __shared__ short lds[];
  short* k_lds = lds;                           // [KB][KS]
  short* v_lds = lds + KB * KS;                 // [KB][VS]
  const int kvh = blockIdx.x, rep = a_.rep;
  const int seq = a_.tiles[2 * blockIdx.y], p0 = a_.tiles[2 * blockIdx.y + 1];
  const Seq sq = load_seq(a_.seq_meta, seq);
  const int64_t ctx0 = PAGED ? 0 : a_.ctx[2 * seq];
  // query p sees keys <= off + p
  const int off = PAGED ? sq.prior : sq.prior - a_.ctx[2 * seq + 1];
  const int32_t* bt =
      PAGED ? a_.block_tables + (int64_t)seq * a_.max_blocks : nullptr;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int qc = lane & 31, hi = lane >> 5;
  const int nq = NW * QW / rep;                 // queries per tile
  const int vr = wave * QW + qc;                // row of the tile
  const int p_last = min(p0 + nq, sq.n) - 1;
  const bool active = vr / rep < nq && p0 + vr / rep < sq.n;
  const int p = active ? p0 + vr / rep : p_last;
  const int h = kvh * rep + vr % rep;
  const int QD = a_.D + a_.rot, D = a_.D, V = a_.V, bs = a_.bs;
  const int window = a_.window;

  bf16x8 qf[DK / 16];
  {
    const short* qr = a_.q + (sq.row0 + p) * a_.q_row + h * QD;
#pragma unroll
    for (int kk = 0; kk < DK / 16; ++kk) {
      const int d = kk * 16 + hi * 8;
      short8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < QD) z = *(const short8*)(qr + d);
      qf[kk] = __builtin_bit_cast(bf16x8, z);
    }
  }
  float m_run = a_.has_sink ? a_.sink : NEG, l_run = a_.has_sink ? 1.f : 0.f;
  f32x16 acc[DV / 32];
#pragma unroll
  for (int t = 0; t < DV / 32; ++t) acc[t] = (f32x16)(0.f);

  auto first_key = [&](int pp) {
    return window > 0 ? max(0, off + pp - window + 1) : 0;
  };
  const int hi_wg = off + p_last + 1;           // one past the last key
  const int lo_wg = first_key(p0) / KB * KB;
  // queries of this wave: [pw0, pw1]
  const int pw0 = p0 + wave * QW / rep;
  const int pw1 = min(p0 + (wave * QW + QW - 1) / rep, p_last);
  const int hi_w = pw0 <= p_last ? off + pw1 + 1 : 0;
  const int lo_w = first_key(pw0);

  short8 kn[NK], vn[NV];
  int kp[PAGED ? NK : 1], vp[PAGED ? NV : 1];   // pages of a tile
  auto find = [&](int t0) {
    if constexpr (PAGED) {
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int t = t0 + (tid + i * NT) / (DK / 8);
        kp[i] = t < hi_wg ? bt[t / bs] : 0;
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int t = t0 + (tid + i * NT) / (DV / 8);
        vp[i] = t < hi_wg ? bt[t / bs] : 0;
      }
    }
  };
  auto page_row = [&](int page, int t) {
    return a_.ka + page * a_.page + kvh * a_.head + t % bs * (D + V);
  };
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int ch = tid + i * NT, row = ch / (DK / 8), d = ch % (DK / 8) * 8;
      const int t = t0 + row;
      kn[i] = (short8){0, 0, 0, 0, 0, 0, 0, 0};
      if (t < hi_wg && d < QD) {
        if constexpr (PAGED)
          kn[i] = *(const short8*)(page_row(kp[i], t) + d);
        else
          kn[i] = *(const short8*)(
              d < D ? a_.ka + (ctx0 + t) * a_.ka_tok + kvh * a_.ka_head + d
                    : a_.kb + (ctx0 + t) * a_.kb_tok + (d - D));
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int ch = tid + i * NT, row = ch / (DV / 8), d = ch % (DV / 8) * 8;
      const int t = t0 + row;
      vn[i] = (short8){0, 0, 0, 0, 0, 0, 0, 0};
      if (t < hi_wg && d < V) {
        if constexpr (PAGED)
          vn[i] = *(const short8*)(page_row(vp[i], t) + D + d);
        else
          vn[i] = *(const short8*)(a_.v + (ctx0 + t) * a_.v_tok +
                                   kvh * a_.v_head + d);
      }
    }
  };
  find(lo_wg);
  fetch(lo_wg);
  find(lo_wg + KB);

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
    if (t0 + KB < hi_wg) {
      fetch(t0 + KB);
      find(t0 + 2 * KB);
    }

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
      const bool inside =
          sub + 31 <= off + pw0 && sub >= first_key(pw1);
      if (inside) {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          x[r] = s[r] * a_.scale_log2;
          mx = fmaxf(mx, x[r]);
        }
      } else {
        const int last = off + p, first = first_key(p);
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int t = sub + (r & 3) + 8 * (r >> 2) + 4 * hi;
          x[r] = t <= last && t >= first ? s[r] * a_.scale_log2 : NEG;
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
    short* o = a_.out + ((int64_t)(sq.row0 + p) * a_.H + h) * V;
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

template <int DK, int DV, bool PAGED>
hipError_t launch(const Prefill& a, int kv_heads, int n_tiles,
                  hipStream_t stream) {
  const int lds = KB * (DK + 8 + DV + 32) * (int)sizeof(short);
  auto fn = context_prefill_kernel<DK, DV, PAGED>;
  hipError_t e = hipFuncSetAttribute(
      (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  if (e != hipSuccess) return e;
  hipLaunchKernelGGL(fn, dim3(kv_heads, n_tiles), dim3(NT), lds, stream, a);
  HIP_CHECK_LAST();
  return hipSuccess;
}

constexpr float LOG2E = 1.4426950408889634f;

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
  Prefill a{};
  a.q = (const short*)q;
  a.q_row = (int64_t)H * (D + rot);
  a.ka = (const short*)kv;
  a.kb = (const short*)lat + lat_w - rot;
  a.v = (const short*)kv + (int64_t)H * D;
  a.ka_tok = a.v_tok = (int64_t)H * (D + V);
  a.ka_head = D;
  a.kb_tok = lat_w;
  a.v_head = V;
  a.ctx = ctx;
  a.bs = 1;
  a.seq_meta = seq_meta;
  a.tiles = tiles;
  a.out = (short*)out;
  a.H = H;
  a.rep = 1;
  a.D = D;
  a.rot = rot;
  a.V = V;
  a.window = window;
  a.scale_log2 = scale * LOG2E;
  const int qd = D + rot;
#define GO(DK)                                                                \
  return V <= 64 ? launch<DK, 64, false>(a, H, n_tiles, stream)               \
                 : launch<DK, 128, false>(a, H, n_tiles, stream)
  if (qd <= 64) GO(64);
  if (qd <= 96) GO(96);
  if (qd <= 128) GO(128);
  GO(192);
#undef GO
}

int lds_grouped_prefill_ok(int D, int V, int rep, int64_t q_stride) {
  return D % 8 == 0 && V % 8 == 0 && q_stride % 8 == 0 && D <= 256 &&
         V <= 256 && rep <= NW * QW;
}

// q: first query of row 0, rows q_stride apart; cache [NB, G, bs, D + V];
// tiles hold 128 / (H / G) queries; out [rows, H V]
hipError_t lds_grouped_prefill(const void* q, int64_t q_stride,
                               const void* cache, const int32_t* block_tables,
                               int max_blocks, int bs,
                               const int32_t* seq_meta, const int32_t* tiles,
                               int n_tiles, void* out, int H, int G, int D,
                               int V, float scale, int has_sink, float sink,
                               hipStream_t stream) {
  if (n_tiles == 0) return hipSuccess;
  if (n_tiles > 65535 || !lds_grouped_prefill_ok(D, V, H / G, q_stride))
    return hipErrorInvalidValue;
  Prefill a{};
  a.q = (const short*)q;
  a.q_row = q_stride;
  a.ka = (const short*)cache;
  a.block_tables = block_tables;
  a.max_blocks = max_blocks;
  a.bs = bs;
  a.head = (int64_t)bs * (D + V);
  a.page = G * a.head;
  a.seq_meta = seq_meta;
  a.tiles = tiles;
  a.out = (short*)out;
  a.H = H;
  a.rep = H / G;
  a.D = D;
  a.V = V;
  a.scale_log2 = scale * LOG2E;
  a.has_sink = has_sink;
  a.sink = sink * LOG2E;
#define GO(DK)                                                                \
  return V <= 64    ? launch<DK, 64, true>(a, G, n_tiles, stream)             \
         : V <= 128 ? launch<DK, 128, true>(a, G, n_tiles, stream)            \
                    : launch<DK, 256, true>(a, G, n_tiles, stream)
  if (D <= 64) GO(64);
  if (D <= 128) GO(128);
  if (D <= 192) GO(192);
  GO(256);
#undef GO
}

}  // extern "C"
