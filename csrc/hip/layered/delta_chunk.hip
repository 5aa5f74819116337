// delta_chunk.hip — the gated delta rule of delta_rule.hip over chunks of 64
// tokens, all in 32-bit on the matrix cores (v_mfma_f32_16x16x4f32).
//
// With G the running sum of log decays inside a chunk (token's own included)
// and S0 the state before it, per head:
//   A[i][j] = sum_d k_i k_j e^(G_i - G_j)   (j < i)
//   P[i][j] = sum_d q_i k_j e^(G_i - G_j)   (j <= i)
//   (I + diag(beta) A) U = diag(beta) (V - (k e^G) S0)
//   O = (q e^G) S0 + P U,   S = e^(G_last) S0 + (k e^(G_last - G))' U
// A and P are products of scaled rows, in blocks of 16 tokens. Off the diagonal
// the sum before the later block is the reference, so no exponent is positive.
// On the diagonal it is the block's middle, as long as no channel decays by
// more than e^-DECAY_LIMIT inside a block; else every pair is taken by itself.
// So any decay down to 0 is right.
//
// delta_chunk_local  everything that does not need S0, one workgroup per
//                    (head, chunk): U0 and W with U = U0 - W S0, P, the
//                    scaled q and k -> workspace
// delta_chunk_scan   one workgroup per (head, 16 columns of S, sequence)
//                    walks the chunks with S in registers
// delta_gate         gated output norm
//
// MFMA operands: lane l gives A[l % 16][k] and B[k][l % 16] with k = l / 16,
// and holds D[4 (l / 16) + r][l % 16] in register r. Taking k = 4 (l / 16) + r
// in step r instead makes a D tile usable as B as it is, and an A operand one
// 16-byte read per four steps.
#include "elem.h"

namespace {

constexpr int C = 64;       // tokens per chunk
constexpr int B = 16;       // tokens per block
constexpr int LT = 512;     // threads of delta_chunk_local
constexpr int ST = 256;     // threads of delta_chunk_scan

__device__ __forceinline__ float4v mfma4(float4v a, float4v b, float4v c) {
#pragma unroll
  for (int r = 0; r < 4; ++r)
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], c, 0, 0, 0);
  return c;
}

// Workspace of one (chunk, head), floats; KP, VP: sizes rounded up. All but
// gl are 16 x 16 tiles in operand order (256 floats, 4 per lane: the scan
// reads a kilobyte per instruction):
//   u0 [VP / 16][4]       D: lane (c, g) holds tokens 4 g .. of channel c
//   w, qe [4][KP / 16]    A: lane (t, g) holds channels 4 g .. of token t
//   kt [KP / 16][4]       A: lane (c, g) holds tokens 4 g .. of channel c
//   p [4][4]              A: lane (t, g) holds columns 4 g .. of token t
struct Work {
  float *u0, *w, *qe, *kt, *p, *gl;
};
__host__ __device__ __forceinline__ int64_t work_size(int KP, int VP) {
  return (int64_t)C * VP + 3 * C * KP + C * C + KP;
}
__device__ __forceinline__ Work work_at(float* ws, int64_t i, int KP, int VP) {
  float* p = ws + i * work_size(KP, VP);
  return {p, p + C * VP, p + C * VP + C * KP, p + C * VP + 2 * C * KP,
          p + C * VP + 3 * C * KP, p + C * VP + 3 * C * KP + C * C};
}

// 4 channels from p, of which the first `left` exist; `whole` rows only hold
// multiples of 4 (and are aligned)
__device__ __forceinline__ float4v load4(const float* p, int left,
                                         bool whole) {
  float4v f = {0.f, 0.f, 0.f, 0.f};
  if (whole) {
    if (left > 0) f = *(const float4v*)p;
  } else {
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (x < left) f[x] = p[x];
  }
  return f;
}
__device__ __forceinline__ float4v load4(const short* p, int left,
                                         bool whole) {
  float4v f = {0.f, 0.f, 0.f, 0.f};
  if (whole) {
    if (left > 0) {
      const short4v v = *(const short4v*)p;
#pragma unroll
      for (int x = 0; x < 4; ++x) f[x] = bf16_to_f32(v[x]);
    }
  } else {
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (x < left) f[x] = bf16_to_f32(p[x]);
  }
  return f;
}

constexpr float DECAY_LIMIT = 24.f;
constexpr int AB = B * (B + 4);     // one 16 x 16 block of beta A in LDS
__device__ __forceinline__ int block_at(int bi, int bj) {
  return (bi * (bi + 1) / 2 + bj) * AB;
}

// grid (H, chunks); chunks [n, 2] = first row, tokens. Everything the waves
// share goes through LDS (80 KB: two workgroups per CU), so its barriers let
// global loads and stores run on.
template <typename T, int KP>
__global__ __launch_bounds__(LT, 4) void delta_chunk_local_kernel(
    const float* __restrict__ q, const float* __restrict__ k,
    const float* __restrict__ v, const T* __restrict__ beta, int64_t bstride,
    const T* __restrict__ decay, const float* __restrict__ dt_bias,
    const float* __restrict__ neg_a, const int32_t* __restrict__ chunks,
    float* __restrict__ ws, int KH, int H, int K, int V, int VP) {
  constexpr int LD = KP + 4;          // row stride in LDS
  extern __shared__ float lds[];
  float* kl = lds;                    // [C][LD]
  float* gl = kl + C * LD;            // log decays summed inside blocks
  float* al = gl + C * LD;            // beta A, lower blocks; the diagonal
                                      // ones become their inverses
  float* bl = al + 10 * AB;           // beta [C]
  int* steep = (int*)(bl + C);        // per wave: a block decays too much
  const int h = blockIdx.x;
  const int kh = h / (H / KH);
  const int64_t row0 = chunks[2 * blockIdx.y];
  const int n = chunks[2 * blockIdx.y + 1];
  const Work wk = work_at(ws, (int64_t)blockIdx.y * H + h, KP, VP);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int col = lane % 16, g4 = 4 * (lane / 16);
  // bases of this chunk and head; offsets from them fit 32 bits
  const float* kc = k + (row0 * KH + kh) * K;
  const float* qc = q + (row0 * KH + kh) * K;
  const float* vc = v + (row0 * H + h) * V;
  const T* dc = decay + (row0 * H + h) * K;
  const unsigned krow = KH * K, drow = H * K, vrow = H * V;
  const bool whole = K % 4 == 0;

  // ---- load; rows and channels past the end are zero. All loads of a
  // thread are under way before the first is used ----
  constexpr int Q4 = C * KP / 4 / LT;            // groups of 4 channels
  const int di = tid / 8, ds = tid % 8;          // diagonal part: token, slice
  constexpr int DS = KP / 32;                    // its groups of 4 channels
  {
    float4v kr[Q4], dr[Q4], bias[Q4];
#pragma unroll
    for (int i = 0; i < Q4; ++i) {
      const unsigned t = (tid + i * LT) / (KP / 4),
                     d = (tid + i * LT) % (KP / 4) * 4;
      const int left = (int)t < n ? K - (int)d : 0;
      kr[i] = load4(kc + t * krow + d, left, whole);
      dr[i] = load4(dc + t * drow + d, left, whole);
      bias[i] = load4(dt_bias + (int64_t)h * K + d, left, whole);
    }
    const float na = neg_a[h];
#pragma unroll
    for (int i = 0; i < Q4; ++i) {
      const int t = (tid + i * LT) / (KP / 4), d = (tid + i * LT) % (KP / 4) * 4;
      float4v gv;
#pragma unroll
      for (int x = 0; x < 4; ++x)
        gv[x] = t < n && d + x < K ? na * softplus_f(dr[i][x] + bias[i][x])
                                   : 0.f;
      *(float4v*)(kl + t * LD + d) = kr[i];
      *(float4v*)(gl + t * LD + d) = gv;
    }
  }
  if (tid < C)
    bl[tid] = tid < n ? sigmoid_f(ld(beta + (row0 + tid) * bstride + h)) : 0.f;
  lds_barrier();
  // ---- running sums inside blocks of 16: differences of small sums stay
  // exact where a chunk's whole sum would have swallowed them ----
  static_assert(4 * KP <= LT, "one pass");
  bool over = false;
  for (int i = tid; i < 4 * KP; i += LT) {
    float* c = gl + (i / KP) * B * LD + i % KP;
    float x[B];
#pragma unroll
    for (int t = 0; t < B; ++t) x[t] = c[t * LD];
#pragma unroll
    for (int t = 1; t < B; ++t) {
      x[t] += x[t - 1];
      c[t * LD] = x[t];
    }
    over = x[B - 1] < -DECAY_LIMIT;
  }
  {
    const bool any = __any(over);
    if (lane == 0) steep[wave] = any;
  }
  lds_barrier();
  bool slow = false;
#pragma unroll
  for (int w = 0; w < LT / WAVE; ++w) slow |= steep[w] != 0;
  // sum over the blocks b0 <= b < b1
  auto blocks = [&](int b0, int b1, int d) {
    float s = 0.f;
    for (int b = b0; b < b1; ++b) s += gl[(b * B + B - 1) * LD + d];
    return s;
  };

  // ---- blocks of A (to LDS) and P: one wave each, bi >= bj ----
  auto block_pair = [&](int bi, int bj) -> float4v {
    const int i = bi * B + col, j = bj * B + col;
    float4v qo[KP / 16];
#pragma unroll
    for (int t = 0; t < KP / 16; ++t)
      qo[t] = load4(qc + i * krow + 16 * t + g4, i < n ? K - 16 * t - g4 : 0,
                    whole);
    float4v a = {0.f, 0.f, 0.f, 0.f}, p = a;
#pragma unroll
    for (int t = 0; t < KP / 16; ++t) {
      const int o = 16 * t + g4;
      const float4v gi = *(const float4v*)(gl + i * LD + o);
      const float4v gj = *(const float4v*)(gl + j * LD + o);
      const float4v ki = *(const float4v*)(kl + i * LD + o);
      const float4v kj = *(const float4v*)(kl + j * LD + o);
      // reference as seen from block bi and from block bj
      float4v ri = {0.f, 0.f, 0.f, 0.f}, rj = ri;
      if (bi == bj)
        ri = rj = *(const float4v*)(gl + (bi * B + B / 2) * LD + o);
      for (int b = bj; b < bi; ++b)
        rj += *(const float4v*)(gl + (b * B + B - 1) * LD + o);
      float4v ka, qa, kb;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float e = __expf(gi[x] - ri[x]);
        ka[x] = ki[x] * e;
        qa[x] = qo[t][x] * e;
        kb[x] = kj[x] * __expf(rj[x] - gj[x]);
      }
      a = mfma4(ka, kb, a);
      p = mfma4(qa, kb, p);
      __builtin_amdgcn_sched_barrier(0);   // keep the reads of later steps
    }                                      // from taking all registers
    float* ab = al + block_at(bi, bj);
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int r = g4 + x;
      if (bi == bj && col > r) p[x] = 0.f;
      ab[r * (B + 4) + col] =
          bi == bj && col >= r ? 0.f : bl[bi * B + r] * a[x];
    }
    return p;
  };
  float4v p0 = {0.f, 0.f, 0.f, 0.f}, p1 = p0;
  const int bi = wave < 1 ? 1 : wave < 3 ? 2 : wave < 6 ? 3 : 2 * (wave - 6);
  const int bj = wave < 6 ? wave - bi * (bi - 1) / 2 : bi;
  if (wave < 6 || !slow) p0 = block_pair(bi, bj);
  if (wave >= 6 && !slow) p1 = block_pair(bi + 1, bj + 1);

  // ---- diagonal blocks pair by pair: 8 threads share token i ----
  float pk[2] = {0.f, 0.f};          // this thread's share of P's row
  if (slow) {
    const int i = di, s = ds, b0 = i / B * B;
    const int top = (wave * 8 + 7) % B + b0;   // largest token of the wave
    float4v gi[DS], ki[DS], qi[DS];
#pragma unroll
    for (int d = 0; d < DS; ++d) {
      gi[d] = *(const float4v*)(gl + i * LD + s * 4 + d * 32);
      ki[d] = *(const float4v*)(kl + i * LD + s * 4 + d * 32);
      qi[d] = load4(qc + i * krow + s * 4 + d * 32,
                    i < n ? K - s * 4 - d * 32 : 0, whole);
    }
    const float beta_i = bl[i];
    float* ab = al + block_at(i / B, i / B) + (i % B) * (B + 4);
#pragma unroll 1
    for (int j = b0; j < b0 + B; ++j) {
      float a = 0.f, p = 0.f;
      if (j <= top) {                // wave-uniform
#pragma unroll
        for (int d = 0; d < DS; ++d) {
          const float4v gj = *(const float4v*)(gl + j * LD + s * 4 + d * 32);
          const float4v kj = *(const float4v*)(kl + j * LD + s * 4 + d * 32);
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            // pairs with j > i are thrown away below; their exponent is cut
            const float e = __expf(fminf(gi[d][x] - gj[x], 0.f)) * kj[x];
            a += ki[d][x] * e;
            p += qi[d][x] * e;
          }
        }
#pragma unroll
        for (int o = 1; o < 8; o *= 2) {
          a += __shfl_xor(a, o, WAVE);
          p += __shfl_xor(p, o, WAVE);
        }
      }
      if (s == 0) ab[j - b0] = j < i ? beta_i * a : 0.f;
      p = j <= i ? p : 0.f;
      if (j - b0 == 2 * s) pk[0] = p;
      if (j - b0 == 2 * s + 1) pk[1] = p;
    }
  }
  lds_barrier();

  // ---- inverses of the unit lower triangular diagonal blocks, in place (a
  // step reads row i before it writes row i; lanes run in step) ----
  if (wave < 4 && lane < B) {
    float* a = al + block_at(wave, wave);
    float x[B];
#pragma unroll
    for (int i = 0; i < B; ++i) {
      float s = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s -= a[i * (B + 4) + j] * x[j];
      x[i] = s;
      a[i * (B + 4) + lane] = s;
    }
  }
  // Loads wait for the stores issued before them, so this wave's first tile
  // of v comes now and every store after it.
  float4v vpre[4];
#pragma unroll
  for (int b = 0; b < 4; ++b)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = b * B + g4 + r, c = wave * 16 + col;
      vpre[b][r] = t < n && c < V ? vc[t * vrow + c] : 0.f;
    }
  // its share of q too
  float4v qr[Q4];
#pragma unroll
  for (int i = 0; i < Q4; ++i) {
    const int tile = wave + i * (LT / WAVE);
    const int t = tile / (KP / 16) * 16 + col, d = tile % (KP / 16) * 16 + g4;
    qr[i] = load4(qc + t * krow + d, t < n ? K - d : 0, whole);
  }
  lds_barrier();

  // ---- forward substitution by blocks, 16 columns of [V | K] at a time ----
  for (int tile = wave; tile < (VP + KP) / 16; tile += LT / WAVE) {
    const bool is_v = tile < VP / 16;            // wave-uniform
    const int c = (is_v ? tile : tile - VP / 16) * 16 + col;
    float4v f[4], x[4];
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = b * B + g4 + r;
        if (is_v)
          f[b][r] = tile == wave         ? vpre[b][r]
                    : t < n && c < V     ? vc[t * vrow + c]
                                         : 0.f;
        else
          f[b][r] = -kl[t * LD + c] * __expf(blocks(0, b, c) + gl[t * LD + c]);
      }
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      float4v acc = *(const float4v*)(bl + b * B + g4) * f[b];
#pragma unroll
      for (int p = 0; p < b; ++p) {
        const float4v a =
            *(const float4v*)(al + block_at(b, p) + col * (B + 4) + g4);
        acc = mfma4(-a, x[p], acc);
      }
      const float4v inv =
          *(const float4v*)(al + block_at(b, b) + col * (B + 4) + g4);
      x[b] = mfma4(inv, acc, (float4v){0.f, 0.f, 0.f, 0.f});
      if (is_v) {
        *(float4v*)(wk.u0 + (tile * 4 + b) * 256 + lane * 4) = x[b];
      } else {
        // -W, turned: rows of D are the lanes of A
        float* o = wk.w + (b * (KP / 16) + tile - VP / 16) * 256;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          o[(g4 + r + 16 * (col / 4)) * 4 + col % 4] = x[b][r];
      }
    }
  }

  // ---- P, scaled q and k, the chunk's decay ----
  if (slow) {
    float* o = wk.p + di / B * (4 + 1) * 256;     // tile (b, b)
    typedef __attribute__((ext_vector_type(2))) float f2;
    *(f2*)(o + (di % B + 16 * (ds / 2)) * 4 + ds % 2 * 2) =
        (f2){pk[0], pk[1]};
  }
  if (wave < 6 || !slow) {
    float* o = wk.p + (bi * 4 + bj) * 256;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int at = (g4 + r + 16 * (col / 4)) * 4 + col % 4;
      o[at] = p0[r];
      if (wave >= 6) o[at + 5 * 256] = p1[r];     // the next diagonal tile
    }
  }
#pragma unroll
  for (int i = 0; i < Q4; ++i) {
    const int tile = wave + i * (LT / WAVE);
    {
      const int t = tile / (KP / 16) * 16 + col,
                d = tile % (KP / 16) * 16 + g4;
      const float4v g = *(const float4v*)(gl + t * LD + d);
      float4v o = qr[i];
      float4v before = {0.f, 0.f, 0.f, 0.f};
      for (int b = 0; b < tile / (KP / 16); ++b)
        before += *(const float4v*)(gl + (b * B + B - 1) * LD + d);
#pragma unroll
      for (int x = 0; x < 4; ++x) o[x] *= __expf(before[x] + g[x]);
      *(float4v*)(wk.qe + tile * 256 + lane * 4) = o;
    }
    {
      const int d = tile / 4 * 16 + col, t = tile % 4 * 16 + g4;
      const float after = blocks(tile % 4, 4, d);
      float4v o;
#pragma unroll
      for (int x = 0; x < 4; ++x)
        o[x] = kl[(t + x) * LD + d] * __expf(after - gl[(t + x) * LD + d]);
      *(float4v*)(wk.kt + tile * 256 + lane * 4) = o;
    }
  }
  for (int d = tid; d < KP; d += LT) wk.gl[d] = __expf(blocks(0, 4, d));
}

// grid (H, VP / 16, sequences); walk [n, 4] = first row, tokens, slot, first
// chunk | (1 << 30 if the state starts at zero)
template <int KT>
__global__ __launch_bounds__(ST) void delta_chunk_scan_kernel(
    float* __restrict__ ws, float* __restrict__ state,  // [slots, H, K, V]
    const int32_t* __restrict__ walk, float* __restrict__ out,  // [rows, H V]
    int H, int K, int V, int VP) {
  constexpr int KP = KT * 16;
  __shared__ float4v s_lds[KT][WAVE], u_lds[4][WAVE];
  const int h = blockIdx.x, lane = threadIdx.x % WAVE;
  const int wave = threadIdx.x / WAVE, col = lane % 16, g4 = 4 * (lane / 16);
  const int c = blockIdx.y * 16 + col;
  const int4 m = ((const int4*)walk)[blockIdx.z];
  const int64_t row0 = m.x;
  const int n = m.y;
  const bool fresh = m.w >> 30;
  const int64_t chunk0 = m.w & ((1 << 30) - 1);
  float* Sp = state + ((int64_t)m.z * H + h) * K * V;

  float4v S[KT];      // every wave has all of its 16 columns
#pragma unroll
  for (int t = 0; t < KT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * t + g4 + r;
      S[t][r] = !fresh && d < K && c < V ? Sp[(int64_t)d * V + c] : 0.f;
    }

  // uniform bases, per-lane offsets that stay the same for every chunk
  const int tw = wave * B;            // this wave's 16 tokens
  const int64_t stride = (int64_t)H * work_size(KP, VP);
  const float* base = ws + (chunk0 * H + h) * work_size(KP, VP);
  const unsigned at_w = wave * KT * 256 + lane * 4, at_g = tw + g4;
  const unsigned at_u = (blockIdx.y * 4 + wave) * 256 + lane * 4;
  const unsigned at_k = wave * 4 * 256 + lane * 4;
  float4v w[KT], qe[KT], u;
  auto fetch = [&](const float* p) {
    const float* pw = p + C * VP;
    const float* pq = pw + C * KP;
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      w[t] = *(const float4v*)(pw + (at_w + 256 * t));
      qe[t] = *(const float4v*)(pq + (at_w + 256 * t));
    }
    u = *(const float4v*)(p + at_u);
  };
  fetch(base);
  float* oc = out + (row0 * H + h) * V;
  const unsigned at_o = (tw + g4) * (H * V) + c, orow = H * V;
  for (int t0 = 0; t0 < n; t0 += C, base += stride, oc += C * orow) {
    // operands of the state update and of P U, used after the first products
    constexpr int MY = (KT + 3) / 4;
    float4v kt[MY][4], decay[MY], p[4];
    const float* pk = base + C * VP + 2 * C * KP;
    const float* pp = pk + C * KP;
    const float* pg = pp + C * C;
#pragma unroll
    for (int i = 0; i < MY; ++i)
      if (wave + 4 * i < KT) {
#pragma unroll
        for (int x = 0; x < 4; ++x)
          kt[i][x] = *(const float4v*)(pk + (at_k + i * 4096 + 256 * x));
        decay[i] = *(const float4v*)(pg + (at_g + i * 4 * B));
      }
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (x <= wave) p[x] = *(const float4v*)(pp + (at_k + 256 * x));
    float4v o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      u = mfma4(w[t], S[t], u);
      o = mfma4(qe[t], S[t], o);
    }
    u_lds[wave][lane] = u;
    // w, qe and u are free now: the next chunk's arrive during the rest
    if (t0 + C < n) fetch(base + stride);
    lds_barrier();
    float4v us[4];
#pragma unroll
    for (int x = 0; x < 4; ++x) us[x] = u_lds[x][lane];
#pragma unroll
    for (int i = 0; i < MY; ++i) {
      const int t = wave + 4 * i;
      if (t < KT) {
        // S[t] with a register index that depends on the wave would spill
        float4v s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int y = 0; y < KT; ++y)
          if (y == t) s = S[y];
        s = s * decay[i];
#pragma unroll
        for (int x = 0; x < 4; ++x) s = mfma4(kt[i][x], us[x], s);
        s_lds[t][lane] = s;
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      if (x <= wave) o = mfma4(p[x], us[x], o);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (t0 + tw + g4 + r < n && c < V) oc[at_o + r * orow] = o[r];
    }
    lds_barrier();
#pragma unroll
    for (int t = 0; t < KT; ++t) S[t] = s_lds[t][lane];
  }

  if (wave == 0) {
#pragma unroll
    for (int t = 0; t < KT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * t + g4 + r;
        if (d < K && c < V) Sp[(int64_t)d * V + c] = S[t][r];
      }
  }
}

// out = o / rms(o) * w * sigmoid(gate) per head; LANES threads per (row,
// head), N channels each at a time
template <typename T, int LANES, int N>
__global__ __launch_bounds__(256) void delta_gate_kernel(
    const float* __restrict__ o, const T* __restrict__ gate,
    const float* __restrict__ norm_w, T* __restrict__ out, int64_t n, int V,
    float eps) {
  const int64_t i =
      (int64_t)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  const int lane = threadIdx.x % LANES;
  const bool in = i < n;
  float ss = 0.f;
  if (in)
    for (int d = lane * N; d < V; d += LANES * N) {
      float f[N];
      ldn<N>(o + i * V + d, f);
#pragma unroll
      for (int x = 0; x < N; ++x) ss += f[x] * f[x];
    }
#pragma unroll
  for (int x = LANES / 2; x > 0; x /= 2) ss += __shfl_xor(ss, x, WAVE);
  if (!in) return;
  const float inv = 1.f / sqrtf(ss / (float)V + eps);
  for (int d = lane * N; d < V; d += LANES * N) {
    float f[N], g[N], w[N];
    ldn<N>(o + i * V + d, f);
    ldn<N>(gate + i * V + d, g);
    ldn<N>(norm_w + d, w);
#pragma unroll
    for (int x = 0; x < N; ++x) f[x] = f[x] * inv * w[x] * sigmoid_f(g[x]);
    stn<N>(out + i * V + d, f);
  }
}

int padded_k(int K) { return K <= 32 ? 32 : K <= 64 ? 64 : 128; }

}  // namespace

extern "C" {

// floats of workspace per (chunk, head); 0: sizes without a chunked form
int64_t lds_delta_chunk_work(int K, int V) {
  return K > 128 ? 0 : work_size(padded_k(K), (V + 15) / 16 * 16);
}

hipError_t lds_delta_chunk(int f32, const float* q, const float* k,
                           const float* v, const void* beta, int64_t bstride,
                           const void* decay, const float* dt_bias,
                           const float* neg_a, float* state,
                           const int32_t* chunks, int n_chunks,
                           const int32_t* walk, int n_seqs, float* ws,
                           float* out, int KH, int H, int K, int V,
                           hipStream_t stream) {
  if (n_chunks == 0) return hipSuccess;
  if (K > 128) return hipErrorInvalidValue;
  const int KP = padded_k(K), VP = (V + 15) / 16 * 16;
  const size_t lds =
      (2 * C * (KP + 4) + 10 * AB + C + LT / WAVE) * sizeof(float);
  const dim3 g1(H, n_chunks), g2(H, VP / 16, n_seqs);
#define LOCAL(T, KPV)                                                         \
  do {                                                                        \
    auto fn = delta_chunk_local_kernel<T, KPV>;                               \
    hipError_t e = hipFuncSetAttribute(                                       \
        (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize,          \
        (int)lds);                                                            \
    if (e != hipSuccess) return e;                                            \
    hipLaunchKernelGGL(fn, g1, dim3(LT), lds, stream, q, k, v,                \
                       (const T*)beta, bstride, (const T*)decay, dt_bias,     \
                       neg_a, chunks, ws, KH, H, K, V, VP);                   \
  } while (0)
#define GO(KPV)                                                               \
  do {                                                                        \
    if (f32) LOCAL(float, KPV); else LOCAL(short, KPV);                       \
    hipLaunchKernelGGL(delta_chunk_scan_kernel<KPV / 16>, g2, dim3(ST), 0,    \
                       stream, ws, state, walk, out, H, K, V, VP);            \
  } while (0)
  if (KP == 32) GO(32); else if (KP == 64) GO(64); else GO(128);
#undef GO
#undef LOCAL
  HIP_CHECK_LAST();
  return hipSuccess;
}

hipError_t lds_delta_gate(int f32, const float* o, const void* gate,
                          const float* norm_w, void* out, int64_t n, int V,
                          float eps, hipStream_t stream) {
  if (n == 0) return hipSuccess;
#define GO2(T, L, N)                                                          \
  hipLaunchKernelGGL((delta_gate_kernel<T, L, N>),                            \
                     dim3((uint32_t)((n + 256 / L - 1) / (256 / L))),         \
                     dim3(256), 0, stream, o, (const T*)gate, norm_w,         \
                     (T*)out, n, V, eps)
#define GO(L, N)                                                              \
  do {                                                                        \
    if (f32) GO2(float, L, N); else GO2(short, L, N);                         \
  } while (0)
  if (V % 8 == 0) GO(16, 8); else GO(64, 1);
#undef GO
#undef GO2
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
