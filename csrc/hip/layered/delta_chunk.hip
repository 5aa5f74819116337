// delta_chunk.hip — the gated delta rule of delta_rule.hip over chunks of 64
// tokens, all in 32-bit on the matrix cores (v_mfma_f32_16x16x4f32).
//
// With G the running sum of log decays inside a chunk (token's own included)
// and S0 the state before it, per head:
//   A[i][j] = sum_d k_i k_j e^(G_i - G_j)   (j < i)
//   P[i][j] = sum_d q_i k_j e^(G_i - G_j)   (j <= i)
//   (I + diag(beta) A) U = diag(beta) (V - (k e^G) S0)
//   O = (q e^G) S0 + P U,   S = e^(G_last) S0 + (k e^(G_last - G))' U
// The exponents are never positive: blocks of 16 tokens off the diagonal take
// the sum before the later block as their reference, blocks on the diagonal
// take every pair by itself. So any decay down to 0 is exact.
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

// workspace of one (chunk, head), floats; KP, VP: sizes rounded up
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

// grid (H, chunks); chunks [n, 2] = first row, tokens
template <typename T, int KP>
__global__ __launch_bounds__(LT) void delta_chunk_local_kernel(
    const float* __restrict__ q, const float* __restrict__ k,
    const float* __restrict__ v, const T* __restrict__ beta, int64_t bstride,
    const T* __restrict__ decay, const float* __restrict__ dt_bias,
    const float* __restrict__ neg_a, const int32_t* __restrict__ chunks,
    float* __restrict__ ws, int KH, int H, int K, int V, int VP) {
  constexpr int LD = KP + 4;          // row stride in LDS
  extern __shared__ float lds[];
  float* kl = lds;                    // [C][LD]
  float* ql = kl + C * LD;
  float* gl = ql + C * LD;            // log decays summed inside blocks
  float* al = gl + C * LD;            // beta A, [C][C + 4]
  float* li = al + C * (C + 4);       // inverse diagonal blocks [4][B][B + 4]
  float* bl = li + 4 * B * (B + 4);   // beta [C]
  const int h = blockIdx.x;
  const int kh = h / (H / KH);
  const int64_t row0 = chunks[2 * blockIdx.y];
  const int n = chunks[2 * blockIdx.y + 1];
  const Work wk = work_at(ws, (int64_t)blockIdx.y * H + h, KP, VP);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int col = lane % 16, g4 = 4 * (lane / 16);

  // ---- load; rows and channels past the end are zero ----
  for (int i = tid; i < C * KP; i += LT) {
    const int t = i / KP, d = i % KP;
    float kv = 0.f, qv = 0.f, lg = 0.f;
    if (t < n && d < K) {
      const int64_t at = ((row0 + t) * KH + kh) * K + d;
      kv = k[at];
      qv = q[at];
      lg = neg_a[h] * softplus_f(ld(decay + ((row0 + t) * H + h) * K + d) +
                                 dt_bias[(int64_t)h * K + d]);
    }
    kl[t * LD + d] = kv;
    ql[t * LD + d] = qv;
    gl[t * LD + d] = lg;
  }
  if (tid < C)
    bl[tid] = tid < n ? sigmoid_f(ld(beta + (row0 + tid) * bstride + h)) : 0.f;
  for (int i = tid; i < C * (C + 4); i += LT) al[i] = 0.f;
  __syncthreads();
  // ---- running sums inside blocks of 16: differences of small sums stay
  // exact where a chunk's whole sum would have swallowed them ----
  for (int i = tid; i < 4 * KP; i += LT) {
    float* c = gl + (i / KP) * B * LD + i % KP;
    float s = 0.f;
    for (int t = 0; t < B; ++t) {
      s += c[t * LD];
      c[t * LD] = s;
    }
  }
  __syncthreads();
  // sum over the blocks b0 <= b < b1
  auto blocks = [&](int b0, int b1, int d) {
    float s = 0.f;
    for (int b = b0; b < b1; ++b) s += gl[(b * B + B - 1) * LD + d];
    return s;
  };

  // ---- diagonal blocks, pair by pair: 8 threads share token i ----
  {
    constexpr int DS = KP / 8;        // channels per thread, 4 at a time
    const int i = tid / 8, s = tid % 8, b0 = i / B * B;
    const int top = (wave * 8 + 7) % B + b0;   // largest token of the wave
    for (int j = b0; j <= top; ++j) {
      float a = 0.f, p = 0.f;
      if (j <= i) {
#pragma unroll
        for (int d = 0; d < DS; d += 4) {
          const int o = s * 4 + d * 8;
          const float4v gi = *(const float4v*)(gl + i * LD + o);
          const float4v gj = *(const float4v*)(gl + j * LD + o);
          const float4v ki = *(const float4v*)(kl + i * LD + o);
          const float4v kj = *(const float4v*)(kl + j * LD + o);
          const float4v qi = *(const float4v*)(ql + i * LD + o);
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            const float e = __expf(gi[x] - gj[x]) * kj[x];
            a += ki[x] * e;
            p += qi[x] * e;
          }
        }
      }
#pragma unroll
      for (int o = 1; o < 8; o *= 2) {
        a += __shfl_xor(a, o, WAVE);
        p += __shfl_xor(p, o, WAVE);
      }
      if (s == 0) {
        if (j < i) al[i * (C + 4) + j] = bl[i] * a;
        wk.p[i * C + j] = j <= i ? p : 0.f;
      }
    }
    if (s == 0)
      for (int j = top + 1; j < b0 + B; ++j) wk.p[i * C + j] = 0.f;
  }

  // ---- blocks below the diagonal: one wave each ----
  if (wave < 6) {
    const int bi = wave < 1 ? 1 : wave < 3 ? 2 : 3;
    const int bj = wave - bi * (bi - 1) / 2;
    const int i = bi * B + col, j = bj * B + col;
    float4v a = {0.f, 0.f, 0.f, 0.f}, p = a;
#pragma unroll
    for (int t = 0; t < KP / 16; ++t) {
      const int o = 16 * t + g4;
      // sum from token j to the end of block bi - 1
      float4v gr = {0.f, 0.f, 0.f, 0.f};
      for (int b = bj; b < bi; ++b)
        gr += *(const float4v*)(gl + (b * B + B - 1) * LD + o);
      const float4v gi = *(const float4v*)(gl + i * LD + o);
      const float4v gj = *(const float4v*)(gl + j * LD + o);
      const float4v ki = *(const float4v*)(kl + i * LD + o);
      const float4v kj = *(const float4v*)(kl + j * LD + o);
      const float4v qi = *(const float4v*)(ql + i * LD + o);
      float4v ka, qa, kb;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float e = __expf(gi[x]);
        ka[x] = ki[x] * e;
        qa[x] = qi[x] * e;
        kb[x] = kj[x] * __expf(gr[x] - gj[x]);
      }
      a = mfma4(ka, kb, a);
      p = mfma4(qa, kb, p);
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int row = bi * B + g4 + x;
      al[row * (C + 4) + bj * B + col] = bl[row] * a[x];
      wk.p[row * C + bj * B + col] = p[x];
    }
  }
  __syncthreads();

  // ---- inverses of the unit lower triangular diagonal blocks ----
  if (wave < 4 && lane < B) {
    const float* a = al + wave * B * (C + 4) + wave * B;
    float x[B];
#pragma unroll
    for (int i = 0; i < B; ++i) {
      float s = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s -= a[i * (C + 4) + j] * x[j];
      x[i] = s;
      li[(wave * B + i) * (B + 4) + lane] = s;
    }
  }
  // ---- scaled q and k for the scan ----
  for (int i = tid; i < C * KP; i += LT) {
    const int t = i / KP, d = i % KP;
    wk.qe[i] = ql[t * LD + d] * __expf(blocks(0, t / B, d) + gl[t * LD + d]);
    const int d2 = i / C, t2 = i % C;
    wk.kt[i] = kl[t2 * LD + d2] *
               __expf(blocks(t2 / B, 4, d2) - gl[t2 * LD + d2]);
  }
  for (int d = tid; d < KP; d += LT) wk.gl[d] = __expf(blocks(0, 4, d));
  __syncthreads();

  // ---- forward substitution by blocks, 16 columns of [V | K] at a time ----
  for (int tile = wave; tile < (VP + KP) / 16; tile += LT / WAVE) {
    const bool is_v = tile < VP / 16;
    const int c = (is_v ? tile : tile - VP / 16) * 16 + col;
    float4v x[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      float4v acc;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = b * B + g4 + r;
        float f = 0.f;
        if (is_v) {
          if (t < n && c < V) f = v[((row0 + t) * H + h) * V + c];
        } else {
          f = -kl[t * LD + c] * __expf(blocks(0, b, c) + gl[t * LD + c]);
        }
        acc[r] = bl[t] * f;
      }
#pragma unroll
      for (int p = 0; p < b; ++p) {
        const float4v a = *(const float4v*)(al + (b * B + col) * (C + 4) +
                                            p * B + g4);
        acc = mfma4(-a, x[p], acc);
      }
      const float4v inv =
          *(const float4v*)(li + (b * B + col) * (B + 4) + g4);
      x[b] = mfma4(inv, acc, (float4v){0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = b * B + g4 + r;
        if (is_v)
          wk.u0[t * VP + c] = x[b][r];
        else
          wk.w[t * KP + c] = x[b][r];     // -W
      }
    }
  }
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

  for (int t0 = 0; t0 < n; t0 += C) {
    const Work wk = work_at(ws, (chunk0 + t0 / C) * H + h, KP, VP);
    const int tw = wave * B;          // this wave's 16 tokens
    float4v w[KT], qe[KT];
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      w[t] = *(const float4v*)(wk.w + (tw + col) * KP + 16 * t + g4);
      qe[t] = *(const float4v*)(wk.qe + (tw + col) * KP + 16 * t + g4);
    }
    float4v u;
#pragma unroll
    for (int r = 0; r < 4; ++r) u[r] = wk.u0[(tw + g4 + r) * VP + c];
    float4v o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      u = mfma4(w[t], S[t], u);
      o = mfma4(qe[t], S[t], o);
    }
    u_lds[wave][lane] = u;
    // the state update's operands while the others finish
    constexpr int MY = (KT + 3) / 4;
    float4v kt[MY][4], decay[MY];
#pragma unroll
    for (int i = 0; i < MY; ++i) {
      const int t = wave + 4 * i;
      if (t < KT) {
#pragma unroll
        for (int x = 0; x < 4; ++x)
          kt[i][x] =
              *(const float4v*)(wk.kt + (16 * t + col) * C + 16 * x + g4);
        decay[i] = *(const float4v*)(wk.gl + 16 * t + g4);
      }
    }
    __syncthreads();
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
      if (x <= wave) {
        const float4v p =
            *(const float4v*)(wk.p + (tw + col) * C + 16 * x + g4);
        o = mfma4(p, us[x], o);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = t0 + tw + g4 + r;
      if (t < n && c < V) out[((row0 + t) * H + h) * V + c] = o[r];
    }
    __syncthreads();
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

// out = o / rms(o) * w * sigmoid(gate) per head; one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_gate_kernel(
    const float* __restrict__ o, const T* __restrict__ gate,
    const float* __restrict__ norm_w, T* __restrict__ out, int64_t n, int V,
    float eps) {
  const int64_t i = (int64_t)blockIdx.x * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  if (i >= n) return;
  float ss = 0.f;
  for (int d = lane; d < V; d += WAVE) ss += o[i * V + d] * o[i * V + d];
  const float inv = 1.f / sqrtf(wave_reduce_sum(ss) / (float)V + eps);
  for (int d = lane; d < V; d += WAVE)
    st(out + i * V + d,
       o[i * V + d] * inv * norm_w[d] * sigmoid_f(ld(gate + i * V + d)));
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
  const size_t lds = (3 * C * (KP + 4) + C * (C + 4) + 4 * B * (B + 4) + C) *
                     sizeof(float);
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
  const dim3 grid((uint32_t)((n + 3) / 4)), block(256);
  if (f32)
    hipLaunchKernelGGL(delta_gate_kernel<float>, grid, block, 0, stream, o,
                       (const float*)gate, norm_w, (float*)out, n, V, eps);
  else
    hipLaunchKernelGGL(delta_gate_kernel<short>, grid, block, 0, stream, o,
                       (const short*)gate, norm_w, (short*)out, n, V, eps);
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
