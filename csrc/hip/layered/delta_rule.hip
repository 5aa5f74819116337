// delta_rule.hip — gated delta rule with one decay per head and key channel.
//
// Per head, with S [K, V] in 32-bit floats, token by token:
//   S <- diag(g) S;  u = beta (v - S'k);  S <- S + k u';  o = S'q
//
// delta_prep     short causal convolutions + silu of q, k, v; unit norms
// delta_conv     convolution inputs kept for the next step
// delta_step     the recurrence itself, one workgroup per (head, sequence),
//                with gates and the gated output norm (decode, short rows)
// The chunked form for long rows is in delta_chunk.hip.
#include "elem.h"

namespace {

constexpr int NT = 256;
constexpr int NWV = NT / WAVE;
constexpr int MAXU = 8;  // unit norm over up to MAXU * 64 channels

// grid (rows, y): waves share the units of one row. Units: KH of q, KH of k
// (K channels each, unit-normed), H of v (V channels).
template <typename T>
__global__ __launch_bounds__(NT) void delta_prep_kernel(
    const T* __restrict__ proj, int64_t pstride,  // [rows, >= C]
    const float* __restrict__ taps,               // [n_taps, C]
    T* __restrict__ conv_state,                   // [slots, n_taps - 1, C]
    const int32_t* __restrict__ row_seq, const int32_t* __restrict__ seq_meta,
    float* __restrict__ q, float* __restrict__ k, float* __restrict__ v,
    int KH, int H, int K, int V, int n_taps, float q_scale, float unit_eps) {
  const int row = blockIdx.x;
  const int lane = threadIdx.x % WAVE;
  const int wave = threadIdx.x / WAVE + blockIdx.y * NWV;
  const int C = 2 * KH * K + H * V;
  const Seq sq = load_seq(seq_meta, row_seq[row]);
  const int pos = row - sq.row0;
  T* state = conv_state + (int64_t)sq.slot * (n_taps - 1) * C;
  const bool roll = sq.n == 1;  // this thread is the only user of its channel

  for (int unit = wave; unit < 2 * KH + H; unit += NWV * gridDim.y) {
    const bool qk = unit < 2 * KH;
    const int len = qk ? K : V;
    const int c0 = qk ? unit * K : 2 * KH * K + (unit - 2 * KH) * V;
    float* dst = unit < KH ? q + ((int64_t)row * KH + unit) * K
                 : qk      ? k + ((int64_t)row * KH + unit - KH) * K
                           : v + ((int64_t)row * H + unit - 2 * KH) * V;
    float keep[MAXU];
    float ss = 0.f;
    auto channel = [&](int d) {
      const int c = c0 + d;
      float acc = 0.f;
      for (int j = 0; j < n_taps; ++j) {
        const int p = pos - (n_taps - 1) + j;
        float in = 0.f;
        if (p >= 0)
          in = ld(proj + (int64_t)(sq.row0 + p) * pstride + c);
        else if (sq.prior > 0)
          in = ld(state + (int64_t)(n_taps - 1 + p) * C + c);
        if (roll && j > 0) st(state + (int64_t)(j - 1) * C + c, in);
        acc += taps[(int64_t)j * C + c] * in;
      }
      return acc * sigmoid_f(acc);
    };
    if (!qk) {
      for (int d = lane; d < len; d += WAVE) dst[d] = channel(d);
      continue;
    }
#pragma unroll
    for (int i = 0; i < MAXU; ++i) {
      const int d = lane + i * WAVE;
      keep[i] = d < len ? channel(d) : 0.f;
      ss += keep[i] * keep[i];
    }
    const float norm = sqrtf(wave_reduce_sum(ss) + unit_eps);
    const float mul = (unit < KH ? q_scale : 1.f) / norm;
#pragma unroll
    for (int i = 0; i < MAXU; ++i) {
      const int d = lane + i * WAVE;
      if (d < len) dst[d] = keep[i] * mul;
    }
  }
}

// The same for sizes in vectors: a thread owns 8 channels and walks RB rows
// with the last TAPS - 1 inputs in registers; K / 8 threads (a power of two)
// share a unit norm. grid (channel blocks, row blocks)
template <typename T, int TAPS>
__global__ __launch_bounds__(NT) void delta_prep_vec_kernel(
    const T* __restrict__ proj, int64_t pstride, const float* __restrict__ taps,
    T* __restrict__ conv_state, const int32_t* __restrict__ row_seq,
    const int32_t* __restrict__ seq_meta, float* __restrict__ q,
    float* __restrict__ k, float* __restrict__ v, int rows, int RB, int KH,
    int H, int K, int V, float q_scale, float unit_eps) {
  const int C = 2 * KH * K + H * V, QK = KH * K;
  const int c = (blockIdx.x * NT + threadIdx.x) * 8;
  const bool in = c < C;
  const int cc = in ? c : 0;
  const bool qk = cc < 2 * QK;
  float w[TAPS][8], x[TAPS][8];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) ldn<8>(taps + (int64_t)j * C + cc, w[j]);
  const int r0 = blockIdx.y * RB, r1 = min(rows, r0 + RB);
  for (int row = r0; row < r1; ++row) {
    const Seq sq = load_seq(seq_meta, row_seq[row]);
    const int pos = row - sq.row0;
    T* state = conv_state + (int64_t)sq.slot * (TAPS - 1) * C + cc;
    if (row == r0 || pos == 0) {
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        const int p = pos - (TAPS - 1) + j;
        if (p >= 0) {
          ldn<8>(proj + (int64_t)(sq.row0 + p) * pstride + cc, x[j]);
        } else if (sq.prior > 0) {
          ldn<8>(state + (int64_t)(TAPS - 1 + p) * C, x[j]);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[j][e] = 0.f;
        }
      }
    }
    ldn<8>(proj + (int64_t)row * pstride + cc, x[TAPS - 1]);
    if (sq.n == 1 && in) {
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) stn<8>(state + (int64_t)j * C, x[j + 1]);
    }
    float f[8], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float a = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) a += w[j][e] * x[j][e];
      f[e] = a * sigmoid_f(a);
      ss += f[e] * f[e];
    }
    for (int o = K / 16; o > 0; o /= 2) ss += __shfl_xor(ss, o, WAVE);
    if (qk) {
      const float m = (cc < QK ? q_scale : 1.f) / sqrtf(ss + unit_eps);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] *= m;
    }
    if (in)
      stn<8>(cc < QK       ? q + (int64_t)row * QK + cc
             : cc < 2 * QK ? k + (int64_t)row * QK + cc - QK
                           : v + (int64_t)row * H * V + cc - 2 * QK,
             f);
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) x[j][e] = x[j + 1][e];
  }
}

// grid (channel blocks, sequences): keep the last n_taps - 1 inputs of every
// sequence with more than one row (single rows roll in delta_prep)
template <typename T>
__global__ __launch_bounds__(NT) void delta_conv_kernel(
    const T* __restrict__ proj, int64_t pstride, T* __restrict__ conv_state,
    const int32_t* __restrict__ seq_meta, int C, int n_taps) {
  const Seq sq = load_seq(seq_meta, blockIdx.y);
  const int c = blockIdx.x * NT + threadIdx.x;
  if (c >= C || sq.n == 1) return;
  T* state = conv_state + (int64_t)sq.slot * (n_taps - 1) * C;
  // entry i takes an input that is newer than entry i: ascending is in place
  for (int i = 0; i < n_taps - 1; ++i) {
    const int p = sq.n - (n_taps - 1) + i;
    float in = 0.f;
    if (p >= 0)
      in = ld(proj + (int64_t)(sq.row0 + p) * pstride + c);
    else if (sq.prior > 0)
      in = ld(state + (int64_t)(n_taps - 1 + p) * C + c);
    st(state + (int64_t)i * C + c, in);
  }
}

// One workgroup per (head, sequence). S is spread over the threads: a thread
// owns 4 columns (lanes_v threads cover V) and every groups-th row.
// RPT: rows per thread. VEC: V % 4 == 0.
template <typename T, int RPT, bool VEC>
__global__ __launch_bounds__(NT) void delta_step_kernel(
    const float* __restrict__ q, const float* __restrict__ k,
    const float* __restrict__ v,                 // [rows, KH|KH|H, K|K|V]
    const T* __restrict__ beta, int64_t bstride,  // [rows, H] before sigmoid
    const T* __restrict__ decay,                 // [rows, H K] before bias
    const float* __restrict__ dt_bias,           // [H K]
    const float* __restrict__ neg_a,             // [H]: -exp(A_log)
    const T* __restrict__ gate,                  // [rows, H V] before sigmoid
    const float* __restrict__ norm_w,            // [V]
    float* __restrict__ state,                   // [slots, H, K, V]
    const int32_t* __restrict__ seq_meta, T* __restrict__ out, int KH, int H,
    int K, int V, int lanes_v, float eps) {
  const int h = blockIdx.x;
  const Seq sq = load_seq(seq_meta, blockIdx.y);
  const int kh = h / (H / KH);
  const int groups = NT / lanes_v;
  const int tv = threadIdx.x % lanes_v, grp = threadIdx.x / lanes_v;
  const int c0 = tv * 4;

  __shared__ float qs[512], ks[512], gs[512];
  __shared__ float sk[4 * NT], so[4 * NT], kq[NT];
  __shared__ float red[NWV];

  float S[RPT][4];
  float* Sp = state + ((int64_t)sq.slot * H + h) * K * V;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = grp + i * groups;
#pragma unroll
    for (int j = 0; j < 4; ++j) S[i][j] = 0.f;
    if (r < K && sq.prior > 0) {
      if constexpr (VEC) {
        if (c0 < V) {
          const float4v t = *(const float4v*)(Sp + (int64_t)r * V + c0);
#pragma unroll
          for (int j = 0; j < 4; ++j) S[i][j] = t[j];
        }
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c0 + j < V) S[i][j] = Sp[(int64_t)r * V + c0 + j];
      }
    }
  }

  for (int t = 0; t < sq.n; ++t) {
    const int64_t row = sq.row0 + t;
    __syncthreads();  // the previous token's readers of shared memory
    for (int d = threadIdx.x; d < K; d += NT) {
      qs[d] = q[(row * KH + kh) * K + d];
      ks[d] = k[(row * KH + kh) * K + d];
      gs[d] = expf(neg_a[h] * softplus_f(ld(decay + (row * H + h) * K + d) +
                                         dt_bias[(int64_t)h * K + d]));
    }
    __syncthreads();
    float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f}, c = 0.f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = grp + i * groups;
      if (r < K) {
        const float g = gs[r], kr = ks[r], qr = qs[r];
        c += kr * qr;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          S[i][j] *= g;
          a[j] += S[i][j] * kr;
          b[j] += S[i][j] * qr;
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sk[(grp * lanes_v + tv) * 4 + j] = a[j];
      so[(grp * lanes_v + tv) * 4 + j] = b[j];
    }
    if (tv == 0) kq[grp] = c;
    __syncthreads();
    // S'k and S'q of the decayed state; the new write adds (k.q) u to o
    float u[4], o[4] = {0.f, 0.f, 0.f, 0.f}, dot = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) u[j] = 0.f;
    for (int p = 0; p < groups; ++p) {
      dot += kq[p];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        u[j] += sk[(p * lanes_v + tv) * 4 + j];
        o[j] += so[(p * lanes_v + tv) * 4 + j];
      }
    }
    const float bt = sigmoid_f(ld(beta + row * bstride + h));
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const bool in = c0 + j < V;
      u[j] = in ? bt * (v[(row * H + h) * V + c0 + j] - u[j]) : 0.f;
      o[j] += dot * u[j];
      if (in && grp == 0) ss += o[j] * o[j];
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = grp + i * groups;
      if (r < K) {
#pragma unroll
        for (int j = 0; j < 4; ++j) S[i][j] += ks[r] * u[j];
      }
    }
    const float inv =
        1.f / sqrtf(block_sum<NWV>(ss, red) / (float)V + eps);
    if (grp == 0) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (c0 + j < V) {
          const int64_t at = (row * H + h) * V + c0 + j;
          st(out + at, o[j] * inv * norm_w[c0 + j] * sigmoid_f(ld(gate + at)));
        }
      }
    }
  }

#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = grp + i * groups;
    if (r < K) {
      if constexpr (VEC) {
        if (c0 < V)
          *(float4v*)(Sp + (int64_t)r * V + c0) =
              (float4v){S[i][0], S[i][1], S[i][2], S[i][3]};
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c0 + j < V) Sp[(int64_t)r * V + c0 + j] = S[i][j];
      }
    }
  }
}

}  // namespace

extern "C" {

hipError_t lds_delta_prep(int f32, const void* proj, int64_t pstride,
                          const float* taps, void* conv_state,
                          const int32_t* row_seq, const int32_t* seq_meta,
                          float* q, float* k, float* v, int rows, int n_seqs,
                          int multi_row, int KH, int H, int K, int V,
                          int n_taps, float q_scale, float unit_eps,
                          hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  if (K > MAXU * WAVE || n_taps < 1) return hipErrorInvalidValue;
  const int units = 2 * KH + H, C = 2 * KH * K + H * V;
  int gy = (units + NWV - 1) / NWV;
  if (rows >= 1024 && gy > 4) gy = 4;
  const dim3 grid(rows, gy), cgrid((C + NT - 1) / NT, n_seqs);
  const bool vec = K % 8 == 0 && V % 8 == 0 && pstride % 8 == 0 &&
                   K / 8 <= WAVE && (K / 8 & (K / 8 - 1)) == 0 &&
                   n_taps >= 2 && n_taps <= 4;
  int rb = 1;       // rows per thread: long walks only with enough of them
  while (rb < 32 && (int64_t)rows * C / 8 / NT / (2 * rb) >= 2048) rb *= 2;
  const dim3 vgrid((C / 8 + NT - 1) / NT, (rows + rb - 1) / rb);
#define VEC(T, TAPS)                                                          \
  hipLaunchKernelGGL((delta_prep_vec_kernel<T, TAPS>), vgrid, dim3(NT), 0,    \
                     stream, (const T*)proj, pstride, taps, (T*)conv_state,   \
                     row_seq, seq_meta, q, k, v, rows, rb, KH, H, K, V,       \
                     q_scale, unit_eps)
#define GO(T)                                                                 \
  do {                                                                        \
    if (vec && n_taps == 2) VEC(T, 2);                                        \
    else if (vec && n_taps == 3) VEC(T, 3);                                   \
    else if (vec) VEC(T, 4);                                                  \
    else                                                                      \
      hipLaunchKernelGGL(delta_prep_kernel<T>, grid, dim3(NT), 0, stream,     \
                         (const T*)proj, pstride, taps, (T*)conv_state,       \
                         row_seq, seq_meta, q, k, v, KH, H, K, V, n_taps,     \
                         q_scale, unit_eps);                                  \
    if (multi_row && n_taps > 1)                                              \
      hipLaunchKernelGGL(delta_conv_kernel<T>, cgrid, dim3(NT), 0, stream,    \
                         (const T*)proj, pstride, (T*)conv_state, seq_meta,   \
                         C, n_taps);                                          \
  } while (0)
  if (f32) GO(float); else GO(short);
#undef VEC
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

hipError_t lds_delta_step(int f32, const float* q, const float* k,
                          const float* v, const void* beta, int64_t bstride,
                          const void* decay, const float* dt_bias,
                          const float* neg_a, const void* gate,
                          const float* norm_w, float* state,
                          const int32_t* seq_meta, void* out, int n_seqs,
                          int KH, int H, int K, int V, float eps,
                          hipStream_t stream) {
  if (n_seqs == 0) return hipSuccess;
  int lanes_v = 1;
  while (lanes_v * 4 < V) lanes_v *= 2;
  if (lanes_v > NT || K > 512) return hipErrorInvalidValue;
  const int groups = NT / lanes_v, need = (K + groups - 1) / groups;
  int rpt = 1;
  while (rpt < need) rpt *= 2;
  const dim3 grid(H, n_seqs);
#define GO2(T, R, VEC)                                                        \
  hipLaunchKernelGGL((delta_step_kernel<T, R, VEC>), grid, dim3(NT), 0,       \
                     stream, q, k, v, (const T*)beta, bstride,                \
                     (const T*)decay, dt_bias, neg_a, (const T*)gate, norm_w, \
                     state, seq_meta, (T*)out, KH, H, K, V, lanes_v, eps)
#define GO1(T, R)                                                             \
  do {                                                                        \
    if (V % 4 == 0) GO2(T, R, true); else GO2(T, R, false);                   \
  } while (0)
#define GO(R)                                                                 \
  do {                                                                        \
    if (f32) GO1(float, R); else GO1(short, R);                               \
  } while (0)
  switch (rpt) {
    case 1: GO(1); break;
    case 2: GO(2); break;
    case 4: GO(4); break;
    case 8: GO(8); break;
    case 16: GO(16); break;
    case 32: GO(32); break;
    case 64: GO(64); break;
    default: return hipErrorInvalidValue;
  }
#undef GO
#undef GO1
#undef GO2
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
