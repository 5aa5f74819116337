// residual_norm.hip — the 32-bit residual stream: embedding, RMS norms on
// both sides of a sublayer, gated activations. HBM-bound; one pass over the
// stream per sublayer.
#include "elem.h"

namespace {

constexpr int NT = 256;
constexpr int KEEP = 4;  // vectors kept in registers per thread

// One workgroup per row of the stream x [T, H] (float).
//   EMBED: x = table[id] * scale
//   else if wb: x += y / rms(y) * (wb + offset)
//   h = x / rms(x) * (wn + offset)
template <typename T, int N, bool EMBED>
__global__ __launch_bounds__(NT) void stream_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const int64_t* __restrict__ ids, const float* __restrict__ wb,
    const float* __restrict__ wn, T* __restrict__ h, int H, float scale,
    float offset, float eps) {
  __shared__ float red[2][NT / WAVE];
  const int64_t row = blockIdx.x;
  float* xr = x + row * H;
  const T* yr = EMBED ? y + ids[row] * H : y + row * H;
  // vector i of this thread starts at element at(i); the first KEEP stay in
  // registers between the passes, the rest are read again
  float keep[KEEP][N];
  auto at = [&](int i) { return (int64_t)(threadIdx.x + i * NT) * N; };
  const bool add = !EMBED && wb;
  float inv_y = 0.f;
  if (add) {
    float ss = 0.f;
    auto square = [&](int i, float* f) {
      ldn<N>(yr + at(i), f);
#pragma unroll
      for (int j = 0; j < N; ++j) ss += f[j] * f[j];
    };
#pragma unroll
    for (int i = 0; i < KEEP; ++i)
      if (at(i) < H) square(i, keep[i]);
    for (int i = KEEP; at(i) < H; ++i) {
      float f[N];
      square(i, f);
    }
    inv_y = 1.f / sqrtf(block_sum<NT / WAVE>(ss, red[0]) / (float)H + eps);
  }
  float ss = 0.f;
  auto update = [&](int i, float* f) {  // f: y's vector in, the stream's out
    if constexpr (EMBED) {
      ldn<N>(yr + at(i), f);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] *= scale;
      stn<N>(xr + at(i), f);
    } else {
      float g[N], w[N];
#pragma unroll
      for (int j = 0; j < N; ++j) g[j] = f[j];
      ldn<N>(xr + at(i), f);
      if (add) {
        ldn<N>(wb + at(i), w);
#pragma unroll
        for (int j = 0; j < N; ++j) f[j] += g[j] * inv_y * (w[j] + offset);
        stn<N>(xr + at(i), f);
      }
    }
#pragma unroll
    for (int j = 0; j < N; ++j) ss += f[j] * f[j];
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (at(i) < H) update(i, keep[i]);
  for (int i = KEEP; at(i) < H; ++i) {
    float f[N];
    if (add) ldn<N>(yr + at(i), f);
    update(i, f);
  }
  const float inv =
      1.f / sqrtf(block_sum<NT / WAVE>(ss, red[1]) / (float)H + eps);
  auto finish = [&](int i, float* f) {
    float w[N];
    ldn<N>(wn + at(i), w);
#pragma unroll
    for (int j = 0; j < N; ++j) f[j] *= inv * (w[j] + offset);
    stn<N>(h + row * H + at(i), f);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (at(i) < H) finish(i, keep[i]);
  for (int i = KEEP; at(i) < H; ++i) {
    float f[N];
    ldn<N>(xr + at(i), f);  // this thread's own store above
    finish(i, f);
  }
}

// y = gelu_tanh(gate) * up on packed [T, 2 I] rows
template <typename T, int N>
__global__ __launch_bounds__(NT) void gelu_mul_kernel(
    const T* __restrict__ gate_up, T* __restrict__ y, int64_t T_, int I) {
  const int nv = I / N;
  const int64_t total = T_ * nv;
  for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * NT) {
    const int64_t row = i / nv;
    const int c = (int)(i % nv) * N;
    float g[N], u[N];
    ldn<N>(gate_up + row * 2 * I + c, g);
    ldn<N>(gate_up + row * 2 * I + I + c, u);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      const float z = g[j];
      // 0.5 (1 + tanh(a)) = 1 / (1 + exp(-2a))
      const float a = 0.7978845608028654f * (z + 0.044715f * z * z * z);
      g[j] = z / (1.f + expf(-2.f * a)) * u[j];
    }
    stn<N>(y + row * I + c, g);
  }
}

}  // namespace

template <typename T>
static hipError_t stream_norm_t(float* x, const void* y, const int64_t* ids,
                                const float* wb, const float* wn, void* h,
                                int64_t rows, int H, float scale, float offset,
                                float eps, hipStream_t stream) {
  const dim3 grid((uint32_t)rows), block(NT);
#define GO(N, E)                                                              \
  hipLaunchKernelGGL((stream_norm_kernel<T, N, E>), grid, block, 0, stream, x, \
                     (const T*)y, ids, wb, wn, (T*)h, H, scale, offset, eps)
  if (H % 8 == 0) {
    if (ids) GO(8, true); else GO(8, false);
  } else {
    if (ids) GO(1, true); else GO(1, false);
  }
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

template <typename T>
static hipError_t gelu_mul_t(const void* gu, void* y, int64_t rows, int I,
                             hipStream_t stream) {
  const int n = I % 8 == 0 ? 8 : 1;
  int64_t blocks = (rows * (I / n) + NT - 1) / NT;
  if (blocks > 4096) blocks = 4096;
  if (n == 8)
    hipLaunchKernelGGL((gelu_mul_kernel<T, 8>), dim3((uint32_t)blocks),
                       dim3(NT), 0, stream, (const T*)gu, (T*)y, rows, I);
  else
    hipLaunchKernelGGL((gelu_mul_kernel<T, 1>), dim3((uint32_t)blocks),
                       dim3(NT), 0, stream, (const T*)gu, (T*)y, rows, I);
  HIP_CHECK_LAST();
  return hipSuccess;
}

extern "C" {

hipError_t lds_stream_norm(int f32, float* x, const void* y,
                           const int64_t* ids, const float* wb,
                           const float* wn, void* h, int64_t rows, int H,
                           float scale, float offset, float eps,
                           hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  return f32 ? stream_norm_t<float>(x, y, ids, wb, wn, h, rows, H, scale,
                                    offset, eps, stream)
             : stream_norm_t<short>(x, y, ids, wb, wn, h, rows, H, scale,
                                    offset, eps, stream);
}

hipError_t lds_gelu_mul(int f32, const void* gate_up, void* y, int64_t rows,
                        int I, hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  return f32 ? gelu_mul_t<float>(gate_up, y, rows, I, stream)
             : gelu_mul_t<short>(gate_up, y, rows, I, stream);
}

}  // extern "C"
