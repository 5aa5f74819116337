// residual_norm.hip — the 32-bit residual stream: embedding, what sublayers
// and loop passes add to it, RMS norms, activations. HBM-bound; one pass over
// the stream per sublayer.
#include "elem.h"

namespace {

constexpr int NT = 256;
constexpr int KEEP = 4;  // vectors kept in registers per thread

enum Mode { EMBED, POST, ADD, LOOP };

template <typename T>
struct Stream {
  float* x;                  // [T, H]
  const T* y;                // [T, H], or the embedding table
  const int64_t* ids;        // EMBED
  const float* pos;          // EMBED: [positions, H] or null
  const int32_t* positions;
  const float* wb;           // POST
  const T* rows;             // POST, ADD: [T n_rows, H], n_rows of each token
  int n_rows;
  const float *a, *b, *v;    // LOOP: [T, H], [T, H], [H]
  const float* wn;           // null: h = x
  T* h;
  int H;
  float scale, offset, eps;
};

// One workgroup per row of the stream.
//   EMBED: x = table[id] * scale + pos[position]
//   POST:  x += y / rms(y) * (wb + offset) + the token's rows
//   ADD:   x += y + the token's rows (either may be missing)
//   LOOP:  x = a + b + v
//   h = x / rms(x) * (wn + offset)
template <typename T, int N, int MODE>
__global__ __launch_bounds__(NT) void stream_norm_kernel(const Stream<T> s) {
  __shared__ float red[2][NT / WAVE];
  const int64_t row = blockIdx.x;
  const int H = s.H;
  float* xr = s.x + row * H;
  const T* yr = MODE == EMBED ? s.y + s.ids[row] * H : s.y + row * H;
  // vector i of this thread starts at element at(i); the first KEEP stay in
  // registers between the passes, the rest are read again
  float keep[KEEP][N];
  auto at = [&](int i) { return (int64_t)(threadIdx.x + i * NT) * N; };
  float inv_y = 0.f;
  if constexpr (MODE == POST) {
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
    inv_y = 1.f / sqrtf(block_sum<NT / WAVE>(ss, red[0]) / (float)H + s.eps);
  }
  float ss = 0.f;
  auto update = [&](int i, float* f) {  // POST: y's vector in; stream's out
    const int64_t c = at(i);
    float g[N];
    if constexpr (MODE == EMBED) {
      ldn<N>(yr + c, f);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] *= s.scale;
      if (s.pos) {
        ldn<N>(s.pos + (int64_t)s.positions[row] * H + c, g);
#pragma unroll
        for (int j = 0; j < N; ++j) f[j] += g[j];
      }
      stn<N>(xr + c, f);
    } else if constexpr (MODE == LOOP) {
      ldn<N>(s.a + row * H + c, f);
      ldn<N>(s.b + row * H + c, g);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] += g[j];
      ldn<N>(s.v + c, g);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] += g[j];
      stn<N>(xr + c, f);
    } else {
      float d[N];                       // what the row gets
#pragma unroll
      for (int j = 0; j < N; ++j) d[j] = 0.f;
      if constexpr (MODE == POST) {
        float w[N];
        ldn<N>(s.wb + c, w);
#pragma unroll
        for (int j = 0; j < N; ++j) d[j] = f[j] * inv_y * (w[j] + s.offset);
      } else if (s.y) {
        ldn<N>(yr + c, d);
      }
      for (int r = 0; r < s.n_rows; ++r) {
        ldn<N>(s.rows + (row * s.n_rows + r) * H + c, g);
#pragma unroll
        for (int j = 0; j < N; ++j) d[j] += g[j];
      }
      ldn<N>(xr + c, f);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] += d[j];
      if (MODE == POST || s.y || s.n_rows) stn<N>(xr + c, f);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) ss += f[j] * f[j];
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (at(i) < H) update(i, keep[i]);
  for (int i = KEEP; at(i) < H; ++i) {
    float f[N];
    if (MODE == POST) ldn<N>(yr + at(i), f);
    update(i, f);
  }
  const float inv = s.wn ? 1.f / sqrtf(block_sum<NT / WAVE>(ss, red[1]) /
                                       (float)H + s.eps)
                         : 1.f;
  auto finish = [&](int i, float* f) {
    if (s.wn) {
      float w[N];
      ldn<N>(s.wn + at(i), w);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] *= inv * (w[j] + s.offset);
    }
    stn<N>(s.h + row * H + at(i), f);
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

// y = act(gate) * up on packed [T, 2 I] rows, or act(x) on [T, I] rows
template <typename T, int N, bool GATED>
__global__ __launch_bounds__(NT) void act_kernel(
    const T* __restrict__ x, T* __restrict__ y, int64_t T_, int I, int act) {
  const int nv = I / N;
  const int64_t total = T_ * nv;
  for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * NT) {
    const int64_t row = i / nv;
    const int c = (int)(i % nv) * N;
    const T* p = x + row * I * (GATED ? 2 : 1) + c;
    float g[N], u[N];
    ldn<N>(p, g);
    if constexpr (GATED) ldn<N>(p + I, u);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      g[j] = activate(act, g[j]);
      if constexpr (GATED) g[j] *= u[j];
    }
    stn<N>(y + row * I + c, g);
  }
}

template <typename T>
hipError_t stream_norm_t(int mode, const void* const* p, int64_t rows,
                         int n_rows, int H, float scale, float offset,
                         float eps, hipStream_t stream) {
  const Stream<T> s{(float*)p[0], (const T*)p[1], (const int64_t*)p[2],
                    (const float*)p[3], (const int32_t*)p[4],
                    (const float*)p[5], (const T*)p[6], n_rows,
                    (const float*)p[7], (const float*)p[8],
                    (const float*)p[9], (const float*)p[10], (T*)p[11], H,
                    scale, offset, eps};
  const dim3 grid((uint32_t)rows), block(NT);
#define GO(N, M)                                                              \
  hipLaunchKernelGGL((stream_norm_kernel<T, N, M>), grid, block, 0, stream, s)
#define GOM(N)                                                                \
  do {                                                                        \
    if (mode == EMBED) GO(N, EMBED); else if (mode == POST) GO(N, POST);      \
    else if (mode == ADD) GO(N, ADD); else GO(N, LOOP);                       \
  } while (0)
  if (H % 8 == 0) GOM(8); else GOM(1);
#undef GOM
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

template <typename T, bool GATED>
hipError_t act_t(const void* x, void* y, int64_t rows, int I, int act,
                 hipStream_t stream) {
  const int n = I % 8 == 0 ? 8 : 1;
  int64_t blocks = (rows * (I / n) + NT - 1) / NT;
  if (blocks > 4096) blocks = 4096;
  const dim3 grid((uint32_t)blocks), block(NT);
  if (n == 8)
    hipLaunchKernelGGL((act_kernel<T, 8, GATED>), grid, block, 0, stream,
                       (const T*)x, (T*)y, rows, I, act);
  else
    hipLaunchKernelGGL((act_kernel<T, 1, GATED>), grid, block, 0, stream,
                       (const T*)x, (T*)y, rows, I, act);
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // namespace

extern "C" {

// ptr: x, y or table, ids, pos, positions, wb, rows, a, b, v, wn, h (null
// where the mode has none): see Stream
hipError_t lds_stream_norm(int f32, int mode, const void* const* ptr,
                           int64_t rows, int n_rows, int H, float scale,
                           float offset, float eps, hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  return f32 ? stream_norm_t<float>(mode, ptr, rows, n_rows, H, scale, offset,
                                    eps, stream)
             : stream_norm_t<short>(mode, ptr, rows, n_rows, H, scale, offset,
                                    eps, stream);
}

hipError_t lds_act(int f32, int gated, const void* x, void* y, int64_t rows,
                   int I, int act, hipStream_t stream) {
  if (rows == 0 || I == 0) return hipSuccess;
  if (gated)
    return f32 ? act_t<float, true>(x, y, rows, I, act, stream)
               : act_t<short, true>(x, y, rows, I, act, stream);
  return f32 ? act_t<float, false>(x, y, rows, I, act, stream)
             : act_t<short, false>(x, y, rows, I, act, stream);
}

}  // extern "C"
