// attention.hip — cache rows of latent attention and of grouped heads, and
// plain attention over either.
//
// Latent attention caches per token: [latent (kv_rank, normed) | rotated key part (rot_dim)],
// pages [n_blocks, block_size, kv_rank + rot_dim]. Rows that come alone (or
// in short portions) attend to the pages directly, with the key projection
// absorbed into the query; long portions expand keys and values first
// (context_prefill.hip). attn_rows is the plain kernel for either form and for
// grouped heads: any size, bf16 or float.
#include "elem.h"

namespace {

constexpr int NT = 256;
constexpr int NWV = NT / WAVE;

// cos_sin: [max_pos, dims / 2, 2]. Rotates pairs (2i, 2i + 1).
template <typename T>
__device__ __forceinline__ void rotate_pair(const T* src, T* dst,
                                            const float* cs) {
  const float u = ld(src), v = ld(src + 1);
  st(dst, u * cs[0] - v * cs[1]);
  st(dst + 1, v * cs[0] + u * cs[1]);
}

// One workgroup per row of [.., q_rank | kv_rank | rot]: norms the query
// latent into cq, norms the latent and rotates the key part into the cache.
template <typename T>
__global__ __launch_bounds__(NT) void latent_prep_kernel(
    const T* __restrict__ proj, int64_t pstride, const float* __restrict__ wq,
    const float* __restrict__ wkv, const float* __restrict__ cos_sin,
    const int32_t* __restrict__ positions, const int64_t* __restrict__ slots,
    T* __restrict__ cq, T* __restrict__ cache, int q_rank, int kv_rank,
    int rot, float eps) {
  __shared__ float red[2][NWV];
  const int64_t row = blockIdx.x;
  const T* p = proj + row * pstride;
  float ss = 0.f;
  for (int d = threadIdx.x; d < q_rank; d += NT) {
    const float x = ld(p + d);
    ss += x * x;
  }
  float inv = 1.f / sqrtf(block_sum<NWV>(ss, red[0]) / (float)q_rank + eps);
  for (int d = threadIdx.x; d < q_rank; d += NT)
    st(cq + row * q_rank + d, ld(p + d) * inv * wq[d]);
  if (!cache) return;
  p += q_rank;
  ss = 0.f;
  for (int d = threadIdx.x; d < kv_rank; d += NT) {
    const float x = ld(p + d);
    ss += x * x;
  }
  inv = 1.f / sqrtf(block_sum<NWV>(ss, red[1]) / (float)kv_rank + eps);
  T* dst = cache + slots[row] * (kv_rank + rot);
  for (int d = threadIdx.x; d < kv_rank; d += NT)
    st(dst + d, ld(p + d) * inv * wkv[d]);
  const float* cs = cos_sin + (int64_t)positions[row] * rot;
  for (int i = threadIdx.x; i < rot / 2; i += NT)
    rotate_pair(p + kv_rank + 2 * i, dst + kv_rank + 2 * i, cs + 2 * i);
}

// In place on the rotated part of q [rows, H, D + rot]; the unrotated part
// of the first n_abs rows is laid out by head for the absorbing product.
template <typename T>
__global__ __launch_bounds__(NT) void rope_part_kernel(
    T* __restrict__ q, T* __restrict__ by_head,  // [H, n_abs, D]
    const float* __restrict__ cos_sin, const int32_t* __restrict__ positions,
    int n_abs, int H, int D, int rot) {
  const int64_t row = blockIdx.x;
  T* qr = q + row * H * (D + rot);
  const float* cs = cos_sin + (int64_t)positions[row] * rot;
  const int half = rot / 2;
  for (int i = threadIdx.x; i < H * half; i += NT) {
    const int h = i / half, d = i % half;
    T* p = qr + (int64_t)h * (D + rot) + D + 2 * d;
    rotate_pair(p, p, cs + 2 * d);
  }
  if (row < n_abs) {
    for (int i = threadIdx.x; i < H * D; i += NT) {
      const int h = i / D, d = i % D;
      by_head[((int64_t)h * n_abs + row) * D + d] =
          qr[(int64_t)h * (D + rot) + d];
    }
  }
}

// [H, n_abs, V] -> rows of [.., H V]
template <typename T>
__global__ __launch_bounds__(NT) void heads_to_rows_kernel(
    const T* __restrict__ src, T* __restrict__ dst, int n_abs, int H, int V) {
  const int64_t row = blockIdx.x;
  for (int i = threadIdx.x; i < H * V; i += NT)
    dst[row * H * V + i] = src[((int64_t)(i / V) * n_abs + row) * V + i % V];
}

// rows of the cache at `slots`, contiguous; unit: bytes moved per lane
template <typename U>
__global__ __launch_bounds__(NT) void gather_rows_kernel(
    const U* __restrict__ cache, const int64_t* __restrict__ slots,
    U* __restrict__ out, int64_t rows, int width) {
  const int64_t total = rows * width;
  for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * NT)
    out[i] = cache[slots[i / width] * width + i % width];
}

// Keys and values as the plain kernel sees them: score = qa.ka + qb.kb.
// Strides in elements; a token is a row of a page (block table given) or a
// context row. `rep` query heads share a key/value head.
template <typename T>
struct View {
  const T *qa, *qb, *ka, *kb, *v;
  int64_t qa_row, qa_head, qb_row, qb_head;
  int64_t ka_tok, ka_head, kb_tok, v_tok, v_head, page;
  int da, db, dv, rep;
  int has_sink;
  float sink;                    // score of a key without a value
};

// One workgroup per (head, row).
//   paged: keys of positions (pos - window, pos] through the block table
//   else:  ctx [n_seqs, 2] = first context row, its position
template <typename T, int MAXV>
__global__ __launch_bounds__(NT) void attn_rows_kernel(
    View<T> a, const int32_t* __restrict__ positions,
    const int32_t* __restrict__ row_seq, int row_base,
    const int32_t* __restrict__ block_tables, int max_blocks, int block_size,
    const int32_t* __restrict__ ctx, int window, float scale,
    T* __restrict__ out, int64_t o_row, int64_t o_head) {
  extern __shared__ float qv[];  // da + db
  __shared__ float p[NT], redm[NWV], reds[NWV];
  const int h = blockIdx.x, kvh = h / a.rep;
  const int64_t i = blockIdx.y;       // row of q and out
  const int64_t row = row_base + i;   // row of the batch
  const int seq = row_seq[row];
  const int pos = positions[row];
  const int lo = window > 0 && pos + 1 > window ? pos + 1 - window : 0;
  const int32_t* bt =
      block_tables ? block_tables + (int64_t)seq * max_blocks : nullptr;
  const int64_t shift =
      bt ? 0 : (int64_t)ctx[2 * seq] - ctx[2 * seq + 1];
  // element offset of a token whose rows are `stride` apart
  auto at = [&](int t, int64_t stride) -> int64_t {
    return bt ? bt[t / block_size] * a.page + t % block_size * stride
              : (t + shift) * stride;
  };
  for (int d = threadIdx.x; d < a.da; d += NT)
    qv[d] = ld(a.qa + i * a.qa_row + h * a.qa_head + d);
  for (int d = threadIdx.x; d < a.db; d += NT)
    qv[a.da + d] = ld(a.qb + i * a.qb_row + h * a.qb_head + d);
  float acc[MAXV];
#pragma unroll
  for (int j = 0; j < MAXV; ++j) acc[j] = 0.f;
  float m = a.has_sink ? a.sink : -INFINITY, l = a.has_sink ? 1.f : 0.f;
  for (int t0 = lo; t0 <= pos; t0 += NT) {
    __syncthreads();
    const int t = t0 + threadIdx.x;
    float s = -INFINITY;
    if (t <= pos) {
      const T* ka = a.ka + at(t, a.ka_tok) + kvh * a.ka_head;
      const T* kb = a.kb + at(t, a.kb_tok);
      float dot = 0.f;
      for (int d = 0; d < a.da; ++d) dot += qv[d] * ld(ka + d);
      for (int d = 0; d < a.db; ++d) dot += qv[a.da + d] * ld(kb + d);
      s = dot * scale;
    }
    float mx = wave_reduce_max(s);
    if (threadIdx.x % WAVE == 0) redm[threadIdx.x / WAVE] = mx;
    __syncthreads();
#pragma unroll
    for (int w = 0; w < NWV; ++w) mx = fmaxf(mx, redm[w]);
    const float mn = fmaxf(m, mx);      // finite: key lo..pos is not empty
    const float alpha = expf(m - mn);   // 0 at the first tile without a sink
    const float e = t <= pos ? expf(s - mn) : 0.f;
    p[threadIdx.x] = e;
    l = l * alpha + block_sum<NWV>(e, reds);
    m = mn;
    const int n = min(NT, pos + 1 - t0);
#pragma unroll
    for (int j = 0; j < MAXV; ++j) {
      const int d = threadIdx.x + j * NT;
      if (d < a.dv) {
        float o = acc[j] * alpha;
        for (int x = 0; x < n; ++x)
          o += p[x] * ld(a.v + at(t0 + x, a.v_tok) + kvh * a.v_head + d);
        acc[j] = o;
      }
    }
  }
#pragma unroll
  for (int j = 0; j < MAXV; ++j) {
    const int d = threadIdx.x + j * NT;
    if (d < a.dv) st(out + i * o_row + h * o_head + d, acc[j] / l);
  }
}

// rows [.., keys of all heads | values of all heads] from column 0 of kv on
// -> pages [NB, G, bs, D + V]; U: the unit moved per lane
template <typename U>
__global__ __launch_bounds__(NT) void store_heads_kernel(
    const U* __restrict__ kv, int64_t stride,
    const int64_t* __restrict__ slots, U* __restrict__ cache, int64_t rows,
    int G, int bs, int D, int V) {
  const int W = D + V, width = G * W;
  const int64_t total = rows * width;
  for (int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * NT) {
    const int64_t row = i / width, slot = slots[row];
    const int c = (int)(i % width), g = c / W, d = c % W;
    cache[((slot / bs * G + g) * bs + slot % bs) * W + d] =
        kv[row * stride + (d < D ? g * D + d : G * D + g * V + (d - D))];
  }
}

template <typename T>
hipError_t attn_rows_t(const void* const* ptr, const int64_t* stride, int da,
                       int db, int dv, int rep, int has_sink, float sink,
                       const int32_t* positions, const int32_t* row_seq,
                       int row_base, const int32_t* block_tables,
                       int max_blocks, int block_size, const int32_t* ctx,
                       int window, float scale, void* out, int64_t o_row,
                       int64_t o_head, int rows, int H, hipStream_t stream) {
  View<T> a{(const T*)ptr[0], (const T*)ptr[1], (const T*)ptr[2],
            (const T*)ptr[3], (const T*)ptr[4],
            stride[0], stride[1], stride[2], stride[3], stride[4], stride[5],
            stride[6], stride[7], stride[8], stride[9], da, db, dv, rep,
            has_sink, sink};
  if (dv > 8 * NT || da + db > 8192) return hipErrorInvalidValue;
  const size_t lds = (size_t)(da + db) * sizeof(float);
  const dim3 block(NT);
  for (int r = 0; r < rows; r += 32768) {  // grid.y limit
    const int n = rows - r < 32768 ? rows - r : 32768;
    const dim3 grid(H, n);
    View<T> b = a;
    b.qa += r * a.qa_row;
    b.qb += r * a.qb_row;
    T* o = (T*)out + r * o_row;
#define GO(M)                                                                 \
  hipLaunchKernelGGL((attn_rows_kernel<T, M>), grid, block, lds, stream, b,   \
                     positions, row_seq, row_base + r, block_tables,          \
                     max_blocks, block_size, ctx, window, scale, o, o_row,    \
                     o_head)
    if (dv <= NT) GO(1); else if (dv <= 2 * NT) GO(2); else GO(8);
#undef GO
  }
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // namespace

extern "C" {

hipError_t lds_latent_prep(int f32, const void* proj, int64_t pstride,
                           const float* wq, const float* wkv,
                           const float* cos_sin, const int32_t* positions,
                           const int64_t* slots, void* cq, void* cache,
                           int rows, int q_rank, int kv_rank, int rot,
                           float eps, hipStream_t stream) {
  if (rows == 0) return hipSuccess;
#define GO(T)                                                                 \
  hipLaunchKernelGGL(latent_prep_kernel<T>, dim3(rows), dim3(NT), 0, stream,  \
                     (const T*)proj, pstride, wq, wkv, cos_sin, positions,    \
                     slots, (T*)cq, (T*)cache, q_rank, kv_rank, rot, eps)
  if (f32) GO(float); else GO(short);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

hipError_t lds_rope_part(int f32, void* q, void* by_head, const float* cos_sin,
                         const int32_t* positions, int rows, int n_abs, int H,
                         int D, int rot, hipStream_t stream) {
  if (rows == 0) return hipSuccess;
#define GO(T)                                                                 \
  hipLaunchKernelGGL(rope_part_kernel<T>, dim3(rows), dim3(NT), 0, stream,    \
                     (T*)q, (T*)by_head, cos_sin, positions, n_abs, H, D, rot)
  if (f32) GO(float); else GO(short);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

hipError_t lds_heads_to_rows(int f32, const void* src, void* dst, int n_abs,
                             int H, int V, hipStream_t stream) {
  if (n_abs == 0) return hipSuccess;
#define GO(T)                                                                 \
  hipLaunchKernelGGL(heads_to_rows_kernel<T>, dim3(n_abs), dim3(NT), 0,       \
                     stream, (const T*)src, (T*)dst, n_abs, H, V)
  if (f32) GO(float); else GO(short);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

hipError_t lds_gather_rows(const void* cache, const int64_t* slots, void* out,
                           int64_t rows, int64_t row_bytes,
                           hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  const int unit = row_bytes % 16 == 0 ? 16 : row_bytes % 4 == 0 ? 4 : 2;
  if (row_bytes % unit) return hipErrorInvalidValue;
  const int width = (int)(row_bytes / unit);
  int64_t blocks = (rows * width + NT - 1) / NT;
  if (blocks > 4096) blocks = 4096;
#define GO(U)                                                                 \
  hipLaunchKernelGGL(gather_rows_kernel<U>, dim3((uint32_t)blocks), dim3(NT), \
                     0, stream, (const U*)cache, slots, (U*)out, rows, width)
  if (unit == 16) GO(short8); else if (unit == 4) GO(float); else GO(short);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

// ptr: qa, qb, ka, kb, v; stride: qa row/head, qb row/head, ka token/head,
// kb token, v token/head, page (elements)
hipError_t lds_attn_rows(int f32, const void* const* ptr,
                         const int64_t* stride, int da, int db, int dv,
                         int rep, int has_sink, float sink,
                         const int32_t* positions, const int32_t* row_seq,
                         int row_base, const int32_t* block_tables,
                         int max_blocks, int block_size, const int32_t* ctx,
                         int window, float scale, void* out, int64_t o_row,
                         int64_t o_head, int rows, int H,
                         hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  auto fn = f32 ? attn_rows_t<float> : attn_rows_t<short>;
  return fn(ptr, stride, da, db, dv, rep, has_sink, sink, positions, row_seq,
            row_base, block_tables, max_blocks, block_size, ctx, window, scale,
            out, o_row, o_head, rows, H, stream);
}

// es: bytes per element
hipError_t lds_store_heads(const void* kv, int64_t stride,
                           const int64_t* slots, void* cache, int64_t rows,
                           int G, int bs, int D, int V, int es,
                           hipStream_t stream) {
  if (rows == 0) return hipSuccess;
  const int n = 16 / es;      // elements of a 16-byte unit
  const int u = D % n == 0 && V % n == 0 && stride % n == 0 &&
                        (uintptr_t)kv % 16 == 0
                    ? n
                    : 1;
  int64_t blocks = (rows * G * (D + V) / u + NT - 1) / NT;
  if (blocks > 4096) blocks = 4096;
#define GO(U)                                                                 \
  hipLaunchKernelGGL(store_heads_kernel<U>, dim3((uint32_t)blocks), dim3(NT), \
                     0, stream, (const U*)kv, stride / u, slots, (U*)cache,   \
                     rows, G, bs, D / u, V / u)
  if (u > 1) GO(short8); else if (es == 4) GO(float); else GO(short);
#undef GO
  HIP_CHECK_LAST();
  return hipSuccess;
}

}  // extern "C"
