// ops_grouped.hip — torch binding of grouped attention and the experts (part
// of `_hip_layered`).
#include "check.h"

extern "C" {
hipError_t lds_store_heads(const void*, int64_t, const int64_t*, void*,
                           int64_t, int, int, int, int, int, hipStream_t);
int lds_grouped_decode_ok(int, int, int64_t);
int lds_grouped_decode_parts(int, int, int, int, int, int);
hipError_t lds_grouped_decode(const void*, int64_t, const void*,
                              const int32_t*, const int32_t*, const int32_t*,
                              void*, float*, float*, int, int, int, int, int,
                              int, int, int, float, int, float, hipStream_t);
int lds_grouped_prefill_ok(int, int, int, int64_t);
hipError_t lds_grouped_prefill(const void*, int64_t, const void*,
                               const int32_t*, int, int, const int32_t*,
                               const int32_t*, int, void*, int, int, int, int,
                               float, int, float, hipStream_t);
hipError_t lds_route(int, const void*, const void*, int32_t*, float*, int64_t,
                     int, int, int, hipStream_t);
int lds_expert_tile(int, int, int, int, int, int, int);
int lds_expert_max_tiles(int, int, int);
hipError_t lds_sort_pairs(const int32_t*, int32_t*, void*, int, int, int,
                          hipStream_t);
hipError_t lds_expert_product(int, int, int, const void*, const void*, void*,
                              const int32_t*, const void*, int, int,
                              const float*, int, int, int, int, hipStream_t);
}

namespace {

using OptFloat = c10::optional<double>;

// sizes of grouped attention
struct Heads {
  int f32;
  int64_t rows, H, G, D, V, bs;
};

Heads heads(const Tensor& proj, const Tensor& cache, int64_t H, int64_t D) {
  const int f32 = act(proj, "proj");
  same_act(cache, f32, "cache");
  TORCH_CHECK(proj.dim() == 2 && cache.dim() == 4, "proj, cache");
  Heads s{f32, proj.size(0), H, cache.size(1), D, cache.size(3) - D,
          cache.size(2)};
  TORCH_CHECK(D > 0 && s.V > 0 && H > 0 && H % s.G == 0 &&
                  proj.size(1) >= H * D, "heads");
  return s;
}

// columns from `col` on: keys of all heads, then values of all heads
void store_heads(Tensor proj, int64_t col, Tensor slots, Tensor cache,
                 int64_t dim) {
  const int f32 = act(proj, "proj");
  same_act(cache, f32, "cache");
  TORCH_CHECK(proj.dim() == 2 && cache.dim() == 4, "proj, cache");
  const int64_t G = cache.size(1), W = cache.size(3);
  TORCH_CHECK(dim >= 0 && dim <= W && col >= 0 &&
                  col + G * W <= proj.size(1), "columns");
  check(slots, at::kLong, "slots");
  sized(slots, {proj.size(0)}, "slots");
  const int es = (int)proj.element_size();
  check_hip(lds_store_heads((const char*)proj.data_ptr() + col * es,
                            proj.size(1), slots.data_ptr<int64_t>(),
                            cache.data_ptr(), proj.size(0), (int)G,
                            (int)cache.size(2), (int)dim, (int)(W - dim), es,
                            cur_stream()),
            "store_heads");
}

// rows [base, base + n) one by one
void plain_rows(const Heads& s, const Tensor& proj, const Tensor& cache,
                const Tensor& positions, const Tensor& row_seq,
                const Tensor& block_tables, int64_t base, int64_t n,
                double scale, OptFloat sink, const Tensor& out) {
  const int64_t es = proj.element_size(), P = proj.size(1), W = s.D + s.V;
  const char* q = (const char*)proj.data_ptr() + base * P * es;
  const char* c = (const char*)cache.data_ptr();
  const void* ptr[5] = {q, q, c, c, c + s.D * es};
  const int64_t stride[10] = {P, s.D, 0, 0, W, s.bs * W, 0, W, s.bs * W,
                              s.G * s.bs * W};
  check_hip(lds_attn_rows(s.f32, ptr, stride, (int)s.D, 0, (int)s.V,
                          (int)(s.H / s.G), sink.has_value(),
                          (float)sink.value_or(0.), ip(positions), ip(row_seq),
                          (int)base, ip(block_tables),
                          (int)block_tables.size(1), (int)s.bs, nullptr, 0,
                          (float)scale,
                          (char*)out.data_ptr() + base * s.H * s.V * es,
                          s.H * s.V, s.V, (int)n, (int)s.H, cur_stream()),
            "attn_rows");
}

// proj [rows, >= H D], queries first; cache [NB, G, bs, D + V]; the first n
// rows of out [rows, H V]. bf16 in tiles where the sizes allow it, else (or
// if `plain`) row by row.
void grouped_decode(Tensor proj, Tensor cache, Tensor positions,
                    Tensor row_seq, Tensor block_tables, int64_t n, int64_t H,
                    int64_t D, double scale, OptFloat sink, int64_t max_ctx,
                    Tensor out, bool plain) {
  const Heads s = heads(proj, cache, H, D);
  same_act(out, s.f32, "out");
  sized(out, {s.rows, H * s.V}, "out");
  check_rows(positions, row_seq, 0, n);
  check(block_tables, at::kInt, "block_tables");
  TORCH_CHECK(n >= 0 && n <= s.rows, "n");
  if (s.f32 || plain ||
      !lds_grouped_decode_ok((int)D, (int)s.V, proj.size(1))) {
    plain_rows(s, proj, cache, positions, row_seq, block_tables, 0, n, scale,
               sink, out);
    return;
  }
  if (n == 0) return;
  const int parts = lds_grouped_decode_parts((int)n, (int)H, (int)s.G, (int)D,
                                             (int)s.V, (int)max_ctx);
  auto f = proj.options().dtype(at::kFloat);
  Tensor po, ml;
  if (parts > 1) {
    po = torch::empty({n, H, parts, s.V}, f);
    ml = torch::empty({n, H, parts, 2}, f);
  }
  check_hip(lds_grouped_decode(
                proj.data_ptr(), proj.size(1), cache.data_ptr(),
                ip(positions), ip(row_seq), ip(block_tables), out.data_ptr(),
                parts > 1 ? fp(po) : nullptr, parts > 1 ? fp(ml) : nullptr,
                (int)n, (int)H, (int)s.G, (int)D, (int)s.V,
                (int)block_tables.size(1), (int)s.bs, parts, (float)scale,
                sink.has_value(), (float)sink.value_or(0.), cur_stream()),
            "grouped_decode");
}

// rows [base, rows); tiles [n, 2] = (sequence, first query of its portion),
// 128 / (H / G) queries each
void grouped_prefill(Tensor proj, Tensor cache, Tensor positions,
                     Tensor row_seq, Tensor block_tables, int64_t base,
                     Tensor seq_meta, Tensor tiles, int64_t H, int64_t D,
                     double scale, OptFloat sink, Tensor out, bool plain) {
  const Heads s = heads(proj, cache, H, D);
  same_act(out, s.f32, "out");
  sized(out, {s.rows, H * s.V}, "out");
  check_rows(positions, row_seq, base, s.rows - base);
  check(block_tables, at::kInt, "block_tables");
  if (s.f32 || plain ||
      !lds_grouped_prefill_ok((int)D, (int)s.V, (int)(H / s.G),
                              proj.size(1))) {
    plain_rows(s, proj, cache, positions, row_seq, block_tables, base,
               s.rows - base, scale, sink, out);
    return;
  }
  check(seq_meta, at::kInt, "seq_meta");
  sized(seq_meta, {block_tables.size(0), 4}, "seq_meta");
  check(tiles, at::kInt, "tiles");
  sized(tiles, {tiles.size(0), 2}, "tiles");
  check_hip(lds_grouped_prefill(
                proj.data_ptr(), proj.size(1), cache.data_ptr(),
                ip(block_tables), (int)block_tables.size(1), (int)s.bs,
                ip(seq_meta), ip(tiles), (int)tiles.size(0), out.data_ptr(),
                (int)H, (int)s.G, (int)D, (int)s.V, (float)scale,
                sink.has_value(), (float)sink.value_or(0.), cur_stream()),
            "grouped_prefill");
}

// -> experts [T, top], their scores [T, top]
std::vector<Tensor> route(Tensor h, Tensor w, int64_t top) {
  const int f32 = act(h, "h");
  same_act(w, f32, "w");
  TORCH_CHECK(h.dim() == 2 && w.dim() == 2, "h, w");
  const int64_t T = h.size(0), K = h.size(1), E = w.size(0);
  sized(w, {E, K}, "w");
  TORCH_CHECK(top >= 1 && top <= E && E <= 8192, "top of experts");
  auto ids = torch::empty({T, top}, h.options().dtype(at::kInt));
  auto wt = torch::empty({T, top}, h.options().dtype(at::kFloat));
  check_hip(lds_route(f32, h.data_ptr(), w.data_ptr(), ip(ids), fp(wt), T,
                      (int)K, (int)E, (int)top, cur_stream()),
            "route");
  return {ids, wt};
}

// h [T, K], ids and weights [T, top], up [E, F, K], down [E, K, F]
// -> [T top, K]
Tensor experts(Tensor h, Tensor ids, Tensor weights, Tensor up, Tensor down,
               int64_t act_code, bool plain) {
  const int f32 = act(h, "h");
  same_act(up, f32, "up");
  same_act(down, f32, "down");
  TORCH_CHECK(h.dim() == 2 && up.dim() == 3, "h, up");
  const int64_t T = h.size(0), K = h.size(1), E = up.size(0), F = up.size(1);
  check(ids, at::kInt, "ids");
  check(weights, at::kFloat, "weights");
  TORCH_CHECK(ids.dim() == 2 && ids.size(0) == T && ids.size(1) > 0, "ids");
  const int64_t top = ids.size(1), P = T * top;
  sized(weights, {T, top}, "weights");
  sized(up, {E, F, K}, "up");
  sized(down, {E, K, F}, "down");
  TORCH_CHECK(P < (1 << 30) && E <= 8192 && act_code >= 0 && act_code < 3,
              "experts");
  auto out = torch::empty({P, K}, h.options());
  if (P == 0) return out;
  const int tile = lds_expert_tile(f32, plain, (int)P, (int)T, (int)E, (int)F,
                                   (int)K);
  const int max_tiles = lds_expert_max_tiles((int)P, (int)E, tile);
  auto order = torch::empty({P}, ids.options());
  auto tiles = torch::empty({1 + max_tiles, 4}, ids.options());
  auto inner = torch::empty({P, F}, h.options());
  check_hip(lds_sort_pairs(ip(ids), ip(order), tiles.data_ptr(), (int)P,
                           (int)E, tile, cur_stream()),
            "sort_pairs");
  check_hip(lds_expert_product(f32, plain, 1, h.data_ptr(), up.data_ptr(),
                               inner.data_ptr(), ip(order), tiles.data_ptr(),
                               max_tiles, tile, fp(weights), (int)F, (int)K,
                               (int)top, (int)act_code, cur_stream()),
            "expert_product");
  check_hip(lds_expert_product(f32, plain, 0, inner.data_ptr(),
                               down.data_ptr(), out.data_ptr(), ip(order),
                               tiles.data_ptr(), max_tiles, tile, fp(weights),
                               (int)K, (int)F, (int)top, (int)act_code,
                               cur_stream()),
            "expert_product");
  return out;
}

}  // namespace

void bind_grouped(pybind11::module& m) {
  m.def("store_heads", &store_heads);
  m.def("grouped_decode", &grouped_decode);
  m.def("grouped_prefill", &grouped_prefill);
  m.def("route", &route);
  m.def("experts", &experts);
}
