// ops.hip — torch binding of the layered-model kernels (`_hip_layered`).
#include "check.h"

extern "C" {
hipError_t lds_stream_norm(int, int, const void* const*, int64_t, int, int,
                           float, float, float, hipStream_t);
hipError_t lds_act(int, int, const void*, void*, int64_t, int, int,
                   hipStream_t);
hipError_t lds_delta_prep(int, const void*, int64_t, const float*, void*,
                          const int32_t*, const int32_t*, float*, float*,
                          float*, int, int, int, int, int, int, int, int,
                          float, float, hipStream_t);
hipError_t lds_delta_step(int, const float*, const float*, const float*,
                          const void*, int64_t, const void*, const float*,
                          const float*, const void*, const float*, float*,
                          const int32_t*, void*, int, int, int, int, int,
                          float, hipStream_t);
int64_t lds_delta_chunk_work(int, int);
hipError_t lds_delta_chunk(int, const float*, const float*, const float*,
                           const void*, int64_t, const void*, const float*,
                           const float*, float*, const int32_t*, int,
                           const int32_t*, int, float*, float*, int, int, int,
                           int, hipStream_t);
hipError_t lds_delta_gate(int, const float*, const void*, const float*, void*,
                          int64_t, int, float, hipStream_t);
hipError_t lds_latent_prep(int, const void*, int64_t, const float*,
                           const float*, const float*, const int32_t*,
                           const int64_t*, void*, void*, int, int, int, int,
                           float, hipStream_t);
hipError_t lds_rope_part(int, void*, void*, const float*, const int32_t*, int,
                         int, int, int, int, hipStream_t);
hipError_t lds_heads_to_rows(int, const void*, void*, int, int, int,
                             hipStream_t);
hipError_t lds_gather_rows(const void*, const int64_t*, void*, int64_t,
                           int64_t, hipStream_t);
int lds_latent_decode_ok(int, int, int);
int lds_latent_decode_parts(int, int, int, int);
hipError_t lds_latent_decode(const void*, const void*, const void*,
                             const int32_t*, const int32_t*, const int32_t*,
                             void*, float*, float*, int, int, int, int, int,
                             int, int, int, int, float, hipStream_t);
int lds_latent_prefill_ok(int, int, int, int);
hipError_t lds_latent_prefill(const void*, const void*, const void*,
                              const int32_t*, const int32_t*, const int32_t*,
                              int, void*, int, int, int, int, int, int, float,
                              hipStream_t);
}

namespace {

void check_batch(const Tensor& row_seq, const Tensor& seq_meta, int64_t rows) {
  check(row_seq, at::kInt, "row_seq");
  check(seq_meta, at::kInt, "seq_meta");
  sized(row_seq, {rows}, "row_seq");
  TORCH_CHECK(seq_meta.dim() == 2 && seq_meta.size(1) == 4, "seq_meta");
}

enum Mode { EMBED, POST, ADD, LOOP };

void* ptr_or_null(const OptTensor& t) { return t ? t->data_ptr() : nullptr; }

void check_norm(const OptTensor& w, int64_t H, const char* name) {
  if (!w) return;
  check(*w, at::kFloat, name);
  sized(*w, {H}, name);
}

// without wn the stream itself comes back
Tensor stream_norm(Tensor x, OptTensor y, OptTensor wb, OptTensor wn,
                   double offset, double eps, bool f32, OptTensor added) {
  check(x, at::kFloat, "x");
  TORCH_CHECK(x.dim() == 2, "x");
  const int64_t rows = x.size(0), H = x.size(1);
  check_norm(wn, H, "wn");
  check_norm(wb, H, "wb");
  if (y) {
    same_act(*y, f32, "y");
    sized(*y, {rows, H}, "y");
  }
  TORCH_CHECK(y || !wb, "wb goes with y");
  int64_t n = 0;
  if (added) {
    same_act(*added, f32, "rows");
    n = rows ? added->size(0) / rows : 0;
    sized(*added, {rows * n, H}, "rows");
  }
  auto h = torch::empty({rows, H},
                        x.options().dtype(f32 ? at::kFloat : at::kBFloat16));
  const void* ptr[12] = {x.data_ptr(), ptr_or_null(y), nullptr, nullptr,
                         nullptr, ptr_or_null(wb), ptr_or_null(added), nullptr,
                         nullptr, nullptr, ptr_or_null(wn), h.data_ptr()};
  check_hip(lds_stream_norm(f32, wb ? POST : ADD, ptr, rows, (int)n, (int)H,
                            1.f, (float)offset, (float)eps, cur_stream()),
            "stream_norm");
  return h;
}

std::vector<Tensor> embed_norm(Tensor ids, Tensor table, double scale,
                               OptTensor wn, double offset, double eps,
                               OptTensor pos, OptTensor positions) {
  check(ids, at::kLong, "ids");
  const int f32 = act(table, "table");
  const int64_t rows = ids.numel(), H = table.size(1);
  check_norm(wn, H, "wn");
  if (pos) {
    check(*pos, at::kFloat, "pos");
    sized(*pos, {pos->size(0), H}, "pos");
    TORCH_CHECK(positions.has_value(), "positions go with pos");
    check(*positions, at::kInt, "positions");
    sized(*positions, {rows}, "positions");
  }
  auto x = torch::empty({rows, H}, table.options().dtype(at::kFloat));
  auto h = torch::empty({rows, H}, table.options());
  const void* ptr[12] = {x.data_ptr(), table.data_ptr(), ids.data_ptr(),
                         ptr_or_null(pos),
                         pos ? positions->data_ptr() : nullptr, nullptr,
                         nullptr, nullptr, nullptr, nullptr, ptr_or_null(wn),
                         h.data_ptr()};
  check_hip(lds_stream_norm(f32, EMBED, ptr, rows, 0, (int)H, (float)scale,
                            (float)offset, (float)eps, cur_stream()),
            "embed_norm");
  return {x, h};
}

// x = a + b + v
Tensor loop_norm(Tensor x, Tensor a, Tensor b, Tensor v, OptTensor wn,
                 double offset, double eps, bool f32) {
  check(x, at::kFloat, "x");
  TORCH_CHECK(x.dim() == 2, "x");
  const int64_t rows = x.size(0), H = x.size(1);
  for (const Tensor& t : {a, b}) {
    check(t, at::kFloat, "a, b");
    sized(t, {rows, H}, "a, b");
  }
  check_norm(v, H, "v");
  check_norm(wn, H, "wn");
  auto h = torch::empty({rows, H},
                        x.options().dtype(f32 ? at::kFloat : at::kBFloat16));
  const void* ptr[12] = {x.data_ptr(), nullptr, nullptr, nullptr, nullptr,
                         nullptr, nullptr, a.data_ptr(), b.data_ptr(),
                         v.data_ptr(), ptr_or_null(wn), h.data_ptr()};
  check_hip(lds_stream_norm(f32, LOOP, ptr, rows, 0, (int)H, 1.f,
                            (float)offset, (float)eps, cur_stream()),
            "loop_norm");
  return h;
}

Tensor act_rows(const Tensor& x, int64_t I, int gated, int64_t code) {
  const int f32 = act(x, "x");
  TORCH_CHECK(code >= 0 && code < 3, "activation ", code);
  auto y = torch::empty({x.size(0), I}, x.options());
  check_hip(lds_act(f32, gated, x.data_ptr(), y.data_ptr(), x.size(0), (int)I,
                    (int)code, cur_stream()),
            "act");
  return y;
}

Tensor gated_act(Tensor gate_up, int64_t code) {
  TORCH_CHECK(gate_up.dim() == 2 && gate_up.size(1) % 2 == 0, "gate_up");
  return act_rows(gate_up, gate_up.size(1) / 2, 1, code);
}

Tensor activate(Tensor x, int64_t code) {
  TORCH_CHECK(x.dim() == 2, "x");
  return act_rows(x, x.size(1), 0, code);
}

std::vector<Tensor> delta_prep(Tensor proj, Tensor taps, Tensor conv_state,
                               Tensor row_seq, Tensor seq_meta,
                               bool multi_row, int64_t KH, int64_t H,
                               int64_t K, int64_t V, double q_scale,
                               double unit_eps) {
  const int f32 = act(proj, "proj");
  const int64_t rows = proj.size(0), n_taps = taps.size(0);
  const int64_t C = 2 * KH * K + H * V;
  check(taps, at::kFloat, "taps");
  sized(taps, {n_taps, C}, "taps");
  same_act(conv_state, f32, "conv_state");
  sized(conv_state, {conv_state.size(0), n_taps - 1, C}, "conv_state");
  TORCH_CHECK(proj.size(1) >= C, "proj is narrower than its channels");
  check_batch(row_seq, seq_meta, rows);
  auto opt = proj.options().dtype(at::kFloat);
  auto q = torch::empty({rows, KH, K}, opt), k = torch::empty({rows, KH, K}, opt);
  auto v = torch::empty({rows, H, V}, opt);
  check_hip(lds_delta_prep(f32, proj.data_ptr(), proj.size(1), fp(taps),
                           conv_state.data_ptr(), ip(row_seq), ip(seq_meta),
                           fp(q), fp(k), fp(v), (int)rows,
                           (int)seq_meta.size(0), multi_row, (int)KH, (int)H,
                           (int)K, (int)V, (int)n_taps, (float)q_scale,
                           (float)unit_eps, cur_stream()),
            "delta_prep");
  return {q, k, v};
}

void check_delta(const Tensor& q, const Tensor& k, const Tensor& v,
                 const Tensor& proj, int64_t beta_col, const Tensor& decay,
                 const Tensor& dt_bias, const Tensor& neg_a,
                 const Tensor& state, int f32) {
  const int64_t rows = q.size(0), KH = q.size(1), K = q.size(2);
  const int64_t H = v.size(1), V = v.size(2);
  check(q, at::kFloat, "q");
  check(k, at::kFloat, "k");
  check(v, at::kFloat, "v");
  sized(k, {rows, KH, K}, "k");
  sized(v, {rows, H, V}, "v");
  TORCH_CHECK(H % KH == 0, "heads per key head");
  same_act(proj, f32, "proj");
  TORCH_CHECK(proj.size(0) == rows && beta_col >= 0 &&
                  beta_col + H <= proj.size(1), "beta columns");
  same_act(decay, f32, "decay");
  sized(decay, {rows, H * K}, "decay");
  check(dt_bias, at::kFloat, "dt_bias");
  sized(dt_bias, {H * K}, "dt_bias");
  check(neg_a, at::kFloat, "neg_a");
  sized(neg_a, {H}, "neg_a");
  check(state, at::kFloat, "state");
  sized(state, {state.size(0), H, K, V}, "state");
}

// the first n_seqs sequences of seq_meta; out gets their rows
void delta_step(Tensor q, Tensor k, Tensor v, Tensor proj, int64_t beta_col,
                Tensor decay, Tensor dt_bias, Tensor neg_a, Tensor gate,
                Tensor norm_w, Tensor state, Tensor seq_meta, int64_t n_seqs,
                Tensor out, double eps) {
  const int f32 = act(out, "out");
  check_delta(q, k, v, proj, beta_col, decay, dt_bias, neg_a, state, f32);
  const int64_t rows = q.size(0), KH = q.size(1), K = q.size(2);
  const int64_t H = v.size(1), V = v.size(2);
  same_act(gate, f32, "gate");
  sized(gate, {rows, H * V}, "gate");
  sized(out, {rows, H * V}, "out");
  check(norm_w, at::kFloat, "norm_w");
  sized(norm_w, {V}, "norm_w");
  check(seq_meta, at::kInt, "seq_meta");
  TORCH_CHECK(n_seqs <= seq_meta.size(0) && seq_meta.size(1) == 4, "n_seqs");
  const char* beta = (const char*)proj.data_ptr() +
                     beta_col * proj.element_size();
  check_hip(lds_delta_step(f32, fp(q), fp(k), fp(v), beta, proj.size(1),
                           decay.data_ptr(), fp(dt_bias), fp(neg_a),
                           gate.data_ptr(), fp(norm_w), fp(state),
                           ip(seq_meta), out.data_ptr(), (int)n_seqs, (int)KH,
                           (int)H, (int)K, (int)V, (float)eps, cur_stream()),
            "delta_step");
}

// chunks [n, 2] = first row, tokens (1..64); walk [s, 4] = first row, tokens,
// slot, first chunk | 1 << 30 for a state that starts at zero. Both on the
// CPU as well (*_host): the kernels index with them unchecked.
void delta_chunk(Tensor q, Tensor k, Tensor v, Tensor proj, int64_t beta_col,
                 Tensor decay, Tensor dt_bias, Tensor neg_a, Tensor state,
                 Tensor chunks, Tensor walk, Tensor chunks_host,
                 Tensor walk_host, Tensor ws, Tensor out) {
  const int f32 = act(proj, "proj");
  check_delta(q, k, v, proj, beta_col, decay, dt_bias, neg_a, state, f32);
  const int64_t rows = q.size(0), KH = q.size(1), K = q.size(2);
  const int64_t H = v.size(1), V = v.size(2);
  check(chunks, at::kInt, "chunks");
  check(walk, at::kInt, "walk");
  const int64_t nc = chunks.size(0), ns = walk.size(0);
  sized(chunks, {nc, 2}, "chunks");
  sized(walk, {ns, 4}, "walk");
  sized(chunks_host, {nc, 2}, "chunks_host");
  sized(walk_host, {ns, 4}, "walk_host");
  const auto c = chunks_host.accessor<int32_t, 2>();
  const auto w = walk_host.accessor<int32_t, 2>();
  for (int64_t i = 0; i < nc; ++i)
    TORCH_CHECK(c[i][0] >= 0 && c[i][1] > 0 && c[i][1] <= 64 &&
                    c[i][0] + c[i][1] <= rows, "chunk ", i);
  for (int64_t i = 0; i < ns; ++i)
    TORCH_CHECK(w[i][0] >= 0 && w[i][1] > 0 && w[i][0] + w[i][1] <= rows &&
                    w[i][2] >= 0 && w[i][2] < state.size(0) &&
                    (w[i][3] & ((1 << 30) - 1)) + (w[i][1] + 63) / 64 <= nc,
                "walk ", i);
  check(ws, at::kFloat, "ws");
  check(out, at::kFloat, "out");
  sized(out, {rows, H * V}, "out");
  const int64_t work = lds_delta_chunk_work((int)K, (int)V);
  TORCH_CHECK(work > 0 && ws.numel() >= work * nc * H, "ws");
  const char* beta = (const char*)proj.data_ptr() +
                     beta_col * proj.element_size();
  check_hip(lds_delta_chunk(f32, fp(q), fp(k), fp(v), beta, proj.size(1),
                            decay.data_ptr(), fp(dt_bias), fp(neg_a),
                            fp(state), ip(chunks), (int)nc, ip(walk), (int)ns,
                            fp(ws), fp(out), (int)KH, (int)H, (int)K, (int)V,
                            cur_stream()),
            "delta_chunk");
}

// rows [base, rows) of o [rows, H V] -> out
void delta_gate(Tensor o, Tensor gate, Tensor norm_w, Tensor out,
                int64_t base, double eps) {
  check(o, at::kFloat, "o");
  const int f32 = act(out, "out");
  same_act(gate, f32, "gate");
  check(norm_w, at::kFloat, "norm_w");
  const int64_t rows = o.size(0), HV = o.size(1), V = norm_w.size(0);
  sized(gate, {rows, HV}, "gate");
  sized(out, {rows, HV}, "out");
  TORCH_CHECK(HV % V == 0 && base >= 0 && base <= rows, "delta_gate");
  const int64_t at = base * HV, es = out.element_size();
  check_hip(lds_delta_gate(f32, fp(o) + at,
                           (const char*)gate.data_ptr() + at * es,
                           fp(norm_w), (char*)out.data_ptr() + at * es,
                           (rows - base) * (HV / V), (int)V, (float)eps,
                           cur_stream()),
            "delta_gate");
}

Tensor latent_prep(Tensor proj, Tensor wq, OptTensor wkv, Tensor cos_sin,
                   Tensor positions, Tensor slots, OptTensor cache,
                   double eps) {
  const int f32 = act(proj, "proj");
  const int64_t rows = proj.size(0), q_rank = wq.size(0);
  check(wq, at::kFloat, "wq");
  check(positions, at::kInt, "positions");
  check(slots, at::kLong, "slots");
  sized(positions, {rows}, "positions");
  sized(slots, {rows}, "slots");
  int64_t kv_rank = 0, rot = 0;
  if (cache) {
    same_act(*cache, f32, "cache");
    check(*wkv, at::kFloat, "wkv");
    check(cos_sin, at::kFloat, "cos_sin");
    kv_rank = wkv->size(0);
    rot = cache->size(2) - kv_rank;
    sized(cos_sin, {cos_sin.size(0), rot / 2, 2}, "cos_sin");
  }
  TORCH_CHECK(rot % 2 == 0, "rotated size");
  sized(proj, {rows, q_rank + kv_rank + rot}, "proj");
  auto cq = torch::empty({rows, q_rank}, proj.options());
  check_hip(lds_latent_prep(f32, proj.data_ptr(), proj.size(1), fp(wq),
                            cache ? fp(*wkv) : nullptr,
                            cache ? fp(cos_sin) : nullptr, ip(positions),
                            slots.data_ptr<int64_t>(), cq.data_ptr(),
                            cache ? cache->data_ptr() : nullptr, (int)rows,
                            (int)q_rank, (int)kv_rank, (int)rot, (float)eps,
                            cur_stream()),
            "latent_prep");
  return cq;
}

// rotates q [rows, H, D + rot] in place; -> [H, n_abs, D]
Tensor rope_part(Tensor q, Tensor cos_sin, Tensor positions, int64_t n_abs) {
  const int f32 = act(q, "q");
  check(cos_sin, at::kFloat, "cos_sin");
  check(positions, at::kInt, "positions");
  const int64_t rows = q.size(0), H = q.size(1);
  const int64_t rot = cos_sin.size(1) * 2, D = q.size(2) - rot;
  sized(cos_sin, {cos_sin.size(0), rot / 2, 2}, "cos_sin");
  sized(positions, {rows}, "positions");
  TORCH_CHECK(D >= 0 && n_abs <= rows, "q");
  auto by_head = torch::empty({H, n_abs, D}, q.options());
  check_hip(lds_rope_part(f32, q.data_ptr(), by_head.data_ptr(), fp(cos_sin),
                          ip(positions), (int)rows, (int)n_abs, (int)H, (int)D,
                          (int)rot, cur_stream()),
            "rope_part");
  return by_head;
}

// src [H, n, V] -> the first n rows of dst [rows, H V]
void heads_to_rows(Tensor src, Tensor dst) {
  const int f32 = act(src, "src");
  same_act(dst, f32, "dst");
  TORCH_CHECK(dst.dim() == 2 && dst.size(0) >= src.size(1) &&
                  dst.size(1) == src.size(0) * src.size(2), "dst");
  check_hip(lds_heads_to_rows(f32, src.data_ptr(), dst.data_ptr(),
                              (int)src.size(1), (int)src.size(0),
                              (int)src.size(2), cur_stream()),
            "heads_to_rows");
}

Tensor gather_rows(Tensor cache, Tensor slots) {
  act(cache, "cache");
  check(slots, at::kLong, "slots");
  const int64_t w = cache.size(-1);
  auto out = torch::empty({slots.numel(), w}, cache.options());
  check_hip(lds_gather_rows(cache.data_ptr(), slots.data_ptr<int64_t>(),
                            out.data_ptr(), slots.numel(),
                            w * cache.element_size(), cur_stream()),
            "gather_rows");
  return out;
}

// q_lat [H, n, R], q [rows, H, D + rot] rotated, cache [NB, BS, R + rot];
// -> [H, n, R], the first n rows of the batch. bf16 in tiles where the sizes
// allow it, else (or if `plain`) row by row.
Tensor latent_decode(Tensor q_lat, Tensor q, Tensor cache, Tensor positions,
                     Tensor row_seq, Tensor block_tables, int64_t window,
                     double scale, int64_t max_ctx, bool plain) {
  const int f32 = act(q_lat, "q_lat");
  same_act(q, f32, "q");
  same_act(cache, f32, "cache");
  check(block_tables, at::kInt, "block_tables");
  const int64_t H = q_lat.size(0), n = q_lat.size(1), R = q_lat.size(2);
  const int64_t W = cache.size(2), rot = W - R, Q = q.size(2);
  check_rows(positions, row_seq, 0, n);
  TORCH_CHECK(rot >= 0 && Q >= rot && q.size(0) >= n && q.size(1) == H, "q");
  auto out = torch::empty_like(q_lat);
  if (!f32 && !plain && lds_latent_decode_ok((int)R, (int)rot, (int)Q)) {
    const int parts = lds_latent_decode_parts((int)n, (int)H, (int)max_ctx,
                                              (int)window);
    auto f = q.options().dtype(at::kFloat);
    Tensor po, ml;
    if (parts > 1) {
      po = torch::empty({n, H, parts, R}, f);
      ml = torch::empty({n, H, parts, 2}, f);
    }
    check_hip(lds_latent_decode(
                  q_lat.data_ptr(), q.data_ptr(), cache.data_ptr(),
                  ip(positions), ip(row_seq), ip(block_tables),
                  out.data_ptr(), parts > 1 ? fp(po) : nullptr,
                  parts > 1 ? fp(ml) : nullptr, (int)n, (int)H, (int)R,
                  (int)rot, (int)Q, (int)block_tables.size(1),
                  (int)cache.size(1), (int)window, parts, (float)scale,
                  cur_stream()),
              "latent_decode");
    return out;
  }
  const int64_t es = q.element_size();
  const char* c = (const char*)cache.data_ptr();
  const void* ptr[5] = {q_lat.data_ptr(),
                        (const char*)q.data_ptr() + (Q - rot) * es, c,
                        c + R * es, c};
  const int64_t stride[10] = {R, n * R, H * Q, Q, W, 0, W, W, 0,
                              cache.size(1) * W};
  check_hip(lds_attn_rows(f32, ptr, stride, (int)R, (int)rot, (int)R, (int)H,
                          0, 0.f,
                          ip(positions), ip(row_seq), 0, ip(block_tables),
                          (int)block_tables.size(1), (int)cache.size(1),
                          nullptr, (int)window, (float)scale, out.data_ptr(),
                          R, n * R, (int)n, (int)H, cur_stream()),
            "attn_rows");
  return out;
}

// rows [base, rows): kv [ctx rows, H D + H V], lat [ctx rows, R + rot],
// ctx [n_seqs, 2] = (first context row, its position); out [rows, H V].
// tiles [n, 2] = (sequence, first row of 128 in its portion).
void latent_prefill(Tensor q, Tensor kv, Tensor lat, Tensor positions,
                    Tensor row_seq, int64_t base, Tensor seq_meta, Tensor ctx,
                    Tensor tiles, int64_t rot, int64_t window, double scale,
                    Tensor out, bool plain) {
  const int f32 = act(q, "q");
  same_act(kv, f32, "kv");
  same_act(lat, f32, "lat");
  same_act(out, f32, "out");
  check(ctx, at::kInt, "ctx");
  const int64_t rows = q.size(0), H = q.size(1), Q = q.size(2), D = Q - rot;
  const int64_t V = out.size(1) / H, W = lat.size(1);
  check_rows(positions, row_seq, base, rows - base);
  sized(kv, {lat.size(0), H * (D + V)}, "kv");
  sized(out, {rows, H * V}, "out");
  TORCH_CHECK(D >= 0 && W >= rot && ctx.dim() == 2 && ctx.size(1) == 2, "ctx");
  if (!f32 && !plain &&
      lds_latent_prefill_ok((int)D, (int)rot, (int)V, (int)(W - rot))) {
    check(seq_meta, at::kInt, "seq_meta");
    check(tiles, at::kInt, "tiles");
    sized(seq_meta, {ctx.size(0), 4}, "seq_meta");
    sized(tiles, {tiles.size(0), 2}, "tiles");
    check_hip(lds_latent_prefill(q.data_ptr(), kv.data_ptr(), lat.data_ptr(),
                                 ip(seq_meta), ip(ctx), ip(tiles),
                                 (int)tiles.size(0), out.data_ptr(), (int)H,
                                 (int)D, (int)rot, (int)V, (int)W,
                                 (int)window, (float)scale, cur_stream()),
              "latent_prefill");
    return;
  }
  const int64_t es = q.element_size(), KV = kv.size(1);
  const char* qp = (const char*)q.data_ptr() + base * H * Q * es;
  const char* kp = (const char*)kv.data_ptr();
  const void* ptr[5] = {qp, qp + D * es, kp,
                        (const char*)lat.data_ptr() + (W - rot) * es,
                        kp + H * D * es};
  const int64_t stride[10] = {H * Q, Q, H * Q, Q, KV, D, W, KV, V, 0};
  check_hip(lds_attn_rows(f32, ptr, stride, (int)D, (int)rot, (int)V, 1, 0,
                          0.f,
                          ip(positions), ip(row_seq), (int)base, nullptr, 0, 1,
                          ip(ctx), (int)window, (float)scale,
                          (char*)out.data_ptr() + base * H * V * es, H * V, V,
                          (int)(rows - base), (int)H, cur_stream()),
            "attn_rows");
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "gfx950 kernels of the layer-listed designs";
  m.def("stream_norm", &stream_norm);
  m.def("embed_norm", &embed_norm);
  m.def("loop_norm", &loop_norm);
  m.def("gated_act", &gated_act);
  m.def("activate", &activate);
  m.def("delta_prep", &delta_prep);
  m.def("delta_step", &delta_step);
  m.def("delta_chunk_work", &lds_delta_chunk_work);
  m.def("delta_chunk", &delta_chunk);
  m.def("delta_gate", &delta_gate);
  m.def("latent_prep", &latent_prep);
  m.def("rope_part", &rope_part);
  m.def("heads_to_rows", &heads_to_rows);
  m.def("gather_rows", &gather_rows);
  m.def("latent_decode", &latent_decode);
  m.def("latent_prefill", &latent_prefill);
  bind_grouped(m);
}
