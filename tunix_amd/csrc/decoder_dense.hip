// Layers of one pass of a TMX_FAMILY_DENSE model.  A layer is a mixer and a feed-forward, with a row kernel between two
// sublayers that applies the first one's result to the residual and makes the second one's input:
//   latent attention   fused projection (query | latent | gate), rotation / norm / cache row and query into the latent
//                      space (one launch up to 128 rows), attention over the cache rows, values (with the output gate
//                      in the epilogue), output projection
//   grouped attention  fused projection (query | key | value heads), norm / rotation / cache rows and attention (one
//                      launch for one token per sequence), output projection
//   feed-forward       gate | up with SwiGLU or up with a squared relu, down
//   residual           streams mixed at every boundary with a norm in front of the sublayers (stream_rows), or one stream
//                      with the norm behind them (residual_rows)
#include <algorithm>

#include "tmx_decoder.h"

namespace tmx {

static size_t act_bytes(const tmx_model_desc* m) { return m->act == TMX_ACT_F32 ? 4 : 2; }

// The different chunk sizes of the layers with grouped attention.
static std::vector<int> chunk_sizes(const tmx_model_desc* m) {
  std::vector<int> out;
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_dense_layer_desc& l = m->dense_layers[i];
    if (l.mixer == TMX_MIXER_HEADS && std::find(out.begin(), out.end(), l.chunk) == out.end()) out.push_back(l.chunk);
  }
  return out;
}

DenseWorkspace dense_carve(const tmx_model_desc* m, int rows, char* base) {
  DenseWorkspace w = {};
  size_t off = 0;
  auto take = [&](size_t bytes) { char* p = (base && bytes) ? base + off : nullptr; off += align256(bytes); return p; };
  const size_t B = rows, Bt = pad_to(rows, 32), Dp = pad_to(m->embed_dim, 64), e = act_bytes(m);
  size_t z = 0, q = 0, lat = 0, val = 0, act = 0, part = 0, splits = 1;
  auto up = [](size_t& d, size_t v) { if (v > d) d = v; };
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_dense_layer_desc& l = m->dense_layers[i];
    up(z, l.in.N);
    up(val, (size_t)l.heads * l.vdim_p);
    up(splits, dense_num_splits(m->act, rows, l.o.K, l.o.N));
    if (l.mixer == TMX_MIXER_HEADS) {
      up(q, (size_t)l.heads * l.dim_p);
      if (m->act == TMX_ACT_BF16) up(part, head_attn_partial_bytes(rows, l.heads, l.vdim_p));
    } else {
      up(q, (size_t)l.heads * (l.rank_p + l.rot_p));
      up(lat, (size_t)l.heads * l.rank_p);
      if (m->act == TMX_ACT_BF16) up(part, latent_attn_partial_bytes(rows, l.heads, l.rank_p));
    }
    if (l.gate_up.w) {
      up(act, l.down.K);
      up(splits, dense_num_splits(m->act, rows, l.down.K, l.down.N));
    }
  }
  take(256);  // status block
  w.xs = (float*)take(B * m->streams * Dp * 4);
  w.xn = take(Bt * Dp * e);
  w.z = take(B * z * e);
  w.q = take(B * q * e);
  w.lat = take(B * lat * e);
  w.val = take(Bt * val * e);
  w.y = take(B * Dp * e);
  w.act = take(Bt * act * e);
  w.place = (int2*)take(chunk_sizes(m).size() * B * 8);
  w.attn_partial = (float*)take(part);
  w.y_part = (float*)take(splits > 1 ? splits * B * Dp * 4 : 0);
  const size_t Vp = pad_to(m->vocab_size, 32);
  w.logits = (float*)take(m->act == TMX_ACT_F32 ? B * Vp * 4 : 0);
  w.head_partial = take(head_partial_bytes(rows, (int)Vp));
  w.total = off;
  return w;
}

static int check_dense(const tmx_dense_desc& d, int K, int N, int heads) {
  if (!d.w) return TMX_ERR_ARG;
  if (d.K != K || d.N != N || d.heads != heads || K % 64 || N % 32) return TMX_ERR_SHAPE;
  return TMX_OK;
}

static int check_latent(const tmx_model_desc* m, int i) {
  const tmx_dense_layer_desc& l = m->dense_layers[i];
  if (l.kv_rank > l.rank_p || l.rot_dim > l.rot_p || l.rot_dim % 2 || !latent_attn_ok(l.rank_p, l.rot_p)) return TMX_ERR_SHAPE;
  if (!l.table || l.kv_layer < 0 || l.kv_layer > i || (l.off_kv >= 0) != (l.kv_layer == i)) return TMX_ERR_ARG;
  const tmx_dense_layer_desc& src = m->dense_layers[l.kv_layer];
  if (src.mixer != TMX_MIXER_LATENT || src.off_kv < 0 || src.rank_p != l.rank_p || src.rot_p != l.rot_p) return TMX_ERR_ARG;
  if (l.off_kv >= 0 && !l.kv_norm_w) return TMX_ERR_ARG;
  int rc;
  if ((rc = check_dense(l.uk, l.dim_p, l.rank_p, l.heads)) || (rc = check_dense(l.uv, l.rank_p, l.vdim_p, l.heads))) return rc;
  // columns of the fused projection stay inside it
  if (l.off_qr < l.heads * l.dim_p || l.off_qr + l.heads * l.rot_dim > l.in.N ||
      (l.off_kv >= 0 && l.off_kv + l.kv_rank + l.rot_dim > l.in.N) ||
      (l.off_gate >= 0 && l.off_gate + l.heads * l.vdim_p > l.in.N))
    return TMX_ERR_SHAPE;
  return TMX_OK;
}

static int check_heads(const tmx_dense_layer_desc& l) {
  if (l.kv_heads <= 0 || l.heads % l.kv_heads || l.dim <= 0 || l.dim > l.dim_p || l.rot_dim < 0 || l.rot_dim % 2 ||
      l.rot_dim > l.dim || l.chunk < 0 || !head_attn_ok(l.dim_p, l.vdim_p))
    return TMX_ERR_SHAPE;
  if (l.rot_dim > 0 && !l.table) return TMX_ERR_ARG;
  return l.in.N == l.heads * l.dim_p + l.kv_heads * (l.dim_p + l.vdim_p) ? TMX_OK : TMX_ERR_SHAPE;
}

int dense_check(const tmx_model_desc* m) {
  if (!m->dense_layers || (!m->norm_after && !m->final_in)) return TMX_ERR_ARG;
  if (m->act != TMX_ACT_BF16 && m->act != TMX_ACT_F32) return TMX_ERR_ARG;
  if (m->streams < 1 || m->streams > TMX_MAX_STREAMS || m->max_positions <= 0 || m->num_layers <= 0) return TMX_ERR_SHAPE;
  if (m->norm_after && (m->streams != 1 || m->pos_embed)) return TMX_ERR_UNSUPPORTED;
  const int Dp = pad_to(m->embed_dim, 64);
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_dense_layer_desc& l = m->dense_layers[i];
    auto streams_ok = [&](const tmx_streams_desc& hc) { return m->norm_after || (hc.in && hc.out && hc.mix); };
    if (!l.norm1_w || !streams_ok(l.hc1)) return TMX_ERR_ARG;
    if (l.heads <= 0 || l.dim_p <= 0 || l.dim_p % 64 || l.vdim_p <= 0 || l.vdim_p % 64) return TMX_ERR_SHAPE;
    int rc;
    if ((rc = check_dense(l.in, Dp, l.in.N, 1)) || (rc = check_dense(l.o, l.heads * l.vdim_p, Dp, 1))) return rc;
    if (l.mixer == TMX_MIXER_LATENT) rc = check_latent(m, i);
    else rc = l.mixer == TMX_MIXER_HEADS ? check_heads(l) : TMX_ERR_UNSUPPORTED;
    if (rc) return rc;
    if (l.gate_up.w) {
      if (!l.norm2_w || !streams_ok(l.hc2)) return TMX_ERR_ARG;
      if (l.ff != TMX_DENSE_SWIGLU && l.ff != TMX_DENSE_RELU2) return TMX_ERR_UNSUPPORTED;
      const int per = l.ff == TMX_DENSE_SWIGLU ? 2 : 1;
      if ((rc = check_dense(l.gate_up, Dp, l.gate_up.N, 1)) || l.gate_up.N % (64 * per)) return rc ? rc : TMX_ERR_SHAPE;
      if ((rc = check_dense(l.down, l.gate_up.N / per, Dp, 1))) return rc;
    }
  }
  return TMX_OK;
}

int dense_layers(hipStream_t st, const tmx_model_desc* m, const tmx_decode_state* s, const DenseWorkspace& w,
                  int n_seq, int T, bool final_norm, Prof* prof) {
  const int M = n_seq * T, C = s->cache_size, L = s->buf_len, Dp = pad_to(m->embed_dim, 64), act = m->act;
  const size_t e = act_bytes(m);
  int rc;
  // up to 128 bf16 rows: the inputs of the plain projections travel in the order the matrix pipe reads them
  const bool tiled = act == TMX_ACT_BF16 && M <= 128;
  auto args = [&](const tmx_dense_desc& d, const void* x, int ldx, int x_head, void* y, int ldy, int y_head, int epi) {
    DenseArgs a = {};
    a.x = x; a.ldx = ldx; a.x_head = x_head;
    a.w = d.w; a.bias = d.bias;
    a.y = y; a.ldy = ldy; a.y_head = y_head;
    a.M = M; a.K = d.K; a.N = d.N; a.heads = d.heads; a.epi = epi;
    return a;
  };
  // a sublayer's last projection, whose result the next stream row kernel adds: w.y, or planes in w.y_part
  int y_splits = 1;
  auto into_streams = [&](const tmx_dense_desc& d, const void* x) {
    DenseArgs a = args(d, x, d.K, 0, w.y, Dp, 0, TMX_DENSE_PLAIN);
    a.x_tiled = tiled;
    a.nsplit = y_splits = dense_num_splits(act, M, d.K, d.N);
    a.y_part = w.y_part;
    return dense_linear(st, act, a);
  };
  // The boundary behind sublayer `prev` (its streams and its norm; null: the embedding) and in front of the next one (or,
  // with `head`, of the final norm).
  const tmx_streams_desc* prev = nullptr;
  const float* prev_norm = nullptr;
  auto boundary = [&](const float* in, const float* norm_w, bool head) {
    if (m->norm_after) {
      ResidualArgs a = {};
      a.x = w.xs; a.xn = w.xn; a.norm_w = head ? norm_w : nullptr;
      a.D = m->embed_dim; a.Dp = Dp; a.eps = m->norm_eps; a.store = !head;
      a.xn_tiled = tiled && !head;
      if (prev) {
        if (y_splits > 1) { a.y_part = w.y_part; a.nsplit = y_splits; }
        else a.y = w.y;
        a.post_w = prev_norm;
      } else {
        a.embed = (const uint16_t*)m->embed; a.embed_scale = m->embed_scale; a.vocab = m->vocab_size;
        a.token_buffer = s->token_buffer; a.step = s->step; a.buf_len = L; a.tpp = T;
      }
      return residual_rows(st, act, a, M);
    }
    StreamArgs a = {};
    a.xs = w.xs; a.in = in; a.norm_w = norm_w; a.xn = w.xn;
    a.S = m->streams; a.D = m->embed_dim; a.Dp = Dp; a.eps = m->norm_eps; a.store = !head;
    a.xn_tiled = tiled && !head;
    if (prev) {
      if (y_splits > 1) { a.y_part = w.y_part; a.nsplit = y_splits; }
      else a.y = w.y;
      a.mix = prev->mix; a.out = prev->out;
    } else {
      a.embed = (const uint16_t*)m->embed; a.pos_embed = (const uint16_t*)m->pos_embed; a.embed_scale = m->embed_scale;
      a.vocab = m->vocab_size; a.max_positions = m->max_positions;
      a.token_buffer = s->token_buffer; a.positions = s->positions; a.step = s->step; a.buf_len = L; a.tpp = T;
    }
    return stream_rows(st, act, a, M);
  };
  std::vector<char*> cache(m->num_layers, nullptr);
  {
    char* p = (char*)s->kv_cache;
    for (int i = 0; i < m->num_layers; ++i) {
      const tmx_dense_layer_desc& l = m->dense_layers[i];
      if (l.mixer == TMX_MIXER_HEADS) {
        cache[i] = p;
        p += (size_t)n_seq * C * l.kv_heads * (l.dim_p + l.vdim_p) * e;
        continue;
      }
      if (l.off_kv < 0) {
        cache[i] = cache[l.kv_layer];
        continue;
      }
      cache[i] = p;
      p += (size_t)n_seq * C * (l.rank_p + l.rot_p) * e;
    }
  }
  // from the fused projection w.z to the input of the output projection w.val
  auto latent_mixer = [&](const tmx_dense_layer_desc& l, char* cache) {
    const int ld = l.rank_p + l.rot_p, H = l.heads;
    {
      LatentRowsArgs a = {};
      a.z = w.z; a.ldz = l.in.N; a.off_qr = l.off_qr; a.off_kv = l.off_kv;
      a.norm_w = l.kv_norm_w; a.eps = m->norm_eps;
      a.table = l.table; a.max_positions = m->max_positions;
      a.positions = s->positions; a.step = s->step; a.buf_len = L; a.tpp = T;
      a.q = w.q; a.cache = cache;
      a.H = H; a.rot = l.rot_dim; a.rank = l.kv_rank; a.rank_p = l.rank_p; a.rot_p = l.rot_p; a.C = C;
      const DenseArgs d = args(l.uk, w.z, l.in.N, l.dim_p, w.q, H * ld, ld, TMX_DENSE_PLAIN);
      if (tiled) {
        TMX_TRY(TMX_K_LATENT_Q, latent_q_rows(st, d, a));
      } else {
        TMX_TRY(TMX_K_ROPE, latent_rows(st, act, a, M));
        TMX_TRY(TMX_K_LATENT_Q, dense_linear(st, act, d));
      }
    }
    {
      LatentAttnArgs a = {};
      a.q = w.q; a.cache = cache; a.sink = l.sink;
      a.input_mask = s->input_mask; a.step = s->step; a.buf_len = L;
      a.out = w.lat; a.partial = w.attn_partial;
      a.n_seq = n_seq; a.tpp = T; a.H = H; a.rank_p = l.rank_p; a.rot_p = l.rot_p; a.C = C; a.scale = l.scale;
      TMX_TRY(TMX_K_ATTN, latent_attention(st, act, a));
    }
    {
      DenseArgs a = args(l.uv, w.lat, H * l.rank_p, l.rank_p, w.val, H * l.vdim_p, l.vdim_p, TMX_DENSE_PLAIN);
      if (l.off_gate >= 0) {
        a.epi = TMX_DENSE_GATED;
        a.gate = (const char*)w.z + (size_t)l.off_gate * e;
        a.ldg = l.in.N;
      }
      a.y_tiled = tiled;
      TMX_TRY(TMX_K_LATENT_V, dense_linear(st, act, a));
    }
    return TMX_OK;
  };
  const std::vector<int> chunks = chunk_sizes(m);
  auto place_of = [&](int chunk) { return w.place + (std::find(chunks.begin(), chunks.end(), chunk) - chunks.begin()) * (size_t)M; };
  for (int chunk : chunks) {
    RowPlacesArgs a = {};
    a.positions = s->positions; a.input_mask = s->input_mask; a.step = s->step; a.buf_len = L; a.tpp = T; a.C = C;
    a.chunk = chunk; a.place = place_of(chunk);
    TMX_TRY(TMX_K_ROPE, row_places(st, a, M));
  }
  auto heads_mixer = [&](const tmx_dense_layer_desc& l, char* kcache) {
    char* vcache = kcache + (size_t)n_seq * C * l.kv_heads * l.dim_p * e;
    HeadRowsArgs r = {};
    r.z = w.z; r.ldz = l.in.N; r.q_norm_w = l.q_norm_w; r.k_norm_w = l.k_norm_w; r.eps = m->norm_eps;
    r.table = l.table; r.max_positions = m->max_positions;
    r.place = place_of(l.chunk); r.step = s->step; r.buf_len = L; r.tpp = T;
    r.q = w.q; r.kcache = kcache; r.vcache = vcache;
    r.H = l.heads; r.Kh = l.kv_heads; r.dim = l.dim; r.dk = l.dim_p; r.dv = l.vdim_p; r.rot = l.rot_dim; r.C = C;
    const bool fused = head_rows_fused(act, T, l.heads, l.kv_heads);
    if (!fused) TMX_TRY(TMX_K_ROPE, head_rows(st, act, r, M));
    HeadAttnArgs a = {};
    a.q = w.q; a.kcache = kcache; a.vcache = vcache; a.sink = l.sink; a.place = r.place;
    a.input_mask = s->input_mask; a.step = s->step; a.buf_len = L;
    a.out = w.val; a.out_tiled = tiled; a.partial = w.attn_partial;
    a.n_seq = n_seq; a.tpp = T; a.H = l.heads; a.Kh = l.kv_heads; a.dk = l.dim_p; a.dv = l.vdim_p; a.C = C;
    a.chunk = l.chunk; a.scale = l.scale;
    TMX_TRY(TMX_K_ATTN, head_attention(st, act, a, fused ? &r : nullptr));
    return TMX_OK;
  };
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_dense_layer_desc& l = m->dense_layers[i];
    TMX_TRY(TMX_K_ROWNORM, boundary(l.hc1.in, l.norm1_w, false));
    {
      DenseArgs a = args(l.in, w.xn, Dp, 0, w.z, l.in.N, 0, TMX_DENSE_PLAIN);
      a.x_tiled = tiled;
      TMX_TRY(TMX_K_QKV, dense_linear(st, act, a));
    }
    rc = l.mixer == TMX_MIXER_HEADS ? heads_mixer(l, cache[i]) : latent_mixer(l, cache[i]);
    if (rc != TMX_OK) return rc;
    TMX_TRY(TMX_K_O, into_streams(l.o, w.val));
    prev = &l.hc1;
    prev_norm = l.norm1_w;
    if (l.gate_up.w) {
      TMX_TRY(TMX_K_ROWNORM, boundary(l.hc2.in, l.norm2_w, false));
      DenseArgs a = args(l.gate_up, w.xn, Dp, 0, w.act, l.down.K, 0, l.ff);
      a.x_tiled = a.y_tiled = tiled;
      TMX_TRY(TMX_K_GATE_UP, dense_linear(st, act, a));
      TMX_TRY(TMX_K_DOWN, into_streams(l.down, w.act));
      prev = &l.hc2;
      prev_norm = l.norm2_w;
    }
    if (prof) TMX_TRY(TMX_K_EMPTY, empty_launch(st));
  }
  if (final_norm) TMX_TRY(TMX_K_ROWNORM, boundary(m->final_in, (const float*)m->final_norm_w, true));
  return TMX_OK;
}

}  // namespace tmx
