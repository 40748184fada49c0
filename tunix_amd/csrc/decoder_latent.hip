// Layers of one pass of a TMX_FAMILY_LATENT model: dense weights, latent attention, several residual streams.
// Per layer: fused projection of the normed input (query | latent | gate), rotation / norm / cache row and query into
// the latent space (one launch up to 128 rows), attention over the cache rows, values (with the output gate in the epilogue), output projection,
// stream row kernel; gate | up with SwiGLU, down, stream row kernel.  A row kernel between two sublayers applies the
// first one's result to the streams and makes the second one's normed input.
#include "tmx_decoder.h"

namespace tmx {

static size_t act_bytes(const tmx_model_desc* m) { return m->act == TMX_ACT_F32 ? 4 : 2; }

LatentWorkspace latent_carve(const tmx_model_desc* m, int rows, char* base) {
  LatentWorkspace w = {};
  size_t off = 0;
  auto take = [&](size_t bytes) { char* p = (base && bytes) ? base + off : nullptr; off += align256(bytes); return p; };
  const size_t B = rows, Bt = pad_to(rows, 32), Dp = pad_to(m->embed_dim, 64), e = act_bytes(m);
  size_t z = 0, q = 0, lat = 0, val = 0, act = 0, part = 0, splits = 1;
  auto up = [](size_t& d, size_t v) { if (v > d) d = v; };
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_latent_layer_desc& l = m->latent_layers[i];
    up(z, l.in.N);
    up(q, (size_t)l.heads * (l.rank_p + l.rot_p));
    up(lat, (size_t)l.heads * l.rank_p);
    up(val, (size_t)l.heads * l.vdim_p);
    up(splits, dense_num_splits(m->act, rows, l.o.K, l.o.N));
    if (l.gate_up.w) {
      up(act, l.gate_up.N / 2);
      up(splits, dense_num_splits(m->act, rows, l.down.K, l.down.N));
    }
    if (m->act == TMX_ACT_BF16) up(part, latent_attn_partial_bytes(rows, l.heads, l.rank_p));
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

int latent_check(const tmx_model_desc* m) {
  if (!m->latent_layers || !m->final_in) return TMX_ERR_ARG;
  if (m->act != TMX_ACT_BF16 && m->act != TMX_ACT_F32) return TMX_ERR_ARG;
  if (m->streams < 1 || m->streams > TMX_MAX_STREAMS || m->max_positions <= 0 || m->num_layers <= 0) return TMX_ERR_SHAPE;
  const int Dp = pad_to(m->embed_dim, 64);
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_latent_layer_desc& l = m->latent_layers[i];
    if (!l.norm1_w || !l.hc1.in || !l.hc1.out || !l.hc1.mix || !l.table) return TMX_ERR_ARG;
    if (l.heads <= 0 || l.dim_p % 64 || l.vdim_p % 64 || l.kv_rank > l.rank_p || l.rot_dim > l.rot_p ||
        l.rot_dim % 2 || !latent_attn_ok(l.rank_p, l.rot_p))
      return TMX_ERR_SHAPE;
    if (l.kv_layer < 0 || l.kv_layer > i || (l.off_kv >= 0) != (l.kv_layer == i)) return TMX_ERR_ARG;
    const tmx_latent_layer_desc& src = m->latent_layers[l.kv_layer];
    if (src.off_kv < 0 || src.rank_p != l.rank_p || src.rot_p != l.rot_p) return TMX_ERR_ARG;
    if (l.off_kv >= 0 && !l.kv_norm_w) return TMX_ERR_ARG;
    int rc;
    if ((rc = check_dense(l.in, Dp, l.in.N, 1)) || (rc = check_dense(l.uk, l.dim_p, l.rank_p, l.heads)) ||
        (rc = check_dense(l.uv, l.rank_p, l.vdim_p, l.heads)) || (rc = check_dense(l.o, l.heads * l.vdim_p, Dp, 1)))
      return rc;
    // columns of the fused projection stay inside it
    if (l.off_qr < l.heads * l.dim_p || l.off_qr + l.heads * l.rot_dim > l.in.N ||
        (l.off_kv >= 0 && l.off_kv + l.kv_rank + l.rot_dim > l.in.N) ||
        (l.off_gate >= 0 && l.off_gate + l.heads * l.vdim_p > l.in.N))
      return TMX_ERR_SHAPE;
    if (l.gate_up.w) {
      if (!l.norm2_w || !l.hc2.in || !l.hc2.out || !l.hc2.mix) return TMX_ERR_ARG;
      if ((rc = check_dense(l.gate_up, Dp, l.gate_up.N, 1)) || l.gate_up.N % 64) return rc ? rc : TMX_ERR_SHAPE;
      if ((rc = check_dense(l.down, l.gate_up.N / 2, Dp, 1))) return rc;
    }
  }
  return TMX_OK;
}

int latent_layers(hipStream_t st, const tmx_model_desc* m, const tmx_decode_state* s, const LatentWorkspace& w,
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
  // The boundary behind sublayer `prev` (null: the embedding) and in front of the next one.
  const tmx_streams_desc* prev = nullptr;
  auto boundary = [&](const float* in, const float* norm_w, bool head) {
    StreamArgs a = {};
    a.xs = w.xs; a.in = in; a.norm_w = norm_w; a.xn = w.xn;
    a.S = m->streams; a.D = m->embed_dim; a.Dp = Dp; a.eps = m->norm_eps; a.store = !head;
    a.xn_tiled = tiled && !head;
    if (prev) {
      if (y_splits > 1) { a.y_part = w.y_part; a.nsplit = y_splits; }
      else a.y = w.y;
      a.mix = prev->mix; a.out = prev->out;
    } else {
      a.embed = (const uint16_t*)m->embed; a.pos_embed = (const uint16_t*)m->pos_embed;
      a.vocab = m->vocab_size; a.max_positions = m->max_positions;
      a.token_buffer = s->token_buffer; a.positions = s->positions; a.step = s->step; a.buf_len = L; a.tpp = T;
    }
    return stream_rows(st, act, a, M);
  };
  std::vector<char*> cache(m->num_layers, nullptr);
  {
    char* p = (char*)s->kv_cache;
    for (int i = 0; i < m->num_layers; ++i) {
      const tmx_latent_layer_desc& l = m->latent_layers[i];
      if (l.off_kv < 0) {
        cache[i] = cache[l.kv_layer];
        continue;
      }
      cache[i] = p;
      p += (size_t)n_seq * C * (l.rank_p + l.rot_p) * e;
    }
  }
  for (int i = 0; i < m->num_layers; ++i) {
    const tmx_latent_layer_desc& l = m->latent_layers[i];
    const int ld = l.rank_p + l.rot_p, H = l.heads;
    TMX_TRY(TMX_K_ROWNORM, boundary(l.hc1.in, l.norm1_w, false));
    {
      DenseArgs a = args(l.in, w.xn, Dp, 0, w.z, l.in.N, 0, TMX_DENSE_PLAIN);
      a.x_tiled = tiled;
      TMX_TRY(TMX_K_QKV, dense_linear(st, act, a));
    }
    {
      LatentRowsArgs a = {};
      a.z = w.z; a.ldz = l.in.N; a.off_qr = l.off_qr; a.off_kv = l.off_kv;
      a.norm_w = l.kv_norm_w; a.eps = m->norm_eps;
      a.table = l.table; a.max_positions = m->max_positions;
      a.positions = s->positions; a.step = s->step; a.buf_len = L; a.tpp = T;
      a.q = w.q; a.cache = cache[i];
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
      a.q = w.q; a.cache = cache[i]; a.sink = l.sink;
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
    TMX_TRY(TMX_K_O, into_streams(l.o, w.val));
    prev = &l.hc1;
    if (l.gate_up.w) {
      const int Fp = l.gate_up.N / 2;
      TMX_TRY(TMX_K_ROWNORM, boundary(l.hc2.in, l.norm2_w, false));
      DenseArgs a = args(l.gate_up, w.xn, Dp, 0, w.act, Fp, 0, TMX_DENSE_SWIGLU);
      a.x_tiled = a.y_tiled = tiled;
      TMX_TRY(TMX_K_GATE_UP, dense_linear(st, act, a));
      TMX_TRY(TMX_K_DOWN, into_streams(l.down, w.act));
      prev = &l.hc2;
    }
    if (prof) TMX_TRY(TMX_K_EMPTY, empty_launch(st));
  }
  if (final_norm) TMX_TRY(TMX_K_ROWNORM, boundary(m->final_in, (const float*)m->final_norm_w, true));
  return TMX_OK;
}

}  // namespace tmx
