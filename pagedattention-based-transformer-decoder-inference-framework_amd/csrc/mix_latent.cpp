// Latent attention in the layer-stack model.
//
//   q | down product (queries turned) -> norm, turn and append the latent row ->
//   [short portions] queries into the latent space per head -> latent attention ->
//     values per head
//   [long portions]  keys and values of the whole context into scratch pages ->
//     grouped-query attention with a key/value head per head
//   -> o product
//
// A token against a cached row costs about H (2 rank + rot) products in the latent
// space and H (dim + rot + vdim) against expanded keys, whose expansion costs
// rank (dim + vdim) per head and row once for all of a portion's tokens.  Both
// give the same up to rounding; single tokens always stay in the latent space.
#include <algorithm>

#include "common.hpp"
#include "layer_stack_impl.hpp"
#include "paged_latent.hpp"

namespace llm {

int LayerStack::init_latent(Layer& l) {
  const LatentSpec& a = l.s.latent;
  l.geo = find_geometry(true, 1, a.rank, a.rot_dim);
  RET_IF(find_rope(a.rope, &l.rope));
  const int dim = up(a.dim, 2), Dp = up(dim + a.rot_dim, 8);
  int min_x = INT_MAX;  // tokens of a portion from which expanding pays
  const long long extra = 2LL * a.rank - a.dim - a.vdim;
  if (extra > 0 && dim + a.rot_dim <= kGqaMaxDim && a.vdim <= kGqaMaxDim)
    min_x = (int)std::max<long long>(kGqaSmallRows + 1, (long long)a.rank * (a.dim + a.vdim) / extra);
  auto p = std::make_unique<Plan>();
  p->latent = true;
  p->R = a.heads;
  p->small_tile = p->small_max = a.heads <= 16 ? 16 : a.heads <= 32 ? 32 : 64;
  p->big_tile = 64;
  p->max_n = min_x == INT_MAX ? INT_MAX : min_x - 1;
  p->max_pd = gqa_part_dim(a.rank);
  l.plan = add_plan(std::move(p));
  if (min_x < INT_MAX) {
    auto x = std::make_unique<Plan>();
    x->expand = true;
    x->G = a.heads;
    x->dim = dim;
    x->rot = a.rot_dim;
    x->Dp = Dp;
    x->Dv = a.vdim;
    x->Dvp = up(a.vdim, 8);
    x->big_tile = gqa_tile_rows(dt_, Dp, x->Dvp, 1 << 20);
    x->min_n = min_x;
    x->max_pd = gqa_part_dim(a.vdim);
    l.plan_x = add_plan(std::move(x));
  }
  ld_q_ = std::max(ld_q_, a.heads * Dp);
  ld_qlat_ = std::max(ld_qlat_, a.heads * geos_[l.geo]->Dp);
  ld_olat_ = std::max(ld_olat_, a.heads * mm_pad(a.rank));
  ld_down_ = std::max(ld_down_, up(a.rank, 2) + a.rot_dim);
  ld_att_ = std::max(ld_att_, mm_pad(a.heads * a.vdim));
  return LLM_OK;
}

int LayerStack::load_latent(const SafeTensors& f, const std::string& mix, Layer& l) {
  const LatentSpec& a = l.s.latent;
  const int H = a.heads, dim = up(a.dim, 2), rank = up(a.rank, 2), qd = a.dim + a.rot_dim;
  // query heads (odd sizes get a zero column), then the latent and its key part
  std::vector<int32_t> map;
  for (int h = 0; h < H; ++h) {
    for (int d = 0; d < dim; ++d) map.push_back(d < a.dim ? h * qd + d : -1);
    for (int d = 0; d < a.rot_dim; ++d) map.push_back(h * qd + a.dim + d);
  }
  for (int d = 0; d < rank; ++d) map.push_back(d < a.rank ? H * qd + d : -1);
  for (int d = 0; d < a.rot_dim; ++d) map.push_back(H * qd + a.rank + d);
  l.n_qkv = (int)map.size();
  RET_IF(load_packed(f, {{mix + "q", H * qd}, {mix + "dkv", a.rank + a.rot_dim}}, cfg_.width, &map,
                     l.qkv));
  RET_IF(load_vector(f, mix + "dkv.norm", a.rank, a.rank, l.latent_norm));
  RET_IF(load_packed(f, {{mix + "o", cfg_.width}}, H * a.vdim, nullptr, l.o));
  if (a.sink) RET_IF(load_vector(f, mix + "sink", H, H, l.sink));

  std::vector<uint16_t> uk, uv;
  RET_IF(f.get_bf16(mix + "uk", {(int64_t)H * a.dim, a.rank}, &uk));
  RET_IF(f.get_bf16(mix + "uv", {(int64_t)H * a.vdim, a.rank}, &uv));
  l.absorb_head = mm_packed_bytes(dt_, a.rank, a.dim);
  l.value_head = mm_packed_bytes(dt_, a.vdim, a.rank);
  RET_IF(l.absorb.alloc(l.absorb_head * H));
  RET_IF(l.value.alloc(l.value_head * H));
  for (int h = 0; h < H; ++h) {
    std::vector<uint16_t> t((size_t)a.rank * a.dim);
    for (int d = 0; d < a.dim; ++d)
      for (int r = 0; r < a.rank; ++r)
        t[(size_t)r * a.dim + d] = uk[((size_t)h * a.dim + d) * a.rank + r];
    RET_IF(pack_host(t, a.dim, nullptr, l.absorb.p + l.absorb_head * h));
    const auto v = uv.begin() + (size_t)h * a.vdim * a.rank;
    RET_IF(pack_host(std::vector<uint16_t>(v, v + (size_t)a.vdim * a.rank), a.rank, nullptr,
                     l.value.p + l.value_head * h));
  }
  if (l.plan_x >= 0) {
    std::vector<int32_t> rows;
    for (int h = 0; h < H; ++h)
      for (int d = 0; d < dim; ++d) rows.push_back(d < a.dim ? h * a.dim + d : -1);
    for (int n = 0; n < H * a.vdim; ++n) rows.push_back(H * a.dim + n);
    RET_IF(load_packed(f, {{mix + "uk", H * a.dim}, {mix + "uv", H * a.vdim}}, a.rank, &rows, l.expand));
  }
  return LLM_OK;
}

void LayerStack::plan_expansion(const std::vector<StepSeq>& batch, Plan& p,
                                std::vector<int32_t>& pos, std::vector<int32_t>& slot,
                                std::vector<int32_t>& entry, std::vector<int32_t>& table) {
  int n = 0;
  p.x_tiles = 0;
  for (const StepSeq& s : batch)
    if (s.n >= p.min_n && s.n <= p.max_n)
      p.x_tiles = std::max(p.x_tiles, (s.p0 + s.n - 1) / kPageTokens + 1);
  int32_t page = 0;
  for (const StepSeq& s : batch) {
    if (s.n < p.min_n || s.n > p.max_n) continue;
    for (int i = 0; i < s.p0 + s.n; ++i) {
      pos.push_back(i);
      slot.push_back(s.slot);
      entry.push_back(n);
    }
    const int tiles = (s.p0 + s.n - 1) / kPageTokens + 1;
    for (int h = 0; h < p.G; ++h)
      for (int t = 0; t < p.x_tiles; ++t) table.push_back(t < tiles ? page++ : -1);
    ++n;
  }
  p.x_rows = (int)pos.size();
  p.x_pages = page;
}

int LayerStack::latent(const Layer& l, const Run& r, int M, hipStream_t st) {
  const LatentSpec& a = l.s.latent;
  const Geometry& g = *geos_[l.geo];
  const int dim = up(a.dim, 2), rank = up(a.rank, 2), Dp = up(dim + a.rot_dim, 8);
  const int ld_att = mm_pad(a.heads * a.vdim);
  const float2* turn = l.rope >= 0 ? ropes_[l.rope]->turn.p : nullptr;
  const Plan& near = *plans_[l.plan];
  const Plan* far = l.plan_x >= 0 && plans_[l.plan_x]->x_rows > 0 ? plans_[l.plan_x].get() : nullptr;

  MmArgs p;
  p.A = h_.p;
  p.lda = ldx_;
  p.W = l.qkv.p;
  p.M = M;
  p.N = l.n_qkv;
  p.K = cfg_.width;
  p.w_nt = w_nt_;
  MmLatent e;
  e.turn = turn;
  e.H = a.heads;
  e.D = dim;
  e.rot = a.rot_dim;
  e.q = q_.p;
  e.ldq = Dp;
  e.q_lat = q_lat_.p;
  e.ld_lat = g.Dp;
  e.lat_rot = latent_rot_at(a.rank);
  e.down = down_.p;
  e.ldd = rank + a.rot_dim;
  LLM_HIP_RET(mm_latent(dt_, p, e, st));

  MmPageRows rows;  // the new tokens' rows
  rows.pos = meta<int32_t>(at_pos_);
  rows.slot = meta<int32_t>(at_slot_);
  rows.table = table_of(g, r);
  rows.max_tiles = g.kv.max_tiles;
  rows.num_pages = (int)g.kv.num_pages;
  rows.pool = g.kv.k_pool;
  rows.page_stride = g.kv.page_stride();
  rows.row = g.Dp;
  LatentAppend ap;
  ap.M = M;
  ap.rank = a.rank;
  ap.rot = a.rot_dim;
  ap.down = down_.p;
  ap.ldd = e.ldd;
  ap.rot_at = rank;
  ap.w = l.latent_norm.p;
  ap.eps = cfg_.eps;
  ap.turn = turn;
  ap.page = rows;
  LLM_HIP_RET(latent_append(dt_, ap, st));

  GqaArgs q;
  q.ldo = ld_att;
  q.scale = a.scale;
  q.sink = a.sink ? l.sink.p : nullptr;
  q.H = a.heads;
  q.part_o = part_o_.p;
  q.part_ml = part_ml_.p;
  const auto at = [&](const Launch& c) {
    q.items = meta<GqaItem>(c.items_at);
    q.n_items = c.n_items;
    q.merges = meta<GqaMerge>(c.merges_at);
    q.n_merges = c.n_merges;
  };
  if (near.n_rows > 0) {
    const int ld_lat = a.heads * g.Dp, ldv = mm_pad(a.rank);
    MmArgs b;
    b.A = q_.p;
    b.lda = a.heads * Dp;
    b.W = l.absorb.p;
    b.M = near.n_rows;
    b.N = a.rank;
    b.K = a.dim;
    b.w_nt = w_nt_;
    MmHeads hd;
    hd.heads = a.heads;
    hd.a_head = Dp;
    hd.w_head = l.absorb_head;
    hd.C = q_lat_.p;
    hd.ldc = ld_lat;
    hd.c_head = g.Dp;
    hd.rows = near.n_rows == M ? nullptr : meta<int32_t>(near.rows_at);
    LLM_HIP_RET(mm_heads(dt_, b, hd, st));

    q.q = q_lat_.p;
    q.out = o_lat_.p;
    q.ldo = a.heads * ldv;
    q.ldh = ldv;
    q.k_pool = rows.pool;
    q.page_stride = rows.page_stride;
    q.table = rows.table;
    q.max_tiles = rows.max_tiles;
    q.num_pages = rows.num_pages;
    q.G = 1;
    q.Dp = g.Dp;
    q.Dv = a.rank;
    for (const Launch* c : {&near.small, &near.big}) {
      if (c->n_items == 0) continue;
      at(*c);
      LLM_HIP_RET(latent_attention(dt_, q, c->tile_rows, st));
    }

    b.A = o_lat_.p;
    b.lda = q.ldo;
    b.W = l.value.p;
    b.N = a.vdim;
    b.K = a.rank;
    hd.a_head = ldv;
    hd.w_head = l.value_head;
    hd.C = att_.p;
    hd.ldc = ld_att;
    hd.c_head = a.vdim;
    LLM_HIP_RET(mm_heads(dt_, b, hd, st));
  }
  if (far) {
    MmPageRows src = rows;
    src.pos = meta<int32_t>(far->x_pos);
    src.slot = meta<int32_t>(far->x_slot);
    MmArgs x;
    x.W = l.expand.p;
    x.M = far->x_rows;
    x.N = a.heads * (dim + a.vdim);
    x.K = a.rank;
    MmQkv kv;
    kv.pos = src.pos;
    kv.slot = meta<int32_t>(far->x_entry);
    kv.G = a.heads;
    kv.D = dim;
    kv.Dv = a.vdim;
    kv.Dp = Dp;
    kv.Dvp = far->Dvp;
    kv.table = meta<int32_t>(far->x_table);
    kv.max_tiles = far->x_tiles;
    kv.num_pages = (int)far->x_pages;
    kv.k_pool = far->pool.p;
    kv.v_pool = far->pool.p + (size_t)kPageTokens * Dp * es_;
    kv.page_stride = (size_t)kPageTokens * (Dp + far->Dvp) * es_;
    LLM_HIP_RET(mm_expand(dt_, x, src, kv, st));
    LatentSpread sp;
    sp.M = far->x_rows;
    sp.H = a.heads;
    sp.rot = a.rot_dim;
    sp.src_at = latent_rot_at(a.rank);
    sp.src = src;
    sp.slot = kv.slot;
    sp.table = kv.table;
    sp.max_tiles = kv.max_tiles;
    sp.num_pages = kv.num_pages;
    sp.k_pool = kv.k_pool;
    sp.page_stride = kv.page_stride;
    sp.Dp = Dp;
    sp.at = dim;
    if (sp.rot > 0) LLM_HIP_RET(latent_spread(dt_, sp, st));

    q.q = q_.p;
    q.out = att_.p;
    q.ldo = ld_att;
    q.ldh = 0;
    q.k_pool = kv.k_pool;
    q.v_pool = kv.v_pool;
    q.page_stride = kv.page_stride;
    q.table = kv.table;
    q.max_tiles = kv.max_tiles;
    q.num_pages = kv.num_pages;
    q.G = a.heads;
    q.Dp = Dp;
    q.Dv = a.vdim;
    q.Dvp = far->Dvp;
    for (const Launch* c : {&far->small, &far->big}) {
      if (c->n_items == 0) continue;
      at(*c);
      LLM_HIP_RET(gqa_attention(dt_, q, c->tile_rows, st));
    }
  }
  return out_product(l, att_.p, ld_att, a.heads * a.vdim, M, st);
}

}  // namespace llm
