// kf_seq.cpp -- see kf_seq.hpp.  Every device action is a kf_* call.
#include "kf_seq.hpp"

#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>

namespace koifish {

static inline void* P(const hGTensor& t) { return t ? t->data : nullptr; }
static inline float* F(const hGTensor& t) { return reinterpret_cast<float*>(P(t)); }
static inline int32_t* I(const hGTensor& t) { return reinterpret_cast<int32_t*>(P(t)); }
static int up(int n, int m) { return (n + m - 1) / m * m; }
// zeroed device memory of n elements
static hGTensor Mem(kf_ctx* c, const char* name, int type, size_t n) {
    auto t = std::make_shared<GTensor>();
    t->name = name, t->type = type == KF_BF16 ? typNUMBER::BF16 : typNUMBER::F32, t->szData = n * (type == KF_BF16 ? 2 : 4);
    t->ne[0] = (int)std::min<size_t>(n, 0x7fffffff);
    if (t->Alloc(c, t->szData) != KF_OK || kf_memset(c, t->data, 0, t->szData) != KF_OK) return nullptr;
    return t;
}

// ------------------------------------------------------------------------------------------------ neurons
int RowProduct::Forw(const void* x, int64_t ldx, int n, void* y, int64_t ldy, int epilogue, int act, const float* res, float alpha, int mode, const kf_rb_experts* ex, float* ssq) {
    kf_rb_product p;
    std::memset(&p, 0, sizeof(p));
    p.w = w->data, p.x = x, p.y = y, p.res = res, p.ldx = ldx, p.ldy = ldy, p.ldr = ldy;
    p.type = hFish->Seq()->card.type, p.m = m, p.k = k, p.n = n, p.epilogue = epilogue, p.act = act, p.mode = mode, p.alpha = alpha, p.ssq = ssq;
    if (epilogue == KF_RB_STORE && act_lo < act_hi) p.act_lo = act_lo, p.act_hi = act_hi, p.act = col_act;
    kf_rb_experts e;
    if (ex) e = *ex, e.w_stride = (int64_t)m * k, p.experts = &e;
    return kf_rb_linear(hFish->ctx, &p);
}
int RowProduct::ForwNormed(RowWork& w, int n, void* y, int64_t ldy, int epilogue, int act) {
    if (!w.pending) return Forw(P(w.h), k, n, y, ldy, epilogue, act);
    const SEQ_CARD& c = hFish->Seq()->card;
    kf_rb_product p;
    std::memset(&p, 0, sizeof(p));
    p.w = this->w->data, p.x = P(w.h), p.y = y, p.ldx = k, p.ldy = ldy, p.type = c.type, p.m = m, p.k = k, p.n = n, p.epilogue = epilogue, p.act = act;
    p.norm_z = F(w.z), p.norm_ssq = F(w.ssq), p.norm_w = P(w.pending->w), p.norm_x = F(w.x), p.norm_eps = c.eps, p.norm_dim = c.width;
    w.pending = nullptr;
    return kf_rb_linear(hFish->ctx, &p);
}
int RowNorm::Forw(const void* z, int n, float* x_out, void* h_out, const float* res, float alpha, int top, const int32_t* rows) {
    const SEQ_CARD& c = hFish->Seq()->card;
    return kf_rb_norm(hFish->ctx, c.type, z, res, alpha, top, w->data, c.eps, dim, ld, n, rows, x_out, h_out);
}
int RowNorm::Rows(RowWork& w, const float* z, int n, const float* add, float* x_out, void* h_out, const int32_t* rows, bool positions) {
    const SeqFish* f = hFish->Seq();
    kf_rb_norming a;
    std::memset(&a, 0, sizeof(a));
    a.z = z, a.add = add, a.rows = rows, a.w = this->w->data, a.x_out = x_out, a.h_out = h_out, a.ld = ld, a.type = f->card.type, a.kind = f->card.norm_kind, a.dim = dim, a.n = n, a.eps = f->card.eps;
    if (positions) a.pos_hi = F(f->pos_hi), a.pos_lo = F(f->pos_lo), a.meta = I(w.meta);
    return kf_rb_norm_rows(hFish->ctx, &a);
}
int SeqFish::Enter(RowWork& w, int n) {
    return card.embed_norm ? embed_norm.Rows(w, F(w.x), n, nullptr, F(w.x), P(w.h), nullptr, card.sinusoid > 0) : KF_OK;
}
int SeqFish::Close(RowWork& w, RowProduct& proj, RowNorm& norm, const void* in, int64_t ldin, int n, bool defer) {
    if (card.add_norm) {
        KF_TRY(proj.Forw(in, ldin, n, F(w.z), proj.m, KF_RB_STORE_F32));
        return norm.Rows(w, F(w.z), n, F(w.x), F(w.x), P(w.h), nullptr, false);
    }
    KF_TRY(proj.Forw(in, ldin, n, F(w.z), proj.m, KF_RB_RESIDUAL, 0, F(w.x), card.alpha, KF_RB_ALL, nullptr, defer ? F(w.ssq) : nullptr));
    if (defer) {
        w.pending = &norm;
        return KF_OK;
    }
    return norm.Forw(F(w.z), n, F(w.x), P(w.h));
}
int RowMixer::Forw(RowWork& w, const KVCache& kv, const RowBatch& b, bool defer) {
    KF_TRY(in.Forw(P(w.h), in.k, b.n, P(w.raw), ldraw, KF_RB_STORE));
    KF_TRY(Mix(w, kv, b));
    return hFish->Seq()->Close(w, proj, norm, P(w.ao), ldout, b.n, defer);
}
void RowMixer::Need(RowNeed& need, int rows, int, bool) const {
    need.raw = std::max(need.raw, (size_t)rows * ldraw), need.ao = std::max(need.ao, (size_t)rows * ldout);
}
kf_rb_attention RowAttention::Args(const RowWork& w, const KVCache& kv) const {
    const SEQ_CARD& card = hFish->Seq()->card;
    const KVCache::Ring& ring = kv.rings[layid - 1];
    kf_rb_attention a;
    std::memset(&a, 0, sizeof(a));
    a.raw = P(w.raw), a.out = P(w.ao), a.k_new = P(w.knew), a.k_cache = kv.Ring0(KVCache::KV_KEY, layid - 1), a.v_cache = kv.Ring0(KVCache::KV_VAL, layid - 1);
    a.q_norm = c.qk_norm ? P(qn) : nullptr, a.k_norm = c.qk_norm ? P(kn) : nullptr, a.rope = rope, a.scratch = P(w.scratch);
    a.ldraw = ldraw, a.ldout = ldout, a.slot_stride = (int64_t)ring.slot_stride(), a.head_stride = (int64_t)ring.head_stride();
    a.type = card.type, a.n_head = c.heads, a.n_kv = c.kv_heads, a.dim = c.dim, a.rot_dims = c.rot.dims, a.chunk = c.chunk, a.cache_rows = ring.rows, a.gated = c.gated;
    a.scale = c.scale, a.eps = card.eps;
    a.v_col = v_col, a.vdim = c.vdim, a.unit = c.qk_unit, a.window = c.window, a.sink = c.sink;
    if (c.kind == MIXER_CARD::PARALLEL) a.scaled = 1, a.out_scale = c.left_scale;
    return a;
}
int RowAttention::Mix(RowWork& w, const KVCache& kv, const RowBatch& b) {
    const kf_rb_attention a = Args(w, kv);
    if (b.n_seq) return kf_rb_attention_prefill(hFish->ctx, &a, I(w.meta), b.n, I(w.seqs), b.n_seq, b.max_n);
    return kf_rb_attention_decode(hFish->ctx, &a, I(w.meta), b.n, b.max_pos);
}
void RowAttention::Need(RowNeed& need, int rows, int n_seq, bool decode) const {
    RowMixer::Need(need, rows, n_seq, decode);
    need.knew = std::max(need.knew, (size_t)rows * c.kv_heads * c.dim);
    if (decode) need.scratch = std::max(need.scratch, kf_rb_attention_scratch(rows, c.heads, c.V()) / 4);
}
int ChannelDelta::Mix(RowWork& w, const KVCache& kv, const RowBatch& b) {
    SeqFish* f = hFish->Seq();
    kf_rb_delta a;
    std::memset(&a, 0, sizeof(a));
    a.raw = P(w.raw), a.out = P(w.ao), a.conv = P(conv), a.w_a2 = P(a2.w), a.w_g2 = P(g2.w), a.a_log = P(a_log), a.dt_bias = P(dt_bias), a.norm_w = P(out_norm);
    a.state = kv.State0(layid - 1), a.hist = kv.Hist0(layid - 1), a.scratch = F(w.recur), a.ldraw = ldraw, a.ldout = ldout, a.hist_slot = (int64_t)kv.recurrent[layid - 1].hist_slot();
    a.type = f->card.type, a.n_head = c.heads, a.n_kv = c.kv_heads, a.dim = c.dim, a.vdim = c.vdim, a.taps = c.taps, a.col_b = col_b, a.col_a = col_a, a.col_g = col_g;
    a.rank_a = c.rank_a, a.rank_g = c.rank_g, a.ld_a = a2.k, a.ld_g = g2.k;
    a.q_scale = 1.0f / std::sqrt((float)c.dim), a.unit_eps = 1e-6f, a.eps = f->card.eps;
    if (!b.n_seq) return kf_rb_delta_decode(f->ctx, &a, I(w.meta), b.n);
    const uint8_t* raw = reinterpret_cast<const uint8_t*>(a.raw);
    KF_TRY(a2.Forw(raw + col_a * f->Elem(), ldraw, b.n, F(w.az), a2.m, KF_RB_STORE_F32));
    KF_TRY(g2.Forw(raw + col_g * f->Elem(), ldraw, b.n, P(w.gz), g2.m, KF_RB_STORE));
    a.a_z = F(w.az), a.g_z = P(w.gz), a.ld_az = a2.m, a.ld_gz = g2.m;
    return kf_rb_delta_prefill(f->ctx, &a, I(w.meta), b.n, I(w.seqs), b.n_seq, b.max_n);
}
void ChannelDelta::Need(RowNeed& need, int rows, int n_seq, bool decode) const {
    RowMixer::Need(need, rows, n_seq, decode);
    if (decode) return;
    need.az = std::max(need.az, (size_t)rows * a2.m), need.gz = std::max(need.gz, (size_t)rows * g2.m);
    need.recur = std::max(need.recur, kf_rb_delta_scratch(hFish->Seq()->card.type, rows, n_seq, c.heads, c.kv_heads, c.dim, c.vdim) / 4);
}
int ParallelMixer::Mix(RowWork& w, const KVCache& kv, const RowBatch& b) {
    SeqFish* f = hFish->Seq();
    kf_rb_decay d;
    std::memset(&d, 0, sizeof(d));
    d.raw = P(w.raw), d.out = reinterpret_cast<uint8_t*>(P(w.ao)) + out_sum * f->Elem(), d.norm_w = P(sum_norm), d.decay = F(decay), d.state = kv.State0(layid - 1), d.scratch = F(w.recur);
    d.ldraw = ldraw, d.ldout = ldout, d.type = f->card.type, d.n_head = c.sum_heads, d.dim = c.sum_dim, d.vdim = c.sum_vdim, d.col_q = col_sum, d.col_g = col_gate;
    d.out_scale = c.right_scale, d.eps = f->card.eps;
    if (!b.n_seq) {
        const kf_rb_attention a = Args(w, kv);
        return kf_rb_attention_decay_decode(f->ctx, &a, &d, I(w.meta), b.n, b.max_pos);
    }
    KF_TRY(RowAttention::Mix(w, kv, b));
    return kf_rb_decay_prefill(f->ctx, &d, I(w.meta), b.n, I(w.seqs), b.n_seq, b.max_n);
}
void ParallelMixer::Need(RowNeed& need, int rows, int n_seq, bool decode) const {
    RowAttention::Need(need, rows, n_seq, decode);
    need.recur = std::max(need.recur, kf_rb_decay_scratch(hFish->Seq()->card.type, rows, n_seq, c.sum_heads, c.sum_dim, c.sum_vdim) / 4);
}
int RowFFN::Forw(RowWork& w, int n) {
    const SEQ_CARD& card = hFish->Seq()->card;
    if (c.kind == FF_CARD::NONE) return KF_OK;
    const int64_t ld = gateup.k;
    if (c.kind == FF_CARD::DENSE) {
        KF_TRY(gateup.ForwNormed(w, n, P(w.act), ldact, KF_RB_GATED, c.act));
        return hFish->Seq()->Close(w, down, norm, P(w.act), ldact, n);
    }
    const bool few = Sums(card.type, n);
    kf_rb_experts e;
    std::memset(&e, 0, sizeof(e));
    e.n_expert = c.experts, e.top = c.top;
    // few rows: an expert never has more pairs than the batch has rows, one tile each; many: 128-pair tiles where the experts fill several
    e.tile = few ? up(n, 16) : (card.type == KF_BF16 && (long long)n * c.top >= 256LL * c.experts ? 128 : 64);
    e.n_tile = kf_rb_list_tiles(n, c.top, c.experts, e.tile);
    e.tile_expert = I(w.tile_expert), e.list = I(w.list), e.ids = I(w.ids), e.weight = F(w.weight);
    KF_TRY(router.Forw(P(w.h), ld, n, F(w.rlogits), router.m, KF_RB_STORE_F32));
    KF_TRY(kf_rb_route(hFish->ctx, card.type, F(w.rlogits), router.m, P(router_b), n, I(w.meta), &e));
    KF_TRY(gateup.Forw(P(w.h), ld, n, P(w.act), ldact, KF_RB_GATED, c.act, nullptr, 0, KF_RB_UP, &e));
    if (few) {
        KF_TRY(down.Forw(P(w.act), ldact, n, F(w.z), ld, KF_RB_RESIDUAL, 0, F(w.x), card.alpha, KF_RB_SUM, &e));
        return norm.Forw(F(w.z), n, F(w.x), P(w.h));
    }
    KF_TRY(down.Forw(P(w.act), ldact, n, P(w.y), ld, KF_RB_STORE, 0, nullptr, 0, KF_RB_DOWN, &e));
    return norm.Forw(P(w.y), n, F(w.x), P(w.h), F(w.x), card.alpha, c.top);
}

// ------------------------------------------------------------------------------------------------ build
SeqSlots::~SeqSlots() {
    for (auto& g : graphs)
        if (g.second) kf_graph_destroy(g.second);
}
SeqFish::~SeqFish() {
    if (ctx) kf_sync(ctx);
    DropGraphs(self);
    for (auto& r : ropes)
        if (r.second) kf_free(ctx, r.second);
    // everything on the device goes before Fish gives the context back
    self.kv = KVCache(), self.dec = RowWork(), self.pick_ws.reset(), self.logits16.reset(), pre = RowWork();
    mixers.clear(), ffs.clear(), targets.clear(), stage.reset(), table.reset(), pos_hi.reset(), pos_lo.reset();
    seq_head = RowProduct(), seq_norm = RowNorm(), embed_norm = RowNorm();
}
void SeqFish::DropGraphs(SeqSlots& s) {
    for (auto& g : s.graphs)
        if (g.second) kf_graph_destroy(g.second);
    s.graphs.clear();
}

// zeroed weight storage; Vector: n elements padded to KF_RB_PAD, the checkpoint's tensor `name` + suffix unless that is NULL
int SeqFish::Vector(hGTensor& t, const std::string& name, int n, const char* suffix) {
    t = Mem(ctx, name.c_str(), card.type, Width(n));
    if (!t) return KF_OUTOF_GPUMEMORY;
    if (suffix) targets[name + suffix] = Target{t, 0, 0, n, 1, 1, -1, false, false};
    return KF_OK;
}
int SeqFish::Product(RowProduct& p, const std::string& name, int m, int k, int experts) {
    p.hFish = this, p.name = name, p.m = m, p.k = k, p.experts = experts;
    p.w = Mem(ctx, name.c_str(), card.type, (size_t)m * k * std::max(experts, 1));
    return p.w ? KF_OK : KF_OUTOF_GPUMEMORY;
}
int SeqFish::Norm(RowNorm& n, const std::string& name) {
    n.hFish = this, n.name = name, n.dim = card.width, n.ld = Width(card.width);
    return Vector(n.w, name, card.width, "");
}
// rows row0 .. of the product behind `p`, columns col0 .. (a multiple of KF_RB_PAD): where the checkpoint's [rows][cols] matrix goes
void SeqFish::Rows(const RowProduct& p, const std::string& name, int row0, int rows, int cols, int col0) {
    const bool tiled = card.type == KF_BF16;
    targets[name] = Target{p.w, tiled ? (size_t)col0 / 32 * 512 : (size_t)col0, row0, rows, cols, p.k, -1, true, false};
}
int SeqFish::BuildMixer(const MIXER_CARD& m, int l, std::unique_ptr<RowMixer>& out) {
    const std::string p = "l" + std::to_string(l) + ".", q = p + "mix.";
    const int W = Width(card.width), C = card.width;
    auto named = [&](RowMixer* x) { x->hFish = this, x->layid = l + 1, x->name = p + "mix", x->c = m; };
    // columns of raw: a part starts at a multiple of eight, what a product reads again at a multiple of the padding
    int at = 0;
    auto part = [&](int n, int align) {
        const int col = up(at, align);
        at = col + n;
        return col;
    };
    if (m.kind == MIXER_CARD::CHANNEL_DELTA) {
        auto a = std::make_unique<ChannelDelta>();
        named(a.get());
        const int qd = m.kv_heads * m.dim, vd = m.heads * m.vdim, channels = 2 * qd + vd;
        part(channels, 1);
        a->col_a = part(Width(m.rank_a), KF_RB_PAD), a->col_g = part(Width(m.rank_g), KF_RB_PAD), a->col_b = part(m.heads, 1);
        a->ldraw = Width(at), a->ldout = Width(vd);
        KF_TRY(Product(a->in, q + "in", a->ldraw, W));
        KF_TRY(Product(a->proj, q + "o", W, a->ldout));
        KF_TRY(Product(a->a2, q + "a2", Width(m.heads * m.dim), Width(m.rank_a)));
        KF_TRY(Product(a->g2, q + "g2", Width(vd), Width(m.rank_g)));
        Rows(a->in, q + "q", 0, qd, C), Rows(a->in, q + "k", qd, qd, C), Rows(a->in, q + "v", 2 * qd, vd, C);
        Rows(a->in, q + "a1", a->col_a, m.rank_a, C), Rows(a->in, q + "g1", a->col_g, m.rank_g, C), Rows(a->in, q + "b", a->col_b, m.heads, C);
        Rows(a->a2, q + "a2", 0, m.heads * m.dim, m.rank_a), Rows(a->g2, q + "g2", 0, vd, m.rank_g), Rows(a->proj, q + "o", 0, C, vd);
        KF_TRY(Vector(a->conv, q + "conv", channels * m.taps, nullptr));
        for (const auto& t : {std::make_pair("q.conv", std::make_pair(0, qd)), std::make_pair("k.conv", std::make_pair(qd, qd)), std::make_pair("v.conv", std::make_pair(2 * qd, vd))})
            targets[q + t.first] = Target{a->conv, (size_t)t.second.first * m.taps, 0, t.second.second, m.taps, m.taps, -1, false, false};
        KF_TRY(Vector(a->a_log, q + "A_log", m.heads, ""));
        KF_TRY(Vector(a->dt_bias, q + "dt_bias", m.heads * m.dim, ""));
        KF_TRY(Vector(a->out_norm, q + "norm", m.vdim, ""));
        KF_TRY(Norm(a->norm, p + "norm1"));
        out = std::move(a);
        return KF_OK;
    }
    // attention, alone or as the left half
    const bool par = m.kind == MIXER_CARD::PARALLEL;
    ParallelMixer* pm = nullptr;
    std::unique_ptr<RowAttention> a;
    if (par) a.reset(pm = new ParallelMixer());
    else a.reset(new RowAttention());
    named(a.get());
    const std::string ql = par ? q + "left." : q, qr = q + "right.";
    const int qd = m.heads * m.dim, kd = m.kv_heads * m.dim, vd = m.kv_heads * m.V(), od = m.heads * m.V(), sq = m.sum_heads * m.sum_dim, sv = m.sum_heads * m.sum_vdim;
    part(qd + kd, 1);
    a->v_col = m.vdim ? part(vd, 8) : 0;
    const int col_gate = m.gated ? part(od, m.vdim ? 8 : 1) : 0;
    if (par) pm->col_sum = part(2 * sq + sv, 8), pm->col_gate = part(sv, 8), pm->out_sum = Width(od);
    a->ldraw = Width(at), a->ldout = par ? Width(pm->out_sum + sv) : Width(od);
    KF_TRY(Product(a->in, q + "in", a->ldraw, W));
    KF_TRY(Product(a->proj, q + "o", W, a->ldout));
    Rows(a->in, ql + "q", 0, qd, C), Rows(a->in, ql + "k", qd, kd, C), Rows(a->proj, ql + "o", 0, C, od);
    if (m.vdim) Rows(a->in, ql + "v", a->v_col, vd, C);
    if (m.gated) Rows(a->in, ql + "g", col_gate, od, C);
    if (par) {
        Rows(a->in, qr + "q", pm->col_sum, sq, C), Rows(a->in, qr + "k", pm->col_sum + sq, sq, C), Rows(a->in, qr + "v", pm->col_sum + 2 * sq, sv, C), Rows(a->in, qr + "g", pm->col_gate, sv, C);
        Rows(a->proj, qr + "o", 0, C, sv, pm->out_sum);
        a->in.act_lo = pm->col_sum, a->in.act_hi = pm->col_sum + 2 * sq + sv, a->in.col_act = KF_RB_SILU;
        KF_TRY(Vector(pm->sum_norm, qr + "norm", sv, ""));
        pm->decay = Mem(ctx, (qr + "decay").c_str(), KF_F32, m.decay.size());
        if (!pm->decay) return KF_OUTOF_GPUMEMORY;
        KF_TRY(kf_h2d(ctx, pm->decay->data, m.decay.data(), m.decay.size() * 4));
    }
    if (m.qk_norm) {
        KF_TRY(Vector(a->qn, ql + "q.norm", m.dim, ""));
        KF_TRY(Vector(a->kn, ql + "k.norm", m.dim, ""));
    }
    KF_TRY(Norm(a->norm, p + "norm1"));
    for (auto& r : ropes)
        if (r.first == m.rot) a->rope = r.second;
    if (!a->rope && m.rot.dims) {
        const ROT_CARD& r = m.rot;
        float* d = nullptr;
        std::vector<float> tab((size_t)card.n_ctx * r.dims, 0.f);
        KF_TRY(kf_rb_rope_table_host(tab.data(), card.n_ctx, r.dims, r.base, r.factor, r.low, r.high, r.original));
        KF_TRY(kf_malloc(ctx, tab.size() * 4, (void**)&d));
        ropes.emplace_back(r, d);
        KF_TRY(kf_h2d(ctx, d, tab.data(), tab.size() * 4));
        a->rope = d;
    }
    out = std::move(a);
    return KF_OK;
}
int SeqFish::BuildSeq(const SEQ_CARD& c, int device, void* stream) {
    card = c;
    config.nEmbed = c.width, config.nLayer = (int)c.layers.size(), config.vocab = c.vocab, config.n_ctx = c.n_ctx, config.rms_eps = config.qk_eps = c.eps;
    config.n_head = c.layers[0].mix.heads, config.n_head_kv = c.layers[0].mix.kv_heads, config.head_dim = c.layers[0].mix.dim, config.n_ff = c.layers[0].ff.ff;
    config.rope_theta = (float)c.layers[0].mix.rot.base, config.tie_word_embeddings = false;
    use_engine = false;
    KF_TRY(kf_init(device, stream, &ctx));
    const int W = Width(c.width), V = Width(c.vocab);
    table = Mem(ctx, "embed", c.type, (size_t)V * W);
    if (!table) return KF_OUTOF_GPUMEMORY;
    targets["embed"] = Target{table, 0, 0, c.vocab, c.width, W, -1, false, false};
    KF_TRY(Product(seq_head, "head", V, W));
    targets["head"] = Target{seq_head.w, 0, 0, c.vocab, c.width, W, -1, true, false};
    KF_TRY(Norm(seq_norm, "final.norm"));
    if (c.embed_norm) KF_TRY(Norm(embed_norm, "embed.norm"));
    if (c.sinusoid > 0) {
        const int n_hi = (c.n_ctx + 63) / 64;
        std::vector<float> hi((size_t)n_hi * W), lo((size_t)64 * W);
        KF_TRY(kf_rb_sinusoid_tables_host(hi.data(), lo.data(), c.n_ctx, c.width, W, c.sinusoid));
        pos_hi = Mem(ctx, "pos_hi", KF_F32, hi.size()), pos_lo = Mem(ctx, "pos_lo", KF_F32, lo.size());
        if (!pos_hi || !pos_lo) return KF_OUTOF_GPUMEMORY;
        KF_TRY(kf_h2d(ctx, pos_hi->data, hi.data(), hi.size() * 4));
        KF_TRY(kf_h2d(ctx, pos_lo->data, lo.data(), lo.size() * 4));
    }
    for (size_t l = 0; l < c.layers.size(); l++) {
        const LAYER_CARD& L = c.layers[l];
        const std::string p = "l" + std::to_string(l) + ".";
        std::unique_ptr<RowMixer> mx;
        KF_TRY(BuildMixer(L.mix, (int)l, mx));
        mixers.push_back(std::move(mx));
        auto f = std::make_unique<RowFFN>();
        f->hFish = this, f->layid = (int)l + 1, f->name = p + "mlp", f->c = L.ff;
        if (L.ff.kind != FF_CARD::NONE) {
            const int ff = Width(L.ff.ff), E = L.ff.kind == FF_CARD::MOE ? L.ff.experts : 0;
            f->ldact = ff;
            KF_TRY(Product(f->gateup, p + "mlp.gateup", 2 * ff, W, E));
            KF_TRY(Product(f->down, p + "mlp.down", W, ff, E));
            for (int e = 0; e < std::max(E, 1); e++) {
                const std::string q = p + "mlp." + (E ? "e" + std::to_string(e) + "." : "");
                const size_t gu = (size_t)e * 2 * ff * W, dn = (size_t)e * W * ff;
                targets[q + "gate"] = Target{f->gateup.w, gu, 0, L.ff.ff, c.width, W, 0, true, false};
                targets[q + "up"] = Target{f->gateup.w, gu, 0, L.ff.ff, c.width, W, 1, true, false};
                targets[q + "down"] = Target{f->down.w, dn, 0, c.width, L.ff.ff, ff, -1, true, false};
            }
            if (E) {
                KF_TRY(Product(f->router, p + "mlp.router", Width(E), W));
                targets[p + "mlp.router"] = Target{f->router.w, 0, 0, E, c.width, W, -1, true, false};
                KF_TRY(Vector(f->router_b, p + "mlp.router.b", E, ""));
            }
            KF_TRY(Norm(f->norm, p + "norm2"));
        }
        ffs.push_back(std::move(f));
    }
    KF_TRY(kf_malloc(ctx, 16, (void**)&d_state));
    KF_TRY(kf_malloc(ctx, (size_t)c.n_ctx * 4, (void**)&d_forced));
    KF_TRY(kf_malloc(ctx, (size_t)c.n_ctx * 4, (void**)&d_tokens_out));
    KF_TRY(kf_memset(ctx, d_state, 0, 16));
    KF_TRY(kf_memset(ctx, d_forced, 0xff, (size_t)c.n_ctx * 4));
    KF_TRY(kf_memset(ctx, d_tokens_out, 0xff, (size_t)c.n_ctx * 4));
    self.d_state = d_state, self.d_forced = d_forced, self.d_tokens_out = d_tokens_out;
    return InitSlots(self, 1);
}

int SeqFish::SetTensor(const std::string& name, int rows, int cols, const void* src, bool is_device) {
    auto it = targets.find(name);
    if (it == targets.end() || rows != it->second.rows || cols != it->second.cols || !src) return KF_INVALID_ARGS;
    Target& t = it->second;
    const size_t bytes = (size_t)rows * cols * 2;
    if (!is_device) {
        if (!stage || stage->szData < bytes) {
            KF_TRY(kf_sync(ctx));
            stage = Mem(ctx, "stage", KF_BF16, bytes / 2);
            if (!stage) return KF_OUTOF_GPUMEMORY;
        }
        KF_TRY(kf_h2d(ctx, stage->data, src, bytes));
        src = stage->data;
    }
    uint8_t* dst = reinterpret_cast<uint8_t*>(t.to->data) + t.offset * Elem();
    const bool vec = !t.product && cols == 1;  // a norm weight or a bias: one row of `rows` values
    KF_TRY(kf_rb_pack(ctx, card.type, reinterpret_cast<const kf_bf16*>(src), vec ? 1 : rows, vec ? rows : cols, dst, vec ? rows : t.ld, t.row0, vec ? -1 : t.half, t.product && card.type == KF_BF16));
    t.set = true;
    return KF_OK;
}
std::string SeqFish::Missing() const {
    for (const auto& t : targets)
        if (!t.second.set) return t.first;
    return "";
}
int SeqFish::Load(K_SafeTensors& st, std::string& err) {
    for (const auto& t : targets) {
        const ST_Tensor* s = st.Find(t.first);
        const int rows = t.second.rows, cols = t.second.cols;
        if (!s) {
            err = "tensor '" + t.first + "' not in the checkpoint";
            return KF_INVALID_ARGS;
        }
        if (s->dtype != "BF16" || s->shape.empty() || s->shape[0] != rows || (s->shape.size() == 1 ? cols != 1 : s->shape.size() != 2 || s->shape[1] != cols)) {
            err = "tensor '" + t.first + "': BF16 [" + std::to_string(rows) + (cols > 1 ? ", " + std::to_string(cols) : "") + "] expected";
            return KF_INVALID_ARGS;
        }
        const int rc = SetTensor(t.first, rows, cols, st.Data(*s), false);
        if (rc != KF_OK) {
            err = "tensor '" + t.first + "': " + kf_last_error();
            return rc;
        }
    }
    for (const auto& s : st.tensors)
        if (!targets.count(s.name)) fprintf(stderr, "%s: tensor '%s' is not part of this design: left out\n", card.arch.c_str(), s.name.c_str());
    KF_TRY(kf_sync(ctx));
    stage.reset();
    return KF_OK;
}

SeqFish* BuildSeqModel(const JSON& cfg, const std::string& dir, int device, void* stream, int type, int max_seq, int* rc_out, std::string& err) {
    auto bail = [&](int rc) -> SeqFish* {
        if (rc_out) *rc_out = rc;
        return nullptr;
    };
    const JSON* arch = cfg.get("architecture");
    seq_card_reader read = arch && arch->kind == JSON::STR ? FindSeqArch(arch->str) : nullptr;
    if (!read) {
        err = "config.json: architecture '" + (arch ? arch->str : std::string()) + "' is not registered";
        return bail(KF_INVALID_ARGS);
    }
    K_SafeTensors st;
    if (!dir.empty()) {
        const int rc = st.OpenDir(dir);
        if (rc != KF_OK) {
            err = st.err;
            return bail(rc);
        }
    }
    // sizes that config.json leaves to the tensors: from the checkpoint, or without one from "tensor_shapes" beside the configuration
    const JSON* given = cfg.get("tensor_shapes");
    const seq_shapes shapes = [&](const std::string& name, int& rows, int& cols) {
        std::vector<double> s;
        if (!dir.empty()) {
            const ST_Tensor* t = st.Find(name);
            if (t) s.assign(t->shape.begin(), t->shape.end());
        } else if (const JSON* t = given ? given->get(name) : nullptr) {
            for (const JSON& v : t->arr) s.push_back(v.num);
        }
        if (s.empty() || s.size() > 2) return false;
        for (double v : s)
            if (!(v >= 1 && v < 2147483648.0)) return false;
        rows = (int)s[0], cols = s.size() > 1 ? (int)s[1] : 1;
        return true;
    };
    SEQ_CARD card;
    card.arch = arch->str;
    if (!read(cfg, shapes, card, err)) return bail(KF_INVALID_ARGS);
    if (type != KF_BF16 && type != KF_F32) {
        err = card.arch + ": storage BF16 or F32";
        return bail(KF_UNSUPPORTED_DATATYPE);
    }
    card.type = type;
    const int max_pos = (int)cfg.number_or("max_position_embeddings", 32768);
    card.n_ctx = max_seq > 0 ? max_seq : max_pos;
    std::unique_ptr<SeqFish> f(new SeqFish());
    int rc = f->BuildSeq(card, device, stream);
    if (rc != KF_OK) {
        err = card.arch + ": " + kf_last_error();
        return bail(rc);
    }
    if (!dir.empty()) {
        rc = f->Load(st, err);
        if (rc != KF_OK) return bail(rc);
    }
    if (rc_out) *rc_out = KF_OK;
    return f.release();
}

// ------------------------------------------------------------------------------------------------ state and work areas
int SeqFish::InitSlots(SeqSlots& s, int n) {
    s.n = n;
    std::vector<KVCache::Ring> rings;
    std::vector<KVCache::Recurrent> recurrent;
    for (const LAYER_CARD& L : card.layers) {
        const MIXER_CARD& m = L.mix;
        KVCache::Recurrent r;
        if (m.kind == MIXER_CARD::CHANNEL_DELTA) r.heads = m.heads, r.dim = m.dim, r.vdim = m.vdim, r.taps = m.taps, r.channels = 2 * m.kv_heads * m.dim + m.heads * m.vdim;
        if (m.kind == MIXER_CARD::PARALLEL) r.heads = m.sum_heads, r.dim = m.sum_dim, r.vdim = m.sum_vdim;
        recurrent.push_back(r);
        rings.push_back(m.kind == MIXER_CARD::CHANNEL_DELTA ? KVCache::Ring() : KVCache::Ring{m.Seen(card.n_ctx), m.kv_heads, std::max(m.dim, m.V()), 0});
    }
    KF_TRY(s.kv.InitRings(ctx, rings, n, card.type));
    KF_TRY(s.kv.InitRecurrent(ctx, recurrent, n, card.type));
    s.pos.assign(n, 0), s.parked.assign(n, 0), s.taken.assign(n, 0);
    s.pick_ws = Mem(ctx, "pick", KF_F32, kf_rb_pick_scratch(n) / 4), s.logits16 = Mem(ctx, "logits16", KF_BF16, card.vocab);
    if (!s.pick_ws || !s.logits16) return KF_OUTOF_GPUMEMORY;
    return Ensure(s.dec, n, 0, n, true);
}
int SeqFish::Ensure(RowWork& w, int rows, int n_seq, int head_rows, bool decode) {
    const int W = Width(card.width), V = Width(card.vocab), T = card.type;
    bool ok = true;
    auto get = [&](hGTensor& t, const char* name, int type, size_t n) {
        if (n == 0 || (t && t->szData >= n * (type == KF_BF16 ? 2 : 4))) return;
        t.reset();
        t = Mem(ctx, name, type, n);
        ok = ok && t;
    };
    if (rows > w.rows || n_seq > w.n_seq || head_rows > w.head_rows) KF_TRY(kf_sync(ctx));
    if (rows > w.rows || n_seq > w.n_seq) {
        rows = std::max(rows, w.rows);
        size_t act = 0, y = 0, rl = 0, pairs = 0, list = 0, tiles = 0;
        RowNeed need;
        for (const auto& a : mixers) a->Need(need, rows, decode ? rows : std::max(n_seq, w.n_seq), decode);
        for (const auto& f : ffs) {
            if (f->c.kind == FF_CARD::NONE) continue;
            const bool moe = f->c.kind == FF_CARD::MOE;
            act = std::max<size_t>(act, (size_t)rows * (moe ? f->c.top : 1) * f->ldact);
            if (!moe) continue;
            rl = std::max<size_t>(rl, (size_t)rows * f->router.m), pairs = std::max<size_t>(pairs, (size_t)rows * f->c.top);
            if (!f->Sums(T, rows)) y = std::max<size_t>(y, (size_t)rows * f->c.top * W);
            for (int tile : {16, 32, 48, 64, 128}) { /* whichever tile a batch of at most `rows` rows picks */
                const size_t n = kf_rb_list_tiles(rows, f->c.top, f->c.experts, tile);
                tiles = std::max(tiles, n), list = std::max(list, n * tile);
            }
        }
        get(w.x, "x", KF_F32, (size_t)rows * W), get(w.z, "z", KF_F32, (size_t)rows * W), get(w.h, "h", T, (size_t)rows * W);
        get(w.raw, "raw", T, need.raw), get(w.ao, "ao", T, need.ao), get(w.knew, "knew", T, need.knew);
        get(w.az, "az", KF_F32, need.az), get(w.gz, "gz", T, need.gz), get(w.recur, "recur", KF_F32, need.recur), get(w.act, "act", T, act), get(w.y, "y", T, y), get(w.rlogits, "rlogits", KF_F32, rl);
        get(w.meta, "meta", KF_F32, (size_t)rows * KF_RB_META), get(w.tok, "tok", KF_F32, rows), get(w.ids, "ids", KF_F32, pairs), get(w.weight, "weight", KF_F32, pairs);
        get(w.list, "list", KF_F32, list), get(w.tile_expert, "tile_expert", KF_F32, tiles), get(w.scratch, "scratch", KF_F32, need.scratch);
        if (decode) get(w.ssq, "ssq", KF_F32, (size_t)(W / 16) * KF_RB_NORM_ROWS);
        w.rows = rows;
    }
    if (n_seq > w.n_seq) get(w.seqs, "seqs", KF_F32, (size_t)n_seq * 4), w.n_seq = n_seq;
    if (head_rows > w.head_rows) {
        get(w.want, "want", KF_F32, (size_t)head_rows * (1 + KF_RB_META) + 4), get(w.hl, "hl", T, (size_t)head_rows * W), get(w.logits, "logits", KF_F32, (size_t)head_rows * V);
        w.head_rows = head_rows;
    }
    return ok ? KF_OK : KF_OUTOF_GPUMEMORY;
}

// ------------------------------------------------------------------------------------------------ steps
int SeqFish::Layers(RowWork& w, const KVCache& kv, const RowBatch& b) {
    const int W = Width(card.width), n = b.n, n_seq = b.n_seq;
    // few rows: the norm in front of a dense gate | up inside that product (in front of the q | k | gate product and of a router the separate launch measured the same or faster)
    const bool fuse = n_seq == 0 && !card.add_norm && kf_rb_linear_norms(card.type, n, W);
    w.pending = nullptr;
    KF_TRY(Enter(w, n));
    for (size_t l = 0; l < mixers.size(); l++) {
        KF_TRY(mixers[l]->Forw(w, kv, b, fuse && ffs[l]->c.kind == FF_CARD::DENSE));
        KF_TRY(ffs[l]->Forw(w, n));
        if (tap && n_seq && n == tap_rows) {
            std::vector<float> rows((size_t)n * W);
            KF_TRY(kf_d2h(ctx, rows.data(), w.x->data, rows.size() * 4));
            for (int r = 0; r < n; r++) std::memcpy(tap + ((size_t)l * n + r) * card.width, rows.data() + (size_t)r * W, (size_t)card.width * 4);
        }
    }
    return KF_OK;
}
int SeqFish::HeadRows(RowWork& w, const int32_t* h_rows, int n) {
    if (h_rows) KF_TRY(kf_h2d(ctx, w.want->data, h_rows, (size_t)n * 4));
    const int32_t* rows = h_rows ? I(w.want) : nullptr;
    KF_TRY(card.norm_kind == KF_RB_RMS ? seq_norm.Forw(F(w.x), n, nullptr, P(w.hl), nullptr, 0, 0, rows) : seq_norm.Rows(w, F(w.x), n, nullptr, nullptr, P(w.hl), rows, false));
    return seq_head.Forw(P(w.hl), seq_head.k, n, F(w.logits), seq_head.m, KF_RB_STORE_F32);
}
int SeqFish::Spans(SeqSlots& s, const SeqSpan* spans, int n_span, const int32_t* want, int n_want, float* out, bool last) {
    if (n_span < 1) return KF_INVALID_ARGS;
    for (int i = 0; i < n_span; i++) {
        const SeqSpan& p = spans[i];
        if (p.slot < 0 || p.slot >= s.n || p.n < 1 || p.pos0 < 0 || p.pos0 + p.n > card.n_ctx || !p.tokens) return KF_INVALID_ARGS;
        for (int j = 0; j < i; j++)
            if (spans[j].slot == p.slot) return KF_INVALID_ARGS;
        for (int t = 0; t < p.n; t++)
            if (p.tokens[t] < 0 || p.tokens[t] >= card.vocab) return KF_INVALID_ARGS;
    }
    for (int i = 0; i < n_want; i++)
        if (want[2 * i] < 0 || want[2 * i] >= n_span || want[2 * i + 1] < 0 || want[2 * i + 1] >= spans[want[2 * i]].n) return KF_INVALID_ARGS;
    const int V = Width(card.vocab), cap = std::max(prefill_chunk, 1);
    std::vector<int> done(n_span, 0);
    for (;;) {
        // a pass: the spans' next tokens, in order, up to `cap` rows
        std::vector<int32_t> meta, tok, seqs;
        std::vector<int> row0(n_span, -1), from(n_span, 0), part;
        int rows = 0, max_n = 0;
        for (int i = 0; i < n_span && rows < cap; i++) {
            const SeqSpan& p = spans[i];
            const int n = std::min(p.n - done[i], cap - rows);
            if (n < 1) continue;
            row0[i] = rows, from[i] = done[i], part.push_back(i);
            for (int t = 0; t < n; t++) {
                const int32_t m[4] = {p.pos0 + done[i] + t, p.slot, p.pos0 + done[i], p.pos0 + done[i] + n - 1};
                meta.insert(meta.end(), m, m + 4), tok.push_back(p.tokens[done[i] + t]);
            }
            const int32_t q[4] = {rows, n, p.pos0 + done[i], p.slot};
            seqs.insert(seqs.end(), q, q + 4);
            rows += n, max_n = std::max(max_n, n), done[i] += n;
        }
        if (!rows) break;
        KF_TRY(Ensure(pre, rows, n_span, 1, false));
        KF_TRY(kf_h2d(ctx, pre.meta->data, meta.data(), meta.size() * 4));
        KF_TRY(kf_h2d(ctx, pre.tok->data, tok.data(), tok.size() * 4));
        KF_TRY(kf_h2d(ctx, pre.seqs->data, seqs.data(), seqs.size() * 4));
        KF_TRY(kf_rb_embed(ctx, card.type, table->data, card.vocab, card.width, Width(card.width), I(pre.tok), rows, F(pre.x), P(pre.h)));
        KF_TRY(Layers(pre, s.kv, RowBatch{rows, (int)part.size(), max_n, 0}));
        // logits asked for, a block of rows at a time
        std::vector<int32_t> list, at;
        for (int i = 0; i < n_want; i++) {
            const int sp = want[2 * i], t = want[2 * i + 1] - from[sp];
            if (row0[sp] >= 0 && t >= 0 && t < done[sp] - from[sp]) list.push_back(row0[sp] + t), at.push_back(i);
        }
        const int block = 512;
        for (size_t b = 0; b < list.size(); b += block) {
            const int n = (int)std::min<size_t>(block, list.size() - b);
            KF_TRY(Ensure(pre, rows, n_span, n, false));
            KF_TRY(HeadRows(pre, list.data() + b, n));
            std::vector<float> lg((size_t)n * V);
            KF_TRY(kf_d2h(ctx, lg.data(), pre.logits->data, lg.size() * 4));
            for (int j = 0; j < n; j++) std::memcpy(out + (size_t)at[b + j] * card.vocab, lg.data() + (size_t)j * V, (size_t)card.vocab * 4);
        }
        if (last) { /* the spans that end in this pass: their last rows' logits into the slots', the greedy pick */
            list.clear(), meta.clear();
            std::vector<int> ends;
            for (int i : part)
                if (done[i] == spans[i].n) {
                    const int32_t m[4] = {spans[i].pos0 + spans[i].n - 1, spans[i].slot, 0, 0};
                    list.push_back(row0[i] + done[i] - from[i] - 1), meta.insert(meta.end(), m, m + 4), ends.push_back(i);
                }
            const int n = (int)list.size();
            if (n) {
                KF_TRY(Ensure(pre, rows, n_span, n, false));
                KF_TRY(HeadRows(pre, list.data(), n));
                int32_t* d_meta = I(pre.want) + up(pre.head_rows, 4);
                KF_TRY(kf_h2d(ctx, d_meta, meta.data(), meta.size() * 4));
                for (int j = 0; j < n; j++) {
                    KF_TRY(kf_d2d(ctx, F(s.dec.logits) + (size_t)spans[ends[j]].slot * V, F(pre.logits) + (size_t)j * V, (size_t)V * 4));
                    KF_TRY(kf_memset32(ctx, s.d_state + 4 * spans[ends[j]].slot + 3, 0, 1));
                }
                KF_TRY(kf_rb_pick(ctx, F(pre.logits), V, card.vocab, n, d_meta, s.d_state, s.d_tokens_out, card.n_ctx, s.pick_ws->data));
            }
        }
    }
    for (int i = 0; i < n_span; i++) s.pos[spans[i].slot] = spans[i].pos0 + spans[i].n;
    return KF_OK;
}
int SeqFish::EnqueueSlots(SeqSlots& s, int bound, bool pick) {
    RowWork& w = s.dec;
    KF_TRY(kf_rb_embed_state(ctx, card.type, table->data, card.vocab, card.width, Width(card.width), s.d_state, s.d_forced, card.n_ctx, card.n_ctx, s.n, F(w.x), P(w.h), I(w.meta)));
    KF_TRY(Layers(w, s.kv, RowBatch{s.n, 0, 0, bound}));
    KF_TRY(HeadRows(w, nullptr, s.n));
    return pick ? kf_rb_pick(ctx, F(w.logits), seq_head.m, card.vocab, s.n, I(w.meta), s.d_state, s.d_tokens_out, card.n_ctx, s.pick_ws->data) : KF_OK;
}
int SeqFish::StepSlots(SeqSlots& s, int steps, bool pick, bool use_graph) {
    for (int i = 0; i < steps; i++) {
        int top = 0;
        for (int j = 0; j < s.n; j++)
            if (!s.parked[j]) top = std::max(top, s.pos[j]);
        top = std::min(top, card.n_ctx - 1);
        int b = 0;
        while ((64 << b) - 1 < top) b++;
        const int bound = std::min((64 << b) - 1, card.n_ctx - 1), key = 2 * b + (pick ? 1 : 0);
        if (use_graph) {
            kf_graph*& g = s.graphs[key];
            if (!g) {
                KF_TRY(EnqueueSlots(s, bound, false)); /* outside the capture first: kernels loaded, attributes set.  Without the pick the states stay and the step repeats itself */
                KF_TRY(kf_graph_begin(ctx));
                const int rc = EnqueueSlots(s, bound, pick), rc2 = kf_graph_end(ctx, &g);
                if (rc != KF_OK || rc2 != KF_OK) {
                    if (rc2 == KF_OK) kf_graph_destroy(g);
                    g = nullptr;
                    return rc != KF_OK ? rc : rc2;
                }
            }
            KF_TRY(kf_graph_launch(ctx, g));
        } else {
            KF_TRY(EnqueueSlots(s, bound, pick));
        }
        for (int j = 0; j < s.n; j++)
            if (!s.parked[j] && s.pos[j] < card.n_ctx) s.pos[j]++;
    }
    return KF_OK;
}
int SeqFish::Logits16(SeqSlots& s, int slot, void** out) {
    KF_TRY(kf_rb_to_bf16(ctx, F(s.dec.logits) + (size_t)slot * seq_head.m, ToX(s.logits16), card.vocab));
    *out = s.logits16->data;
    return KF_OK;
}
int SeqFish::Draw(SeqSlots& s, int slot, const CHAT_SAMPLER& sp, uint64_t* d_rng) {
    void* lg = nullptr;
    KF_TRY(Logits16(s, slot, &lg));
    return (sp.true_topk ? kf_sample_topk : kf_sample)(ctx, reinterpret_cast<kf_bf16*>(lg), card.vocab, sp.top_k, sp.temperature, sp.top_p, d_rng, nullptr, s.d_state + 4 * slot,
                                                       s.d_tokens_out + (size_t)slot * card.n_ctx, s.d_forced + (size_t)slot * card.n_ctx, card.n_ctx);
}

// ------------------------------------------------------------------------------------------------ the single-sequence surface
int SeqFish::EnqueueStep(int bound) {
    KF_TRY(EnqueueSlots(self, bound, samp_params.greedy()));
    return samp_params.greedy() ? KF_OK : Draw(self, 0, samp_params, d_rng);
}
int SeqFish::Warm(int bound) { return EnqueueSlots(self, bound, false); }
int SeqFish::ForwardOnRLS(int token, int pos) {
    if (pos < 0 || pos >= config.n_ctx || token < 0 || token >= config.vocab) return KF_INVALID_ARGS;
    tok_pos = pos;
    KF_TRY(kf_memset32(ctx, d_forced + pos, -1, 1)); /* the token of the call is the step's */
    KF_TRY(kf_set_state(ctx, d_state, token, pos));
    return EnqueueStep(pos_bound());
}
int SeqFish::Prefill(const int* tokens, int n, int pos0) {
    if (n < 1) return KF_INVALID_ARGS;
    const SeqSpan sp{0, pos0, n, tokens};
    KF_TRY(Spans(self, &sp, 1, nullptr, 0, nullptr, true));
    tok_pos = pos0 + n - 1;
    if (samp_params.greedy()) return KF_OK;
    KF_TRY(SetState(tokens[n - 1], pos0 + n - 1)); /* the greedy pick moved the state: draw instead */
    return Draw(self, 0, samp_params, d_rng);
}
void* SeqFish::LogitsPtr() {
    void* p = nullptr;
    return Logits16(self, 0, &p) == KF_OK ? p : nullptr;
}

}  // namespace koifish
