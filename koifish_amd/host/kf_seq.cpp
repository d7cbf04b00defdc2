// kf_seq.cpp -- see kf_seq.hpp.  Every device action is a kf_* call.
#include "kf_seq.hpp"

#include <algorithm>
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
int ChunkAttention::Forw(RowWork& w, const KVCache& kv, int n, int n_seq, int max_n, int max_pos, bool defer) {
    const SEQ_CARD& card = hFish->Seq()->card;
    KF_TRY(qkg.Forw(P(w.h), qkg.k, n, P(w.raw), ldraw, KF_RB_STORE));
    const KVCache::Ring& ring = kv.rings[layid - 1];
    kf_rb_attention a;
    std::memset(&a, 0, sizeof(a));
    a.raw = P(w.raw), a.out = P(w.ao), a.k_new = P(w.knew), a.k_cache = kv.Ring0(KVCache::KV_KEY, layid - 1), a.v_cache = kv.Ring0(KVCache::KV_VAL, layid - 1);
    a.q_norm = c.qk_norm ? P(qn) : nullptr, a.k_norm = c.qk_norm ? P(kn) : nullptr, a.rope = rope, a.scratch = P(w.scratch);
    a.ldraw = ldraw, a.ldout = ldout, a.slot_stride = (int64_t)ring.slot_stride(), a.head_stride = (int64_t)ring.head_stride();
    a.type = card.type, a.n_head = c.heads, a.n_kv = c.kv_heads, a.dim = c.dim, a.rot_dims = c.rot.dims, a.chunk = c.chunk, a.cache_rows = ring.rows, a.gated = c.gated;
    a.scale = c.scale, a.eps = card.eps;
    if (n_seq) KF_TRY(kf_rb_attention_prefill(hFish->ctx, &a, I(w.meta), n, I(w.seqs), n_seq, max_n));
    else KF_TRY(kf_rb_attention_decode(hFish->ctx, &a, I(w.meta), n, max_pos));
    KF_TRY(proj.Forw(P(w.ao), ldout, n, F(w.z), proj.m, KF_RB_RESIDUAL, 0, F(w.x), card.alpha, KF_RB_ALL, nullptr, defer ? F(w.ssq) : nullptr));
    if (defer) {
        w.pending = &norm;
        return KF_OK;
    }
    return norm.Forw(F(w.z), n, F(w.x), P(w.h));
}
int RowFFN::Forw(RowWork& w, int n) {
    const SEQ_CARD& card = hFish->Seq()->card;
    if (c.kind == FF_CARD::NONE) return KF_OK;
    const int64_t ld = gateup.k;
    if (c.kind == FF_CARD::DENSE) {
        KF_TRY(gateup.ForwNormed(w, n, P(w.act), ldact, KF_RB_GATED, c.act));
        KF_TRY(down.Forw(P(w.act), ldact, n, F(w.z), ld, KF_RB_RESIDUAL, 0, F(w.x), card.alpha));
        return norm.Forw(F(w.z), n, F(w.x), P(w.h));
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
    mixers.clear(), ffs.clear(), targets.clear(), stage.reset(), table.reset();
    seq_head = RowProduct(), seq_norm = RowNorm();
}
void SeqFish::DropGraphs(SeqSlots& s) {
    for (auto& g : s.graphs)
        if (g.second) kf_graph_destroy(g.second);
    s.graphs.clear();
}

int SeqFish::BuildSeq(const SEQ_CARD& c, int device, void* stream) {
    card = c;
    config.nEmbed = c.width, config.nLayer = (int)c.layers.size(), config.vocab = c.vocab, config.n_ctx = c.n_ctx, config.rms_eps = config.qk_eps = c.eps;
    config.n_head = c.layers[0].mix.heads, config.n_head_kv = c.layers[0].mix.kv_heads, config.head_dim = c.layers[0].mix.dim, config.n_ff = c.layers[0].ff.ff;
    config.rope_theta = (float)c.layers[0].mix.rot.base, config.tie_word_embeddings = false;
    use_engine = false;
    KF_TRY(kf_init(device, stream, &ctx));
    const int W = Width(c.width), V = Width(c.vocab), tp = c.type;
    bool ok = true;
    auto mem = [&](const std::string& name, size_t n) {
        hGTensor t = Mem(ctx, name.c_str(), tp, n);
        ok = ok && t;
        return t;
    };
    auto product = [&](RowProduct& p, const std::string& name, int m, int k, int experts = 0) {
        p.hFish = this, p.name = name, p.m = m, p.k = k, p.experts = experts;
        p.w = mem(name, (size_t)m * k * std::max(experts, 1));
    };
    auto norm = [&](RowNorm& n, const std::string& name) {
        n.hFish = this, n.name = name, n.dim = c.width, n.ld = W, n.w = mem(name, W);
        targets[name] = Target{n.w, 0, 0, c.width, 1, 1, -1, false, false};
    };
    table = mem("embed", (size_t)V * W);
    targets["embed"] = Target{table, 0, 0, c.vocab, c.width, W, -1, false, false};
    product(seq_head, "head", V, W);
    targets["head"] = Target{seq_head.w, 0, 0, c.vocab, c.width, W, -1, true, false};
    norm(seq_norm, "final.norm");
    for (size_t l = 0; l < c.layers.size(); l++) {
        const LAYER_CARD& L = c.layers[l];
        const std::string p = "l" + std::to_string(l) + ".";
        auto a = std::make_unique<ChunkAttention>();
        a->hFish = this, a->layid = (int)l + 1, a->name = p + "mix", a->c = L.mix;
        const int qd = L.mix.heads * L.mix.dim, kd = L.mix.kv_heads * L.mix.dim, rows = qd + kd + (L.mix.gated ? qd : 0);
        a->ldraw = Width(rows), a->ldout = Width(qd);
        product(a->qkg, p + "mix.qkg", a->ldraw, W);
        product(a->proj, p + "mix.o", W, a->ldout);
        targets[p + "mix.q"] = Target{a->qkg.w, 0, 0, qd, c.width, W, -1, true, false};
        targets[p + "mix.k"] = Target{a->qkg.w, 0, qd, kd, c.width, W, -1, true, false};
        if (L.mix.gated) targets[p + "mix.g"] = Target{a->qkg.w, 0, qd + kd, qd, c.width, W, -1, true, false};
        targets[p + "mix.o"] = Target{a->proj.w, 0, 0, c.width, qd, a->ldout, -1, true, false};
        if (L.mix.qk_norm) {
            a->qn = mem(p + "mix.q.norm", Width(L.mix.dim)), a->kn = mem(p + "mix.k.norm", Width(L.mix.dim));
            targets[p + "mix.q.norm"] = Target{a->qn, 0, 0, L.mix.dim, 1, 1, -1, false, false};
            targets[p + "mix.k.norm"] = Target{a->kn, 0, 0, L.mix.dim, 1, 1, -1, false, false};
        }
        norm(a->norm, p + "norm1");
        for (auto& r : ropes)
            if (r.first == L.mix.rot) a->rope = r.second;
        if (!a->rope) {
            const ROT_CARD& r = L.mix.rot;
            float* d = nullptr;
            std::vector<float> tab((size_t)c.n_ctx * std::max(r.dims, 2), 0.f);
            if (r.dims) KF_TRY(kf_rb_rope_table_host(tab.data(), c.n_ctx, r.dims, r.base, r.factor, r.low, r.high, r.original));
            KF_TRY(kf_malloc(ctx, tab.size() * 4, (void**)&d));
            ropes.emplace_back(r, d);
            KF_TRY(kf_h2d(ctx, d, tab.data(), tab.size() * 4));
            a->rope = d;
        }
        mixers.push_back(std::move(a));
        auto f = std::make_unique<RowFFN>();
        f->hFish = this, f->layid = (int)l + 1, f->name = p + "mlp", f->c = L.ff;
        if (L.ff.kind != FF_CARD::NONE) {
            const int ff = Width(L.ff.ff), E = L.ff.kind == FF_CARD::MOE ? L.ff.experts : 0;
            f->ldact = ff;
            product(f->gateup, p + "mlp.gateup", 2 * ff, W, E);
            product(f->down, p + "mlp.down", W, ff, E);
            for (int e = 0; e < std::max(E, 1); e++) {
                const std::string q = p + "mlp." + (E ? "e" + std::to_string(e) + "." : "");
                const size_t gu = (size_t)e * 2 * ff * W, dn = (size_t)e * W * ff;
                targets[q + "gate"] = Target{f->gateup.w, gu, 0, L.ff.ff, c.width, W, 0, true, false};
                targets[q + "up"] = Target{f->gateup.w, gu, 0, L.ff.ff, c.width, W, 1, true, false};
                targets[q + "down"] = Target{f->down.w, dn, 0, c.width, L.ff.ff, ff, -1, true, false};
            }
            if (E) {
                product(f->router, p + "mlp.router", Width(E), W);
                f->router_b = mem(p + "mlp.router.b", Width(E));
                targets[p + "mlp.router"] = Target{f->router.w, 0, 0, E, c.width, W, -1, true, false};
                targets[p + "mlp.router.b"] = Target{f->router_b, 0, 0, E, 1, 1, -1, false, false};
            }
            norm(f->norm, p + "norm2");
        }
        ffs.push_back(std::move(f));
    }
    if (!ok) return KF_OUTOF_GPUMEMORY;
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
    SEQ_CARD card;
    card.arch = arch->str;
    if (!read(cfg, card, err)) return bail(KF_INVALID_ARGS);
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
        K_SafeTensors st;
        rc = st.OpenDir(dir);
        if (rc != KF_OK) err = st.err;
        else rc = f->Load(st, err);
        if (rc != KF_OK) return bail(rc);
    }
    if (rc_out) *rc_out = KF_OK;
    return f.release();
}

// ------------------------------------------------------------------------------------------------ state and work areas
int SeqFish::InitSlots(SeqSlots& s, int n) {
    s.n = n;
    std::vector<KVCache::Ring> rings;
    for (const LAYER_CARD& L : card.layers) rings.push_back(KVCache::Ring{L.mix.chunk > 0 ? std::min(L.mix.chunk, card.n_ctx) : card.n_ctx, L.mix.kv_heads, L.mix.dim, 0});
    KF_TRY(s.kv.InitRings(ctx, rings, n, card.type));
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
    if (rows > w.rows) {
        size_t raw = 0, ao = 0, kn = 0, act = 0, y = 0, rl = 0, pairs = 0, list = 0, tiles = 0, scratch = 0;
        for (const auto& a : mixers) {
            raw = std::max<size_t>(raw, (size_t)rows * a->ldraw), ao = std::max<size_t>(ao, (size_t)rows * a->ldout), kn = std::max<size_t>(kn, (size_t)rows * a->c.kv_heads * a->c.dim);
            if (decode) scratch = std::max(scratch, kf_rb_attention_scratch(rows, a->c.heads, a->c.dim) / 4);
        }
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
        get(w.raw, "raw", T, raw), get(w.ao, "ao", T, ao), get(w.knew, "knew", T, kn), get(w.act, "act", T, act), get(w.y, "y", T, y), get(w.rlogits, "rlogits", KF_F32, rl);
        get(w.meta, "meta", KF_F32, (size_t)rows * KF_RB_META), get(w.tok, "tok", KF_F32, rows), get(w.ids, "ids", KF_F32, pairs), get(w.weight, "weight", KF_F32, pairs);
        get(w.list, "list", KF_F32, list), get(w.tile_expert, "tile_expert", KF_F32, tiles), get(w.scratch, "scratch", KF_F32, scratch);
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
int SeqFish::Layers(RowWork& w, const KVCache& kv, int n, int n_seq, int max_n, int max_pos) {
    const int W = Width(card.width);
    // few rows: the norm in front of a dense gate | up inside that product (in front of the q | k | gate product and of a router the separate launch measured the same or faster)
    const bool fuse = n_seq == 0 && kf_rb_linear_norms(card.type, n, W);
    w.pending = nullptr;
    for (size_t l = 0; l < mixers.size(); l++) {
        KF_TRY(mixers[l]->Forw(w, kv, n, n_seq, max_n, max_pos, fuse && ffs[l]->c.kind == FF_CARD::DENSE));
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
    KF_TRY(seq_norm.Forw(F(w.x), n, nullptr, P(w.hl), nullptr, 0, 0, h_rows ? I(w.want) : nullptr));
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
        KF_TRY(Layers(pre, s.kv, rows, (int)part.size(), max_n, 0));
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
    KF_TRY(Layers(w, s.kv, s.n, 0, 0, bound));
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
