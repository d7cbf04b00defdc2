// kf_tizusun.cpp -- the registry of layer-by-layer designs and the reader of Tizusun's config.json.
//
// Tizusun: a post-norm decoder (every sublayer f: x' = norm(alpha x + f(x)), 32-bit x).  Mixer: kf_rb_attention with gate, q/k norms and chunks of `mask.size`.
// Feed-forward: none, one ReLU-gated matrix triple, or routed SiLU-gated triples.
#include "kf_seq.hpp"

namespace koifish {

bool CardNumber(const JSON* o, const char* key, double lo, double& out, std::string& err, const std::string& where) {
    const JSON* v = o ? o->get(key) : nullptr;
    if (!v || v->kind != JSON::NUM || !(v->num >= lo)) {
        err = "config.json: " + where + "." + key + " is missing or out of range";
        return false;
    }
    out = v->num;
    return true;
}
bool CardNumber(const JSON* o, const char* key, int lo, int& out, std::string& err, const std::string& where) {
    double v;
    if (!CardNumber(o, key, (double)lo, v, err, where)) return false;
    if (v != (double)(int)v) {
        err = "config.json: " + where + "." + key + " is not an integer";
        return false;
    }
    out = (int)v;
    return true;
}

bool ReadTizusun(const JSON& cfg, const seq_shapes&, SEQ_CARD& card, std::string& err) {
    const auto need = [](auto&&... a) { return CardNumber(a...); };
    double eps, alpha;
    if (!need(&cfg, "width", 1, card.width, err, "") || !need(&cfg, "vocab", 1, card.vocab, err, "") || !need(cfg.get("norm"), "eps", 0.0, eps, err, "norm")) return false;
    if (!need(&cfg, "postln_alpha", -1e30, alpha, err, "")) return false;
    card.eps = (float)eps, card.alpha = (float)alpha;
    const JSON* layers = cfg.get("layers");
    if (!layers || layers->kind != JSON::ARR || layers->arr.empty()) {
        err = "config.json: no layers";
        return false;
    }
    for (size_t l = 0; l < layers->arr.size(); l++) {
        const JSON& e = layers->arr[l];
        const std::string at = "layers[" + std::to_string(l) + "]";
        const JSON *type = e.get("type"), *mx = e.get("mixer"), *mlp = e.get("mlp");
        if (!type || type->str != "attention") {
            err = "config.json: " + at + ": mixer type '" + (type ? type->str : "") + "' (served: attention)";
            return false;
        }
        LAYER_CARD L;
        MIXER_CARD& m = L.mix;
        int vdim = 0;
        double scale;
        const JSON* rot = mx ? mx->get("rot") : nullptr;
        if (!need(mx, "heads", 1, m.heads, err, at + ".mixer") || !need(mx, "kv_heads", 1, m.kv_heads, err, at + ".mixer") || !need(mx, "dim", 1, m.dim, err, at + ".mixer") ||
            !need(mx, "scale", -1e30, scale, err, at + ".mixer") || (mx->get("mask") && !need(mx->get("mask"), "size", 1, m.chunk, err, at + ".mixer.mask")) ||
            !need(rot, "dims", 0, m.rot.dims, err, at + ".mixer.rot") || !need(rot, "base", 0.0, m.rot.base, err, at + ".mixer.rot"))
            return false;
        vdim = (int)mx->number_or("vdim", m.dim);
        m.scale = (float)scale, m.gated = true, m.qk_norm = true;
        if (vdim != m.dim || m.heads % m.kv_heads || m.rot.dims > m.dim || (m.rot.dims & 1)) {
            err = "config.json: " + at + ".mixer: " + std::to_string(m.heads) + " / " + std::to_string(m.kv_heads) + " heads of " + std::to_string(m.dim) + " / " + std::to_string(vdim) + ", " +
                  std::to_string(m.rot.dims) + " rotated (values are the keys: equal sizes; heads divide; an even number rotated)";
            return false;
        }
        if (const JSON* s = rot->get("scaling")) {
            if (s->kind == JSON::OBJ && (!need(s, "factor", 0.0, m.rot.factor, err, at + ".mixer.rot.scaling") || !need(s, "low", 0.0, m.rot.low, err, at + ".mixer.rot.scaling") ||
                                         !need(s, "high", 0.0, m.rot.high, err, at + ".mixer.rot.scaling") || !need(s, "original", 0.0, m.rot.original, err, at + ".mixer.rot.scaling")))
                return false;
        }
        if (mlp && mlp->kind == JSON::OBJ) {
            const JSON* kind = mlp->get("kind");
            const std::string k = kind ? kind->str : "";
            if (k == "dense") {
                L.ff.kind = FF_CARD::DENSE, L.ff.act = KF_RB_RELU;
                if (!need(mlp, "ff", 1, L.ff.ff, err, at + ".mlp")) return false;
            } else if (k == "moe") {
                L.ff.kind = FF_CARD::MOE, L.ff.act = KF_RB_SILU;
                if (!need(mlp->get("expert"), "ff", 1, L.ff.ff, err, at + ".mlp.expert") || !need(mlp->get("router"), "experts", 1, L.ff.experts, err, at + ".mlp.router") ||
                    !need(mlp->get("router"), "top", 1, L.ff.top, err, at + ".mlp.router"))
                    return false;
                if (L.ff.top > L.ff.experts) {
                    err = "config.json: " + at + ".mlp.router: top " + std::to_string(L.ff.top) + " of " + std::to_string(L.ff.experts) + " experts";
                    return false;
                }
            } else {
                err = "config.json: " + at + ".mlp.kind '" + k + "' (served: dense, moe)";
                return false;
            }
        }
        card.layers.push_back(L);
    }
    return true;
}

static const struct {
    const char* name;
    seq_card_reader read;
} kSeqArchs[] = {{"Tizusun", ReadTizusun}, {"Bolopel", ReadBolopel}};
seq_card_reader FindSeqArch(const std::string& architecture) {
    for (const auto& e : kSeqArchs)
        if (architecture == e.name) return e.read;
    return nullptr;
}

}  // namespace koifish
