// kf_bolopel.cpp -- the reader of Bolopel's config.json.
//
// Bolopel: sinusoidal position vectors and a norm behind the embedding; every sublayer f adds its normed output, x' = x + norm(f(x)) (layer norm, 32-bit x).  Mixers:
//   channel_delta  the gated delta rule with a decay per key channel behind a short convolution (kf_rb_delta)
//   parallel       windowed attention with a sink and unit q / k (kf_rb_attention) beside a sum with one decay per head (kf_rb_decay)
// Feed-forward: none or a SiLU-gated triple.  The ranks of the decay's and the gate's factors are read from the tensors' shapes.
#include "kf_seq.hpp"

namespace koifish {

static bool read_delta(const JSON* mx, const seq_shapes& shapes, const std::string& prefix, MIXER_CARD& m, std::string& err, const std::string& at) {
    m.kind = MIXER_CARD::CHANNEL_DELTA;
    if (!CardNumber(mx, "heads", 1, m.heads, err, at) || !CardNumber(mx, "kv_heads", 1, m.kv_heads, err, at) || !CardNumber(mx, "dim", 1, m.dim, err, at) || !CardNumber(mx, "vdim", 1, m.vdim, err, at) ||
        !CardNumber(mx, "conv", 1, m.taps, err, at))
        return false;
    if (m.heads % m.kv_heads) {
        err = "config.json: " + at + ": " + std::to_string(m.heads) + " heads over " + std::to_string(m.kv_heads) + " kv_heads";
        return false;
    }
    for (auto& f : {std::make_pair("a1", &m.rank_a), std::make_pair("g1", &m.rank_g)}) {
        int cols = 0;
        const std::string name = prefix + "mix." + f.first;
        if (!shapes || !shapes(name, *f.second, cols) || *f.second < 1) {
            err = "tensor '" + name + "' not in the checkpoint (its rows are a size of the layer)";
            return false;
        }
    }
    return true;
}
static bool read_parallel(const JSON* mx, MIXER_CARD& m, std::string& err, const std::string& at) {
    m.kind = MIXER_CARD::PARALLEL, m.qk_unit = m.sink = true;
    const JSON *l = mx ? mx->get("left") : nullptr, *r = mx ? mx->get("right") : nullptr;
    double scale, ls, rs;
    if (!CardNumber(l, "heads", 1, m.heads, err, at + ".left") || !CardNumber(l, "kv_heads", 1, m.kv_heads, err, at + ".left") || !CardNumber(l, "dim", 1, m.dim, err, at + ".left") ||
        !CardNumber(l, "vdim", 1, m.vdim, err, at + ".left") || !CardNumber(l, "scale", -1e30, scale, err, at + ".left") ||
        !CardNumber(l->get("mask"), "size", 1, m.window, err, at + ".left.mask") || !CardNumber(r, "heads", 1, m.sum_heads, err, at + ".right") ||
        !CardNumber(r, "dim", 1, m.sum_dim, err, at + ".right") || !CardNumber(r, "vdim", 1, m.sum_vdim, err, at + ".right") || !CardNumber(mx, "left_scale", -1e30, ls, err, at) ||
        !CardNumber(mx, "right_scale", -1e30, rs, err, at))
        return false;
    m.scale = (float)scale, m.left_scale = (float)ls, m.right_scale = (float)rs;
    if (m.heads % m.kv_heads) {
        err = "config.json: " + at + ".left: " + std::to_string(m.heads) + " heads over " + std::to_string(m.kv_heads) + " kv_heads";
        return false;
    }
    const JSON* d = r->get("decay");
    if (!d || d->kind != JSON::ARR || (int)d->arr.size() != m.sum_heads) {
        err = "config.json: " + at + ".right.decay: a number per head";
        return false;
    }
    for (const JSON& v : d->arr) {
        if (v.kind != JSON::NUM) {
            err = "config.json: " + at + ".right.decay: a number per head";
            return false;
        }
        m.decay.push_back((float)v.num);
    }
    return true;
}

bool ReadBolopel(const JSON& cfg, const seq_shapes& shapes, SEQ_CARD& card, std::string& err) {
    double eps;
    if (!CardNumber(&cfg, "width", 1, card.width, err, "") || !CardNumber(&cfg, "vocab", 1, card.vocab, err, "") || !CardNumber(cfg.get("norm"), "eps", 0.0, eps, err, "norm")) return false;
    card.eps = (float)eps, card.add_norm = true, card.norm_kind = KF_RB_LAYER, card.sinusoid = 10000.0, card.embed_norm = true;
    const JSON* layers = cfg.get("layers");
    if (!layers || layers->kind != JSON::ARR || layers->arr.empty()) {
        err = "config.json: no layers";
        return false;
    }
    for (size_t l = 0; l < layers->arr.size(); l++) {
        const JSON& e = layers->arr[l];
        const std::string at = "layers[" + std::to_string(l) + "]";
        const JSON *type = e.get("type"), *mlp = e.get("mlp");
        const std::string t = type ? type->str : "";
        LAYER_CARD L;
        if (t == "channel_delta") {
            if (!read_delta(e.get("mixer"), shapes, "l" + std::to_string(l) + ".", L.mix, err, at + ".mixer")) return false;
        } else if (t == "parallel") {
            if (!read_parallel(e.get("mixer"), L.mix, err, at + ".mixer")) return false;
        } else {
            err = "config.json: " + at + ": mixer type '" + t + "' (served: channel_delta, parallel)";
            return false;
        }
        if (mlp && mlp->kind == JSON::OBJ) {
            const JSON* kind = mlp->get("kind");
            if (!kind || kind->str != "dense") {
                err = "config.json: " + at + ".mlp.kind '" + (kind ? kind->str : "") + "' (served: dense)";
                return false;
            }
            L.ff.kind = FF_CARD::DENSE, L.ff.act = KF_RB_SILU;
            if (!CardNumber(mlp, "ff", 1, L.ff.ff, err, at + ".mlp")) return false;
        }
        card.layers.push_back(L);
    }
    return true;
}

}  // namespace koifish
