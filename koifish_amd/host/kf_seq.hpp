// kf_seq.hpp -- decoders described layer by layer (every layer its own mixer and feed-forward sizes), on the row-batch operators of include/kf_rb.h.
//
// A SeqFish is a Fish: the flat kfh_* surface (generate, prefill, run_steps, sampler, forced ids, graphs) and the slot scheduler (XcdReplicas: prompts in a queue, one slot
// per live request) drive it as they drive the Qwen3 decoder.  What differs is below the step: a 32-bit residual stream, bf16 or fp32 storage, state rings sized by what
// a layer can see, and steps over any set of slots at once.
#pragma once
#include <algorithm>
#include <functional>
#include <map>
#include <string>
#include <vector>

#include "../../include/kf_rb.h"
#include "kf_host.hpp"
#include "kf_safetensors.hpp"

namespace koifish {

struct ROT_CARD {
    int dims = 0;
    double base = 10000, factor = 1, low = 1, high = 4, original = 1;
    bool operator==(const ROT_CARD& o) const { return dims == o.dims && base == o.base && factor == o.factor && low == o.low && high == o.high && original == o.original; }
};
struct MIXER_CARD {
    enum KIND { ATTENTION = 0, CHANNEL_DELTA, PARALLEL } kind = ATTENTION;
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;  // attention: vdim 0: the values are the projected keys
    // attention, alone or beside a decayed sum (PARALLEL)
    int chunk = 0, window = 0;  // neither: plain causal
    float scale = 1;
    bool gated = false, qk_norm = false, qk_unit = false, sink = false;  // norms of q and k: with weights, without
    ROT_CARD rot;
    // CHANNEL_DELTA: gated delta rule behind a short convolution; the ranks of the decay's and the output gate's factors
    int taps = 0, rank_a = 0, rank_g = 0;
    // PARALLEL: left_scale * attention + right_scale * decayed sum
    int sum_heads = 0, sum_dim = 0, sum_vdim = 0;
    std::vector<float> decay;
    float left_scale = 1, right_scale = 1;
    int Seen(int n_ctx) const { return chunk > 0 ? std::min(chunk, n_ctx) : window > 0 ? std::min(window, n_ctx) : n_ctx; }  // positions a query can see
    int V() const { return vdim ? vdim : dim; }
};
struct FF_CARD {
    enum KIND { NONE = 0, DENSE, MOE } kind = NONE;
    int ff = 0, act = KF_RB_SILU, experts = 0, top = 0;
};
struct LAYER_CARD {
    MIXER_CARD mix;
    FF_CARD ff;
};
struct SEQ_CARD {
    std::string arch;
    int width = 0, vocab = 0, n_ctx = 0, type = KF_BF16;
    float eps = 1e-6f;
    // a sublayer f: x' = norm(alpha x + f(x)), or add_norm: x' = x + norm(f(x))
    float alpha = 1;
    bool add_norm = false;
    int norm_kind = KF_RB_RMS;
    double sinusoid = 0;      // base of position vectors added to the embedding; 0: none
    bool embed_norm = false;  // a norm behind the embedding
    std::vector<LAYER_CARD> layers;
};

// activations of a row batch; one set for the decode steps (captured graphs hold its addresses), one for prompts
struct RowNorm;
struct RowWork {
    RowNorm* pending = nullptr;  // decode: z holds a residual sum whose norm the next product forms itself
    int rows = 0, n_seq = 0, head_rows = 0;
    hGTensor ssq;                                                      // decode: z's sums of squares
    hGTensor x, z, h, raw, knew, ao, act, y, rlogits, scratch;         // residual and its sum (fp32), bf16 / fp32 rows, expert outputs, router logits, key-range partials
    hGTensor meta, seqs, tok, ids, weight, list, tile_expert, want, hl;  // int32 tables; hl: the rows the head reads
    hGTensor logits;                                                     // fp32 [head_rows][padded vocab]
    hGTensor az, gz, recur;                                              // recurrent layers: products of the low-rank factors, scratch
};
struct RowBatch {  // n rows; n_seq 0: a decode step, one row per slot, positions up to max_pos; otherwise the next rows of n_seq sequences, the longest max_n
    int n = 0, n_seq = 0, max_n = 0, max_pos = 0;
};
struct RowNeed {  // the most elements any mixer needs of a work area
    size_t raw = 0, ao = 0, knew = 0, scratch = 0, az = 0, gz = 0, recur = 0;
};

// the state of n slots: K / V rings, decode states, logits, the step graphs
struct SeqSlots {
    int n = 0;
    KVCache kv;
    int32_t *d_state = nullptr, *d_forced = nullptr, *d_tokens_out = nullptr;  // [n][4], [n][n_ctx], [n][n_ctx]: the owner's
    RowWork dec;
    hGTensor pick_ws, logits16;         // [1][vocab] bf16: what kf_sample reads
    std::vector<int> pos;               // upper bound of every slot's position
    std::vector<char> parked, taken;
    std::map<int, kf_graph*> graphs;    // step graphs: 2 * bucket + (1: with the greedy pick)
    ~SeqSlots();
};

struct SeqSpan {  // the next n tokens of the sequence in a slot
    int slot = 0, pos0 = 0, n = 0;
    const int32_t* tokens = nullptr;
};

struct SeqFish;
struct RowProduct : GeNeuron {  // padded weight [m][k] (x experts)
    hGTensor w;
    int m = 0, k = 0, experts = 0;
    int act_lo = 0, act_hi = 0, col_act = 0;  // KF_RB_STORE: columns [act_lo, act_hi) pass through col_act
    int Forw(const void* x, int64_t ldx, int n, void* y, int64_t ldy, int epilogue, int act = 0, const float* res = nullptr, float alpha = 0, int mode = KF_RB_ALL,
             const kf_rb_experts* ex = nullptr, float* ssq = nullptr);
    int ForwNormed(RowWork& w, int n, void* y, int64_t ldy, int epilogue, int act = 0);  // of w.h, the pending norm first
};
struct RowNorm : GeNeuron {
    hGTensor w;
    int dim = 0, ld = 0;
    int Forw(const void* z, int n, float* x_out, void* h_out, const float* res = nullptr, float alpha = 0, int top = 0, const int32_t* rows = nullptr);
    int Rows(RowWork& w, const float* z, int n, const float* add, float* x_out, void* h_out, const int32_t* rows, bool positions);  // kf_rb_norm_rows, the design's kind of norm
};
// a mixer: one product of h -> raw, what the kind does with raw -> ao, the product back, the sublayer's norm
struct RowMixer : GeNeuron {
    MIXER_CARD c;
    RowProduct in, proj;
    RowNorm norm;
    int ldraw = 0, ldout = 0;
    virtual int Mix(RowWork& w, const KVCache& kv, const RowBatch& b) = 0;
    virtual void Need(RowNeed& need, int rows, int n_seq, bool decode) const;
    int Forw(RowWork& w, const KVCache& kv, const RowBatch& b, bool defer);  // defer: leave the norm pending
};
// attention: grouped heads, chunks or a window, optional norms, rotation, output gate and sink; values the projected keys or their own columns
struct RowAttention : RowMixer {
    hGTensor qn, kn;
    const float* rope = nullptr;
    int v_col = 0;
    kf_rb_attention Args(const RowWork& w, const KVCache& kv) const;
    int Mix(RowWork& w, const KVCache& kv, const RowBatch& b) override;
    void Need(RowNeed& need, int rows, int n_seq, bool decode) const override;
};
// the gated delta rule with a decay per key channel
struct ChannelDelta : RowMixer {
    RowProduct a2, g2;
    hGTensor conv, a_log, dt_bias, out_norm;
    int col_a = 0, col_g = 0, col_b = 0;
    int Mix(RowWork& w, const KVCache& kv, const RowBatch& b) override;
    void Need(RowNeed& need, int rows, int n_seq, bool decode) const override;
};
// attention and a decayed sum side by side on the same input: one product in front, one behind (their outputs side by side, scaled)
struct ParallelMixer : RowAttention {
    hGTensor sum_norm, decay;
    int col_sum = 0, col_gate = 0, out_sum = 0;
    int Mix(RowWork& w, const KVCache& kv, const RowBatch& b) override;
    void Need(RowNeed& need, int rows, int n_seq, bool decode) const override;
};
struct RowFFN : GeNeuron {  // dense gated feed-forward, or routed experts
    FF_CARD c;
    RowProduct gateup, down, router;
    hGTensor router_b;
    RowNorm norm;
    int ldact = 0;
    int Forw(RowWork& w, int n);
    bool Sums(int type, int n) const { return type == KF_BF16 && n <= KF_RB_DECODE_MAX && n * c.top <= KF_RB_SUM_PAIRS; }  // the experts' outputs summed inside one product
};

struct SeqFish : Fish {
    SEQ_CARD card;
    SeqSlots self;  // the single-sequence surface: slot 0
    RowWork pre;
    RowProduct seq_head;
    RowNorm seq_norm;
    hGTensor table;
    RowNorm embed_norm;
    hGTensor pos_hi, pos_lo;  // position vectors (kf_rb_sinusoid_tables_host)
    std::vector<std::unique_ptr<RowMixer>> mixers;
    std::vector<std::unique_ptr<RowFFN>> ffs;
    std::vector<std::pair<ROT_CARD, float*>> ropes;
    struct Target {  // where a named tensor of the checkpoint goes
        hGTensor to;
        size_t offset = 0;  // elements in front of the matrix
        int row0 = 0, rows = 0, cols = 0, ld = 0, half = -1;
        bool product = false, set = false;
    };
    std::map<std::string, Target> targets;
    hGTensor stage;
    float* tap = nullptr;  // host [layers][tap_rows][width]: the residual stream after every layer of a prompt pass of exactly tap_rows rows (diagnosis)
    int tap_rows = 0;

    ~SeqFish() override;
    const char* Arch() const override { return card.arch.c_str(); }
    SeqFish* Seq() override { return this; }
    int BuildSeq(const SEQ_CARD& c, int device, void* stream);
    int BuildMixer(const MIXER_CARD& m, int layer, std::unique_ptr<RowMixer>& out);
    int Vector(hGTensor& t, const std::string& name, int n, const char* suffix);
    int Product(RowProduct& p, const std::string& name, int m, int k, int experts = 0);
    int Norm(RowNorm& n, const std::string& name);
    void Rows(const RowProduct& p, const std::string& name, int row0, int rows, int cols, int col0 = 0);
    int SetTensor(const std::string& name, int rows, int cols, const void* bf16, bool is_device);
    int Load(K_SafeTensors& st, std::string& err);
    std::string Missing() const;  // "" when every tensor has been set
    int Width(int n) const { return (n + KF_RB_PAD - 1) / KF_RB_PAD * KF_RB_PAD; }
    size_t Elem() const { return card.type == KF_F32 ? 4 : 2; }

    int InitSlots(SeqSlots& s, int n);
    int Ensure(RowWork& w, int rows, int n_seq, int head_rows, bool decode);
    int Enter(RowWork& w, int n);  // position vectors and the norm behind the embedding, where the design has them
    // the end of a sublayer: the product of `in` and the residual, normed as the design does (defer: the norm left pending)
    int Close(RowWork& w, RowProduct& proj, RowNorm& norm, const void* in, int64_t ldin, int n, bool defer = false);
    int Layers(RowWork& w, const KVCache& kv, const RowBatch& b);
    int HeadRows(RowWork& w, const int32_t* h_rows, int n);  // rows of w.x (host list, NULL: 0 .. n - 1) -> w.logits
    // n_span spans in one batch (cut into passes of at most prefill_chunk rows); want: (span, offset) pairs whose logits go to out [n_want][vocab] (host);
    // last: the last row of every span is picked, drawn from or left to the caller's sampler (state, ids out, slot logits)
    int Spans(SeqSlots& s, const SeqSpan* spans, int n_span, const int32_t* want, int n_want, float* out, bool last);
    int EnqueueSlots(SeqSlots& s, int bound, bool pick);
    int StepSlots(SeqSlots& s, int steps, bool pick, bool use_graph);
    int Draw(SeqSlots& s, int slot, const CHAT_SAMPLER& sp, uint64_t* d_rng);
    int Logits16(SeqSlots& s, int slot, void** out);  // the slot's logits rounded to bf16
    void DropGraphs(SeqSlots& s);

    int EnqueueStep(int bound) override;
    int Warm(int bound) override;
    int ForwardOnRLS(int token, int pos) override;
    int Prefill(const int* tokens, int n, int pos0) override;
    bool OneLaunchStep() override { return false; }
    void* LogitsPtr() override;
};

// the registry: config.json's architecture name -> its card.  shapes(name, rows, cols): the shape of a checkpoint's tensor, for sizes that config.json leaves to them
typedef std::function<bool(const std::string& name, int& rows, int& cols)> seq_shapes;
typedef bool (*seq_card_reader)(const JSON& cfg, const seq_shapes& shapes, SEQ_CARD& card, std::string& err);
seq_card_reader FindSeqArch(const std::string& architecture);
bool ReadTizusun(const JSON& cfg, const seq_shapes& shapes, SEQ_CARD& card, std::string& err);
bool ReadBolopel(const JSON& cfg, const seq_shapes& shapes, SEQ_CARD& card, std::string& err);
// a number of config.json, at least `lo`; err names what is missing or out of range
bool CardNumber(const JSON* o, const char* key, double lo, double& out, std::string& err, const std::string& where);
bool CardNumber(const JSON* o, const char* key, int lo, int& out, std::string& err, const std::string& where);
SeqFish* BuildSeqModel(const JSON& cfg, const std::string& dir, int device, void* stream, int type, int max_seq, int* rc, std::string& err);

}  // namespace koifish
