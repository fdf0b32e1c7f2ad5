// Lufatar: a decoder whose layers read the residual stream twice, through a grouped norm and a short filter over time each,
// for a mixer and for a mixture of experts that run side by side; behind them every token adds a vector of its own, gated
// by its row.  The mixer is attention with rotated unit queries and keys, scores mixed over the heads before a soft-max that
// may give its weight to nothing.  Embeddings of token pairs go beside the tokens' own, and a stretch of layers may run
// several times in a row, each pass with its own caches and filter inputs.
//
// Every layer run is four backend calls (blocks.hpp): norms, filters and the products behind them, the mixer, the two
// sublayers' way into the residual stream, and the tokens' own vectors.
#pragma once

#include "layers.hpp"

namespace cgh {

struct LufatarLayer {
    blocks::AttentionOptions attention;
    blocks::ExpertOptions experts;
    size_t count = 0, ff = 0; // experts and their inner size; 0: no feed-forward
};

struct LufatarConfig {
    static constexpr float kGateSlope = 1.702f; // of the experts' gated activation

    std::vector<LufatarLayer> layers;
    size_t vocab = 0, width = 0, taps = 0, side = 0, buckets = 0, mul_prev = 0, mul_cur = 0, groups = 1;
    LayerLoop loop;
    float eps = 0.0f, mult = 1.0f;

    static LufatarConfig read(const Json &j) {
        LufatarConfig c;
        c.vocab = j.at("vocab").nat();
        c.width = j.at("width").nat();
        c.eps = (float)j.at("norm").at("eps").real();
        c.groups = j.at("norm").at("groups").nat();
        c.mult = (float)j.at("residual_mult").real();
        c.taps = j.at("canon").at("taps").nat();
        c.side = j.at("token_side").at("dim").nat();
        const Json &pairs = j.at("embedding").at("bigram");
        c.buckets = pairs.at("buckets").nat();
        c.mul_prev = pairs.at("mul_prev").nat();
        c.mul_cur = pairs.at("mul_cur").nat();
        if (!c.vocab || !c.width || !c.taps || !c.side || !c.buckets) throw ConfigError("config: sizes must be positive");
        if (!c.groups || c.width % c.groups) throw ConfigError("config: the norm's groups do not divide the width");
        for (const Json &l : j.at("layers").list()) {
            LufatarLayer o;
            if (l.at("type").str() != "attention") throw ConfigError("config: unknown mixer '" + l.at("type").str() + "'");
            const Json &m = l.at("mixer"), &rot = m.at("rot");
            blocks::AttentionOptions &a = o.attention;
            a.heads = m.at("heads").nat();
            a.kv_heads = m.at("kv_heads").nat();
            a.dim = m.at("dim").nat();
            a.vdim = m.at("vdim").nat();
            a.scale = (float)m.at("scale").real();
            a.norm_eps = c.eps;
            a.rot_dims = rot.at("dims").nat();
            a.rot_base = rot.at("base").real();
            a.unit_heads = a.mix_scores = a.zero_sink = true;
            if (!a.heads || !a.kv_heads || !a.dim || !a.vdim || a.heads % a.kv_heads) throw ConfigError("config: the heads of a mixer do not fit together");
            if (a.rot_dims > a.dim || a.rot_dims % 2 || !(a.rot_base > 0.0)) throw ConfigError("config: the rotation does not fit the heads");
            if (const Json *f = l.find("mlp")) {
                if (f->at("kind").str() != "moe") throw ConfigError("config: unknown feed-forward '" + f->at("kind").str() + "'");
                const Json &r = f->at("router");
                o.ff = f->at("expert").at("ff").nat();
                o.count = r.at("experts").nat();
                o.experts.limit = (float)f->at("expert").at("limit").real();
                o.experts.slope = kGateSlope;
                o.experts.top = r.at("top").nat();
                if (const Json *g = r.find("groups")) {
                    o.experts.groups = g->at("count").nat();
                    o.experts.keep = g->at("keep").nat();
                }
                const blocks::ExpertOptions &e = o.experts;
                if (!o.ff || !o.count || !e.groups || o.count % e.groups || !e.keep || e.keep > e.groups || !e.top || e.top > o.count / e.groups * e.keep)
                    throw ConfigError("config: the experts and their groups do not fit together");
            }
            c.layers.push_back(o);
        }
        c.loop = LayerLoop::read(j, c.layers.size());
        return c;
    }
};

class LufatarModel : public LayeredModel {
  public:
    LufatarModel(Interpreter &i, const LufatarConfig &c, cg_dtype weights) : LayeredModel(i, weights), c_(c), runs_(c.loop.runs(c.layers.size())) {}
    size_t vocab_size() const override { return c_.vocab; }

    // the last token, then per layer run: keys, values, the filters' last inputs
    State empty_state(size_t B) override {
        Backend &be = i_.backend;
        State s;
        s.tensors.push_back(be.zeros(Shape{B, 0}, CG_U32));
        for (const auto &r : runs_) {
            const blocks::AttentionOptions &a = c_.layers[r.layer].attention;
            s.tensors.push_back(be.zeros(Shape{B, a.kv_heads, 0, a.dim}, CG_F32));
            s.tensors.push_back(be.zeros(Shape{B, a.kv_heads, 0, a.vdim}, CG_F32));
            s.tensors.push_back(be.zeros(Shape{B, c_.taps - 1, c_.width}, CG_F32));
        }
        return s;
    }

  protected:
    Parts def(Tensor ids, std::vector<Tensor> state, size_t position, size_t, const Want &want) override {
        using namespace ops;
        I &i = i_;
        Parts p;
        std::vector<Tensor> e = blocks::pair_embedding(i, ids, std::move(state[0]), i.param("embed"), i.param("bigram"), c_.mul_prev, c_.mul_cur);
        Tensor x = std::move(e[0]);
        const Shape xs = shape(x);
        p.state.push_back(std::move(e[1]));
        for (size_t r = 0; r < runs_.size(); r++) {
            if (runs_[r].begins >= 0) {
                Tensor step = reshape(i, Shape{c_.width}, slice(i, 0, (size_t)runs_[r].begins, 1, i.param("loop.step")));
                x = add(i, std::move(x), broadcast(i, xs, std::move(step)));
            }
            Tensor *s = &state[3 * r + 1];
            x = layer(runs_[r].layer, position, std::move(x), r + 1 == runs_.size() ? std::move(ids) : ids, s);
            for (size_t k = 0; k < 3; k++) p.state.push_back(std::move(s[k]));
        }
        if (!want.tokens && !want.logits) return p;
        blocks::LinearOptions opt;
        opt.eps = c_.eps;
        opt.groups = c_.groups;
        p.out = head(std::move(x), want, opt);
        return p;
    }

    void prepare_weights() override {
        const size_t W = c_.width;
        auto stored = [&](const std::string &name, const Shape &s) {
            expect(name, s);
            store(name);
        };
        stored("embed", {c_.vocab, W});
        stored("bigram", {c_.buckets + 1, W});
        stored("side.embed", {c_.vocab, c_.layers.size() * c_.side});
        stored("head", {c_.vocab, W});
        expect("final.norm", {W});
        if (c_.loop.times) expect("loop.step", {c_.loop.times, W});
        for (size_t l = 0; l < c_.layers.size(); l++) {
            const LufatarLayer &c = c_.layers[l];
            const blocks::AttentionOptions &a = c.attention;
            const std::string p = "l" + std::to_string(l), m = p + ".mix", f = p + ".mlp";
            expect(p + ".norm1", {W});
            expect(p + ".canon1", {W, c_.taps});
            expect(m + ".q", {a.heads * a.dim, W});
            expect(m + ".k", {a.kv_heads * a.dim, W});
            expect(m + ".v", {a.kv_heads * a.vdim, W});
            stack(p + ".in", {m + ".q", m + ".k", m + ".v"});
            expect(m + ".talk", {a.heads, a.heads});
            stored(m + ".o", {W, a.heads * a.vdim});
            if (c.count) {
                expect(p + ".norm2", {W});
                expect(p + ".canon2", {W, c_.taps});
                stored(f + ".router", {c.count, W}); // (bfloat16 products are exact in the 32-bit sums)
                expect(f + ".correction", {c.count});
                std::vector<std::string> first, second;
                for (size_t e = 0; e < c.count; e++) {
                    const std::string x = f + ".e" + std::to_string(e);
                    for (const char *n : {".gate", ".up"}) {
                        expect(x + n, {c.ff, W});
                        first.push_back(x + n);
                    }
                    expect(x + ".down", {W, c.ff});
                    second.push_back(x + ".down");
                }
                stack(f + ".first", first, 1);
                stack(f + ".second", second, 1);
            }
            stored(p + ".side.gate", {c_.side, W});
            stored(p + ".side.proj", {W, c_.side});
            expect(p + ".side.norm", {W});
        }
    }

  private:
    Tensor layer(size_t l, size_t position, Tensor x, Tensor ids, Tensor *s) {
        using namespace ops;
        I &i = i_;
        const LufatarLayer &c = c_.layers[l];
        const std::string p = "l" + std::to_string(l), m = p + ".mix", f = p + ".mlp";
        std::vector<blocks::ConvInput> in;
        in.push_back({i.param(p + ".norm1"), i.param(p + ".canon1"), i.param(p + ".in"), false});
        if (c.count) in.push_back({i.param(p + ".norm2"), i.param(p + ".canon2"), i.param(f + ".router"), true});
        std::vector<Tensor> h = blocks::conv_linear(i, x, std::move(s[2]), std::move(in), weights_, c_.groups, c_.eps);
        s[2] = std::move(h.back());
        blocks::AttentionTensors t;
        t.q = part_of(h[0], p + ".in", m + ".q");
        t.k = part_of(h[0], p + ".in", m + ".k");
        t.v = part_of(h[0], p + ".in", m + ".v");
        t.talk = i.param(m + ".talk");
        t.k_cache = std::move(s[0]);
        t.v_cache = std::move(s[1]);
        std::vector<Tensor> a = blocks::attention(i, std::move(t), c.attention, position);
        s[0] = std::move(a[1]);
        s[1] = std::move(a[2]);
        std::vector<blocks::Branch> br;
        br.push_back({std::move(a[0]), i.param(m + ".o"), Tensor(), Tensor(), Tensor()});
        blocks::Experts ex;
        if (c.count) {
            ex.h = std::move(h[2]);
            ex.logits = std::move(h[1]);
            ex.correction = i.param(f + ".correction");
            ex.gate_up = reshape(i, Shape{c.count, 2, c.ff, c_.width}, i.param(f + ".first"));
            ex.down = reshape(i, Shape{c.count, c_.width, c.ff}, i.param(f + ".second"));
            ex.options = c.experts;
        }
        x = blocks::residual(i, std::move(x), std::move(br), c_.eps, c_.mult, std::move(ex));
        blocks::SideOptions side;
        side.first = l * c_.side;
        side.eps = c_.eps;
        side.scale = c_.mult;
        return blocks::token_side(i, std::move(x), std::move(ids), i.param("side.embed"), i.param(p + ".side.gate"), i.param(p + ".side.proj"),
                                  i.param(p + ".side.norm"), side);
    }

    LufatarConfig c_;
    std::vector<LayerLoop::Run> runs_;
};

} // namespace cgh
