// Loretar: a decoder whose layers mix tokens either with sliding-window attention (distance bias, query temperature,
// norms over the whole query / key projection, talking heads) or with a gated delta rule that decays every key channel on
// its own; the mixer and the feed-forward read the same normed input and reach the residual stream through gates, and a
// stretch of layers may run several times in a row, each pass with its own cache and state.
//
// Every layer run is three backend calls (blocks.hpp): the norm and all products that read its output, the mixer, and the
// two sublayers' output products with the gated residual sum.  For the first of them the weight matrices that read the
// same input are kept as one matrix; a parameter that went into it stays available under its name as a view.
#pragma once

#include "layers.hpp"

namespace cgh {

struct LoretarLayer {
    enum Mixer { ATTENTION, CHANNEL_DELTA } mixer = ATTENTION;
    blocks::AttentionOptions attention;
    blocks::DeltaOptions delta;
    size_t taps = 1; // of the short convolutions
    size_t ff = 0;   // 0: no feed-forward
    size_t inner() const { return mixer == ATTENTION ? attention.heads * attention.vdim : delta.heads * delta.vdim; }
};

struct LoretarConfig {
    std::vector<LoretarLayer> layers;
    size_t vocab = 0, width = 0;
    LayerLoop loop;
    float eps = 0.0f, logit_scale = 1.0f;

    static LoretarConfig read(const Json &j) {
        LoretarConfig c;
        c.vocab = j.at("vocab").nat();
        c.width = j.at("width").nat();
        c.eps = (float)j.at("norm").at("eps").real();
        if (const Json *s = j.find("logit_scale")) c.logit_scale = (float)s->real();
        for (const Json &l : j.at("layers").list()) {
            LoretarLayer o;
            const std::string &type = l.at("type").str();
            const Json &m = l.at("mixer");
            const size_t heads = m.at("heads").nat(), kv = m.at("kv_heads").nat(), dim = m.at("dim").nat(), vdim = m.at("vdim").nat();
            if (!heads || !kv || !dim || !vdim || heads % kv) throw ConfigError("config: the heads of a mixer do not fit together");
            if (type == "attention") {
                blocks::AttentionOptions &a = o.attention;
                a.heads = heads;
                a.kv_heads = kv;
                a.dim = dim;
                a.vdim = vdim;
                a.scale = (float)m.at("scale").real();
                a.norm_eps = c.eps;
                a.distance_bias = true;
                if (const Json *mask = m.find("mask")) {
                    a.window = mask->at("size").nat();
                    if (!a.window) throw ConfigError("config: a window of no tokens");
                }
                if (const Json *t = m.find("q_temp")) {
                    a.temp_coef = (float)t->at("coef").real();
                    a.temp_every = t->at("every").nat();
                    if (!a.temp_every) throw ConfigError("config: q_temp.every must be positive");
                }
            } else if (type == "channel_delta") {
                o.mixer = LoretarLayer::CHANNEL_DELTA;
                o.delta = {heads, kv, dim, vdim, c.eps};
                o.taps = m.at("conv").nat();
                if (!o.taps) throw ConfigError("config: a convolution of no taps");
            } else {
                throw ConfigError("config: unknown mixer '" + type + "'");
            }
            if (const Json *f = l.find("mlp")) {
                if (f->at("kind").str() != "dense") throw ConfigError("config: unknown feed-forward '" + f->at("kind").str() + "'");
                o.ff = f->at("ff").nat();
                if (!o.ff) throw ConfigError("config: a feed-forward of no values");
            }
            c.layers.push_back(o);
        }
        c.loop = LayerLoop::read(j, c.layers.size());
        if (!c.vocab || !c.width) throw ConfigError("config: sizes must be positive");
        return c;
    }
};

class LoretarModel : public LayeredModel {
  public:
    LoretarModel(Interpreter &i, const LoretarConfig &c, cg_dtype weights) : LayeredModel(i, weights), c_(c), runs_(c.loop.runs(c.layers.size())) {}
    size_t vocab_size() const override { return c_.vocab; }

    State empty_state(size_t B) override {
        State s;
        for (const auto &r : runs_) {
            const LoretarLayer &l = c_.layers[r.layer];
            if (l.mixer == LoretarLayer::ATTENTION) {
                s.tensors.push_back(i_.backend.zeros(Shape{B, l.attention.kv_heads, 0, l.attention.dim}, CG_F32));
                s.tensors.push_back(i_.backend.zeros(Shape{B, l.attention.kv_heads, 0, l.attention.vdim}, CG_F32));
            } else {
                const blocks::DeltaOptions &d = l.delta;
                s.tensors.push_back(i_.backend.zeros(Shape{B, d.heads, d.dim, d.vdim}, CG_F32));
                s.tensors.push_back(i_.backend.zeros(Shape{B, l.taps - 1, 2 * d.kv_heads * d.dim + d.heads * d.vdim}, CG_F32));
            }
        }
        return s;
    }

  protected:
    Parts def(Tensor ids, std::vector<Tensor> state, size_t position, size_t, const Want &want) override {
        using namespace ops;
        I &i = i_;
        const Shape xs = shape(ids);
        const size_t B = xs[0], S = xs[1], W = c_.width;
        Tensor x = reshape(i, Shape{B * S}, std::move(ids));
        x = cast(i, index(i, 0, std::move(x), i.param("embed")), CG_F32);
        x = reshape(i, Shape{B, S, W}, std::move(x));
        Tensor x0;
        if (c_.loop.times) x0 = x;
        Parts p;
        for (size_t r = 0; r < runs_.size(); r++) {
            const int begins = runs_[r].begins;
            if (begins >= 0) { // x <- loop.in [x; x0] + loop.step[pass]
                Tensor step = reshape(i, Shape{W}, slice(i, 0, (size_t)begins, 1, i.param("loop.step")));
                Tensor again = begins + 1 == (int)c_.loop.times ? std::move(x0) : x0;
                x = blocks::linear(i, std::move(x), std::move(again), Tensor(), i.param("loop.in"), std::move(step), {});
            }
            Tensor s0 = std::move(state[2 * r]), s1 = std::move(state[2 * r + 1]);
            x = layer(runs_[r].layer, position, std::move(x), &s0, &s1);
            p.state.push_back(std::move(s0));
            p.state.push_back(std::move(s1));
        }
        if (!want.tokens && !want.logits) return p;
        blocks::LinearOptions opt;
        opt.eps = c_.eps;
        opt.scale = c_.logit_scale;
        p.out = head(std::move(x), want, opt);
        return p;
    }

    // The weight matrices that read a layer's normed input become one, everything that is multiplied takes the form it is
    // multiplied in, and the shapes are checked against the configuration.
    void prepare_weights() override {
        expect("embed", {c_.vocab, c_.width});
        expect("head", {c_.vocab, c_.width});
        expect("final.norm", {c_.width});
        store("embed");
        store("head");
        if (c_.loop.times) {
            expect("loop.in", {c_.width, 2 * c_.width});
            expect("loop.step", {c_.loop.times, c_.width});
            store("loop.in");
        }
        for (size_t l = 0; l < c_.layers.size(); l++) {
            const LoretarLayer &c = c_.layers[l];
            const std::string p = "l" + std::to_string(l), m = p + ".mix";
            std::vector<std::string> parts;
            auto rows = [&](const std::string &name, size_t n) {
                expect(name, {n, c_.width});
                parts.push_back(name);
            };
            expect(p + ".norm1", {c_.width});
            if (c.mixer == LoretarLayer::ATTENTION) {
                const blocks::AttentionOptions &a = c.attention;
                rows(m + ".q", a.heads * a.dim);
                rows(m + ".k", a.kv_heads * a.dim);
                rows(m + ".v", a.kv_heads * a.vdim);
                expect(m + ".q.norm", {a.heads * a.dim});
                expect(m + ".k.norm", {a.kv_heads * a.dim});
                expect(m + ".talk", {a.heads, a.heads});
            } else {
                const blocks::DeltaOptions &d = c.delta;
                const size_t kc = d.kv_heads * d.dim, vc = d.heads * d.vdim;
                rows(m + ".q", kc);
                rows(m + ".k", kc);
                rows(m + ".v", vc);
                rows(m + ".a1", dims(m + ".a1")[0]);
                rows(m + ".g1", dims(m + ".g1")[0]);
                rows(m + ".b", d.heads);
                expect(m + ".q.conv", {kc, c.taps});
                expect(m + ".k.conv", {kc, c.taps});
                expect(m + ".v.conv", {vc, c.taps});
                expect(m + ".a2", {d.heads * d.dim, dims(m + ".a1")[0]});
                expect(m + ".g2", {vc, dims(m + ".g1")[0]});
                expect(m + ".A_log", {d.heads});
                expect(m + ".dt_bias", {d.heads * d.dim});
                expect(m + ".norm", {d.vdim});
            }
            expect(m + ".o", {c_.width, c.inner()});
            store(m + ".o");
            if (c.ff) {
                rows(p + ".mlp.up", c.ff);
                expect(p + ".mlp.down", {c_.width, c.ff});
                expect(p + ".mlp.act", {4});
                store(p + ".mlp.down");
            }
            rows(p + ".rg1", c_.width);
            expect(p + ".rg1.b", {c_.width});
            if (c.ff) {
                rows(p + ".rg2", c_.width);
                expect(p + ".rg2.b", {c_.width});
            }
            stack(p + ".in", parts);
        }
    }

  private:
    Tensor layer(size_t l, size_t position, Tensor x, Tensor *s0, Tensor *s1) {
        using namespace ops;
        I &i = i_;
        const LoretarLayer &c = c_.layers[l];
        const std::string p = "l" + std::to_string(l), m = p + ".mix";
        blocks::LinearOptions opt;
        opt.eps = c_.eps;
        Tensor h = blocks::linear(i, x, Tensor(), i.param(p + ".norm1"), i.param(p + ".in"), Tensor(), opt);
        auto part = [&](const std::string &name) { return part_of(h, p + ".in", name); };
        std::vector<Tensor> r;
        if (c.mixer == LoretarLayer::ATTENTION) {
            blocks::AttentionTensors t{part(m + ".q"),          part(m + ".k"),          part(m + ".v"), i.param(m + ".q.norm"),
                                       i.param(m + ".k.norm"), i.param(m + ".talk"), std::move(*s0), std::move(*s1)};
            r = blocks::attention(i, std::move(t), c.attention, position);
        } else {
            blocks::DeltaTensors t{part(m + ".q"),         part(m + ".k"),        part(m + ".v"),      i.param(m + ".q.conv"), i.param(m + ".k.conv"),
                                   i.param(m + ".v.conv"), part(m + ".b"),        part(m + ".a1"),     i.param(m + ".a2"),     i.param(m + ".A_log"),
                                   i.param(m + ".dt_bias"), part(m + ".g1"),      i.param(m + ".g2"), i.param(m + ".norm"),   std::move(*s0),
                                   std::move(*s1)};
            r = blocks::channel_delta(i, std::move(t), c.delta);
        }
        *s0 = std::move(r[1]);
        *s1 = std::move(r[2]);
        std::vector<blocks::Branch> br;
        br.push_back({std::move(r[0]), i.param(m + ".o"), part(p + ".rg1"), i.param(p + ".rg1.b"), Tensor()});
        if (c.ff) br.push_back({part(p + ".mlp.up"), i.param(p + ".mlp.down"), part(p + ".rg2"), i.param(p + ".rg2.b"), i.param(p + ".mlp.act")});
        return blocks::residual(i, std::move(x), std::move(br), c_.eps);
    }

    LoretarConfig c_;
    std::vector<LayerLoop::Run> runs_;
};

} // namespace cgh
