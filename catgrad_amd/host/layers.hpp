// What the models made of decoder blocks (blocks.hpp) have in common: a list of layers of which a stretch may run several
// times in a row, and weights that are checked, kept in the form they are multiplied in, and packed when several of them
// read the same input.
#pragma once

#include "blocks.hpp"
#include "json.hpp"
#include "model.hpp"
#include "nn.hpp"

namespace cgh {

// Layers start .. stop - 1 run `times` times in a row (0: no layer runs more than once), then the rest follow.
struct LayerLoop {
    size_t start = 0, stop = 0, times = 0;

    static LayerLoop read(const Json &config, size_t layers) {
        LayerLoop l;
        if (const Json *lp = config.find("loop")) {
            l.start = lp->at("start").nat();
            l.stop = lp->at("stop").nat();
            l.times = lp->at("times").nat();
            if (l.start >= l.stop || l.stop > layers || !l.times) throw ConfigError("config: the loop does not fit the layers");
        }
        return l;
    }

    // One evaluation of a layer; `begins`: the pass of the loop that starts with it, or -1.
    struct Run {
        size_t layer;
        int begins;
    };
    std::vector<Run> runs(size_t layers) const {
        std::vector<Run> r;
        const size_t from = times ? start : layers, to = times ? stop : layers;
        for (size_t l = 0; l < from; l++) r.push_back({l, -1});
        for (size_t t = 0; t < times; t++)
            for (size_t l = from; l < to; l++) r.push_back({l, l == from ? (int)t : -1});
        for (size_t l = to; l < layers; l++) r.push_back({l, -1});
        return r;
    }
};

class LayeredModel : public Model {
  public:
    // weights: CG_F32, or CG_BF16 for matrices held and multiplied at bfloat16 precision
    LayeredModel(Interpreter &i, cg_dtype weights) : Model(i), weights_(weights) {}
    bool selects_rows() const override { return true; }
    void parameters_changed() override { prepared_ = false; }

  protected:
    void prepare() override {
        if (prepared_) return;
        in_.clear();
        prepare_weights();
        i_.backend.sync();
        prepared_ = true;
    }
    // checks the parameters' shapes against the configuration, stores and packs them
    virtual void prepare_weights() = 0;

    Shape dims(const std::string &name) {
        auto it = i_.parameters.find(name);
        if (it == i_.parameters.end()) throw InterpreterError("MissingParameter: " + name);
        Shape s = it->second.shape();
        if (s.empty()) throw InterpreterError("parameter " + name + " has no extents");
        return s;
    }
    void expect(const std::string &name, const Shape &s) {
        if (dims(name) != s) throw InterpreterError("parameter " + name + " does not have the shape the configuration asks for");
    }
    // Computed at once: a view of a deferred tensor would compute it again for itself.  A small matrix is part of one that is
    // large enough for the backend to keep it in two bytes a value.
    static constexpr size_t kNarrowFrom = 65536;
    Tensor stored_form(Tensor t) {
        Backend &be = i_.backend;
        const Shape s = t.shape();
        const bool small = weights_ != CG_F32 && s.size() == 2 && s[0] * s[1] < kNarrowFrom;
        if (small) t = be.concat(be.cast(std::move(t), CG_F32), be.zeros(Shape{(kNarrowFrom + s[1] - 1) / s[1], s[1]}, CG_F32), 0);
        t = be.cast(std::move(t), weights_);
        be.realize(t);
        return small ? be.slice(std::move(t), 0, 0, s[0]) : t;
    }
    void store(const std::string &name) { i_.parameters[name] = stored_form(std::move(i_.parameters[name])); }

    // The matrices `parts` [.., cols] one below the other as parameter `name`, each beginning at a multiple of `align`
    // rows; the parts' own names become views of it.
    void stack(const std::string &name, const std::vector<std::string> &parts, size_t align = 8) {
        Backend &be = i_.backend;
        std::map<std::string, Part> where;
        Tensor all;
        size_t at = 0;
        const size_t cols = dims(parts[0])[1];
        auto append = [&](Tensor t) { all = all ? be.concat(std::move(all), std::move(t), 0) : std::move(t); };
        for (const std::string &part : parts) {
            Tensor t = be.cast(std::move(i_.parameters[part]), CG_F32);
            const size_t n = t.shape()[0], pad = (align - n % align) % align;
            append(std::move(t));
            if (pad) append(be.zeros(Shape{pad, cols}, CG_F32));
            where[part] = {at, n};
            at += n + pad;
        }
        all = stored_form(std::move(all));
        for (const std::string &part : parts) i_.parameters[part] = be.slice(all, 0, where[part].at, where[part].n);
        i_.parameters[name] = std::move(all);
        in_[name] = std::move(where);
    }
    // the columns of a product with stack `name` that belong to `part`
    Tensor part_of(const Tensor &product, const std::string &name, const std::string &part) {
        const Part &w = in_.at(name).at(part);
        return ops::slice(i_, 2, w.at, w.n, product);
    }

    // The rows of x [B, S, W] that the caller wants, through the norm and the vocabulary projection.
    RunOut head(Tensor x, const Want &want, const blocks::LinearOptions &opt) {
        RunOut o;
        const Shape s = x.shape();
        if (want.rows) {
            x = ops::reshape(i_, Shape{s[0] * s[1], s[2]}, std::move(x));
            Tensor rows = i_.backend.ndarray_from_vec_u32(want.rows->data(), want.rows->size(), Shape{want.rows->size()});
            x = nn::unsqueeze(i_, 0, ops::index(i_, 0, std::move(rows), std::move(x)));
        }
        x = blocks::linear(i_, std::move(x), Tensor(), i_.param("final.norm"), i_.param("head"), Tensor(), opt);
        if (want.logits) o.logits = x;
        if (want.tokens) o.tokens = ops::argmax(i_, std::move(x));
        return o;
    }

    cg_dtype weights_;

  private:
    struct Part { // rows of a stack: columns of the product with it
        size_t at, n;
    };
    std::map<std::string, std::map<std::string, Part>> in_;
    bool prepared_ = false;
};

} // namespace cgh
