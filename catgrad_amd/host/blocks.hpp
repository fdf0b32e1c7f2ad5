// Steps of a decoder layer that are one backend call each (the last section of include/catgrad_hip.h) as operations of
// the interpreter: run where they stand, or recorded like any other operation.  Every mechanism is a parameter; a tensor
// that is not there (`Tensor()`) or a zero switches it off.
#pragma once

#include <algorithm>

#include "graph.hpp"

namespace cgh {
namespace blocks {
using I = Interpreter;

// The operands of a block in a fixed order, some of them absent: what is there travels through the interpreter.
struct Operands {
    std::vector<Value> values;
    std::vector<int> slot; // per position: index into the operands handed to `run`, or -1
    void add(Tensor t) {
        slot.push_back(t ? (int)values.size() : -1);
        if (t) values.emplace_back(std::move(t));
    }
    static cg_tensor *raw(std::vector<Tensor> &in, const std::vector<int> &slot, size_t k) {
        return slot[k] < 0 ? nullptr : in[slot[k]].into_raw();
    }
};

template <class F>
inline std::vector<Tensor> issue(I &i, Operands o, std::vector<std::pair<Shape, cg_dtype>> types, F &&call) {
    auto b = std::make_shared<BlockOp>();
    b->types = std::move(types);
    b->run = [slot = o.slot, call](Backend &be, std::vector<Tensor> in) {
        return call(be, [&](size_t k) { return Operands::raw(in, slot, k); });
    };
    Op op(TensorOp::Block);
    op.block = b;
    std::vector<Tensor> r;
    for (Value &v : i.run(op, std::move(o.values))) r.push_back(std::move(v.tensor));
    return r;
}

// scale * norm(x | x2) . w^T + bias; the RMS norm is there when gamma is
struct LinearOptions {
    float eps = 0.0f, scale = 1.0f;
    size_t groups = 1; // of the norm
};
inline Tensor linear(I &i, Tensor x, Tensor x2, Tensor gamma, Tensor w, Tensor bias, LinearOptions opt) {
    Shape s = x.shape();
    s.back() = w.shape()[0];
    Operands o;
    o.add(std::move(x));
    o.add(std::move(x2));
    o.add(std::move(gamma));
    o.add(std::move(w));
    o.add(std::move(bias));
    return std::move(issue(i, std::move(o), {{s, CG_F32}}, [opt](Backend &be, auto &&raw) {
        cg_linear_args a{raw(0), raw(1), raw(2), raw(3), raw(4), opt.eps, opt.scale, opt.groups};
        std::vector<Tensor> r;
        r.push_back(be.block_linear(a));
        return r;
    })[0]);
}

// rows of `table`, plus those of `pairs` that a token and the one before it choose -> {rows [B, S, width], last tokens [B, 1]}
inline std::vector<Tensor> pair_embedding(I &i, Tensor ids, Tensor previous, Tensor table, Tensor pairs, size_t mul_prev, size_t mul_cur) {
    const Shape s = ids.shape();
    std::vector<std::pair<Shape, cg_dtype>> types = {{{s[0], s[1], table.shape()[1]}, CG_F32}, {{s[0], 1}, CG_U32}};
    Operands o;
    for (Tensor *x : {&ids, &previous, &table, &pairs}) o.add(std::move(*x));
    return issue(i, std::move(o), std::move(types), [mul_prev, mul_cur](Backend &be, auto &&raw) {
        cg_pair_embedding_args a{raw(0), raw(1), raw(2), raw(3), mul_prev, mul_cur};
        return be.block_pair_embedding(a);
    });
}

// Products that read the same rows through a norm and a short filter over time each.
struct ConvInput {
    Tensor gamma, conv, w;
    bool keep; // the normed and filtered rows are a result too, of dtype `kept`
};
// -> {products, kept rows, state}
inline std::vector<Tensor> conv_linear(I &i, Tensor x, Tensor state, std::vector<ConvInput> in, cg_dtype kept, size_t groups, float eps) {
    const Shape s = x.shape();
    const size_t n = in.size();
    std::vector<std::pair<Shape, cg_dtype>> types;
    std::vector<bool> keep;
    for (const ConvInput &c : in) {
        types.push_back({{s[0], s[1], c.w.shape()[0]}, CG_F32});
        keep.push_back(c.keep);
    }
    for (const ConvInput &c : in)
        if (c.keep) types.push_back({s, kept});
    types.push_back({state.shape(), CG_F32});
    Operands o;
    o.add(std::move(x));
    o.add(std::move(state));
    for (ConvInput &c : in) {
        o.add(std::move(c.gamma));
        o.add(std::move(c.conv));
        o.add(std::move(c.w));
    }
    return issue(i, std::move(o), std::move(types), [n, keep, kept, groups, eps](Backend &be, auto &&raw) {
        cg_conv_linear_args a{};
        a.x = raw(0);
        a.state = raw(1);
        for (size_t k = 0; k < n; k++) a.in[k] = {raw(3 * k + 2), raw(3 * k + 3), raw(3 * k + 4), keep[k], kept == CG_BF16};
        a.n = n;
        a.groups = groups;
        a.eps = eps;
        return be.block_conv_linear(a);
    });
}

// x plus what every token's own part of a table, gated by x, adds to it
struct SideOptions {
    size_t first = 0; // column of the table
    float eps = 0.0f, scale = 1.0f;
};
inline Tensor token_side(I &i, Tensor x, Tensor ids, Tensor table, Tensor gate, Tensor proj, Tensor norm, SideOptions opt) {
    const Shape s = x.shape();
    Operands o;
    for (Tensor *t : {&x, &ids, &table, &gate, &proj, &norm}) o.add(std::move(*t));
    return std::move(issue(i, std::move(o), {{s, CG_F32}}, [opt](Backend &be, auto &&raw) {
        cg_token_side_args a{raw(0), raw(1), raw(2), raw(3), raw(4), raw(5), opt.first, opt.eps, opt.scale};
        std::vector<Tensor> r;
        r.push_back(be.block_token_side(a));
        return r;
    })[0]);
}

// A mixture of experts as a term of the residual sum; h absent: none.
struct ExpertOptions {
    size_t top = 0, groups = 1, keep = 1;
    float limit = 0.0f, slope = 0.0f;
};
struct Experts {
    Tensor h, logits, correction, gate_up, down;
    ExpertOptions options;
};

// One sublayer's result on its way into the residual stream: act(y) . w^T, times sigmoid(gate + gate_bias)
struct Branch {
    Tensor y, w, gate, gate_bias, poly;
};
// x + scale * (the branches + the experts)
inline Tensor residual(I &i, Tensor x, std::vector<Branch> br, float eps, float scale = 1.0f, Experts ex = {}) {
    const Shape s = x.shape();
    const size_t n = br.size();
    const bool mixture = (bool)ex.h;
    const ExpertOptions eo = ex.options;
    Operands o;
    o.add(std::move(x));
    for (Branch &b : br) {
        o.add(std::move(b.y));
        o.add(std::move(b.w));
        o.add(std::move(b.gate));
        o.add(std::move(b.gate_bias));
        o.add(std::move(b.poly));
    }
    for (Tensor *t : {&ex.h, &ex.logits, &ex.correction, &ex.gate_up, &ex.down}) o.add(std::move(*t));
    return std::move(issue(i, std::move(o), {{s, CG_F32}}, [n, eps, scale, mixture, eo](Backend &be, auto &&raw) {
        std::vector<cg_branch> c(n);
        for (size_t k = 0; k < n; k++) c[k] = {raw(5 * k + 1), raw(5 * k + 2), raw(5 * k + 3), raw(5 * k + 4), raw(5 * k + 5)};
        const size_t e = 5 * n + 1;
        cg_experts m{raw(e), raw(e + 1), raw(e + 2), raw(e + 3), raw(e + 4), eo.top, eo.groups, eo.keep, eo.limit, eo.slope};
        std::vector<Tensor> r;
        r.push_back(be.block_residual(be.adopt(raw(0)), c, eps, scale, mixture ? &m : nullptr));
        return r;
    })[0]);
}

struct AttentionOptions {
    size_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    float scale = 1.0f;
    size_t window = 0; // 0: every earlier position is visible
    float temp_coef = 0.0f;
    size_t temp_every = 0; // 0: no query temperature
    bool distance_bias = false;
    float norm_eps = 0.0f;
    size_t rot_dims = 0; // 0: no rotation
    double rot_base = 0.0;
    bool unit_heads = false, mix_scores = false, zero_sink = false;
};
struct AttentionTensors {
    Tensor q, k, v, q_norm, k_norm, talk, k_cache, v_cache;
};
// -> {output [B, S, heads * vdim], k cache, v cache}
inline std::vector<Tensor> attention(I &i, AttentionTensors t, const AttentionOptions &opt, size_t position) {
    const Shape qs = t.q.shape();
    const size_t B = qs[0], S = qs[1], all = t.k_cache.shape()[2] + S;
    const size_t keep = opt.window ? std::min(all, opt.window - 1) : all;
    std::vector<std::pair<Shape, cg_dtype>> types = {{{B, S, opt.heads * opt.vdim}, CG_F32},
                                                     {{B, opt.kv_heads, keep, opt.dim}, CG_F32},
                                                     {{B, opt.kv_heads, keep, opt.vdim}, CG_F32}};
    Operands o;
    for (Tensor *x : {&t.q, &t.k, &t.v, &t.q_norm, &t.k_norm, &t.talk, &t.k_cache, &t.v_cache}) o.add(std::move(*x));
    return issue(i, std::move(o), std::move(types), [opt, position](Backend &be, auto &&raw) {
        cg_attention_args a{raw(0),   raw(1),     raw(2),   raw(3),   raw(4),     raw(5),         raw(6),    raw(7),       opt.heads,     opt.kv_heads,
                            opt.dim, opt.vdim, position, opt.window, opt.temp_every, opt.scale, opt.norm_eps, opt.temp_coef, opt.distance_bias,
                            opt.rot_dims, opt.rot_base, opt.unit_heads, opt.mix_scores, opt.zero_sink};
        return be.block_attention(a);
    });
}

struct DeltaOptions {
    size_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    float eps = 0.0f;
};
struct DeltaTensors {
    Tensor q, k, v, conv_q, conv_k, conv_v, beta, decay, decay_w, a_log, dt_bias, gate, gate_w, norm, state, conv_state;
};
// -> {output [B, S, heads * vdim], state, convolution state}
inline std::vector<Tensor> channel_delta(I &i, DeltaTensors t, const DeltaOptions &opt) {
    const Shape qs = t.q.shape();
    std::vector<std::pair<Shape, cg_dtype>> types = {{{qs[0], qs[1], opt.heads * opt.vdim}, CG_F32}, {t.state.shape(), CG_F32}, {t.conv_state.shape(), CG_F32}};
    Operands o;
    for (Tensor *x : {&t.q, &t.k, &t.v, &t.conv_q, &t.conv_k, &t.conv_v, &t.beta, &t.decay, &t.decay_w, &t.a_log, &t.dt_bias, &t.gate, &t.gate_w,
                      &t.norm, &t.state, &t.conv_state})
        o.add(std::move(*x));
    return issue(i, std::move(o), std::move(types), [opt](Backend &be, auto &&raw) {
        cg_channel_delta_args a{raw(0), raw(1),  raw(2),  raw(3),  raw(4),  raw(5),  raw(6),    raw(7),       raw(8),  raw(9),   raw(10),
                                raw(11), raw(12), raw(13), raw(14), raw(15), opt.heads, opt.kv_heads, opt.dim, opt.vdim, opt.eps};
        return be.block_channel_delta(a);
    });
}

} // namespace blocks
} // namespace cgh
