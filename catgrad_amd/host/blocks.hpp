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
        cg_linear_args a{raw(0), raw(1), raw(2), raw(3), raw(4), opt.eps, opt.scale};
        std::vector<Tensor> r;
        r.push_back(be.block_linear(a));
        return r;
    })[0]);
}

// One sublayer's result on its way into the residual stream: act(y) . w^T, times sigmoid(gate + gate_bias)
struct Branch {
    Tensor y, w, gate, gate_bias, poly;
};
inline Tensor residual(I &i, Tensor x, std::vector<Branch> br, float eps) {
    const Shape s = x.shape();
    const size_t n = br.size();
    Operands o;
    o.add(std::move(x));
    for (Branch &b : br) {
        o.add(std::move(b.y));
        o.add(std::move(b.w));
        o.add(std::move(b.gate));
        o.add(std::move(b.gate_bias));
        o.add(std::move(b.poly));
    }
    return std::move(issue(i, std::move(o), {{s, CG_F32}}, [n, eps](Backend &be, auto &&raw) {
        std::vector<cg_branch> c(n);
        for (size_t k = 0; k < n; k++) c[k] = {raw(5 * k + 1), raw(5 * k + 2), raw(5 * k + 3), raw(5 * k + 4), raw(5 * k + 5)};
        std::vector<Tensor> r;
        r.push_back(be.block_residual(be.adopt(raw(0)), c, eps));
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
                            opt.dim, opt.vdim, position, opt.window, opt.temp_every, opt.scale, opt.norm_eps, opt.temp_coef, opt.distance_bias};
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
