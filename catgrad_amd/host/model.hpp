// What every decoder model of this driver offers: an empty state for B sequences, and a run that takes [B, S] new tokens
// and the state behind which they stand and leaves the state moved on — a whole prompt, a portion of one, or one token.
// The greedy generate loop and its timing protocol (catgrad-llm/examples/llama/main.rs:876-940,955-1037;
// catgrad-llm/src/utils/mod.rs:528-583) work on this interface alone.
#pragma once

#include <chrono>

#include "graph.hpp"

namespace cgh {

// What a model carries from run to run: caches, recurrent states, and how many tokens they stand behind.
struct State {
    std::vector<Tensor> tensors;
    size_t position = 0;
};

// Which results a run is asked for.  rows: positions b * S + s that go through the vocabulary projection (null: all).
struct Want {
    const std::vector<uint32_t> *rows = nullptr;
    bool tokens = true;  // their arg-max ids
    bool logits = false; // the logits themselves
};

struct RunOut {
    Tensor tokens; // u32 [B, S, 1], or [1, rows, 1]
    Tensor logits; // f32 [B, S, vocab], or [1, rows, vocab]
};

class Model {
  public:
    explicit Model(Interpreter &i) : i_(i) {}
    virtual ~Model() = default;
    virtual size_t vocab_size() const = 0;
    virtual State empty_state(size_t B) = 0;
    // The parameters of the interpreter are not those of the last run any more.
    virtual void parameters_changed() {}
    // True when rows that nobody asked for skip the vocabulary projection.
    virtual bool selects_rows() const { return false; }

    // `Interpreter::run(term, inputs)` for the model's term.  With Interpreter::schedule 0 the operations run as the
    // graph builder issues them; with 1 the pass is first recorded as a term and then evaluated in the layers of the
    // reference's evaluator, with its value map (graph.hpp); with 2 recorded and evaluated in the order of recording.
    // The run's inputs are clones of the caller's state (main.rs:1007), which is replaced when the run has succeeded.
    RunOut run(Tensor ids, State &state, size_t max_positions, const Want &want) {
        prepare();
        const size_t S = ids.shape()[1];
        Parts p;
        if (i_.schedule == 0 || i_.recorder) p = def(std::move(ids), state.tensors, state.position, max_positions, want);
        else p = run_recorded(std::move(ids), state.tensors, state.position, max_positions, want);
        state.tensors = std::move(p.state);
        state.position += S;
        return std::move(p.out);
    }

  protected:
    struct Parts {
        RunOut out;
        std::vector<Tensor> state;
    };
    // `DynModule::def`: the model's operations on the run's inputs
    virtual Parts def(Tensor ids, std::vector<Tensor> state, size_t position, size_t max_positions, const Want &want) = 0;
    virtual void prepare() {}
    Interpreter &i_;

  private:
    Parts run_recorded(Tensor ids, const std::vector<Tensor> &state, size_t position, size_t max_positions, const Want &want) {
        Term term;
        Tensor sx = term.source(ids.shape(), ids.dtype());
        std::vector<Tensor> ss;
        for (const Tensor &t : state) ss.push_back(term.source(t.shape(), t.dtype()));
        Parts p;
        i_.recorder = &term;
        try {
            p = def(std::move(sx), std::move(ss), position, max_positions, want);
        } catch (...) {
            i_.recorder = nullptr;
            throw;
        }
        i_.recorder = nullptr;
        std::vector<Tensor> outs = std::move(p.state);
        const size_t n = outs.size();
        const bool tok = (bool)p.out.tokens, lg = (bool)p.out.logits;
        if (tok) outs.push_back(std::move(p.out.tokens));
        if (lg) outs.push_back(std::move(p.out.logits));
        term.finish(std::move(outs));
        std::vector<Tensor> in;
        in.push_back(std::move(ids));
        for (const Tensor &t : state) in.push_back(t);
        std::vector<Tensor> r = term.run(i_, std::move(in), i_.schedule == 2);
        Parts q;
        for (size_t k = 0; k < n; k++) q.state.push_back(std::move(r[k]));
        if (tok) q.out.tokens = std::move(r[n]);
        if (lg) q.out.logits = std::move(r[n + (tok ? 1 : 0)]);
        return q;
    }
};

struct GenerateStats {
    double prefill_s = 0, decode_s = 0;
    uint64_t prefill_calls = 0, decode_calls = 0;
};

// Greedy generation for a batch of B equal-length prompts.  One prefill run, then `steps` decode runs; each run ends
// with the only device-to-host read of the step, `to_vec` of the argmax tokens, of which the last position of every
// sequence is the next input (main.rs:1031-1037 generalised from batch 1 to B rows).
// out_tokens receives (steps + 1) x B ids: the token produced by the prefill, then one
// per decode run.  Prefill time includes the first read-back, as in main.rs:914-917.
// prefill_logits, when given, receives the logits [B, S, vocab] of the prefill run (read back after the
// timed part of that run; for parity checks).
inline void generate(Model &m, Interpreter &i, const uint32_t *prompt, size_t B, size_t S, size_t steps,
                     size_t max_positions, uint32_t *out_tokens, GenerateStats *st, std::vector<uint32_t> *prefill_logits = nullptr) {
    State state = m.empty_state(B);
    std::vector<uint32_t> ids(prompt, prompt + B * S);
    size_t cur = S;
    auto t0 = std::chrono::steady_clock::now();
    uint64_t calls0 = i.backend.calls;
    for (size_t it = 0; it <= steps; it++) {
        Tensor x = i.backend.ndarray_from_vec_u32(ids.data(), ids.size(), Shape{B, cur});
        Want want;
        want.logits = it == 0 && prefill_logits;
        std::vector<uint32_t> last;
        if (m.selects_rows() && !want.logits && cur > 1) {
            for (size_t b = 0; b < B; b++) last.push_back((uint32_t)(b * cur + cur - 1));
            want.rows = &last;
        }
        RunOut o = m.run(std::move(x), state, max_positions, want);
        std::vector<uint32_t> tok = i.backend.to_vec_bits(std::move(o.tokens));
        const size_t per = tok.size() / B;
        ids.resize(B);
        for (size_t b = 0; b < B; b++) {
            ids[b] = tok[b * per + (per - 1)];
            out_tokens[it * B + b] = ids[b];
        }
        cur = 1;
        if (it == 0) {
            auto t1 = std::chrono::steady_clock::now();
            st->prefill_s = std::chrono::duration<double>(t1 - t0).count();
            st->prefill_calls = i.backend.calls - calls0;
            if (prefill_logits) *prefill_logits = i.backend.to_vec_bits(std::move(o.logits));
            calls0 = i.backend.calls;
            t0 = std::chrono::steady_clock::now();
        }
    }
    st->decode_s = std::chrono::duration<double>(std::chrono::steady_clock::now() - t0).count();
    st->decode_calls = i.backend.calls - calls0;
}

} // namespace cgh
