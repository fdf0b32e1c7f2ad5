// Model graphs of the benchmark configurations as eager interpreter programs:
//   LlamaModel  catgrad-llm-models/src/models/llama.rs:144-386
//   Qwen3Model  catgrad-llm-models/src/models/qwen3.rs:100-123,196-434 (dense path)
//   HiddenMlp   catgrad/examples/hidden.rs:103-132 with nn::linear + nn::Sigmoid
#pragma once

#include "model.hpp"
#include "nn.hpp"

namespace cgh {

struct LlmConfig { // the fields of LlamaConfig / Qwen3Config that the dense graphs read
    int arch = 0; // 0 llama, 1 qwen3
    size_t hidden_size = 0, num_hidden_layers = 0, num_attention_heads = 0, num_key_value_heads = 0;
    size_t head_dim = 0, intermediate_size = 0, vocab_size = 0;
    float rms_norm_eps = 1e-5f, rope_theta = 10000.0f;
    int tie_word_embeddings = 0;
};

class LlmModel : public Model {
  public:
    LlmModel(Interpreter &i, const LlmConfig &c) : Model(i), c_(c) {}
    const LlmConfig &config() const { return c_; }
    std::string root() const { return c_.arch == 0 ? "llama" : "qwen3"; }
    size_t vocab_size() const override { return c_.vocab_size; }
    State empty_state(size_t B) override { // empty_state_cache (utils/mod.rs:570-583) with the batch axis set to B
        Shape kv{c_.num_hidden_layers, B, c_.num_key_value_heads, 0, c_.head_dim};
        State s;
        s.tensors.push_back(i_.backend.zeros(kv, CG_F32));
        s.tensors.push_back(i_.backend.zeros(kv, CG_F32));
        return s;
    }

  protected:
    // `DynModule::def` for inputs [x u32[B,S], in_k, in_v f32[L,B,kvH,P,hd], Nat(max_positions)]
    // The logits, when asked for, are a clone of the lm_head output (for parity checks).
    Parts def(Tensor x, std::vector<Tensor> state, size_t, size_t max_positions, const Want &want) override {
        using namespace nn;
        Tensor in_k = std::move(state[0]), in_v = std::move(state[1]);
        I &i = i_;
        const std::string model = root() + ".model";
        // rope tables + per-layer cache views: Cache::init (helpers/cache.rs:86-103)
        auto tables = rope_tables_default(i, c_.rope_theta, max_positions, c_.head_dim, 1.0f);
        KVCache cache(i, c_.num_hidden_layers, in_k, in_v);
        size_t pos = shape(in_k)[3];
        in_k = Tensor();
        in_v = Tensor();
        x = embeddings(i, model + ".embed_tokens", std::move(x));
        size_t s = shape(x)[1];
        Tensor mask = causal_mask(i, s, pos);
        for (size_t l = 0; l < c_.num_hidden_layers; l++)
            x = layer(l, mask, cache, tables.first, tables.second, pos, model + ".layers." + std::to_string(l), std::move(x));
        mask = Tensor();
        x = rmsnorm(i, c_.rms_norm_eps, model + ".norm", std::move(x));
        const std::string lm_head = c_.tie_word_embeddings ? model + ".embed_tokens" : root() + ".lm_head";
        x = linear_no_bias(i, c_.hidden_size, c_.vocab_size, lm_head, std::move(x));
        if (want.rows) { // [B, S, vocab] -> [1, rows, vocab]: the graph projects every position, the chosen ones are gathered
            Shape ls = shape(x);
            x = reshape(i, Shape{ls[0] * ls[1], ls[2]}, std::move(x));
            Tensor ids = i.backend.ndarray_from_vec_u32(want.rows->data(), want.rows->size(), Shape{want.rows->size()});
            x = unsqueeze(i, 0, index(i, 0, std::move(ids), std::move(x)));
        }
        Parts p;
        if (want.logits) p.out.logits = x;
        if (want.tokens) p.out.tokens = argmax(i, std::move(x));
        auto kv = cache.output(i);
        p.state.push_back(std::move(kv.first));
        p.state.push_back(std::move(kv.second));
        return p;
    }

  private:
    // llama.rs:349-386 / qwen3.rs:330-372
    Tensor layer(size_t l, const Tensor &mask, nn::KVCache &cache, const Tensor &cos_t, const Tensor &sin_t, size_t pos,
                 const std::string &p, Tensor x) {
        using namespace nn;
        I &i = i_;
        Tensor res = x;
        x = rmsnorm(i, c_.rms_norm_eps, p + ".input_layernorm", std::move(x));
        x = attention(l, mask, cache, cos_t, sin_t, pos, p + ".self_attn", std::move(x));
        x = add(i, std::move(res), std::move(x));
        res = x;
        x = rmsnorm(i, c_.rms_norm_eps, p + ".post_attention_layernorm", std::move(x));
        x = mlp(p + ".mlp", std::move(x));
        return add(i, std::move(x), std::move(res));
    }

    // llama.rs:230-253 / qwen3.rs:100-123
    Tensor mlp(const std::string &p, Tensor x) {
        using namespace nn;
        I &i = i_;
        Tensor gate = linear_no_bias(i, c_.hidden_size, c_.intermediate_size, p + ".gate_proj", x);
        Tensor up = linear_no_bias(i, c_.hidden_size, c_.intermediate_size, p + ".up_proj", std::move(x));
        x = mul(i, silu(i, std::move(gate)), std::move(up));
        return linear_no_bias(i, c_.intermediate_size, c_.hidden_size, p + ".down_proj", std::move(x));
    }

    // llama.rs:255-347 / qwen3.rs:196-328
    Tensor attention(size_t l, const Tensor &mask, nn::KVCache &cache, const Tensor &cos_t, const Tensor &sin_t,
                     size_t pos, const std::string &p, Tensor x) {
        using namespace nn;
        I &i = i_;
        const size_t dim = c_.hidden_size, nh = c_.num_attention_heads, nkv = c_.num_key_value_heads;
        const size_t hd = c_.head_dim, rep = nh / nkv;
        Shape xs = shape(x);
        const size_t b = xs[0], s = xs[1];
        Tensor q = linear_no_bias(i, dim, nh * hd, p + ".q_proj", x);
        Tensor k = linear_no_bias(i, dim, nkv * hd, p + ".k_proj", x);
        Tensor v = linear_no_bias(i, dim, nkv * hd, p + ".v_proj", std::move(x));
        q = reshape(i, Shape{b, s, nh, hd}, std::move(q));
        k = reshape(i, Shape{b, s, nkv, hd}, std::move(k));
        v = reshape(i, Shape{b, s, nkv, hd}, std::move(v));
        q = transpose(i, 1, 2, std::move(q));
        k = transpose(i, 1, 2, std::move(k));
        v = transpose(i, 1, 2, std::move(v));
        if (c_.arch == 1) { // Qwen3 QK-norm over head_dim (qwen3.rs:249-279)
            q = reshape(i, Shape{b * s * nh, hd}, std::move(q));
            k = reshape(i, Shape{b * s * nkv, hd}, std::move(k));
            q = rmsnorm(i, c_.rms_norm_eps, p + ".q_norm", std::move(q));
            k = rmsnorm(i, c_.rms_norm_eps, p + ".k_norm", std::move(k));
            q = reshape(i, Shape{b, nh, s, hd}, std::move(q));
            k = reshape(i, Shape{b, nkv, s, hd}, std::move(k));
        }
        q = apply_rope_embedding(i, pos, hd, cos_t, sin_t, std::move(q));
        k = apply_rope_embedding(i, pos, hd, cos_t, sin_t, std::move(k));
        auto kv = cache.update(i, l, std::move(k), std::move(v));
        k = repeat_kv(i, rep, std::move(kv.first));
        v = repeat_kv(i, rep, std::move(kv.second));
        Tensor tk = transpose(i, 2, 3, std::move(k));
        Tensor attn = matmul(i, std::move(q), std::move(tk));
        Shape sh = shape(attn);
        Tensor denom = constant(i, std::sqrt((float)hd), sh);
        denom = cast(i, std::move(denom), dtype(attn));
        attn = div(i, std::move(attn), std::move(denom));
        Tensor am = cast(i, mask, dtype(attn));
        am = broadcast(i, sh, std::move(am));
        attn = add(i, std::move(attn), std::move(am));
        attn = softmax(i, std::move(attn));
        attn = matmul(i, std::move(attn), std::move(v));
        attn = transpose(i, 1, 2, std::move(attn));
        attn = reshape(i, Shape{b, s, nh * hd}, std::move(attn));
        return linear_no_bias(i, nh * hd, dim, p + ".o_proj", std::move(attn));
    }

    LlmConfig c_;
};

// hidden.rs:103-132 shaped MLP: Linear(in, hidden) -> nn::Sigmoid -> Linear(hidden, out).
inline Tensor hidden_mlp(Interpreter &i, size_t in_dim, size_t hidden, size_t out_dim, Tensor x) {
    x = nn::linear(i, in_dim, hidden, "mlp.l1", std::move(x));
    x = nn::sigmoid_module(i, std::move(x));
    return nn::linear(i, hidden, out_dim, "mlp.l2", std::move(x));
}

} // namespace cgh
