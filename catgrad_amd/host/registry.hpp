// The models this driver knows, by what a model folder's config.json says: "architecture" (or the "model_type" /
// "architectures" of a Llama or Qwen3 checkpoint).
#pragma once

#include <memory>

#include "loretar.hpp"
#include "lufatar.hpp"
#include "models.hpp"

namespace cgh {

// llama.rs:13-60, qwen3.rs:14-60: the fields the dense graphs read
inline LlmConfig read_llm_config(const Json &j, int arch) {
    LlmConfig c;
    c.arch = arch;
    c.hidden_size = j.at("hidden_size").nat();
    c.num_hidden_layers = j.at("num_hidden_layers").nat();
    c.num_attention_heads = j.at("num_attention_heads").nat();
    const Json *kv = j.find("num_key_value_heads"), *hd = j.find("head_dim"), *tie = j.find("tie_word_embeddings");
    c.num_key_value_heads = kv ? kv->nat() : c.num_attention_heads;
    if (!c.num_attention_heads || !c.num_key_value_heads) throw ConfigError("config: no attention heads");
    c.head_dim = hd ? hd->nat() : c.hidden_size / c.num_attention_heads;
    c.intermediate_size = j.at("intermediate_size").nat();
    c.vocab_size = j.at("vocab_size").nat();
    c.rms_norm_eps = (float)j.at("rms_norm_eps").real();
    c.rope_theta = (float)j.at("rope_theta").real();
    c.tie_word_embeddings = tie && tie->flag();
    return c;
}

// weights: CG_F32, or CG_BF16 for matrices at bfloat16 precision (models that have such a form)
inline std::unique_ptr<Model> make_model(Interpreter &i, const Json &config, cg_dtype weights) {
    std::string name;
    if (const Json *a = config.find("architecture")) name = a->str();
    else if (const Json *t = config.find("model_type")) name = t->str();
    else if (const Json *l = config.find("architectures"))
        if (!l->list().empty()) name = l->list()[0].str();
    if (name == "Loretar") return std::make_unique<LoretarModel>(i, LoretarConfig::read(config), weights);
    if (name == "Lufatar") return std::make_unique<LufatarModel>(i, LufatarConfig::read(config), weights);
    int arch = name == "llama" || name == "LlamaForCausalLM" ? 0 : name == "qwen3" || name == "Qwen3ForCausalLM" ? 1 : -1;
    if (arch < 0) throw ConfigError("config: unknown architecture '" + name + "'");
    if (weights != CG_F32) throw ConfigError("config: this architecture runs in f32 only");
    return std::make_unique<LlmModel>(i, read_llm_config(config, arch));
}

} // namespace cgh
