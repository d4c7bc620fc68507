// capi_llama.cpp -- C ABI of the serving runtime that belongs to the LLaMA
// family: typed model creation and SSM exchange over its communicators.
#include "json.h"
#include "request_manager.h"

// HF LLaMA config.json keys (checkpoint.py llama_config_from_hf)
static ffmi_status llama_from_json(const ffmi::Json &c, const ffmi_model_opts *o,
                                   ffmi_model **out) {
  ffmi_llama_config cfg{};
  if (!c.get("num_hidden_layers", &cfg.num_layers) || !c.get("vocab_size", &cfg.vocab_size) ||
      !c.get("num_attention_heads", &cfg.num_heads) || !c.get("hidden_size", &cfg.hidden) ||
      !c.get("intermediate_size", &cfg.intermediate) || !c.get("rms_norm_eps", &cfg.rms_eps)) {
    ffmi_set_last_error("config.json: a LLaMA size is missing", __FILE__, __LINE__);
    return FFMI_ERR_INVALID;
  }
  if (!c.get("num_key_value_heads", &cfg.num_kv_heads)) cfg.num_kv_heads = cfg.num_heads;
  cfg.rope_theta = 10000.0f;
  const ffmi::Json *rp = c.find("rope_parameters"), *sc = c.find("rope_scaling");
  if (!c.get("rope_theta", &cfg.rope_theta) && rp) rp->get("rope_theta", &cfg.rope_theta);
  if (!sc || sc->is_null()) sc = rp;
  std::string kind = sc ? sc->text("rope_type") : "";
  if (kind.empty() && sc) kind = sc->text("type");
  if (kind == "llama3") {
    cfg.rope_llama3 = 1;
    if (!sc->get("factor", &cfg.rope_factor) ||
        !sc->get("low_freq_factor", &cfg.rope_low_freq_factor) ||
        !sc->get("high_freq_factor", &cfg.rope_high_freq_factor) ||
        !sc->get("original_max_position_embeddings", &cfg.rope_original_max_pos))
      return FFMI_ERR_INVALID;
  } else if (!kind.empty() && kind != "default") {
    ffmi_set_last_error("config.json: unsupported rope scaling", __FILE__, __LINE__);
    return FFMI_ERR_UNSUPPORTED;
  }
  return ffmi_model_create(&cfg, o, out);
}
static ffmi::ModelRegistrar g_llama("LlamaForCausalLM", llama_from_json);

extern "C" ffmi_status ffmi_model_create(const ffmi_llama_config *cfg, const ffmi_model_opts *o,
                                         ffmi_model **out) {
  if (o && o->full_precision) return ffmi::create_llama_f32(cfg, o, out);
  return ffmi::create_llama_gpu(cfg, o, out);
}

static int comm_allgather_cb(void *ctx, const void *mine, size_t bytes, void *all) {
  return ffmi_comm_allgather(static_cast<ffmi_comm *>(ctx), mine, bytes, all) == FFMI_OK ? 0 : 1;
}

extern "C" ffmi_status ffmi_rm_set_ssm_exchange_comm(ffmi_rm *rm, ffmi_comm *comm) {
  if (!rm || !comm) return FFMI_ERR_INVALID;
  rm->rm.set_ssm_exchange(ffmi::comm_size(comm), ffmi::comm_rank(comm), comm_allgather_cb, comm);
  return FFMI_OK;
}
