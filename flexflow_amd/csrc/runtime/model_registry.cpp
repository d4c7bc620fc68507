// model_registry.cpp -- model classes by the architecture config.json names.
#include "json.h"
#include "model.h"

namespace ffmi {

static std::map<std::string, ModelFactory> &registry() {
  static std::map<std::string, ModelFactory> r;
  return r;
}

ModelRegistrar::ModelRegistrar(const char *architecture, ModelFactory f) {
  registry()[architecture] = f;
}

ffmi_status create_model_from_json(const char *config_json, const ffmi_model_opts *o,
                                   ffmi_model **out) {
  Json c;
  if (!Json::parse(config_json, strlen(config_json), &c) || c.type != Json::OBJ) {
    ffmi_set_last_error("config.json: not a JSON object", __FILE__, __LINE__);
    return FFMI_ERR_INVALID;
  }
  std::string name = c.text("architecture");
  if (name.empty()) {
    const Json *a = c.find("architectures");
    if (a && a->type == Json::ARR && !a->arr.empty()) name = a->arr[0].str;
  }
  auto it = registry().find(name);
  if (it == registry().end()) {
    ffmi_set_last_error(("config.json: no model class for architecture '" + name + "'").c_str(),
                        __FILE__, __LINE__);
    return FFMI_ERR_UNSUPPORTED;
  }
  return it->second(c, o, out);
}

}  // namespace ffmi
