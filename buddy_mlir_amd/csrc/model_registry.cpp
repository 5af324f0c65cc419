// model_registry.cpp -- sessions from model folders.
#include "model_registry.h"

#include <utility>
#include <vector>

namespace bh {
namespace {
// built on first use: registrations run in no particular order
std::vector<std::pair<std::string, ModelFactory>> &models() {
  static std::vector<std::pair<std::string, ModelFactory>> m;
  return m;
}
} // namespace

ModelRegistration::ModelRegistration(const char *architecture, ModelFactory factory) {
  models().emplace_back(architecture, factory);
}
} // namespace bh

extern "C" {

buddy_hip_session *buddy_hip_session_create_from_folder(const char *folder,
                                                        const buddy_hip_model_options *options) try {
  if (!folder) {
    bh::fail(BUDDY_HIP_ERR_ARG, "create_from_folder: null folder");
    return nullptr;
  }
  bh::ModelOptions o;
  if (options) {
    if ((options->dtype != BUDDY_HIP_MODEL_BF16 && options->dtype != BUDDY_HIP_MODEL_F32) ||
        options->max_len < 0 || options->prefill_block < 0) {
      bh::fail(BUDDY_HIP_ERR_ARG, "create_from_folder: bad option");
      return nullptr;
    }
    o.f32 = options->dtype == BUDDY_HIP_MODEL_F32;
    if (options->max_len)
      o.max_len = options->max_len;
    if (options->prefill_block)
      o.prefill_block = options->prefill_block;
    o.stream = bh::as_stream(options->stream);
  }
  const bh::ModelFolder files(folder);
  const std::string name = files.architecture();
  for (const auto &m : bh::models())
    if (m.first == name) {
      if (buddy_hip_device_count() == 0) {
        bh::fail(BUDDY_HIP_ERR_NO_DEVICE, "create_from_folder: no HIP device");
        return nullptr;
      }
      return bh::as_handle(m.second(files, o));
    }
  bh::fail(BUDDY_HIP_ERR_ARG, "create_from_folder: no model class for architecture \"%s\"",
           name.c_str());
  return nullptr;
} BH_CATCH_NULL("buddy_hip_session_create_from_folder")

const char *buddy_hip_model_architecture(int index) {
  const auto &m = bh::models();
  return index >= 0 && (size_t)index < m.size() ? m[(size_t)index].first.c_str() : nullptr;
}
}
