// model_registry.h -- model classes by the architecture name of a config.json.
#pragma once

#include "model_folder.h"
#include "session_base.h"

namespace bh {

struct ModelOptions {
  bool f32 = false;
  int max_len = 4096, prefill_block = 2048;
  hipStream_t stream = nullptr;
};

// Builds the session of a folder: null, with the message recorded, on failure; may
// throw std::runtime_error about the folder's contents.
using ModelFactory = Session *(*)(const ModelFolder &folder, const ModelOptions &options);

// A model class registers itself when the library is loaded, with a static object
// of this type in its own source file.
struct ModelRegistration {
  ModelRegistration(const char *architecture, ModelFactory factory);
};

} // namespace bh
