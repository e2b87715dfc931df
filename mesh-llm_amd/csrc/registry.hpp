// The architectures this library runs: name -> container the weights come in and the runner that computes the layers.
#pragma once

#include <string>

namespace mesh {

enum ModelContainer { CONTAINER_GGUF = 0, CONTAINER_FOLDER = 1 };     // one .gguf file | config.json + model.safetensors
enum ModelFamily {
    FAMILY_KQUANT = 0,      // pre-norm decoder over K-quant weights (stage.hip)
    FAMILY_HYBRID = 1       // layers of several kinds over bf16 weights, described one by one (hybrid.hpp)
};

struct ModelArch {
    const char *name;
    ModelContainer container;
    ModelFamily family;
};

// nullptr if the library has no runner for this name in this container
const ModelArch *find_arch(const std::string &name, ModelContainer container);
// "a, b and c": the names of one container, for messages
std::string arch_names(ModelContainer container);

}  // namespace mesh
