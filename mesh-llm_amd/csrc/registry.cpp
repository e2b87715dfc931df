#include "registry.hpp"

namespace mesh {

static const ModelArch ARCHS[] = {
    {"llama", CONTAINER_GGUF, FAMILY_KQUANT},
    {"qwen2", CONTAINER_GGUF, FAMILY_KQUANT},
    {"qwen3", CONTAINER_GGUF, FAMILY_KQUANT},
    {"qwen3moe", CONTAINER_GGUF, FAMILY_KQUANT},
    {"Nadosun", CONTAINER_FOLDER, FAMILY_HYBRID},
    {"Nutavik", CONTAINER_FOLDER, FAMILY_HYBRID},
};

const ModelArch *find_arch(const std::string &name, ModelContainer container) {
    for (const ModelArch &a : ARCHS)
        if (a.container == container && name == a.name) return &a;
    return nullptr;
}

std::string arch_names(ModelContainer container) {
    std::string s;
    for (const ModelArch &a : ARCHS) {
        if (a.container != container) continue;
        if (!s.empty()) s += ", ";
        s += a.name;
    }
    return s;
}

}  // namespace mesh
