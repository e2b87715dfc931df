// See safetensors.hpp.  Host-only.
#include "safetensors.hpp"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cerrno>
#include <cstring>

#include "json.hpp"
#include "mesh_common.hpp"

namespace mesh {

static uint64_t dtype_bytes(const std::string &d) {
    if (d == "F64" || d == "I64" || d == "U64") return 8;
    if (d == "F32" || d == "I32" || d == "U32") return 4;
    if (d == "BF16" || d == "F16" || d == "I16" || d == "U16") return 2;
    if (d == "I8" || d == "U8" || d == "BOOL" || d == "F8_E4M3" || d == "F8_E5M2") return 1;
    return 0;
}

SafetensorsFile::~SafetensorsFile() {
    if (map_) munmap(const_cast<uint8_t *>(map_), size_);
    if (fd_ >= 0) close(fd_);
}

int SafetensorsFile::open(const char *path) {
    fd_ = ::open(path, O_RDONLY | O_CLOEXEC);
    if (fd_ < 0) return fail(MESH_ERR_IO, "safetensors: cannot open '%s': %s", path, strerror(errno));
    struct stat st;
    if (fstat(fd_, &st) != 0) return fail(MESH_ERR_IO, "safetensors: fstat('%s') failed: %s", path, strerror(errno));
    size_ = (uint64_t)st.st_size;
    if (size_ < 8) return fail(MESH_ERR_FORMAT, "safetensors: '%s' is too short", path);
    void *m = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd_, 0);
    if (m == MAP_FAILED) return fail(MESH_ERR_IO, "safetensors: mmap('%s') failed: %s", path, strerror(errno));
    map_ = static_cast<const uint8_t *>(m);
    uint64_t head = 0;
    for (int i = 0; i < 8; ++i) head |= (uint64_t)map_[i] << (8 * i);
    if (head > size_ - 8) return fail(MESH_ERR_FORMAT, "safetensors: the header of '%s' leaves the file", path);
    data_ = 8 + head;
    JsonValue root;
    std::string err;
    if (!json_parse(reinterpret_cast<const char *>(map_) + 8, (size_t)head, root, err) || root.kind != JsonValue::OBJECT)
        return fail(MESH_ERR_FORMAT, "safetensors: bad header in '%s': %s", path, err.empty() ? "not an object" : err.c_str());
    const uint64_t avail = size_ - data_;
    for (const auto &kv : root.fields) {
        if (kv.first == "__metadata__") continue;
        const JsonValue *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *off = kv.second.get("data_offsets");
        SafeTensor t;
        uint64_t b = 0, e = 0;
        bool ok = dt && dt->kind == JsonValue::STRING && sh && sh->kind == JsonValue::ARRAY && off && off->items.size() == 2 &&
                  off->items[0].as_count(avail, b) && off->items[1].as_count(avail, e) && b <= e;
        uint64_t n = 1;
        if (ok) {
            for (const JsonValue &d : sh->items) {
                uint64_t v = 0;
                if (!d.as_count(uint64_t(1) << 40, v) || (v && n > (uint64_t(1) << 44) / v)) { ok = false; break; }
                t.shape.push_back(v);
                n *= v;
            }
        }
        if (ok) {
            t.dtype = dt->str;
            t.begin = b;
            t.nbytes = e - b;
            const uint64_t eb = dtype_bytes(t.dtype);
            ok = eb == 0 || t.nbytes == n * eb;
        }
        if (!ok) return fail(MESH_ERR_FORMAT, "safetensors: entry '%s' of '%s' is inconsistent", kv.first.c_str(), path);
        tensors_[kv.first] = std::move(t);
    }
    return MESH_OK;
}

const SafeTensor *SafetensorsFile::find(const std::string &name) const {
    auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
}

}  // namespace mesh
