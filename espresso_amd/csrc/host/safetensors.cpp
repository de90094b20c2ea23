#include "safetensors.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <cstring>

#include "json_min.h"

namespace esp {

size_t safetensors_dtype_bytes(const std::string &t) {
    if (t == "F64" || t == "I64" || t == "U64") return 8;
    if (t == "F32" || t == "I32" || t == "U32") return 4;
    if (t == "BF16" || t == "F16" || t == "I16" || t == "U16") return 2;
    if (t == "I8" || t == "U8" || t == "BOOL") return 1;
    return 0;
}

size_t TensorView::elements() const {
    size_t n = 1;
    for (int64_t d : shape) n *= (size_t)d;
    return n;
}

SafetensorsFile::~SafetensorsFile() {
    if (map_) munmap(map_, map_bytes_);
}

const TensorView *SafetensorsFile::find(const std::string &name) const {
    auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
}

bool SafetensorsFile::open(const std::string &path, std::unique_ptr<SafetensorsFile> *out, std::string *error) {
    auto bad = [&](const std::string &what) { if (error) *error = path + ": " + what; return false; };
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return bad("cannot be opened");
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) { close(fd); return bad("too short for a safetensors file"); }
    std::unique_ptr<SafetensorsFile> f(new SafetensorsFile());
    f->map_bytes_ = (size_t)st.st_size;
    void *m = mmap(nullptr, f->map_bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (m == MAP_FAILED) return bad("cannot be mapped");
    f->map_ = m;
    const uint8_t *base = static_cast<const uint8_t *>(m);
    uint64_t header = 0;
    for (int i = 7; i >= 0; i--) header = header << 8 | base[i];
    if (header > f->map_bytes_ - 8) return bad("header runs past the end of the file");
    JsonNode root;
    std::string perr;
    if (!json_parse(std::string(reinterpret_cast<const char *>(base) + 8, (size_t)header), &root, &perr) || !root.is(JsonNode::Object))
        return bad("header is not a JSON object " + perr);
    const uint8_t *data = base + 8 + header;
    const size_t data_bytes = f->map_bytes_ - 8 - (size_t)header;
    for (const auto &m2 : root.members) {
        if (m2.first == "__metadata__") continue;
        const JsonNode *dt = m2.second.find("dtype"), *sh = m2.second.find("shape"), *off = m2.second.find("data_offsets");
        if (!dt || !dt->is(JsonNode::String) || !sh || !sh->is(JsonNode::Array) || !off || !off->is(JsonNode::Array) || off->items.size() != 2)
            return bad("entry " + m2.first + " is incomplete");
        TensorView t;
        t.dtype = dt->text;
        for (const JsonNode &d : sh->items) {
            if (!d.is(JsonNode::Number) || d.number < 0 || d.number != std::floor(d.number)) return bad("shape of " + m2.first);
            t.shape.push_back((int64_t)d.number);
        }
        const double lo = off->items[0].number, hi = off->items[1].number;
        if (!off->items[0].is(JsonNode::Number) || !off->items[1].is(JsonNode::Number) || lo < 0 || hi < lo || hi > (double)data_bytes)
            return bad("data of " + m2.first + " lies outside the file");
        t.data = data + (size_t)lo;
        t.bytes = (size_t)(hi - lo);
        const size_t elem = safetensors_dtype_bytes(t.dtype);
        if (elem == 0) return bad("unknown dtype " + t.dtype + " of " + m2.first);
        if (t.elements() * elem != t.bytes) return bad("byte range of " + m2.first + " does not fit its shape");
        f->tensors_[m2.first] = t;
    }
    *out = std::move(f);
    return true;
}

}  // namespace esp
