// Weight files of the layered models.  Host code only.
//
//   u64 (little-endian) header length, JSON header {name: {"dtype", "shape", "data_offsets": [a, b]}},
//   then the data; offsets count from the end of the header.  The key "__metadata__" is skipped.
// Nothing is trusted: the header must lie inside the file, every tensor inside the data, and its
// byte count must be its shape times its element size.
#include "layered.hpp"

#include <algorithm>
#include <cerrno>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace coeus {

SafeTensors::~SafeTensors() {
    if (map_) (void)munmap(map_, size_);
}

static uint64_t element_size(const std::string &dtype) {
    if (dtype == "F64" || dtype == "I64" || dtype == "U64") return 8;
    if (dtype == "F32" || dtype == "I32" || dtype == "U32") return 4;
    if (dtype == "F16" || dtype == "BF16" || dtype == "I16" || dtype == "U16") return 2;
    if (dtype == "I8" || dtype == "U8" || dtype == "BOOL") return 1;
    return 0;
}

// A JSON number that is a count: whole, not negative, exactly representable.
static bool to_u64(const Json &j, uint64_t &out) {
    if (j.type != Json::Number || !(j.num >= 0.0) || j.num > 9007199254740992.0) return false;
    out = (uint64_t)j.num;
    return (double)out == j.num;
}

int SafeTensors::open(const std::string &path) {
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return fail(COEUS_INVALID_INPUT, "Failed to open %s: %s", path.c_str(), std::strerror(errno));
    struct stat sb;
    if (fstat(fd, &sb) != 0 || sb.st_size < 8) {
        ::close(fd);
        return fail(COEUS_INVALID_INPUT, "%s is too short for a weight file", path.c_str());
    }
    size_ = (uint64_t)sb.st_size;
    void *p = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (p == MAP_FAILED) return fail(COEUS_INVALID_INPUT, "Failed to map %s: %s", path.c_str(), std::strerror(errno));
    map_ = p;
    const uint8_t *base = (const uint8_t *)p;
    uint64_t hlen = 0;
    for (int i = 0; i < 8; i++) hlen |= (uint64_t)base[i] << (8 * i);
    if (hlen > size_ - 8) return fail(COEUS_INVALID_INPUT, "%s: the header does not fit the file", path.c_str());
    Json head;
    std::string err;
    if (!json_parse((const char *)base + 8, hlen, head, err) || head.type != Json::Object)
        return fail(COEUS_INVALID_INPUT, "%s: bad header: %s", path.c_str(), err.empty() ? "not an object" : err.c_str());
    const uint8_t *data = base + 8 + hlen;
    const uint64_t room = size_ - 8 - hlen;
    for (const auto &kv : head.fields) {
        if (kv.first == "__metadata__") continue;
        const Json *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *off = kv.second.get("data_offsets");
        uint64_t a = 0, b = 0;
        if (!dt || dt->type != Json::String || !sh || sh->type != Json::Array || !off || off->type != Json::Array ||
            off->items.size() != 2 || !to_u64(off->items[0], a) || !to_u64(off->items[1], b) || a > b || b > room)
            return fail(COEUS_INVALID_INPUT, "%s: bad entry for tensor %s", path.c_str(), kv.first.c_str());
        SafeTensor t;
        t.dtype = dt->str;
        t.data = data + a;
        t.bytes = b - a;
        uint64_t elems = 1;
        bool ok = element_size(t.dtype) != 0;
        for (const Json &d : sh->items) {
            uint64_t v = 0;
            ok = ok && to_u64(d, v) && (v == 0 || elems <= (1ull << 48) / v);
            if (!ok) break;
            elems *= v;
            t.shape.push_back(v);
        }
        if (!ok || elems * element_size(t.dtype) != t.bytes)
            return fail(COEUS_INVALID_INPUT, "%s: shape and size of tensor %s do not agree", path.c_str(), kv.first.c_str());
        tensors_.emplace_back(kv.first, std::move(t));
    }
    std::sort(tensors_.begin(), tensors_.end(), [](const auto &x, const auto &y) { return x.first < y.first; });
    return COEUS_OK;
}

const SafeTensor *SafeTensors::find(const std::string &name) const {
    auto it = std::lower_bound(tensors_.begin(), tensors_.end(), name,
                               [](const auto &x, const std::string &n) { return x.first < n; });
    return it != tensors_.end() && it->first == name ? &it->second : nullptr;
}

int check_tensors(const SafeTensors &file, const std::vector<TensorSpec> &want) {
    for (const TensorSpec &w : want) {
        const SafeTensor *t = file.find(w.name);
        if (!t) return fail(COEUS_INVALID_INPUT, "The weight file has no tensor %s", w.name.c_str());
        const bool shape_ok = w.cols ? t->shape.size() == 2 && t->shape[0] == w.rows && t->shape[1] == w.cols
                                     : t->shape.size() == 1 && t->shape[0] == w.rows;
        if (!shape_ok)
            return fail(COEUS_INVALID_INPUT, "Tensor %s does not have the shape [%llu%s%s] that the configuration asks for",
                        w.name.c_str(), (unsigned long long)w.rows, w.cols ? ", " : "",
                        w.cols ? std::to_string(w.cols).c_str() : "");
        if (t->dtype != "BF16" && t->dtype != "F32")
            return fail(COEUS_INVALID_INPUT, "Tensor %s has type %s; BF16 and F32 are read", w.name.c_str(), t->dtype.c_str());
    }
    return COEUS_OK;
}

int read_text_file(const std::string &path, std::string &out) {
    FILE *f = std::fopen(path.c_str(), "rb");
    if (!f) return fail(COEUS_INVALID_INPUT, "Failed to open %s: %s", path.c_str(), std::strerror(errno));
    out.clear();
    char buf[4096];
    size_t n;
    while ((n = std::fread(buf, 1, sizeof(buf), f)) > 0) {
        out.append(buf, n);
        if (out.size() > (64u << 20)) break;
    }
    const bool bad = std::ferror(f) != 0 || out.size() > (64u << 20);
    std::fclose(f);
    if (bad) return fail(COEUS_INVALID_INPUT, "Failed to read %s", path.c_str());
    return COEUS_OK;
}

}  // namespace coeus
