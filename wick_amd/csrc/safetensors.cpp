// Model folder reader behind include/wick_safetensors.h (host only).
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cerrno>
#include <cmath>
#include <cstdio>
#include <cstring>
#include <memory>

#include "model_folder.h"

using wick_rocm::Json;
using wick_rocm::JsonParser;

namespace {

thread_local std::string g_error;

enum { kOk = 0, kInvalidArg = -1, kIo = -2, kFormat = -3, kNotFound = -4, kUnsupported = -5 };  // the values of wick_gguf_status

int fail(int code, const std::string& what) {
    g_error = what;
    return code;
}

bool read_text(const std::string& path, std::string& out) {
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) return false;
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0) out.append(buf, n);
    const bool ok = !ferror(f);
    fclose(f);
    return ok;
}

bool whole(const Json& v, uint64_t& out) {
    if (v.kind != Json::kNumber || !(v.number >= 0.0) || v.number > 9007199254740992.0 || v.number != std::floor(v.number)) return false;
    out = (uint64_t)v.number;
    return true;
}

int parse_tensors(wick_safetensors* s, const Json& header, const uint8_t* data, uint64_t data_bytes) {
    if (header.kind != Json::kObject) return fail(kFormat, "safetensors: the header is not an object");
    for (const auto& m : header.members) {
        if (m.first == "__metadata__") continue;
        const std::string where = "safetensors: tensor " + m.first + ": ";
        const Json *dt = m.second.find("dtype"), *shape = m.second.find("shape"), *off = m.second.find("data_offsets");
        if (!dt || dt->kind != Json::kString || !shape || shape->kind != Json::kArray || !off || off->kind != Json::kArray || off->items.size() != 2)
            return fail(kFormat, where + "incomplete entry");
        wick_safetensors::Tensor t;
        t.name = m.first;
        uint64_t elem;
        if (dt->string == "BF16") t.dtype = WICK_SAFETENSORS_BF16, elem = 2;
        else if (dt->string == "F32") t.dtype = WICK_SAFETENSORS_F32, elem = 4;
        else if (dt->string == "I32") t.dtype = WICK_SAFETENSORS_I32, elem = 4;
        else return fail(kUnsupported, where + "dtype " + dt->string + " (BF16, F32 and I32 are read)");
        if (shape->items.size() > 8) return fail(kFormat, where + "more than 8 dimensions");
        uint64_t count = 1, b = 0, e = 0;
        for (const Json& d : shape->items) {
            uint64_t v;
            if (!whole(d, v)) return fail(kFormat, where + "bad shape");
            if (v != 0 && count > data_bytes / v) return fail(kFormat, where + "larger than the file");
            count *= v;
            t.shape.push_back(v);
        }
        if (!whole(off->items[0], b) || !whole(off->items[1], e) || b > e || e > data_bytes || (e - b) / elem != count || (e - b) % elem != 0)
            return fail(kFormat, where + "byte range does not fit its shape or the file");
        t.data = data + b, t.nbytes = (size_t)(e - b);
        if (!s->index.emplace(t.name, s->tensors.size()).second) return fail(kFormat, where + "listed twice");
        s->tensors.push_back(std::move(t));
    }
    return kOk;
}

}  // namespace

wick_safetensors::~wick_safetensors() {
    if (map) munmap(const_cast<uint8_t*>(map), map_bytes);
}

extern "C" {

const char* wick_safetensors_last_error(void) { return g_error.c_str(); }

int wick_safetensors_open(const char* dir, wick_safetensors** out) {
    if (!dir || !out) return fail(kInvalidArg, "safetensors: null argument");
    *out = nullptr;
    std::unique_ptr<wick_safetensors> s(new wick_safetensors);
    const std::string base(dir), cfg = base + "/config.json", st = base + "/model.safetensors";
    if (!read_text(cfg, s->config_text)) return fail(kIo, "cannot read " + cfg + ": " + strerror(errno));
    std::string err;
    if (!JsonParser::parse(s->config_text.data(), s->config_text.size(), s->config, err)) return fail(kFormat, cfg + ": " + err);
    const Json* arch = s->config.find("architecture");
    if (!arch || arch->kind != Json::kString) return fail(kFormat, cfg + ": no \"architecture\"");
    s->architecture = arch->string;

    const int fd = open(st.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return fail(kIo, "cannot open " + st + ": " + strerror(errno));
    struct stat sb;
    if (fstat(fd, &sb) != 0 || sb.st_size < 8) {
        close(fd);
        return fail(kFormat, st + ": too short");
    }
    void* p = mmap(nullptr, (size_t)sb.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
    const int mmap_errno = errno;
    close(fd);
    if (p == MAP_FAILED) return fail(kIo, "cannot map " + st + ": " + strerror(mmap_errno));
    s->map = static_cast<const uint8_t*>(p), s->map_bytes = (size_t)sb.st_size;
    uint64_t hlen = 0;
    for (int i = 0; i < 8; i++) hlen |= (uint64_t)s->map[i] << (8 * i);
    if (hlen > s->map_bytes - 8 || hlen > (512u << 20)) return fail(kFormat, st + ": header length beyond the file");
    Json header;
    if (!JsonParser::parse(reinterpret_cast<const char*>(s->map) + 8, (size_t)hlen, header, err)) return fail(kFormat, st + ": " + err);
    if (int rc = parse_tensors(s.get(), header, s->map + 8 + hlen, s->map_bytes - 8 - hlen)) return rc;
    *out = s.release();
    return kOk;
}

void wick_safetensors_close(wick_safetensors* s) { delete s; }

const char* wick_safetensors_architecture(const wick_safetensors* s) { return s ? s->architecture.c_str() : nullptr; }

const char* wick_safetensors_config(const wick_safetensors* s, size_t* nbytes) {
    if (!s) return nullptr;
    if (nbytes) *nbytes = s->config_text.size();
    return s->config_text.c_str();
}

uint64_t wick_safetensors_tensor_count(const wick_safetensors* s) { return s ? s->tensors.size() : 0; }

const char* wick_safetensors_tensor_name(const wick_safetensors* s, uint64_t index) {
    return s && index < s->tensors.size() ? s->tensors[index].name.c_str() : nullptr;
}

int wick_safetensors_tensor(const wick_safetensors* s, const char* name, int* dtype, uint32_t* n_dims, uint64_t* dims, const void** data,
                            size_t* nbytes) {
    if (!s || !name) return fail(kInvalidArg, "safetensors: null argument");
    const wick_safetensors::Tensor* t = s->find(name);
    if (!t) return fail(kNotFound, std::string("safetensors: no tensor ") + name);
    if (dtype) *dtype = t->dtype;
    if (n_dims) *n_dims = (uint32_t)t->shape.size();
    if (dims)
        for (size_t i = 0; i < t->shape.size(); i++) dims[i] = t->shape[i];
    if (data) *data = t->data;
    if (nbytes) *nbytes = t->nbytes;
    return kOk;
}

}  // extern "C"
