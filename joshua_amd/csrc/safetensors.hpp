// A safetensors file mapped read-only: an 8-byte little-endian header length, a JSON header
// (name -> dtype, shape, data_offsets), the data.  Host only.
#pragma once
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <map>
#include <memory>

#include "json.hpp"

namespace jq {

struct SafeTensor {
    enum Type { F32, F16, BF16, I32 };
    Type type;
    std::vector<uint64_t> shape;
    const uint8_t *data;  // any alignment
    uint64_t elems;
};

struct SafeTensors {
    std::map<std::string, SafeTensor> tensors;
    void *map = nullptr;
    size_t size = 0;
    SafeTensors() = default;
    SafeTensors(const SafeTensors &) = delete;
    SafeTensors &operator=(const SafeTensors &) = delete;
    ~SafeTensors() {
        if (map) munmap(map, size);
    }
};

// Elements [at, at + n) of a floating-point tensor as f32.
inline bool safetensor_to_f32(const SafeTensor &t, uint64_t at, uint64_t n, float *out) {
    if (at > t.elems || n > t.elems - at) return false;
    switch (t.type) {
    case SafeTensor::F32: memcpy(out, t.data + 4 * at, 4 * n); return true;
    case SafeTensor::BF16:
        for (uint64_t i = 0; i < n; i++) {
            uint16_t h;
            memcpy(&h, t.data + 2 * (at + i), 2);
            const uint32_t u = (uint32_t)h << 16;
            memcpy(out + i, &u, 4);
        }
        return true;
    case SafeTensor::F16:
        for (uint64_t i = 0; i < n; i++) {
            _Float16 h;
            memcpy(&h, t.data + 2 * (at + i), 2);
            out[i] = (float)h;
        }
        return true;
    default: return false;
    }
}

inline std::unique_ptr<SafeTensors> safetensors_open(const std::string &path, std::string *err) {
    auto bad = [&](const std::string &w) {
        *err = path + ": " + w;
        return std::unique_ptr<SafeTensors>();
    };
    const int fd = open(path.c_str(), O_RDONLY);
    if (fd < 0) return bad(strerror(errno));
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) {
        close(fd);
        return bad("not a safetensors file");
    }
    auto f = std::make_unique<SafeTensors>();
    f->size = (size_t)st.st_size;
    void *map = mmap(nullptr, f->size, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (map == MAP_FAILED) return bad(strerror(errno));
    f->map = map;
    const uint8_t *base = (const uint8_t *)map;
    uint64_t hlen = 0;
    for (int i = 7; i >= 0; i--) hlen = hlen << 8 | base[i];
    if (hlen > f->size - 8) return bad("the header runs past the end of the file");
    Json h;
    std::string jerr;
    if (!json_parse((const char *)base + 8, (size_t)hlen, &h, &jerr)) return bad(jerr);
    if (h.kind != Json::OBJECT) return bad("the header is not an object");
    const uint64_t room = f->size - 8 - hlen;
    for (const auto &m : h.members) {
        if (m.first == "__metadata__") continue;
        const Json *ty = m.second.find("dtype"), *sh = m.second.find("shape"), *off = m.second.find("data_offsets");
        if (!ty || !sh || !off || ty->kind != Json::STRING || sh->kind != Json::ARRAY || off->items.size() != 2)
            return bad("incomplete entry `" + m.first + "`");
        SafeTensor t;
        uint64_t width = 4;
        if (ty->str == "F32") t.type = SafeTensor::F32;
        else if (ty->str == "F16") t.type = SafeTensor::F16, width = 2;
        else if (ty->str == "BF16") t.type = SafeTensor::BF16, width = 2;
        else if (ty->str == "I32") t.type = SafeTensor::I32;
        else continue;  // a type no loader here asks for
        t.elems = 1;
        for (const Json &d : sh->items) {
            if (d.kind != Json::NUMBER || d.num < 0 || d.num > 1e15) return bad("bad shape of `" + m.first + "`");
            t.shape.push_back((uint64_t)d.num);
            if (d.num > 0 && t.elems > (uint64_t)1e15 / (uint64_t)d.num) return bad("bad shape of `" + m.first + "`");
            t.elems *= (uint64_t)d.num;
        }
        const double lo = off->items[0].num, hi = off->items[1].num;
        if (!(lo >= 0) || !(hi >= lo) || hi > (double)room || (uint64_t)hi - (uint64_t)lo != t.elems * width)
            return bad("bad offsets of `" + m.first + "`");
        t.data = base + 8 + hlen + (uint64_t)lo;
        f->tensors[m.first] = std::move(t);
    }
    return f;
}

}  // namespace jq
