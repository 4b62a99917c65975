// safetensors.cpp -- see safetensors.hpp.
#include "safetensors.hpp"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstring>

#include "json.hpp"

namespace bitnet_host {

SafeTensors::~SafeTensors() {
    if (map_) munmap(const_cast<uint8_t *>(map_), len_);
}

bool SafeTensors::open(const std::string &path, std::string &err) {
    const int fd = ::open(path.c_str(), O_RDONLY);
    struct stat st;
    if (fd < 0 || fstat(fd, &st) != 0 || st.st_size < 8) {
        if (fd >= 0) ::close(fd);
        err = path + ": cannot be read";
        return false;
    }
    len_ = (size_t)st.st_size;
    void *m = mmap(nullptr, len_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (m == MAP_FAILED) {
        err = path + ": cannot be mapped";
        return false;
    }
    map_ = static_cast<const uint8_t *>(m);
    uint64_t head = 0;
    for (int i = 7; i >= 0; --i) head = head << 8 | map_[i];
    if (head > len_ - 8) {
        err = path + ": header longer than the file";
        return false;
    }
    Json j;
    if (!Json::parse(reinterpret_cast<const char *>(map_ + 8), (size_t)head, j, err)) return false;
    const size_t data = 8 + (size_t)head, room = len_ - data;
    static const std::map<std::string, size_t> sizes = {{"BF16", 2}, {"F16", 2}, {"F32", 4}, {"I32", 4}, {"I64", 8}, {"F64", 8}, {"U8", 1}, {"I8", 1}};
    for (const auto &m2 : j.members) {
        if (m2.first == "__metadata__") continue;
        const Json *dt = m2.second.find("dtype"), *sh = m2.second.find("shape"), *off = m2.second.find("data_offsets");
        if (!dt || !sh || !off || off->items.size() != 2) {
            err = path + ": " + m2.first + ": incomplete entry";
            return false;
        }
        SafeTensor t;
        t.dtype = dt->str;
        uint64_t n = 1;
        for (const Json &d : sh->items) {
            if (d.num < 0 || d.num > 1e12 || (d.num > 0 && n > 1e15 / d.num)) {
                err = path + ": " + m2.first + ": bad shape";
                return false;
            }
            t.shape.push_back((uint64_t)d.num);
            n *= (uint64_t)d.num;
        }
        const double a = off->items[0].num, b = off->items[1].num;
        const auto es = sizes.find(t.dtype);
        if (a < 0 || b < a || b > (double)room || (es != sizes.end() && (uint64_t)(b - a) != n * es->second)) {
            err = path + ": " + m2.first + ": bad byte range";
            return false;
        }
        t.data = map_ + data + (size_t)a;
        t.bytes = (size_t)(b - a);
        tensors_[m2.first] = t;
    }
    return true;
}

const SafeTensor *SafeTensors::find(const std::string &name) const {
    const auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
}

static std::string shape_text(const std::vector<uint64_t> &s) {
    std::string t = "[";
    for (size_t i = 0; i < s.size(); ++i) t += (i ? ", " : "") + std::to_string(s[i]);
    return t + "]";
}

const uint16_t *SafeTensors::matrix(const std::string &name, size_t rows, size_t cols, std::string &err) const {
    const SafeTensor *t = find(name);
    if (!t || t->dtype != "BF16" || t->shape.size() != 2 || t->shape[0] != rows || t->shape[1] != cols) {
        err = name + ": expected BF16 [" + std::to_string(rows) + ", " + std::to_string(cols) + "], found " +
              (t ? t->dtype + " " + shape_text(t->shape) : std::string("nothing"));
        return nullptr;
    }
    return reinterpret_cast<const uint16_t *>(t->data);
}

bool SafeTensors::vector(const std::string &name, size_t n, std::vector<float> &out, std::string &err) const {
    const SafeTensor *t = find(name);
    if (!t || (t->dtype != "BF16" && t->dtype != "F32") || t->shape.size() != 1 || t->shape[0] != n) {
        err = name + ": expected BF16 or F32 [" + std::to_string(n) + "], found " + (t ? t->dtype + " " + shape_text(t->shape) : std::string("nothing"));
        return false;
    }
    out.resize(n);
    if (t->dtype == "F32") {
        memcpy(out.data(), t->data, n * 4);
    } else {
        for (size_t i = 0; i < n; ++i) {
            uint16_t h;
            memcpy(&h, t->data + 2 * i, 2);
            out[i] = bf16_value(h);
        }
    }
    return true;
}

}  // namespace bitnet_host
