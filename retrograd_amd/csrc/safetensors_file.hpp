// safetensors container access: a read-only mapping and a name -> tensor index. Layout: u64 little-endian length of a
// JSON object, the object (name -> dtype, shape, data_offsets relative to its end), then the payloads.
#pragma once

#include "json_schema.hpp"

#include <cstdint>
#include <cstring>
#include <stdexcept>
#include <string>
#include <unordered_map>
#include <vector>

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace retro {

struct StTensor {
    std::string name, dtype;
    std::vector<int64_t> shape;
    const uint8_t * data = nullptr;
    size_t nbytes = 0;
};

class SafetensorsFile {
public:
    explicit SafetensorsFile(const std::string & path) : path_(path) {
        fd_ = ::open(path.c_str(), O_RDONLY);
        if (fd_ < 0) throw std::runtime_error("cannot open " + path);
        struct stat st {};
        if (::fstat(fd_, &st) != 0 || st.st_size < 8) {
            ::close(fd_);
            throw std::runtime_error("cannot read " + path);
        }
        size_ = (size_t)st.st_size;
        void * p = ::mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd_, 0);
        if (p == MAP_FAILED) {
            ::close(fd_);
            throw std::runtime_error("cannot map " + path);
        }
        map_ = (const uint8_t *)p;
        try {
            read_all();
        } catch (...) {
            ::munmap((void *)map_, size_);
            ::close(fd_);
            throw;
        }
    }
    ~SafetensorsFile() {
        ::munmap((void *)map_, size_);
        ::close(fd_);
    }
    SafetensorsFile(const SafetensorsFile &) = delete;
    SafetensorsFile & operator=(const SafetensorsFile &) = delete;

    const StTensor * find(const std::string & name) const {
        auto it = by_name_.find(name);
        return it == by_name_.end() ? nullptr : &tensors_[it->second];
    }
    const StTensor & require(const std::string & name, const std::vector<int64_t> & shape) const {
        const StTensor * t = find(name);
        if (!t) throw std::runtime_error("model is missing tensor " + name);
        if (t->shape != shape) throw std::runtime_error("tensor " + name + " has an unexpected shape");
        return *t;
    }
    uint64_t tensor_bytes() const { return tensor_bytes_; }

private:
    static size_t elem_bytes(const std::string & dtype) {
        if (dtype == "F64" || dtype == "I64" || dtype == "U64") return 8;
        if (dtype == "F32" || dtype == "I32" || dtype == "U32") return 4;
        if (dtype == "BF16" || dtype == "F16" || dtype == "I16" || dtype == "U16") return 2;
        if (dtype == "BOOL" || dtype == "I8" || dtype == "U8" || dtype.compare(0, 2, "F8") == 0) return 1;
        throw std::runtime_error("unknown safetensors dtype " + dtype);
    }
    static int64_t whole(const JsonValue & v, const std::string & what) {
        if (v.kind != JsonValue::NUMBER || v.num < 0 || v.num > 9e15 || v.num != (double)(int64_t)v.num) throw std::runtime_error(what + " must be a whole number");
        return (int64_t)v.num;
    }
    void read_all() {
        uint64_t n = 0;
        std::memcpy(&n, map_, 8);
        if (n > size_ - 8) throw std::runtime_error(path_ + ": the safetensors header runs past the file");
        const JsonValue head = JsonParser::parse(std::string((const char *)map_ + 8, (size_t)n));
        if (head.kind != JsonValue::OBJECT) throw std::runtime_error(path_ + ": the safetensors header is no JSON object");
        const uint8_t * data0 = map_ + 8 + n;
        const size_t room = size_ - 8 - (size_t)n;
        for (const auto & m : head.members) {
            if (m.first == "__metadata__") continue;
            const JsonValue * dt = m.second.get("dtype"), * sh = m.second.get("shape"), * off = m.second.get("data_offsets");
            if (!dt || !sh || !off || off->items.size() != 2) throw std::runtime_error("tensor " + m.first + " is described incompletely");
            StTensor t;
            t.name = m.first;
            t.dtype = dt->text;
            size_t elems = 1;
            for (const JsonValue & d : sh->items) {
                t.shape.push_back(whole(d, "a dimension of tensor " + m.first));
                if (t.shape.back() != 0 && elems > ((size_t)1 << 46) / (size_t)t.shape.back()) throw std::runtime_error("tensor " + t.name + " is larger than any file");
                elems *= (size_t)t.shape.back();
            }
            const size_t lo = (size_t)whole(off->items[0], "an offset of tensor " + m.first), hi = (size_t)whole(off->items[1], "an offset of tensor " + m.first);
            if (lo > hi || hi > room) throw std::runtime_error("tensor " + t.name + " runs past the file");
            t.nbytes = hi - lo;
            if (t.nbytes != elems * elem_bytes(t.dtype)) throw std::runtime_error("tensor " + t.name + " has an unexpected size");
            t.data = data0 + lo;
            tensor_bytes_ += t.nbytes;
            by_name_[t.name] = tensors_.size();
            tensors_.push_back(std::move(t));
        }
    }

    std::string path_;
    int fd_ = -1;
    size_t size_ = 0;
    const uint8_t * map_ = nullptr;
    std::vector<StTensor> tensors_;
    std::unordered_map<std::string, size_t> by_name_;
    uint64_t tensor_bytes_ = 0;
};

}  // namespace retro
