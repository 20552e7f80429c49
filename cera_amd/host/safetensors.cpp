#include "safetensors.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstring>

#include "json.h"

namespace cera {
namespace {

uint64_t dtype_bytes(const std::string& d) {
    if (d == "BF16" || d == "F16" || d == "I16" || d == "U16") return 2;
    if (d == "F32" || d == "I32" || d == "U32") return 4;
    if (d == "F64" || d == "I64" || d == "U64") return 8;
    if (d == "I8" || d == "U8" || d == "BOOL") return 1;
    return 0;
}

}  // namespace

std::unique_ptr<SafeTensors> SafeTensors::open(const std::string& path, std::string* err) {
    auto fail = [&](const std::string& m) {
        if (err) *err = path + ": " + m;
        return nullptr;
    };
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return fail(std::strerror(errno));
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) {
        ::close(fd);
        return fail("not a safetensors file");
    }
    std::unique_ptr<SafeTensors> f(new SafeTensors());
    f->size_ = static_cast<uint64_t>(st.st_size);
    f->map_ = mmap(nullptr, f->size_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (f->map_ == MAP_FAILED) {
        f->map_ = nullptr;
        return fail("mmap failed");
    }
    const unsigned char* base = static_cast<const unsigned char*>(f->map_);
    uint64_t n = 0;
    for (int i = 7; i >= 0; --i) n = (n << 8) | base[i];
    if (n > f->size_ - 8) return fail("header length beyond the file");
    Json h;
    std::string e;
    if (!Json::parse(std::string_view(reinterpret_cast<const char*>(base) + 8, n), &h, &e)) return fail(e);
    if (h.type != Json::Object) return fail("header is not an object");
    const uint64_t data = 8 + n, room = f->size_ - data;
    for (const auto& kv : h.obj) {
        if (kv.first == "__metadata__") continue;
        const Json *dt = kv.second.find("dtype"), *sh = kv.second.find("shape"), *of = kv.second.find("data_offsets");
        if (!dt || dt->type != Json::String || !sh || sh->type != Json::Array || !of || of->type != Json::Array || of->arr.size() != 2)
            return fail("tensor " + kv.first + ": incomplete entry");
        SafeTensor t;
        t.dtype = dt->str;
        const uint64_t esz = dtype_bytes(t.dtype);
        if (!esz) return fail("tensor " + kv.first + ": unknown dtype " + t.dtype);
        uint64_t elems = 1;
        for (const Json& d : sh->arr) {
            if (!d.is_int || d.integer < 0 || (d.integer && elems > UINT64_MAX / 16 / static_cast<uint64_t>(d.integer)))
                return fail("tensor " + kv.first + ": bad shape");
            t.shape.push_back(static_cast<uint64_t>(d.integer));
            elems *= static_cast<uint64_t>(d.integer);
        }
        const Json &b = of->arr[0], &en = of->arr[1];
        if (!b.is_int || !en.is_int || b.integer < 0 || en.integer < b.integer || static_cast<uint64_t>(en.integer) > room)
            return fail("tensor " + kv.first + ": offsets outside the file");
        t.nbytes = static_cast<uint64_t>(en.integer - b.integer);
        if (t.nbytes != elems * esz) return fail("tensor " + kv.first + ": byte count does not fit its shape");
        t.data = base + data + b.integer;
        f->tensors_[kv.first] = std::move(t);
    }
    return f;
}

SafeTensors::~SafeTensors() {
    if (map_) munmap(map_, size_);
}

const SafeTensor* SafeTensors::find(const std::string& name) const {
    auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
}

}  // namespace cera
