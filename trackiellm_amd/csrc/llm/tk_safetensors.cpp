#include "tk_safetensors.h"

#include <fcntl.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include "../common/tk_json.h"

using namespace tk_json;

TkSafetensorsFile::~TkSafetensorsFile() {
    if (map_) (void)munmap(map_, size_);
}

const TkSafeTensor* TkSafetensorsFile::find(const std::string& name) const {
    auto it = tensors.find(name);
    return it == tensors.end() ? nullptr : &it->second;
}

static size_t dtype_bytes(const std::string& d) {
    if (d == "BF16" || d == "F16" || d == "I16" || d == "U16") return 2;
    if (d == "F32" || d == "I32" || d == "U32") return 4;
    if (d == "F64" || d == "I64" || d == "U64") return 8;
    if (d == "I8" || d == "U8" || d == "BOOL" || d == "F8_E4M3" || d == "F8_E5M2") return 1;
    return 0;
}

bool TkSafetensorsFile::open(const std::string& path) {
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) { error = "cannot open " + path; return false; }
    struct stat st;
    if (fstat(fd, &st) != 0 || !S_ISREG(st.st_mode) || st.st_size < 8) { ::close(fd); error = path + " is not a safetensors file"; return false; }
    size_ = (size_t)st.st_size;
    map_ = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (map_ == MAP_FAILED) { map_ = nullptr; error = "cannot map " + path; return false; }
    const uint8_t* p = (const uint8_t*)map_;
    uint64_t hlen = 0;
    for (int i = 7; i >= 0; --i) hlen = hlen << 8 | p[i];
    if (hlen > size_ - 8) { error = path + ": header length is outside the file"; return false; }
    JVal root;
    JParser ps{(const char*)p + 8, (const char*)p + 8 + hlen};
    if (!ps.value(&root) || root.kind != JVal::JOBJ) { error = path + ": header is not a JSON object"; return false; }
    const uint8_t* base = p + 8 + hlen;
    const double room = (double)(size_ - 8 - hlen);
    for (const auto& kv : root.obj) {
        if (kv.first == "__metadata__") continue;
        const JVal *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *of = kv.second.get("data_offsets");
        auto bad = [&](const char* why) { error = path + ": tensor " + kv.first + ": " + why; return false; };
        if (!dt || dt->kind != JVal::JSTR || !sh || sh->kind != JVal::JARR || !of || of->kind != JVal::JARR || of->arr.size() != 2) return bad("incomplete entry");
        TkSafeTensor t;
        t.dtype = dt->str;
        double n = 1.0;
        for (const JVal& d : sh->arr) {
            if (d.kind != JVal::JNUM || d.num < 0 || d.num > 1e15) return bad("bad shape");
            t.shape.push_back((int64_t)d.num);
            n *= d.num;
        }
        const double a = of->arr[0].num, b = of->arr[1].num;
        if (of->arr[0].kind != JVal::JNUM || of->arr[1].kind != JVal::JNUM || !(a >= 0) || !(b >= a) || b > room) return bad("data outside the file");
        const size_t eb = dtype_bytes(t.dtype);
        if (!eb || n * (double)eb != b - a) return bad("size does not fit its shape");
        t.data = base + (size_t)a;
        t.nbytes = (size_t)(b - a);
        tensors[kv.first] = std::move(t);
    }
    return true;
}
