/*
 * tk_safetensors.h — reader of safetensors files (an 8-byte little-endian header length, a JSON header name -> {dtype, shape,
 * data_offsets}, the data), memory-mapped.  Host only.
 */
#ifndef TK_SAFETENSORS_H
#define TK_SAFETENSORS_H

#include <stddef.h>
#include <stdint.h>

#include <map>
#include <string>
#include <vector>

struct TkSafeTensor {
    std::string dtype;            /* "BF16", "F32", ... */
    std::vector<int64_t> shape;
    const uint8_t* data = nullptr; /* into the mapping */
    size_t nbytes = 0;
    int64_t dim(size_t i) const { return i < shape.size() ? shape[i] : 1; }
    int64_t elems() const { int64_t n = 1; for (int64_t d : shape) n *= d; return n; }
};

class TkSafetensorsFile {
public:
    ~TkSafetensorsFile();
    bool open(const std::string& path);
    const TkSafeTensor* find(const std::string& name) const;
    std::map<std::string, TkSafeTensor> tensors;
    std::string error;

private:
    void* map_ = nullptr;
    size_t size_ = 0;
};

#endif
