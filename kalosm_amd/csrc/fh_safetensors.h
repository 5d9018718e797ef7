// Safetensors files (host code): eight bytes little-endian header length, a JSON header name -> dtype, shape,
// data_offsets, then the tensors.  The file is mapped read-only; tensors are pointers into the mapping.
#pragma once
#include "fh_internal.h"

#include <string>
#include <vector>

struct FhSafetensors {
    struct Entry {
        std::string name, dtype;
        int ggml_type = -1; // F32, F16, BF16, I32; -1: another type
        std::vector<int64_t> shape;
        const void *data = nullptr;
        size_t bytes = 0;
    };
    std::vector<Entry> entries; // in header order

    FhSafetensors() = default;
    FhSafetensors(const FhSafetensors &) = delete;
    ~FhSafetensors();
    fh_status open(const char *path);

  private:
    void *map = nullptr;
    size_t map_len = 0;
};

struct fh_decoder;
fh_status fh_decoder_load_safetensors(fh_decoder *m, const char *path);
fh_status fh_read_file(const char *path, std::string &out);
