// Safetensors reader (fh_safetensors.h) and its entry point for one tensor directory.
#include "fh_safetensors.h"
#include "fh_json.h"

#include <cerrno>
#include <cstdio>
#include <cstring>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

FhSafetensors::~FhSafetensors() {
    if (map) (void)munmap(map, map_len);
}

fh_status fh_read_file(const char *path, std::string &out) {
    FILE *f = fopen(path, "rb");
    if (!f) FH_FAIL(FH_ERR_IO, "%s: %s", path, strerror(errno));
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0) out.append(buf, n);
    const bool bad = ferror(f) != 0;
    fclose(f);
    if (bad) FH_FAIL(FH_ERR_IO, "%s: read error", path);
    return FH_OK;
}

fh_status FhSafetensors::open(const char *path) {
    const int fd = ::open(path, O_RDONLY | O_CLOEXEC);
    if (fd < 0) FH_FAIL(FH_ERR_IO, "%s: %s", path, strerror(errno));
    struct stat sb;
    if (fstat(fd, &sb) != 0 || sb.st_size < 8) {
        ::close(fd);
        FH_FAIL(FH_ERR_IO, "%s: not a safetensors file", path);
    }
    map_len = (size_t)sb.st_size;
    map = mmap(nullptr, map_len, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (map == MAP_FAILED) {
        map = nullptr;
        FH_FAIL(FH_ERR_IO, "%s: mmap failed: %s", path, strerror(errno));
    }
    uint64_t hl;
    memcpy(&hl, map, 8);
    FH_REQUIRE(hl <= map_len - 8, "%s: header of %llu bytes in a file of %zu", path, (unsigned long long)hl, map_len);
    const char *text = (const char *)map + 8;
    const uint8_t *data = (const uint8_t *)map + 8 + hl;
    const size_t data_len = map_len - 8 - (size_t)hl;
    FhJson j;
    std::string err;
    if (!FhJson::parse(text, (size_t)hl, j, err)) FH_FAIL(FH_ERR_INVALID, "%s: header: %s", path, err.c_str());
    FH_REQUIRE(j.is_object(), "%s: header is not an object", path);
    for (auto &m : j.members) {
        if (m.first == "__metadata__") continue;
        const FhJson *dt = m.second.find("dtype"), *sh = m.second.find("shape"), *of = m.second.find("data_offsets");
        FH_REQUIRE(dt && dt->is_string() && sh && sh->is_array() && of && of->is_array() && of->items.size() == 2,
                   "%s: tensor %s has no dtype, shape or data_offsets", path, m.first.c_str());
        Entry e;
        e.name = m.first;
        e.dtype = dt->str;
        size_t width = 0;
        if (e.dtype == "F32") e.ggml_type = FH_W_F32, width = 4;
        else if (e.dtype == "F16") e.ggml_type = FH_W_F16, width = 2;
        else if (e.dtype == "BF16") e.ggml_type = FH_BF16, width = 2;
        else if (e.dtype == "I32") e.ggml_type = FH_GGML_I32, width = 4;
        double count = 1;
        for (auto &d : sh->items) {
            FH_REQUIRE(d.is_number() && d.num >= 0 && d.num < 2147483648.0 && d.num == std::floor(d.num), "%s: tensor %s: bad shape",
                       path, e.name.c_str());
            e.shape.push_back((int64_t)d.num);
            count *= d.num;
        }
        const double a = of->items[0].num, b = of->items[1].num;
        FH_REQUIRE(a >= 0 && b >= a && b <= (double)data_len, "%s: tensor %s lies outside the file", path, e.name.c_str());
        e.data = data + (size_t)a;
        e.bytes = (size_t)(b - a);
        FH_REQUIRE(e.ggml_type < 0 || count * (double)width == b - a, "%s: tensor %s: %zu bytes do not fit its shape", path,
                   e.name.c_str(), e.bytes);
        entries.push_back(std::move(e));
    }
    return FH_OK;
}
