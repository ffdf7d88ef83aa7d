// Model folders: config.json and model.safetensors (a 64-bit length and a JSON header of that size, naming
// each tensor's dtype, shape and byte range, then the data).  Host code only; the file stays mapped while a session
// uploads from it.
#include "model_folder.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cerrno>
#include <cstring>

RmiSafetensors::~RmiSafetensors() {
    if (map_) munmap(map_, bytes_);
}

bool RmiSafetensors::open(const char *path) {
    const int fd = ::open(path, O_RDONLY | O_CLOEXEC);
    if (fd < 0) {
        rmi_set_error("%s: %s", path, strerror(errno));
        return false;
    }
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) {
        rmi_set_error("%s: too short for a safetensors file", path);
        close(fd);
        return false;
    }
    bytes_ = size_t(st.st_size);
    void *m = mmap(nullptr, bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (m == MAP_FAILED) {
        rmi_set_error("%s: mmap: %s", path, strerror(errno));
        return false;
    }
    map_ = m;
    const uint8_t *base = static_cast<const uint8_t *>(m);
    uint64_t head = 0;
    memcpy(&head, base, 8);
    if (head > bytes_ - 8) {
        rmi_set_error("%s: the header runs past the end of the file", path);
        return false;
    }
    RmiJson j;
    std::string why;
    if (!RmiJson::parse(reinterpret_cast<const char *>(base + 8), size_t(head), &j, &why) || j.type != RmiJson::kObject) {
        rmi_set_error("%s: bad header: %s", path, why.empty() ? "not an object" : why.c_str());
        return false;
    }
    const uint64_t room = bytes_ - 8 - head;
    for (const auto &m2 : j.members) {
        if (m2.first == "__metadata__") continue;
        const RmiJson *dt = m2.second.get("dtype"), *sh = m2.second.get("shape"), *off = m2.second.get("data_offsets");
        RmiTensor t;
        bool ok = dt && sh && off && sh->type == RmiJson::kArray && off->items.size() == 2;
        uint64_t elem = 0;
        if (ok) {
            const std::string &d = dt->text;
            t.dtype = d == "BF16" ? RmiTensor::kBf16 : d == "F16" ? RmiTensor::kF16 : d == "F32" ? RmiTensor::kF32
                      : d == "I32" ? RmiTensor::kI32 : RmiTensor::kOther;
            elem = t.dtype == RmiTensor::kBf16 || t.dtype == RmiTensor::kF16 ? 2 : t.dtype == RmiTensor::kOther ? 0 : 4;
            t.count = 1;
            for (const RmiJson &s : sh->items) {
                ok = ok && s.type == RmiJson::kNumber && s.number >= 0 && s.number < 9e15;
                t.shape.push_back(ok ? uint64_t(s.number) : 0);
                ok = ok && !__builtin_mul_overflow(t.count, t.shape.back(), &t.count);
            }
            const double b = off->items[0].number, e = off->items[1].number;
            uint64_t want = 0;
            ok = ok && b >= 0 && e >= b && e <= double(room) && !__builtin_mul_overflow(t.count, elem, &want) &&
                 (elem == 0 || uint64_t(e) - uint64_t(b) == want);
            if (ok) t.data = base + 8 + head + uint64_t(b);
        }
        if (!ok) {
            rmi_set_error("%s: bad entry for tensor %s", path, m2.first.c_str());
            return false;
        }
        tensors_.emplace(m2.first, std::move(t));
    }
    return true;
}

const RmiTensor *RmiSafetensors::find(const std::string &name) const {
    const auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
}

bool rmi_read_config(const char *dir, RmiJson *out) {
    const std::string path = std::string(dir) + "/config.json";
    FILE *f = fopen(path.c_str(), "rb");
    if (!f) {
        rmi_set_error("%s: %s", path.c_str(), strerror(errno));
        return false;
    }
    std::string text;
    char buf[65536];
    for (size_t n; (n = fread(buf, 1, sizeof buf, f)) > 0;) text.append(buf, n);
    fclose(f);
    std::string why;
    if (!RmiJson::parse(text.data(), text.size(), out, &why) || out->type != RmiJson::kObject) {
        rmi_set_error("%s: %s", path.c_str(), why.empty() ? "not an object" : why.c_str());
        return false;
    }
    return true;
}

bool RmiModelFolder::open(const char *dir) {
    return rmi_read_config(dir, &config) && tensors.open((std::string(dir) + "/model.safetensors").c_str());
}

float rmi_tensor_f32(const RmiTensor &t, uint64_t i) {
    uint16_t h;
    float f;
    switch (t.dtype) {
        case RmiTensor::kBf16: {
            memcpy(&h, t.data + 2 * i, 2);
            const uint32_t b = uint32_t(h) << 16;
            memcpy(&f, &b, 4);
            return f;
        }
        case RmiTensor::kF16: {
            memcpy(&h, t.data + 2 * i, 2);
            _Float16 x;
            memcpy(&x, &h, 2);
            return float(x);
        }
        case RmiTensor::kF32: memcpy(&f, t.data + 4 * i, 4); return f;
        default: return 0.0f;
    }
}

void rmi_tensor_bf16(const RmiTensor &t, uint64_t at, uint64_t n, uint16_t *dst) {
    if (t.dtype == RmiTensor::kBf16) {
        memcpy(dst, t.data + 2 * at, 2 * n);
        return;
    }
    for (uint64_t i = 0; i < n; i++) {
        const float v = rmi_tensor_f32(t, at + i);
        uint32_t b;
        memcpy(&b, &v, 4);
        dst[i] = uint16_t((b + 0x7fff + ((b >> 16) & 1)) >> 16);
    }
}

extern "C" int64_t rmi_hip_model_folder_architecture(const char *dir, char *buf, size_t cap) {
    RmiJson c;
    if (!dir || !rmi_read_config(dir, &c)) return -1;
    const RmiJson *a = c.get("architecture");
    if (!a || a->type != RmiJson::kString) {
        rmi_set_error("%s: config.json names no architecture", dir);
        return -1;
    }
    if (buf && cap) snprintf(buf, cap, "%s", a->text.c_str());
    return int64_t(a->text.size());
}
