// Tensor sources: the safetensors reader (8-byte little-endian header length, a JSON header of name -> dtype, shape,
// data_offsets, then the data) and the random one.
#include "tensor_source.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <cstring>

#include "json.h"

namespace a81w41 {
namespace {

class Safetensors : public TensorSource {
   public:
    ~Safetensors() override {
        if (map_) munmap(const_cast<uint8_t*>(map_), size_);
    }
    int open(const std::string& file) {
        const int fd = ::open(file.c_str(), O_RDONLY | O_CLOEXEC);
        if (fd < 0) return failf(A81W41_ERR_IO, "cannot open %s", file.c_str());
        struct stat st {};
        void* p = MAP_FAILED;
        if (fstat(fd, &st) == 0 && st.st_size >= 8) p = mmap(nullptr, (size_t)st.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
        ::close(fd);
        if (p == MAP_FAILED) return failf(A81W41_ERR_IO, "cannot read %s", file.c_str());
        map_ = static_cast<const uint8_t*>(p);
        size_ = (size_t)st.st_size;
        uint64_t n = 0;
        for (int i = 7; i >= 0; i--) n = n << 8 | map_[i];
        if (n > size_ - 8) return failf(A81W41_ERR_IO, "%s: the header is longer than the file", file.c_str());
        data_ = map_ + 8 + n;
        data_bytes_ = size_ - 8 - n;
        try {
            header_ = Json::parse(std::string(reinterpret_cast<const char*>(map_ + 8), n));
            (void)header_.object();
        } catch (const std::exception& e) {
            return failf(A81W41_ERR_IO, "%s: %s", file.c_str(), e.what());
        }
        return 0;
    }
    int matrix(const std::string& name, int rows, int cols, std::vector<float>& out) override {
        std::string type;
        const uint8_t* p = nullptr;
        A81W41_TRY(find(name, rows, cols, &type, &p));
        const size_t n = (size_t)(rows ? rows : 1) * cols;
        out.resize(n);
        if (type == "BF16") {
            for (size_t i = 0; i < n; i++) {
                uint16_t h;
                memcpy(&h, p + 2 * i, 2);
                const uint32_t u = (uint32_t)h << 16;
                memcpy(&out[i], &u, 4);
            }
        } else if (type == "F32") {
            memcpy(out.data(), p, 4 * n);
        } else {
            return failf(A81W41_ERR_IO, "tensor '%s' has type %s, BF16 or F32 is expected", name.c_str(), type.c_str());
        }
        return 0;
    }
    int table(const std::string& name, int rows, int cols, int limit, std::vector<int>& out) override {
        std::string type;
        const uint8_t* p = nullptr;
        A81W41_TRY(find(name, rows, cols, &type, &p));
        if (type != "I32") return failf(A81W41_ERR_IO, "tensor '%s' has type %s, I32 is expected", name.c_str(), type.c_str());
        out.resize((size_t)rows * cols);
        memcpy(out.data(), p, 4 * out.size());
        for (int v : out)
            if (v < 0 || v >= limit) return failf(A81W41_ERR_IO, "tensor '%s' holds %d, outside 0 .. %d", name.c_str(), v, limit - 1);
        return 0;
    }

   private:
    int find(const std::string& name, int rows, int cols, std::string* type, const uint8_t** p) {
        if (!header_.has(name)) return failf(A81W41_ERR_IO, "no tensor '%s'", name.c_str());
        try {
            const Json& t = header_.at(name);
            *type = t.at("dtype").string();
            const auto& shape = t.at("shape").array();
            const bool fits = rows ? shape.size() == 2 && shape[0].integer() == rows && shape[1].integer() == cols
                                   : shape.size() == 1 && shape[0].integer() == cols;
            if (!fits) return failf(A81W41_ERR_IO, "tensor '%s' is not of shape [%d, %d]", name.c_str(), rows, cols);
            const auto& off = t.at("data_offsets").array();
            const long long a = off.at(0).integer(), b = off.at(1).integer();
            const size_t bytes = (size_t)(rows ? rows : 1) * cols * (*type == "BF16" ? 2 : 4);
            if (a < 0 || b < a || (size_t)b > data_bytes_ || (size_t)(b - a) != bytes)
                return failf(A81W41_ERR_IO, "tensor '%s' lies outside the file", name.c_str());
            *p = data_ + a;
        } catch (const std::exception& e) {
            return failf(A81W41_ERR_IO, "tensor '%s': %s", name.c_str(), e.what());
        }
        return 0;
    }
    const uint8_t *map_ = nullptr, *data_ = nullptr;
    size_t size_ = 0, data_bytes_ = 0;
    Json header_;
};

class RandomTensors : public TensorSource {
   public:
    explicit RandomTensors(uint64_t seed) : state_(seed * 0x9E3779B97F4A7C15ull + 0x1234567ull) {}
    int matrix(const std::string&, int rows, int cols, std::vector<float>& out) override {
        out.resize((size_t)(rows ? rows : 1) * cols);
        // uniform on +-sqrt(3) has standard deviation 1
        const float a = (rows ? 1.0f / std::sqrt((float)cols) : 0.2f) * 1.7320508f, b = rows ? 0.f : 1.f;
        for (float& v : out) v = b + a * ((float)(int32_t)(next() >> 32) * (1.0f / 2147483648.0f));
        return 0;
    }
    int table(const std::string&, int rows, int cols, int limit, std::vector<int>& out) override {
        out.resize((size_t)rows * cols);
        for (int r = 0; r < rows; r++) {
            const int first = (int)(next() >> 33) % limit;
            for (int c = 0; c < cols; c++) out[(size_t)r * cols + c] = (first + c) % limit;
        }
        return 0;
    }

   private:
    uint64_t next() {
        state_ = state_ * 6364136223846793005ull + 1442695040888963407ull;
        return state_;
    }
    uint64_t state_;
};

}  // namespace

int open_safetensors(const std::string& file, std::unique_ptr<TensorSource>* out) {
    auto t = std::make_unique<Safetensors>();
    A81W41_TRY(t->open(file));
    *out = std::move(t);
    return 0;
}

std::unique_ptr<TensorSource> random_tensors(uint64_t seed) { return std::make_unique<RandomTensors>(seed); }

}  // namespace a81w41
