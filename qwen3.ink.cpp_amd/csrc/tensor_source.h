// Where a model's tensors come from: a safetensors file, or seeded random numbers of the asked shapes.
#pragma once
#include <cstdint>
#include <memory>
#include <string>
#include <vector>

#include "decoder_session.h"

namespace a81w41 {

class TensorSource {
   public:
    virtual ~TensorSource() = default;
    // [rows][cols] as float; rows == 0: a vector of cols elements.
    virtual int matrix(const std::string& name, int rows, int cols, std::vector<float>& out) = 0;
    // [rows][cols] int32 with entries in 0 .. limit - 1.
    virtual int table(const std::string& name, int rows, int cols, int limit, std::vector<int>& out) = 0;
};

// The file is mapped, not read as a whole.
int open_safetensors(const std::string& file, std::unique_ptr<TensorSource>* out);
// Matrices of standard deviation cols^-1/2, vectors around 1, table rows of distinct entries.
std::unique_ptr<TensorSource> random_tensors(uint64_t seed);

}  // namespace a81w41
