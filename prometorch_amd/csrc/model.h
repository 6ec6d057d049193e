// A loaded model: what it was read from, its device allocations and its decoder.  Shared by the loaders.
#pragma once
#include "ptm_common.h"

#include <list>
#include <vector>

struct ptm_model {
    ptm_gguf* file = nullptr;
    std::vector<void*> device_allocs;
    std::vector<ptm_layer> layers;
    std::vector<ptm_block> blocks;
    std::list<std::vector<float>> host_vectors;  // small arrays the blocks point to
    ptm_decode_config cfg{};
    ptm_decoder* dec = nullptr;
};

namespace ptm {
// device copy of `bytes` host bytes (src NULL: zeros), owned by the model
int model_upload(ptm_model* m, const void* src, size_t bytes, void** dev);
}
