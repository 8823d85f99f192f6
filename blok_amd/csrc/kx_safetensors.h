// kx_safetensors.h -- the tensors of the safetensors files of a directory, as records the loader takes (kx_load.h).
#pragma once
#include <string>
#include <unordered_map>
#include "kx_index.h"

// name -> record; dtype "bf16", "f32" or "i32", shape "4096x1024"
typedef std::unordered_map<std::string, KxTensorRec> KxTensorMap;
// A file is an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets) and the data.
int kx_safetensors_scan(const std::string &dir, KxTensorMap &out);
