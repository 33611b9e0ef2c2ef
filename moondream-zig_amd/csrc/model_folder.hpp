// A model folder: config.json and model.safetensors.  Host code only.
#pragma once
#include <cstdint>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "json_value.hpp"
#include "layer_list.hpp"

// safetensors: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets), the data.
struct StTensor {
    std::string dtype;
    std::vector<size_t> shape;
    const unsigned char *data = nullptr; // into the mapping; may be odd
    size_t bytes = 0;
};
struct SafeTensors {
    ~SafeTensors();
    int open(const std::string &path, std::string *err); // a MOON_* status
    const StTensor *find(const std::string &name) const;
    std::map<std::string, StTensor> tensors;

  private:
    void *map = nullptr;
    size_t size = 0;
};

// A design of the registry: how its config.json describes layers and what its tensors are called.
struct TensorNames {
    std::string (*embed)(), (*head)(), (*final_norm)();
    std::string (*norm)(size_t layer);
    std::string (*mixer)(size_t layer, const char *what);            // q k v o g sink vmix q.norm k.norm temp; see also below
    std::string (*ff)(size_t layer, const char *what);               // gate up down router correction
    std::string (*expert)(size_t layer, size_t e, const char *what); // gate up down
    const char *bias_suffix;                                         // of a norm's bias
    // where a mixer has a delta rule beside the attention: what comes before the names of each (the delta rule's are q k v, each with
    // .conv, b A_log a1 a2 dt_bias g1 g2 norm o; out is the norm of each one's output)
    const char *attention_part = "", *delta_part = "";
};
struct Design {
    const char *name; // config.json "architecture"
    bool (*parse)(const Json &config, LayerListSpec *spec, std::string *err);
    TensorNames names;
};
const Design *find_design(const std::string &architecture);
std::string known_designs();

// config.json text -> design and description
int parse_model_config(const char *text, size_t len, const Design **design, LayerListSpec *spec, std::string *err);
// the whole folder: config.json parsed, the tensor file mapped and checked against it (a MOON_* status)
int read_model_folder(const std::string &dir, const Design **design, LayerListSpec *spec, SafeTensors *file, std::string *err);
