// Models described by config.json + model.safetensors: a JSON reader, a safetensors reader, and the registry that turns an
// architecture name into a layer plan (include/xft_hip.h, "layer plans").  Plain C++, no HIP headers.
#pragma once
#include <cstdint>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "../../../include/xft_hip.h"

namespace xfthost {

// A parsed JSON value.  Lookups that do not fit (missing key, wrong type) print what was asked for and end the process, the
// way the other loaders treat a broken model directory; get() and has() are for optional keys.
class Json {
public:
    enum Kind { Null, Bool, Number, String, Array, Object };
    Kind kind = Null;
    bool flag = false;
    double number = 0;
    std::string text;
    std::vector<Json> items;
    std::map<std::string, Json> fields;

    static bool parse(const std::string &src, Json &out, std::string &error);
    bool has(const std::string &key) const; // present and not null
    const Json &at(const std::string &key) const;
    long integer(const std::string &key) const;
    double real(const std::string &key) const;
    const std::string &string(const std::string &key) const;
};

// One tensor of a safetensors file (8 bytes header length, the JSON header, the data)
struct TensorRef {
    std::string dtype;
    std::vector<long> shape;
    const unsigned char *data = nullptr;
    size_t bytes = 0;
    long count() const;
};

class SafeTensors {
public:
    ~SafeTensors();
    // maps the file; false: not readable or not such a file (error says why)
    bool open(const std::string &path, std::string &error);
    const TensorRef *find(const std::string &name) const;
    const std::map<std::string, TensorRef> &all() const { return tensors; }

private:
    void *base = nullptr;
    size_t length = 0;
    std::map<std::string, TensorRef> tensors;
};

struct PlanSpec {
    xfthip_plan_config cfg {};
    std::vector<xfthip_plan_layer> layers;
    std::vector<int> record; // of every layer of the model, where some have two mixers (empty: one record a layer)
};

// is there a config.json whose architecture this build knows; its name
bool plan_architecture(const std::string &dir, std::string &name);
// reads config.json and the tensors' shapes into a plan's description, then hands the tensors over; exits on a broken directory
xfthip_plan_t load_plan(const std::string &dir, PlanSpec &spec);

} // namespace xfthost
