// A small bounded JSON reader for model folders: config.json and the header of a safetensors file.
#pragma once

#include <cstdint>
#include <map>
#include <string>
#include <vector>

namespace mesh {

struct JsonValue {
    enum Kind { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } kind = NUL;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<JsonValue> items;
    std::map<std::string, JsonValue> fields;

    bool is_null() const { return kind == NUL; }
    // member of an object, nullptr if absent or not an object
    const JsonValue *get(const char *name) const;
    // a non-negative whole number up to `max`
    bool as_count(uint64_t max, uint64_t &out) const;
};

// The whole text is one value.  false: malformed (what and where in `err`), nested deeper than 64, or trailing text.
bool json_parse(const char *text, size_t n, JsonValue &out, std::string &err);

}  // namespace mesh
