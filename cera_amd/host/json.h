// A small JSON reader (RFC 8259): whole documents in memory, numbers as double plus their exact
// integer where they are one.
#pragma once
#include <cstdint>
#include <string>
#include <string_view>
#include <utility>
#include <vector>

namespace cera {

class Json {
public:
    enum Type { Null, Bool, Number, String, Array, Object };
    Type type = Null;
    bool b = false;
    double num = 0.0;
    int64_t integer = 0;      // Number: valid when is_int
    bool is_int = false;
    std::string str;
    std::vector<Json> arr;
    std::vector<std::pair<std::string, Json>> obj;   // in document order

    // false + *err (with the byte offset) on malformed input; trailing non-space is an error
    static bool parse(std::string_view text, Json* out, std::string* err);
    const Json* find(const std::string& key) const;   // nullptr: not an object, or no such key
    bool is_null() const { return type == Null; }
};

}  // namespace cera
