// json.h — a reader for the JSON this program meets: model configurations, safetensors headers, trace steps.
#pragma once

#include <cstddef>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

#include "types.h"

namespace json {

// malformed text, or a value that is absent or of another kind than asked for
struct error : std::runtime_error {
    using std::runtime_error::runtime_error;
};

class value {
public:
    enum class kind { null, boolean, number, string, array, object };

    [[nodiscard]] kind type() const { return kind_; }
    [[nodiscard]] bool is_null() const { return kind_ == kind::null; }
    [[nodiscard]] bool has(const std::string &key) const { return find(key) != nullptr; }
    [[nodiscard]] const value *find(const std::string &key) const;      // null when absent (or not an object)
    [[nodiscard]] const value &at(const std::string &key) const;
    [[nodiscard]] double number() const;
    [[nodiscard]] u64 integer() const;          // a whole number that is not negative
    [[nodiscard]] u32 size_value() const;       // the same, fitting 32 bits
    [[nodiscard]] const std::string &text() const;
    [[nodiscard]] const std::vector<value> &items() const;
    [[nodiscard]] const std::vector<std::pair<std::string, value>> &members() const;

private:
    friend class parser;
    kind kind_ = kind::null;
    bool bool_ = false;
    double number_ = 0;
    std::string text_;
    std::vector<value> items_;
    std::vector<std::pair<std::string, value>> members_;
};

value parse(const char *begin, std::size_t size);
inline value parse(const std::string &s) { return parse(s.data(), s.size()); }

}  // namespace json
