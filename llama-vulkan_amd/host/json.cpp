#include "json.h"

#include <cmath>
#include <cstdlib>
#include <cstring>

namespace json {

const value *value::find(const std::string &key) const
{
    for (const auto &m : members_)
        if (m.first == key) return &m.second;
    return nullptr;
}

const value &value::at(const std::string &key) const
{
    const value *v = find(key);
    if (!v) throw error("no \"" + key + "\"");
    return *v;
}

double value::number() const
{
    if (kind_ != kind::number) throw error("not a number");
    return number_;
}

u64 value::integer() const
{
    const double v = number();
    if (!(v >= 0) || v > 9007199254740992.0 || v != std::floor(v)) throw error("not a whole number");
    return static_cast<u64>(v);
}

u32 value::size_value() const
{
    const u64 v = integer();
    if (v > 0xffffffffu) throw error("number out of range");
    return static_cast<u32>(v);
}

const std::string &value::text() const
{
    if (kind_ != kind::string) throw error("not a string");
    return text_;
}

const std::vector<value> &value::items() const
{
    if (kind_ != kind::array) throw error("not an array");
    return items_;
}

const std::vector<std::pair<std::string, value>> &value::members() const
{
    if (kind_ != kind::object) throw error("not an object");
    return members_;
}

class parser {
public:
    parser(const char *p, std::size_t n) : at_(p), end_(p + n) {}
    value document()
    {
        value v = element(0);
        space();
        if (at_ != end_) throw error("text after the end of the document");
        return v;
    }

private:
    const char *at_, *end_;

    void space()
    {
        while (at_ != end_ && (*at_ == ' ' || *at_ == '\t' || *at_ == '\n' || *at_ == '\r')) ++at_;
    }
    char peek()
    {
        space();
        if (at_ == end_) throw error("unexpected end of text");
        return *at_;
    }
    bool take(char c)
    {
        if (peek() != c) return false;
        ++at_;
        return true;
    }
    void expect(char c)
    {
        if (!take(c)) throw error(std::string("expected '") + c + "'");
    }
    void word(const char *w)
    {
        const std::size_t n = std::strlen(w);
        if (static_cast<std::size_t>(end_ - at_) < n || std::memcmp(at_, w, n) != 0) throw error("unknown word");
        at_ += n;
    }

    value element(int depth)
    {
        if (depth > 200) throw error("nested too deeply");
        value v;
        switch (peek()) {
        case '{':
            ++at_;
            v.kind_ = value::kind::object;
            if (take('}')) return v;
            do {
                if (peek() != '"') throw error("expected a key");
                std::string key = quoted();
                expect(':');
                v.members_.emplace_back(std::move(key), element(depth + 1));
            } while (take(','));
            expect('}');
            return v;
        case '[':
            ++at_;
            v.kind_ = value::kind::array;
            if (take(']')) return v;
            do v.items_.push_back(element(depth + 1));
            while (take(','));
            expect(']');
            return v;
        case '"':
            v.kind_ = value::kind::string;
            v.text_ = quoted();
            return v;
        case 't':
            word("true");
            v.kind_ = value::kind::boolean;
            v.bool_ = true;
            return v;
        case 'f':
            word("false");
            v.kind_ = value::kind::boolean;
            return v;
        case 'n':
            word("null");
            return v;
        default: return numeral();
        }
    }

    value numeral()
    {
        const char *from = at_;
        while (at_ != end_ && std::strchr("+-.0123456789eE", *at_) && *at_) ++at_;
        const std::string s(from, at_);
        char *stop = nullptr;
        value v;
        v.kind_ = value::kind::number;
        v.number_ = std::strtod(s.c_str(), &stop);
        if (s.empty() || *stop) throw error("malformed number");
        return v;
    }

    u32 hex4()
    {
        if (end_ - at_ < 4) throw error("malformed escape");
        u32 c = 0;
        for (int i = 0; i < 4; ++i, ++at_) {
            const char h = *at_;
            c = c * 16 + static_cast<u32>(h >= '0' && h <= '9' ? h - '0' : h >= 'a' && h <= 'f' ? h - 'a' + 10 : h >= 'A' && h <= 'F' ? h - 'A' + 10 : throw error("malformed escape"));
        }
        return c;
    }

    static void utf8(std::string &out, u32 c)
    {
        if (c < 0x80) out += static_cast<char>(c);
        else if (c < 0x800) {
            out += static_cast<char>(0xc0 | c >> 6);
            out += static_cast<char>(0x80 | (c & 0x3f));
        } else if (c < 0x10000) {
            out += static_cast<char>(0xe0 | c >> 12);
            out += static_cast<char>(0x80 | (c >> 6 & 0x3f));
            out += static_cast<char>(0x80 | (c & 0x3f));
        } else {
            out += static_cast<char>(0xf0 | c >> 18);
            out += static_cast<char>(0x80 | (c >> 12 & 0x3f));
            out += static_cast<char>(0x80 | (c >> 6 & 0x3f));
            out += static_cast<char>(0x80 | (c & 0x3f));
        }
    }

    std::string quoted()
    {
        std::string s;
        for (++at_;;) {
            if (at_ == end_) throw error("unterminated string");
            const char c = *at_++;
            if (c == '"') return s;
            if (c != '\\') {
                s += c;
                continue;
            }
            if (at_ == end_) throw error("unterminated string");
            switch (const char e = *at_++) {
            case '"': case '\\': case '/': s += e; break;
            case 'b': s += '\b'; break;
            case 'f': s += '\f'; break;
            case 'n': s += '\n'; break;
            case 'r': s += '\r'; break;
            case 't': s += '\t'; break;
            case 'u': {
                u32 c1 = hex4();
                if (c1 >= 0xd800 && c1 < 0xdc00 && end_ - at_ >= 6 && at_[0] == '\\' && at_[1] == 'u') {
                    at_ += 2;
                    c1 = 0x10000 + ((c1 - 0xd800) << 10) + ((hex4() - 0xdc00) & 0x3ff);
                }
                utf8(s, c1);
                break;
            }
            default: throw error("malformed escape");
            }
        }
    }
};

value parse(const char *begin, std::size_t size) { return parser(begin, size).document(); }

}  // namespace json
