#include "safetensors.h"

#include <cerrno>
#include <cstring>
#include <exception>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include "json.h"

safetensors_file::safetensors_file(const std::string &path)
{
    const int fd = ::open(path.c_str(), O_RDONLY);
    struct stat st{};
    if (fd < 0 || fstat(fd, &st) < 0) {
        problem = "Cannot open " + path + ": " + std::strerror(errno);
        if (fd >= 0) ::close(fd);
        return;
    }
    mapping_size = static_cast<std::size_t>(st.st_size);
    void *m = mapping_size ? mmap(nullptr, mapping_size, PROT_READ, MAP_SHARED, fd, 0) : MAP_FAILED;
    ::close(fd);
    if (m == MAP_FAILED) {
        mapping_size = 0;
        problem = "Cannot map " + path;
        return;
    }
    mapping = static_cast<u8 *>(m);
    try {
        parse();
    } catch (const std::exception &e) {
        problem = "Malformed " + path + ": " + e.what();
        table.clear();
    }
}

safetensors_file::~safetensors_file()
{
    if (mapping) munmap(mapping, mapping_size);
}

void safetensors_file::parse()
{
    u64 header = 0;
    if (mapping_size < 8) throw json::error("shorter than its header");
    for (int i = 7; i >= 0; --i) header = header << 8 | mapping[i];
    if (header > mapping_size - 8) throw json::error("header length exceeds the file");
    const u64 base = 8 + header, room = mapping_size - base;
    const json::value doc = json::parse(reinterpret_cast<const char *>(mapping) + 8, header);
    for (const auto &m : doc.members()) {
        if (m.first == "__metadata__") continue;
        safetensors_entry e;
        e.name = m.first;
        e.dtype = m.second.at("dtype").text();
        for (const json::value &v : m.second.at("shape").items()) e.shape.push_back(v.integer());
        const auto &off = m.second.at("data_offsets").items();
        if (off.size() != 2) throw json::error("data_offsets of " + e.name);
        const u64 lo = off[0].integer(), hi = off[1].integer();
        if (lo > hi || hi > room) throw json::error(e.name + " runs past the end of the file");
        e.offset = base + lo;
        e.size = hi - lo;
        table.push_back(std::move(e));
    }
}
