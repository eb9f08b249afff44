// Driver for the sanitizer run of the host parser and tokenizer: opens every file named on the command line, and
// for files that parse walks the tensor table, tokenizes a few strings and converts them back.  Built by
// tests/test_host_sanitizers.py with -fsanitize=address,undefined; a finding aborts with a non-zero exit code.
#include <cstdio>
#include <string>
#include <vector>

#include "block_model_file.h"
#include "ggml_file.h"
#include "llava_hip.h"

// the parsers are linked without the device library; nothing here uploads
extern "C" int lv_model_upload(lv_ctx *, const void *, uint64_t, const lv_hparams *, const lv_tensor_desc *, uint32_t, lv_model **) { return LV_ERR_STATE; }
extern "C" int lv_block_model_upload(lv_ctx *, const void *base, uint64_t size, const lv_block_hparams *, const lv_block_spec *, const lv_tensor_desc *t, uint32_t n,
                                     int, lv_model **)
{
    // every tensor the folder offers lies inside its file
    unsigned sum = 0;
    for (uint32_t i = 0; i < n; ++i)
        if (t[i].size) sum += static_cast<const unsigned char *>(base)[t[i].offset] + static_cast<const unsigned char *>(base)[t[i].offset + t[i].size - 1];
    return size + sum ? LV_ERR_STATE : LV_OK;
}

int main(int argc, char **argv)
{
    unsigned long opened = 0, checksum = 0;
    for (int i = 1; i < argc; ++i) {
        const std::string path = argv[i];
        if (path.size() > 7 && path.compare(path.size() - 7, 7, ".folder") == 0) {
            block_model_file f(path);
            if (!f.is_open()) continue;
            ++opened;
            lv_model *m = nullptr;
            std::vector<u32> ids;
            checksum += static_cast<unsigned long>(f.upload(nullptr, LV_BF16, &m)) + f.tokenize(ids, "1 2,3\n4", true);
            continue;
        }
        ggml_file f(argv[i]);
        if (!f.is_open()) continue;
        ++opened;
        const unsigned char *base = static_cast<const unsigned char *>(f.data());
        for (const ggml_data_descriptor &d : f.get_tables()) {
            // first and last byte of every payload lie inside the mapping
            if (d.size) checksum += base[d.offset] + base[d.offset + d.size - 1];
            checksum += f.find_buffer_descriptor(d.name) != nullptr;
        }
        for (const char *text : {"", "hello world", " hello", "ab", "\xe6\x97\xa5\xe6\x9c\xac", "\xff\xfe", "aaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaaa"}) {
            std::vector<u32> ids;
            f.tokenize(ids, text, true);
            checksum += f.tokens_to_text(ids.data(), static_cast<u32>(ids.size())).size();
        }
    }
    std::printf("opened %lu of %d, checksum %lu\n", opened, argc - 1, checksum);
    return 0;
}
