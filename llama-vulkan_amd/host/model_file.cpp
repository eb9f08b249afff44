#include "model_file.h"

#include <sys/stat.h>

#include "block_model_file.h"
#include "ggml_file.h"

std::unique_ptr<model_file> model_file::open(const std::string &path)
{
    struct stat st{};
    if (stat(path.c_str(), &st) == 0 && S_ISDIR(st.st_mode)) return std::make_unique<block_model_file>(path);
    return std::make_unique<ggml_file>(path.c_str());
}
