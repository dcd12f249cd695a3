#include "weights.h"

#include <fcntl.h>
#include <hip/hip_runtime.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <algorithm>
#include <cmath>
#include <cstring>
#include <fstream>
#include <functional>
#include <set>
#include <sstream>
#include <thread>

namespace minillm {

// ---------------------------------------------------------------------------------------------
// safetensors
// ---------------------------------------------------------------------------------------------
static size_t dtype_bytes(const std::string& dt, const std::string& path, const std::string& name) {
    if (dt == "F32" || dt == "I32") return 4;
    if (dt == "BF16" || dt == "F16") return 2;
    if (dt == "F64" || dt == "I64") return 8;
    if (dt == "U8" || dt == "BOOL" || dt == "I8") return 1;
    throw WeightsError(path + ": tensor '" + name + "' has unsupported dtype " + dt);
}

SafetensorsFile::SafetensorsFile(const std::string& path) : path_(path) {
    const int fd = ::open(path.c_str(), O_RDONLY);
    if (fd < 0) throw WeightsError(path + ": cannot be opened");
    struct stat st;
    if (fstat(fd, &st) != 0) { ::close(fd); throw WeightsError(path + ": cannot be examined"); }
    size_ = static_cast<size_t>(st.st_size);
    if (size_ < 8) { ::close(fd); throw WeightsError(path + ": too short to be a safetensors file (" + std::to_string(size_) + " bytes)"); }
    map_ = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (map_ == MAP_FAILED) { map_ = nullptr; throw WeightsError(path + ": cannot be mapped"); }
    const unsigned char* base = static_cast<const unsigned char*>(map_);
    uint64_t hlen = 0;
    for (int i = 7; i >= 0; --i) hlen = (hlen << 8) | base[i];
    // (compared without adding to hlen, which may be anything up to 2^64 - 1; headers beyond 100 MB are refused
    // as the format's own library does)
    if (hlen == 0 || hlen > size_ - 8)
        throw WeightsError(path + ": header length " + std::to_string(hlen) + " exceeds the file size " + std::to_string(size_));
    if (hlen > 100u * 1000u * 1000u) throw WeightsError(path + ": header of " + std::to_string(hlen) + " bytes is larger than 100 MB");
    Json header;
    try {
        header = Json::parse(std::string(reinterpret_cast<const char*>(base + 8), hlen));
    } catch (const JsonError& e) {
        throw WeightsError(path + ": header is not valid JSON (" + e.what() + ")");
    }
    if (!header.is_object()) throw WeightsError(path + ": header is not a JSON object");
    const size_t data_start = 8 + hlen, data_len = size_ - data_start;
    for (const auto& kv : header.members()) {
        if (kv.first == "__metadata__") continue;
        StoredTensor t;
        try {
            t.dtype = kv.second.at("dtype").string();
            for (const Json& s : kv.second.at("shape").array()) t.shape.push_back(s.integer());
            const auto& off = kv.second.at("data_offsets").array();
            if (off.size() != 2) throw JsonError("data_offsets must have two entries");
            const int64_t b = off[0].integer(), e = off[1].integer();
            const int64_t numel = t.numel();
            const size_t esz = dtype_bytes(t.dtype, path, kv.first);
            if (numel < 0 || static_cast<uint64_t>(numel) > UINT64_MAX / 8)
                throw WeightsError(path + ": tensor '" + kv.first + "' has a negative dimension or more elements than can be counted");
            const size_t want = static_cast<size_t>(numel) * esz;
            if (b < 0 || e < b || static_cast<size_t>(e) > data_len)
                throw WeightsError(path + ": tensor '" + kv.first + "' has offsets [" + std::to_string(b) + ", " + std::to_string(e) +
                                   ") outside the file's " + std::to_string(data_len) + " data bytes");
            if (static_cast<size_t>(e - b) != want)
                throw WeightsError(path + ": tensor '" + kv.first + "' holds " + std::to_string(e - b) + " bytes, its shape and dtype need " +
                                   std::to_string(want));
            t.data = base + data_start + b;
            t.bytes = static_cast<size_t>(e - b);
        } catch (const JsonError& e) {
            throw WeightsError(path + ": entry of tensor '" + kv.first + "' is malformed (" + e.what() + ")");
        }
        tensors_.emplace(kv.first, std::move(t));
    }
}

SafetensorsFile::~SafetensorsFile() {
    if (map_ != nullptr) munmap(map_, size_);
}

void save_safetensors(const std::string& path, const std::map<std::string, TensorToStore>& tensors,
                      const std::map<std::string, std::string>& metadata) {
    Json header = Json::object();
    if (!metadata.empty()) {
        Json m = Json::object();
        for (const auto& kv : metadata) m.set(kv.first, Json::of(kv.second));
        header.set("__metadata__", m);
    }
    int64_t off = 0;
    for (const auto& kv : tensors) {       // std::map: sorted names
        Json e = Json::object();
        e.set("dtype", Json::of(kv.second.dtype));
        std::vector<Json> shape;
        for (int64_t s : kv.second.shape) shape.push_back(Json::of(s));
        e.set("shape", Json::array_of(shape));
        const int64_t n = static_cast<int64_t>(kv.second.bytes.size());
        e.set("data_offsets", Json::array_of({Json::of(off), Json::of(off + n)}));
        off += n;
        header.set(kv.first, e);
    }
    std::string h = header.dump();
    while (h.size() % 8 != 0) h += ' ';
    std::ofstream f(path, std::ios::binary);
    if (!f) throw WeightsError(path + ": cannot be written");
    uint64_t hlen = h.size();
    unsigned char len[8];
    for (int i = 0; i < 8; ++i) len[i] = static_cast<unsigned char>(hlen >> (8 * i));
    f.write(reinterpret_cast<const char*>(len), 8);
    f.write(h.data(), static_cast<std::streamsize>(h.size()));
    for (const auto& kv : tensors) f.write(reinterpret_cast<const char*>(kv.second.bytes.data()), static_cast<std::streamsize>(kv.second.bytes.size()));
    if (!f) throw WeightsError(path + ": write failed");
}

// ---------------------------------------------------------------------------------------------
// numbers
// ---------------------------------------------------------------------------------------------
uint64_t splitmix64(uint64_t x) {
    uint64_t z = x + 0x9E3779B97F4A7C15ull;
    z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
    z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
    return z ^ (z >> 31);
}

uint64_t fnv1a64(const std::string& s) {
    uint64_t h = 0xCBF29CE484222325ull;
    for (const unsigned char c : s) h = (h ^ c) * 0x100000001B3ull;
    return h;
}

void normal_values(uint64_t seed, const std::string& name, int64_t first, int64_t n, double mean, double std,
                   float* out) {
    const uint64_t key = splitmix64(seed) ^ fnv1a64(name);
    const double inv = 1.0 / 9007199254740992.0;
    const double two_pi = 6.283185307179586476925286766559;
    auto piece = [&](int64_t lo, int64_t hi) {
        for (int64_t k = lo; k < hi; ++k) {
            const uint64_t i = static_cast<uint64_t>(first + k);
            const uint64_t a = splitmix64(key + 2 * i), b = splitmix64(key + 2 * i + 1);
            const double u1 = (static_cast<double>(a >> 11) + 1.0) * inv, u2 = static_cast<double>(b >> 11) * inv;
            out[k] = static_cast<float>(mean + std * (std::sqrt(-2.0 * std::log(u1)) * std::cos(two_pi * u2)));
        }
    };
    const int workers = n > (1 << 18) ? static_cast<int>(std::min<unsigned>(16, std::max(1u, std::thread::hardware_concurrency()))) : 1;
    if (workers <= 1) { piece(0, n); return; }
    std::vector<std::thread> pool;
    const int64_t per = (n + workers - 1) / workers;
    for (int w = 0; w < workers; ++w) {
        const int64_t lo = w * per, hi = std::min<int64_t>(n, lo + per);
        if (lo < hi) pool.emplace_back(piece, lo, hi);
    }
    for (auto& t : pool) t.join();
}

uint16_t float_to_bf16_bits(float f) {
    uint32_t u;
    std::memcpy(&u, &f, 4);
    if ((u & 0x7F800000u) == 0x7F800000u && (u & 0x007FFFFFu)) return static_cast<uint16_t>((u >> 16) | 0x40);   // NaN
    const uint32_t round = 0x7FFFu + ((u >> 16) & 1u);
    return static_cast<uint16_t>((u + round) >> 16);
}

float bf16_bits_to_float(uint16_t b) {
    const uint32_t u = static_cast<uint32_t>(b) << 16;
    float f;
    std::memcpy(&f, &u, 4);
    return f;
}

float f16_bits_to_float(uint16_t h) {
    const uint32_t sign = (h >> 15) & 1u, exp = (h >> 10) & 0x1Fu, man = h & 0x3FFu;
    float v;
    if (exp == 0) v = std::ldexp(static_cast<float>(man), -24);
    else if (exp == 31) v = man ? NAN : INFINITY;
    else v = std::ldexp(static_cast<float>(man | 0x400u), static_cast<int>(exp) - 25);
    return sign ? -v : v;
}

// ---------------------------------------------------------------------------------------------
// sources
// ---------------------------------------------------------------------------------------------
static bool file_exists(const std::string& p) {
    struct stat st;
    return stat(p.c_str(), &st) == 0 && S_ISREG(st.st_mode);
}

static std::string read_text(const std::string& path) {
    std::ifstream f(path);
    if (!f) throw WeightsError(path + ": cannot be read");
    std::stringstream ss;
    ss << f.rdbuf();
    return ss.str();
}

CheckpointSource::CheckpointSource(const std::string& model_dir) : dir_(model_dir) {
    const std::string single = model_dir + "/model.safetensors", index = model_dir + "/model.safetensors.index.json";
    std::vector<std::string> paths;
    if (file_exists(single)) {
        paths.push_back(single);
    } else if (file_exists(index)) {
        std::set<std::string> shards;
        try {
            const Json j = Json::parse(read_text(index));
            for (const auto& kv : j.at("weight_map").members()) shards.insert(kv.second.string());
        } catch (const JsonError& e) {
            throw WeightsError(index + ": " + e.what());
        }
        for (const auto& s : shards) paths.push_back(model_dir + "/" + s);
    } else {
        throw WeightsError(model_dir + ": neither model.safetensors nor model.safetensors.index.json is there");
    }
    for (const auto& p : paths) {
        files_.emplace_back(new SafetensorsFile(p));
        for (const auto& kv : files_.back()->tensors()) {
            if (all_.count(kv.first)) throw WeightsError(model_dir + ": tensor '" + kv.first + "' appears in two files");
            all_[kv.first] = &kv.second;
        }
    }
}

std::vector<std::string> CheckpointSource::names() const {
    std::vector<std::string> n;
    for (const auto& kv : all_) n.push_back(kv.first);
    return n;
}

const std::vector<int64_t>* CheckpointSource::shape_of(const std::string& name) const {
    auto it = all_.find(name);
    return it == all_.end() ? nullptr : &it->second->shape;
}

void CheckpointSource::read(const ParamSpec& spec, const std::string& stored_name, std::vector<float>& out) const {
    const StoredTensor& t = *all_.at(stored_name);
    const int64_t n = t.numel();
    out.resize(static_cast<size_t>(n));
    if (t.dtype == "F32") {
        std::memcpy(out.data(), t.data, static_cast<size_t>(n) * 4);
    } else if (t.dtype == "BF16") {
        const uint16_t* p = reinterpret_cast<const uint16_t*>(t.data);
        for (int64_t i = 0; i < n; ++i) out[i] = bf16_bits_to_float(p[i]);
    } else if (t.dtype == "F16") {
        const uint16_t* p = reinterpret_cast<const uint16_t*>(t.data);
        for (int64_t i = 0; i < n; ++i) out[i] = f16_bits_to_float(p[i]);
    } else {
        throw WeightsError(dir_ + ": tensor '" + spec.name + "' must be floating point (F32, BF16 or F16), found " + t.dtype);
    }
}

RandomSource::RandomSource(uint64_t seed, const std::string& weights_dtype) : seed_(seed) {
    if (weights_dtype != "bfloat16" && weights_dtype != "float32")
        throw WeightsError("random weights are stored as bfloat16 or float32, not '" + weights_dtype + "'");
    round_bf16_ = weights_dtype == "bfloat16";
}

void RandomSource::read(const ParamSpec& spec, const std::string&, std::vector<float>& out) const {
    int64_t n = 1;
    for (int64_t s : spec.shape) n *= s;
    out.resize(static_cast<size_t>(n));
    normal_values(seed_, spec.name, 0, n, spec.mean, spec.std, out.data());
    if (round_bf16_ && spec.role == ParamSpec::Matrix)
        for (auto& v : out) v = bf16_bits_to_float(float_to_bf16_bits(v));
}

// ---------------------------------------------------------------------------------------------
// device tensors
// ---------------------------------------------------------------------------------------------
DeviceTensors::~DeviceTensors() {
    for (void* p : ptrs_) (void)hipFree(p);
}

Tensor2 DeviceTensors::join_rows(const std::vector<Tensor2>& parts) {
    if (parts.empty()) throw WeightsError("join_rows: nothing to join");
    int64_t rows = 0;
    for (const Tensor2& t : parts) {
        if (t.dtype != parts[0].dtype || t.cols != parts[0].cols || !t.contiguous()) throw WeightsError("join_rows: the parts must be contiguous, of one dtype and width");
        rows += t.rows;
    }
    const size_t row_bytes = static_cast<size_t>(parts[0].cols) * parts[0].esz();
    char* base = static_cast<char*>(allocate(static_cast<size_t>(rows) * row_bytes, false));
    size_t at = 0;
    for (const Tensor2& t : parts) {
        const size_t bytes = static_cast<size_t>(t.rows) * row_bytes;
        if (bytes > 0 && hipMemcpy(base + at, t.data, bytes, hipMemcpyDeviceToDevice) != hipSuccess) throw WeightsError("join_rows: the copy on the device failed");
        at += bytes;
    }
    return Tensor2(base, parts[0].dtype, rows, parts[0].cols);
}

Tensor2 DeviceTensors::repeat(const Tensor2& v, int times) {
    if (v.dtype != F32 || !v.contiguous() || times < 1) throw WeightsError("repeat: a contiguous float32 vector and a positive count are needed");
    const size_t n = static_cast<size_t>(v.rows) * v.cols;
    char* base = static_cast<char*>(allocate(n * 4 * times, false));
    for (int i = 0; i < times; ++i)
        if (n > 0 && hipMemcpy(base + i * n * 4, v.data, n * 4, hipMemcpyDeviceToDevice) != hipSuccess) throw WeightsError("repeat: the copy on the device failed");
    return Tensor2(base, F32, 1, static_cast<int64_t>(n) * times);
}

Tensor2 DeviceTensors::join_cols(const std::vector<Tensor2>& parts) {
    if (parts.empty()) throw WeightsError("join_cols: nothing to join");
    int64_t cols = 0;
    for (const Tensor2& t : parts) {
        if (t.dtype != parts[0].dtype || t.rows != parts[0].rows || !t.contiguous()) throw WeightsError("join_cols: the parts must be contiguous, of one dtype and height");
        cols += t.cols;
    }
    const size_t esz = parts[0].esz(), row_bytes = static_cast<size_t>(cols) * esz;
    char* base = static_cast<char*>(allocate(static_cast<size_t>(parts[0].rows) * row_bytes, false));
    size_t at = 0;
    for (const Tensor2& t : parts) {
        const size_t width = static_cast<size_t>(t.cols) * esz;
        if (width > 0 && t.rows > 0 &&
            hipMemcpy2D(base + at, row_bytes, t.data, width, width, static_cast<size_t>(t.rows), hipMemcpyDeviceToDevice) != hipSuccess)
            throw WeightsError("join_cols: the copy on the device failed");
        at += width;
    }
    return Tensor2(base, parts[0].dtype, parts[0].rows, cols);
}

Tensor2 DeviceTensors::pad_row_blocks(const Tensor2& t, int64_t block, int64_t padded) {
    if (block < 1 || padded < block || t.rows % block != 0 || !t.contiguous()) throw WeightsError("pad_row_blocks: contiguous rows in whole blocks are needed");
    const int64_t n = t.rows / block;
    const size_t row_bytes = static_cast<size_t>(t.cols) * t.esz();
    char* base = static_cast<char*>(allocate(static_cast<size_t>(n * padded) * row_bytes, true));
    for (int64_t b = 0; b < n; ++b)
        if (row_bytes > 0 && hipMemcpy(base + static_cast<size_t>(b * padded) * row_bytes, static_cast<const char*>(t.data) + static_cast<size_t>(b * block) * row_bytes,
                                       static_cast<size_t>(block) * row_bytes, hipMemcpyDeviceToDevice) != hipSuccess)
            throw WeightsError("pad_row_blocks: the copy on the device failed");
    return Tensor2(base, t.dtype, n * padded, t.cols);
}

Tensor2 DeviceTensors::pad_col_blocks(const Tensor2& t, int64_t block, int64_t padded) {
    if (block < 1 || padded < block || t.cols % block != 0 || !t.contiguous()) throw WeightsError("pad_col_blocks: contiguous columns in whole blocks are needed");
    const int64_t n = t.cols / block;
    const size_t esz = t.esz(), src_pitch = static_cast<size_t>(t.cols) * esz, dst_pitch = static_cast<size_t>(n * padded) * esz;
    char* base = static_cast<char*>(allocate(static_cast<size_t>(t.rows) * dst_pitch, true));
    for (int64_t b = 0; b < n; ++b)
        if (t.rows > 0 && hipMemcpy2D(base + static_cast<size_t>(b * padded) * esz, dst_pitch, static_cast<const char*>(t.data) + static_cast<size_t>(b * block) * esz, src_pitch,
                                      static_cast<size_t>(block) * esz, static_cast<size_t>(t.rows), hipMemcpyDeviceToDevice) != hipSuccess)
            throw WeightsError("pad_col_blocks: the copy on the device failed");
    return Tensor2(base, t.dtype, t.rows, n * padded);
}

Tensor2 DeviceTensors::pad_row_parts(const Tensor2& t, const std::vector<int64_t>& parts, const std::vector<int64_t>& padded) {
    int64_t block = 0, out_block = 0;
    bool ok = !parts.empty() && parts.size() == padded.size() && t.contiguous();
    for (size_t i = 0; ok && i < parts.size(); ++i) {
        ok = parts[i] >= 0 && padded[i] >= parts[i];
        block += parts[i];
        out_block += padded[i];
    }
    if (!ok || block < 1 || t.rows % block != 0) throw WeightsError("pad_row_parts: contiguous rows in whole blocks are needed");
    const int64_t n = t.rows / block;
    const size_t row_bytes = static_cast<size_t>(t.cols) * t.esz();
    char* base = static_cast<char*>(allocate(static_cast<size_t>(n * out_block) * row_bytes, true));
    for (int64_t b = 0; b < n; ++b) {
        int64_t from = b * block, to = b * out_block;
        for (size_t i = 0; i < parts.size(); ++i) {
            if (parts[i] > 0 && row_bytes > 0 &&
                hipMemcpy(base + static_cast<size_t>(to) * row_bytes, static_cast<const char*>(t.data) + static_cast<size_t>(from) * row_bytes,
                          static_cast<size_t>(parts[i]) * row_bytes, hipMemcpyDeviceToDevice) != hipSuccess)
                throw WeightsError("pad_row_parts: the copy on the device failed");
            from += parts[i];
            to += padded[i];
        }
    }
    return Tensor2(base, t.dtype, n * out_block, t.cols);
}

// Runs of neighbours among the picked indices are copied together: f(first in the result, first in the source, length).
template <typename F>
static void runs_of(const std::vector<int64_t>& picked, int64_t limit, const char* what, F&& f) {
    for (size_t i = 0; i < picked.size();) {
        if (picked[i] < -1 || picked[i] >= limit) throw WeightsError(std::string(what) + ": an index beyond the tensor");
        size_t n = 1;
        if (picked[i] >= 0)
            while (i + n < picked.size() && picked[i + n] == picked[i] + static_cast<int64_t>(n)) ++n;
        if (picked[i] >= 0) {
            if (picked[i] + static_cast<int64_t>(n) > limit) throw WeightsError(std::string(what) + ": an index beyond the tensor");
            f(i, picked[i], n);
        }
        i += n;
    }
}

Tensor2 DeviceTensors::pick_rows(const Tensor2& t, const std::vector<int64_t>& rows) {
    if (!t.contiguous()) throw WeightsError("pick_rows: a contiguous tensor is needed");
    const size_t row_bytes = static_cast<size_t>(t.cols) * t.esz();
    char* base = static_cast<char*>(allocate(rows.size() * row_bytes, true));
    runs_of(rows, t.rows, "pick_rows", [&](size_t to, int64_t from, size_t n) {
        if (hipMemcpy(base + to * row_bytes, static_cast<const char*>(t.data) + static_cast<size_t>(from) * row_bytes, n * row_bytes, hipMemcpyDeviceToDevice) != hipSuccess)
            throw WeightsError("pick_rows: the copy on the device failed");
    });
    return Tensor2(base, t.dtype, static_cast<int64_t>(rows.size()), t.cols);
}

Tensor2 DeviceTensors::pick_cols(const Tensor2& t, const std::vector<int64_t>& cols) {
    if (!t.contiguous()) throw WeightsError("pick_cols: a contiguous tensor is needed");
    const size_t esz = t.esz(), to_pitch = cols.size() * esz, from_pitch = static_cast<size_t>(t.cols) * esz;
    char* base = static_cast<char*>(allocate(static_cast<size_t>(t.rows) * to_pitch, true));
    runs_of(cols, t.cols, "pick_cols", [&](size_t to, int64_t from, size_t n) {
        if (t.rows > 0 && hipMemcpy2D(base + to * esz, to_pitch, static_cast<const char*>(t.data) + static_cast<size_t>(from) * esz, from_pitch, n * esz, static_cast<size_t>(t.rows),
                                      hipMemcpyDeviceToDevice) != hipSuccess)
            throw WeightsError("pick_cols: the copy on the device failed");
    });
    return Tensor2(base, t.dtype, t.rows, static_cast<int64_t>(cols.size()));
}

Tensor2 DeviceTensors::operand_tiles(const Tensor2& t, int64_t rows, int64_t cols) {
    if (t.dtype != BF16 || !t.contiguous() || rows % 16 != 0 || cols % 32 != 0 || rows < t.rows || cols < t.cols)
        throw WeightsError("operand_tiles: a contiguous bfloat16 matrix and sizes in whole tiles are needed");
    std::vector<uint16_t> from(static_cast<size_t>(t.rows) * t.cols), to(static_cast<size_t>(rows) * cols, 0);
    if (!from.empty() && hipMemcpy(from.data(), t.data, from.size() * 2, hipMemcpyDeviceToHost) != hipSuccess) throw WeightsError("operand_tiles: the copy from the device failed");
    size_t at = 0;
    for (int64_t r0 = 0; r0 < rows; r0 += 16)
        for (int64_t c0 = 0; c0 < cols; c0 += 32)
            for (int lane = 0; lane < 64; ++lane)
                for (int i = 0; i < 8; ++i, ++at) {
                    const int64_t r = r0 + lane % 16, c = c0 + 8 * (lane / 16) + i;
                    if (r < t.rows && c < t.cols) to[at] = from[static_cast<size_t>(r) * t.cols + c];
                }
    void* dev = allocate(to.size() * 2, false);
    if (!to.empty() && hipMemcpy(dev, to.data(), to.size() * 2, hipMemcpyHostToDevice) != hipSuccess) throw WeightsError("operand_tiles: the copy to the device failed");
    return Tensor2(dev, BF16, rows, cols);
}

Tensor2 DeviceTensors::gram_tiles(const Tensor2& w, int64_t n) {
    if (w.dtype != BF16 || !w.contiguous() || n % 16 != 0 || n < w.cols) throw WeightsError("gram_tiles: a contiguous bfloat16 matrix and a size in whole tiles are needed");
    std::vector<uint16_t> from(static_cast<size_t>(w.rows) * w.cols);
    if (!from.empty() && hipMemcpy(from.data(), w.data, from.size() * 2, hipMemcpyDeviceToHost) != hipSuccess) throw WeightsError("gram_tiles: the copy from the device failed");
    const size_t C = static_cast<size_t>(w.cols);
    std::vector<double> g(C * C, 0.0), row(C);
    for (int64_t r = 0; r < w.rows; ++r) {
        for (size_t c = 0; c < C; ++c) row[c] = bf16_bits_to_float(from[static_cast<size_t>(r) * C + c]);
        for (size_t a = 0; a < C; ++a)
            for (size_t b = 0; b < C; ++b) g[a * C + b] += row[a] * row[b];
    }
    std::vector<float> tiles(static_cast<size_t>(n) * n, 0.f);
    size_t at = 0;
    for (int64_t r0 = 0; r0 < n; r0 += 16)
        for (int64_t c0 = 0; c0 < n; c0 += 4)
            for (int lane = 0; lane < 64; ++lane, ++at) {
                const int64_t r = r0 + lane % 16, c = c0 + lane / 16;
                if (r < w.cols && c < w.cols) tiles[at] = static_cast<float>(g[static_cast<size_t>(r) * C + static_cast<size_t>(c)]);
            }
    return upload(tiles, n, n, F32);
}

Tensor2 DeviceTensors::scaled(const Tensor2& v, float factor) {
    const size_t n = static_cast<size_t>(v.rows) * v.cols;
    if (v.dtype != F32 || !v.contiguous()) throw WeightsError("scaled: a contiguous float32 vector is needed");
    std::vector<float> host(n);
    if (n > 0 && hipMemcpy(host.data(), v.data, n * 4, hipMemcpyDeviceToHost) != hipSuccess) throw WeightsError("scaled: the copy from the device failed");
    for (float& f : host) f *= factor;
    return upload(host, 1, static_cast<int64_t>(n), F32);
}

Tensor2 DeviceTensors::zeros(int64_t n) {
    if (n < 0) throw WeightsError("zeros: a negative size");
    return Tensor2(allocate(static_cast<size_t>(n) * 4, true), F32, 1, n);
}

void* DeviceTensors::allocate(size_t bytes, bool zero) {
    void* p = nullptr;
    hipError_t e = hipMalloc(&p, std::max<size_t>(bytes, 16));
    if (e != hipSuccess) throw WeightsError("hipMalloc of " + std::to_string(bytes) + " bytes failed: " + hipGetErrorString(e));
    if (zero) {
        e = hipMemset(p, 0, std::max<size_t>(bytes, 16));
        if (e != hipSuccess) throw WeightsError(std::string("hipMemset failed: ") + hipGetErrorString(e));
    }
    ptrs_.push_back(p);
    bytes_ += bytes;
    return p;
}

Tensor2 DeviceTensors::upload(const std::vector<float>& values, int64_t rows, int64_t cols, int dtype) {
    const size_t n = static_cast<size_t>(rows) * cols;
    if (values.size() != n) throw WeightsError("upload: size mismatch");
    void* dev = allocate(n * dtype_size(dtype), false);
    hipError_t e;
    if (dtype == F32) {
        e = hipMemcpy(dev, values.data(), n * 4, hipMemcpyHostToDevice);
    } else {
        std::vector<uint16_t> half(n);
        for (size_t i = 0; i < n; ++i) half[i] = float_to_bf16_bits(values[i]);
        e = hipMemcpy(dev, half.data(), n * 2, hipMemcpyHostToDevice);
    }
    if (e != hipSuccess) throw WeightsError(std::string("copy to the device failed: ") + hipGetErrorString(e));
    return Tensor2(dev, dtype, rows, cols);
}

// ---------------------------------------------------------------------------------------------
// loading
// ---------------------------------------------------------------------------------------------
static std::string shape_text(const std::vector<int64_t>& s) {
    std::string t = "[";
    for (size_t i = 0; i < s.size(); ++i) t += (i ? ", " : "") + std::to_string(s[i]);
    return t + "]";
}

std::map<std::string, std::string> check_checkpoint(const std::vector<ParamSpec>& specs, const TensorSource& source,
                                                    const std::vector<std::string>& optional_prefixes,
                                                    const std::function<bool(const std::string&)>& ignored,
                                                    const std::string& where) {
    std::map<std::string, const ParamSpec*> by_name;
    for (const auto& s : specs) by_name[s.name] = &s;
    std::map<std::string, std::string> available;     // short name -> stored name
    {
        for (const std::string& name : source.names()) {
            std::string short_name = name;
            if (!by_name.count(name)) {
                for (const auto& p : optional_prefixes)
                    if (name.compare(0, p.size(), p) == 0) { short_name = name.substr(p.size()); break; }
            }
            if (ignored && ignored(short_name)) continue;
            available[short_name] = name;
        }
        std::vector<std::string> missing, unexpected, wrong;
        for (const auto& s : specs) {
            auto it = available.find(s.name);
            if (it == available.end()) { missing.push_back(s.name); continue; }
            const std::vector<int64_t>* shape = source.shape_of(it->second);
            bool fits = shape != nullptr && shape->size() == s.shape.size();
            for (size_t k = 0; fits && k < s.shape.size(); ++k)
                fits = static_cast<int>(k) == s.free_dim ? (*shape)[k] >= 1 : (*shape)[k] == s.shape[k];
            if (!fits)
                wrong.push_back(s.name + ": expected " + shape_text(s.shape) + ", found " + (shape ? shape_text(*shape) : "nothing"));
        }
        for (const auto& kv : available)
            if (!by_name.count(kv.first)) unexpected.push_back(kv.first);
        if (!missing.empty() || !unexpected.empty() || !wrong.empty()) {
            auto join = [](const std::vector<std::string>& v, const char* sep) {
                std::string t;
                for (size_t i = 0; i < v.size(); ++i) t += (i ? sep : "") + v[i];
                return t;
            };
            std::string msg = where + ": the checkpoint does not fit the model";
            if (!missing.empty()) msg += "\n  missing tensors (" + std::to_string(missing.size()) + "): " + join(missing, ", ");
            if (!unexpected.empty()) msg += "\n  unexpected tensors (" + std::to_string(unexpected.size()) + "): " + join(unexpected, ", ");
            if (!wrong.empty()) msg += "\n  wrong shapes (" + std::to_string(wrong.size()) + "): " + join(wrong, "; ");
            throw WeightsError(msg);
        }
    }
    return available;
}

std::map<std::string, Tensor2> load_tensors(const std::vector<ParamSpec>& specs, const TensorSource& source,
                                            int compute_dtype, DeviceTensors& store,
                                            const std::vector<std::string>& optional_prefixes,
                                            const std::function<bool(const std::string&)>& ignored,
                                            const std::string& where) {
    std::map<std::string, std::string> available;     // short name -> stored name
    if (!source.generates()) available = check_checkpoint(specs, source, optional_prefixes, ignored, where);
    std::map<std::string, Tensor2> out;
    std::vector<float> values, turned;
    for (const auto& s : specs) {
        source.read(s, source.generates() ? s.name : available.at(s.name), values);
        int64_t rows = 1, cols = 1;
        // (a dimension that the checkpoint decides is read off the stored tensor)
        std::vector<int64_t> shape = s.shape;
        if (!source.generates() && s.free_dim >= 0)
            if (const std::vector<int64_t>* stored = source.shape_of(available.at(s.name))) shape = *stored;
        if (shape.empty()) cols = 1;                      // one number
        else if (shape.size() == 1) cols = shape[0];
        else if (shape.size() == 2) { rows = shape[0]; cols = shape[1]; }
        else throw WeightsError(where + ": tensor '" + s.name + "' has " + std::to_string(shape.size()) + " dimensions; at most two are expected");
        if (s.add != 0.0)
            for (auto& v : values) v = static_cast<float>(v + s.add);
        const std::vector<float>* src = &values;
        if (s.transpose) {
            turned.resize(values.size());
            for (int64_t r = 0; r < rows; ++r)
                for (int64_t c = 0; c < cols; ++c) turned[static_cast<size_t>(c) * rows + r] = values[static_cast<size_t>(r) * cols + c];
            std::swap(rows, cols);
            src = &turned;
        }
        out[s.name] = store.upload(*src, rows, cols, s.role == ParamSpec::Matrix ? compute_dtype : F32);
    }
    return out;
}

void write_random_model(const std::string& out_dir, const Json& config, const std::vector<ParamSpec>& specs,
                        uint64_t seed, const std::string& weights_dtype) {
    RandomSource src(seed, weights_dtype);
    std::map<std::string, TensorToStore> tensors;
    std::vector<float> values;
    for (const auto& s : specs) {
        src.read(s, s.name, values);
        TensorToStore t;
        t.shape = s.shape;
        if (s.role == ParamSpec::Matrix && weights_dtype == "bfloat16") {
            t.dtype = "BF16";
            t.bytes.resize(values.size() * 2);
            uint16_t* p = reinterpret_cast<uint16_t*>(t.bytes.data());
            for (size_t i = 0; i < values.size(); ++i) p[i] = float_to_bf16_bits(values[i]);
        } else {
            t.dtype = "F32";
            t.bytes.resize(values.size() * 4);
            std::memcpy(t.bytes.data(), values.data(), values.size() * 4);
        }
        tensors.emplace(s.name, std::move(t));
    }
    ::mkdir(out_dir.c_str(), 0755);
    Json cfg = config;
    cfg.set("torch_dtype", Json::of(weights_dtype));
    std::ofstream f(out_dir + "/config.json");
    if (!f) throw WeightsError(out_dir + "/config.json: cannot be written");
    f << cfg.dump() << "\n";
    save_safetensors(out_dir + "/model.safetensors", tensors, {{"format", "pt"}, {"seed", std::to_string(seed)}});
}

}  // namespace minillm
