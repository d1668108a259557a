// Read-only private mapping of a whole file (util/file_descriptor.hh + MMap_Region in the reference).
#pragma once

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cerrno>
#include <cstdint>
#include <cstring>
#include <filesystem>
#include <string>

namespace glint {

class MappedFile
{
public:
  MappedFile() = default;
  MappedFile( const MappedFile& ) = delete;
  MappedFile& operator=( const MappedFile& ) = delete;
  ~MappedFile() { close(); }

  static constexpr uint64_t ANY_SIZE = ~0ull;

  // empty string on success
  std::string open( const std::filesystem::path& path, uint64_t expected_bytes = ANY_SIZE )
  {
    close();
    std::error_code ec;
    const auto size = std::filesystem::file_size( path, ec );
    if ( ec ) {
      return "cannot stat " + path.string() + ": " + ec.message();
    }
    if ( expected_bytes != ANY_SIZE && size != expected_bytes ) {
      return "file " + path.string() + " is not the expected size (" + std::to_string( size ) + " bytes, " + std::to_string( expected_bytes ) + " expected)";
    }
    fd_ = ::open( path.c_str(), O_RDONLY );
    if ( fd_ < 0 ) {
      return "cannot open " + path.string() + ": " + std::strerror( errno );
    }
    if ( size == 0 ) {
      return {};
    }
    void* p = ::mmap( nullptr, size, PROT_READ, MAP_PRIVATE, fd_, 0 );
    if ( p == MAP_FAILED ) {
      const std::string msg = "cannot map " + path.string() + ": " + std::strerror( errno );
      close();
      return msg;
    }
    addr_ = static_cast<const uint8_t*>( p );
    len_ = size;
    return {};
  }

  void close()
  {
    if ( addr_ != nullptr ) {
      ::munmap( const_cast<uint8_t*>( addr_ ), len_ );
      addr_ = nullptr;
      len_ = 0;
    }
    if ( fd_ >= 0 ) {
      ::close( fd_ );
      fd_ = -1;
    }
  }

  [[nodiscard]] const uint8_t* addr() const { return addr_; }
  [[nodiscard]] uint64_t len() const { return len_; }

private:
  int fd_ { -1 };
  const uint8_t* addr_ { nullptr };
  uint64_t len_ { 0 };
};

} // namespace glint
