// Reader of a safetensors file: an 8-byte little-endian length, that many bytes of JSON (tensor name -> dtype, shape, data_offsets
// counted from the end of the JSON), then the data.  The file stays mapped; tensors are views into it.
#pragma once

#include <bit>
#include <cstring>
#include <filesystem>
#include <map>
#include <string>
#include <vector>

#include "glint/json.hh"
#include "glint/mapped_file.hh"
#include "glint/types.hh"

namespace glint {

static_assert( std::endian::native == std::endian::little, "tensor data is little-endian" );

class SafeTensors
{
public:
  struct Tensor
  {
    std::string dtype {};
    std::vector<uint64_t> shape {};
    const uint8_t* data { nullptr };
    uint64_t bytes { 0 };
    uint64_t elements() const
    {
      uint64_t n = 1;
      for ( const uint64_t d : shape ) {
        n *= d;
      }
      return n;
    }
  };

  // empty string on success
  std::string open( const std::filesystem::path& path )
  {
    tensors_.clear();
    if ( auto err = file_.open( path ); !err.empty() ) {
      return err;
    }
    const std::string what = path.string() + ": ";
    uint64_t header = 0;
    if ( file_.len() < sizeof( header ) ) {
      return what + "too short for a header";
    }
    std::memcpy( &header, file_.addr(), sizeof( header ) );
    if ( header > file_.len() - sizeof( header ) ) {
      return what + "the header is longer than the file";
    }
    const uint8_t* data = file_.addr() + sizeof( header ) + header;
    const uint64_t data_len = file_.len() - sizeof( header ) - header;
    try {
      const Json root = Json::parse( { reinterpret_cast<const char*>( file_.addr() ) + sizeof( header ), header } );
      for ( const auto& [name, entry] : root.object() ) {
        if ( name == "__metadata__" ) {
          continue;
        }
        Tensor t;
        t.dtype = entry["dtype"].string();
        for ( const Json& d : entry["shape"].array() ) {
          t.shape.push_back( d.integer() );
        }
        const auto& span = entry["data_offsets"].array();
        const uint64_t begin = span.at( 0 ).integer(), end = span.at( 1 ).integer();
        const uint64_t element = element_size( t.dtype );
        if ( begin > end || end > data_len || element == 0 || end - begin != t.elements() * element ) {
          return what + "tensor " + name + " has a bad type or range";
        }
        t.data = data + begin;
        t.bytes = end - begin;
        tensors_.emplace( name, std::move( t ) );
      }
    } catch ( const std::exception& e ) {
      return what + e.what();
    }
    return {};
  }

  // nullptr when absent
  const Tensor* find( const std::string& name ) const
  {
    const auto it = tensors_.find( name );
    return it == tensors_.end() ? nullptr : &it->second;
  }

  static uint64_t element_size( const std::string& dtype )
  {
    if ( dtype == "BF16" || dtype == "F16" ) {
      return 2;
    }
    return dtype == "F32" || dtype == "I32" ? 4 : 0;
  }

  // element i of a floating-point tensor
  static float value( const Tensor& t, const uint64_t i )
  {
    if ( t.dtype == "F32" ) {
      float v;
      std::memcpy( &v, t.data + 4 * i, sizeof( v ) );
      return v;
    }
    uint16_t bits;
    std::memcpy( &bits, t.data + 2 * i, sizeof( bits ) );
    if ( t.dtype == "BF16" ) {
      return std::bit_cast<float>( static_cast<uint32_t>( bits ) << 16 );
    }
    return static_cast<float>( std::bit_cast<float16_t>( bits ) );
  }

private:
  MappedFile file_ {};
  std::map<std::string, Tensor> tensors_ {};
};

} // namespace glint
