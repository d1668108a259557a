// Reading a run-time sized design's configuration: what the designs' readers share.
#pragma once

#include <cstdint>
#include <filesystem>
#include <fstream>
#include <sstream>
#include <string>

#include "glint/json.hh"
#include "glint/types.hh"

namespace glint {

// a whole number in [least, 2^30)
inline uint32_t json_size( const Json& v, const char* what, const uint32_t least = 1 )
{
  const uint64_t n = v[what].integer();
  if ( n < least || n > 0x3fffffffull ) {
    throw JsonError( std::string( what ) + " is out of range" );
  }
  return static_cast<uint32_t>( n );
}

// Config::from_json over the text of a config.json; empty string on success
template<typename Config>
std::string parse_config( const std::string& text, Config& out )
{
  try {
    out = Config::from_json( Json::parse( text ) );
    return {};
  } catch ( const std::exception& e ) {
    return std::string( "config.json: " ) + e.what();
  }
}

// "kind" and size of a layer's feed-forward: its hidden size, 0 where the layer has none
inline uint32_t dense_feed_forward( const Json& layer )
{
  const Json* mlp = layer.find( "mlp" );
  if ( mlp == nullptr || mlp->is_null() ) {
    return 0;
  }
  if ( ( *mlp )["kind"].string() != "dense" ) {
    throw JsonError( "unknown feed-forward kind \"" + ( *mlp )["kind"].string() + "\"" );
  }
  return json_size( *mlp, "ff" );
}

// text of a file; false when it cannot be read
inline bool read_text_file( const std::filesystem::path& path, std::string& out )
{
  std::ifstream in { path, std::ios::binary };
  if ( !in ) {
    return false;
  }
  std::ostringstream text;
  text << in.rdbuf();
  out = text.str();
  return true;
}

// "architecture" of the config.json of a model directory; empty when there is none
inline std::string architecture_of( const std::filesystem::path& model_dir )
{
  std::string text;
  if ( !read_text_file( model_dir / "config.json", text ) ) {
    return {};
  }
  try {
    return Json::parse( text )["architecture"].string();
  } catch ( const std::exception& ) {
    return {};
  }
}

} // namespace glint
