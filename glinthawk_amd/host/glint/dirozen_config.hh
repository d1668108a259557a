// Configuration of the Dirozen design, read from a model directory's config.json: a decoder-only model of parallel layers, attention and
// an optional gated feed-forward side by side behind one norm.  Keys serve as values too, positions enter through the queries' temperature.
#pragma once

#include <cstdint>
#include <string>
#include <vector>

#include "glint/design_config.hh"

namespace glint {

namespace configs {
struct Dirozen // the tag its states and settings are typed with
{
  constexpr static bool sized_at_run_time = true;
};
} // namespace configs

struct DirozenConfig
{
  struct Layer
  {
    uint32_t heads {}, kv_heads {}, dim {};
    float scale {};
    float temp_coef {};
    uint32_t temp_every {}; // 0: queries without a temperature
    uint32_t ff { 0 };      // 0: no feed-forward
  };

  uint32_t width {}, vocab {};
  uint32_t max_positions {}; // of a context: nothing in the model bounds them
  float eps {};
  std::vector<Layer> layers {};

  // empty string on success
  static std::string parse( const std::string& text, DirozenConfig& out ) { return parse_config( text, out ); }

  static DirozenConfig from_json( const Json& j )
  {
    DirozenConfig c;
    c.width = json_size( j, "width" );
    c.vocab = json_size( j, "vocab" );
    c.eps = static_cast<float>( j["norm"]["eps"].number() );
    for ( const Json& l : j["layers"].array() ) {
      if ( l["type"].string() != "attention" ) {
        throw JsonError( "unknown layer type \"" + l["type"].string() + "\"" );
      }
      const Json& m = l["mixer"];
      Layer layer;
      layer.heads = json_size( m, "heads" );
      layer.kv_heads = json_size( m, "kv_heads" );
      layer.dim = json_size( m, "dim" );
      layer.scale = static_cast<float>( m["scale"].number() );
      if ( layer.heads % layer.kv_heads != 0 ) {
        throw JsonError( "attention: heads must be a multiple of kv_heads" );
      }
      if ( json_size( m, "vdim" ) != layer.dim ) {
        throw JsonError( "attention: values are keys, so vdim must equal dim" );
      }
      if ( const Json* t = m.find( "q_temp" ); t != nullptr && !t->is_null() ) {
        layer.temp_coef = static_cast<float>( ( *t )["coef"].number() );
        layer.temp_every = json_size( *t, "every" );
      }
      layer.ff = dense_feed_forward( l );
      c.layers.push_back( layer );
    }
    if ( c.layers.empty() ) {
      throw JsonError( "no layers" );
    }
    return c;
  }
};

} // namespace glint
