// Configuration of the Famidra design, read from a model directory's config.json: a decoder-only model whose layers each name their
// mixer (matrix-memory LSTM, or windowed attention with a bias by distance) and an optional gated feed-forward, with a run of layers
// that is passed several times with the same weights.
#pragma once

#include <algorithm>
#include <cmath>
#include <cstdint>
#include <optional>
#include <string>
#include <vector>

#include "glint/design_config.hh"

namespace glint {

namespace configs {
struct Famidra // the tag its states and settings are typed with
{
  constexpr static bool sized_at_run_time = true;
};
} // namespace configs

// sizes and constants of the mixers and of the feed-forward
struct MlstmConfig
{
  uint32_t heads {}, dim {}, vdim {};
  float gate_cap {};
};
struct WindowAttentionConfig
{
  uint32_t heads {}, kv_heads {}, dim {}, vdim {};
  float scale {};
  double bias_max {};                  // distance from which on the bias is the table's last row
  uint32_t window {}, keep_first {};   // window 0: no window
};

struct FamidraConfig
{
  struct Layer
  {
    std::optional<MlstmConfig> mlstm {};
    std::optional<WindowAttentionConfig> attention {};
    uint32_t ff { 0 }; // 0: no feed-forward
  };
  // one run of a layer: a looped layer runs once a pass, each with a cache or state of its own
  struct Run
  {
    uint32_t layer {};
    int32_t pass { -1 };           // -1: outside the loop
    bool first_of_pass { false };
  };

  uint32_t width {}, vocab {}, max_positions {};
  float eps {}, logit_scale { 1.0f };
  std::vector<Layer> layers {};
  bool looped { false };
  uint32_t loop_start {}, loop_stop {}, loop_times {};

  std::vector<Run> runs() const
  {
    std::vector<Run> out;
    auto plain = [&]( uint32_t from, uint32_t to ) {
      for ( uint32_t l = from; l < to; l++ ) {
        out.push_back( { l, -1, false } );
      }
    };
    if ( !looped ) {
      plain( 0, static_cast<uint32_t>( layers.size() ) );
      return out;
    }
    plain( 0, loop_start );
    for ( uint32_t t = 0; t < loop_times; t++ ) {
      for ( uint32_t l = loop_start; l < loop_stop; l++ ) {
        out.push_back( { l, static_cast<int32_t>( t ), l == loop_start } );
      }
    }
    plain( loop_stop, static_cast<uint32_t>( layers.size() ) );
    return out;
  }

  // empty string on success
  static std::string parse( const std::string& text, FamidraConfig& out ) { return parse_config( text, out ); }

  static FamidraConfig from_json( const Json& j )
  {
    FamidraConfig c;
    c.width = json_size( j, "width" );
    c.vocab = json_size( j, "vocab" );
    c.max_positions = json_size( j, "max_positions" );
    c.eps = static_cast<float>( j["norm"]["eps"].number() );
    if ( const Json* s = j.find( "logit_scale" ); s != nullptr && !s->is_null() ) {
      c.logit_scale = static_cast<float>( s->number() );
    }
    for ( const Json& l : j["layers"].array() ) {
      Layer layer;
      const Json& m = l["mixer"];
      const std::string& type = l["type"].string();
      if ( type == "mlstm" ) {
        layer.mlstm = MlstmConfig { json_size( m, "heads" ), json_size( m, "dim" ), json_size( m, "vdim" ), static_cast<float>( m["gate_cap"].number() ) };
        if ( !( layer.mlstm->gate_cap > 0 ) ) {
          throw JsonError( "gate_cap must be positive" );
        }
      } else if ( type == "attention" ) {
        WindowAttentionConfig a;
        a.heads = json_size( m, "heads" );
        a.kv_heads = json_size( m, "kv_heads" );
        a.dim = json_size( m, "dim" );
        a.vdim = json_size( m, "vdim" );
        a.scale = static_cast<float>( m["scale"].number() );
        a.bias_max = m["bias_max"].number();
        if ( a.heads % a.kv_heads != 0 || !( a.bias_max > 0 && a.bias_max < 1e8 ) ) {
          throw JsonError( "attention: heads must be a multiple of kv_heads and bias_max positive" );
        }
        if ( const Json* mask = m.find( "mask" ); mask != nullptr && !mask->is_null() ) {
          a.window = json_size( *mask, "size" );
          a.keep_first = mask->find( "keep_first" ) != nullptr ? json_size( *mask, "keep_first", 0 ) : 0;
        }
        layer.attention = a;
      } else {
        throw JsonError( "unknown layer type \"" + type + "\"" );
      }
      layer.ff = dense_feed_forward( l );
      c.layers.push_back( layer );
    }
    if ( c.layers.empty() ) {
      throw JsonError( "no layers" );
    }
    if ( const Json* loop = j.find( "loop" ); loop != nullptr && !loop->is_null() ) {
      c.looped = true;
      c.loop_start = json_size( *loop, "start", 0 );
      c.loop_stop = json_size( *loop, "stop" );
      c.loop_times = json_size( *loop, "times" );
      if ( c.loop_start >= c.loop_stop || c.loop_stop > c.layers.size() || (uint64_t)c.loop_times * ( c.loop_stop - c.loop_start ) > 65536 ) {
        throw JsonError( "loop does not fit the layers" );
      }
    }
    return c;
  }
};

// The row of a distance-bias table a distance falls into: a row a distance up to half of the table, from there on rows whose widths
// grow with the logarithm of the distance, the last one without an end.  (The small term keeps distances whose exact value is a whole
// number on the upper side of the rounding.)
inline uint32_t distance_bucket( const uint64_t distance, const uint32_t rows, const double bias_max )
{
  const uint32_t half = rows / 2;
  if ( distance < half ) {
    return static_cast<uint32_t>( distance );
  }
  if ( half == 0 ) {
    return rows - 1;
  }
  const double at = std::log( static_cast<double>( distance ) / half ) / std::log( bias_max / half ) * ( rows - half );
  return !( at < rows - 1 - half ) ? rows - 1 : half + static_cast<uint32_t>( std::max( 0.0, at ) + 1e-9 );
}

} // namespace glint
