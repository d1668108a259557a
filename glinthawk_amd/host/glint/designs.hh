// Registry of the designs whose sizes come from a model directory: config.json names the architecture, the registry picks the driver
// and instantiates it for the storage type and the kind of contexts.  (The Llama2 family is registered by shape name: its sizes are
// compile-time constants.)
#pragma once

#include <filesystem>
#include <memory>
#include <string>

#include "glint/dirozen.hh"
#include "glint/famidra.hh"
#include "glint/stage.hh"

namespace glint {

struct DesignOptions
{
  DataType dtype { DataType::BFloat16 };
  bool paged { false };
  uint64_t concurrency_limit { 1 };
  uint64_t max_context_count { 1 };
  uint32_t max_positions { 0 }; // of a context, for designs whose config.json does not bound them; 0: DEFAULT_POSITIONS
  ModelOptions model {};        // model.randomize: draw the weights, only config.json is read
};
constexpr uint32_t DEFAULT_POSITIONS = 4096;

inline bool is_known_design( const std::string& architecture ) { return architecture == "Famidra" || architecture == "Dirozen"; }

// use() for one design: its driver for the storage type and the kind of contexts
template<template<typename, typename> class Model, typename Config, typename Use>
std::string with_design_config( const Config& config, const DesignOptions& o, const std::string& architecture, Use&& use )
{
  DesignSettings settings;
  settings.concurrency_limit = o.concurrency_limit;
  settings.max_context_count = o.max_context_count;
  settings.randomize_parameters = o.model.randomize;
  auto run = [&]<typename DType>( DType ) -> std::string {
    if ( o.paged ) {
      return use( std::type_identity<Model<DType, hip::DynamicLayeredContext>> {}, config, settings, o.model );
    }
    return use( std::type_identity<Model<DType, hip::LayeredContext>> {}, config, settings, o.model );
  };
  switch ( o.dtype ) {
    case DataType::BFloat16: return run( bfloat16_t {} );
    case DataType::Float32: return run( float32_t {} );
    default: return architecture + " runs in bfloat16 or float32";
  }
}

// use( Model type tag, config, settings, model options ) for the design in `model_dir`; empty string on success
template<typename Use>
std::string with_design( const std::filesystem::path& model_dir, const DesignOptions& o, Use&& use )
{
  std::string text;
  if ( !read_text_file( model_dir / "config.json", text ) ) {
    return "cannot read " + ( model_dir / "config.json" ).string();
  }
  const std::string architecture = architecture_of( model_dir );
  if ( !is_known_design( architecture ) ) {
    return "unknown architecture \"" + architecture + "\"";
  }
  if ( architecture == "Dirozen" ) {
    DirozenConfig config;
    if ( auto err = DirozenConfig::parse( text, config ); !err.empty() ) {
      return err;
    }
    config.max_positions = o.max_positions > 0 ? o.max_positions : DEFAULT_POSITIONS;
    return with_design_config<Dirozen>( config, o, architecture, use );
  }
  FamidraConfig config;
  if ( auto err = FamidraConfig::parse( text, config ); !err.empty() ) {
    return err;
  }
  return with_design_config<Famidra>( config, o, architecture, use );
}

// a stage over the design in `model_dir`, weights loaded (or drawn); nullptr and the reason on failure
inline std::unique_ptr<StageBase> open_design_stage( const std::filesystem::path& model_dir, const DesignOptions& o, std::string& why )
{
  std::unique_ptr<StageBase> stage;
  why = with_design( model_dir, o, [&]( auto tag, const auto& config, const auto& settings, const ModelOptions& options ) -> std::string {
    using Model = typename decltype( tag )::type;
    auto made = std::make_unique<DesignStage<Model>>( config, settings, options );
    if ( !settings.randomize_parameters ) {
      if ( auto err = made->model.load( model_dir ); !err.empty() ) {
        return err;
      }
    }
    stage = std::move( made );
    return {};
  } );
  return stage;
}

} // namespace glint
